"""Borosun on the framework's CPU path (PyTorch ops, fp32) against the plain oracle in
tests/oracles: every mechanism alone, then the whole model through the engine."""

import pytest
import torch

import borosun_cases as K
import borosun_common as C

F32 = torch.float32
CONFIGS = [C.config_a, C.config_b, C.config_c, C.config_d]


@pytest.mark.parametrize("case", [K.case_gated_residual, K.case_side_output, K.case_act_mul_embed,
                                  K.case_prep, K.case_gla_scan], ids=lambda f: f.__name__)
def test_mechanism(case):
    case("cpu", F32)


def test_frequencies():
    K.case_frequencies()


def test_prep_without_convolution_and_normed():
    K.case_prep("cpu", F32, H=3, G=3, D=8, Dv=12, dims=8, taps=0, normed=True)
    K.case_prep("cpu", F32, H=2, G=2, D=6, Dv=4, dims=6, taps=1)
    K.case_prep("cpu", F32, H=2, G=1, D=6, Dv=4, dims=0, taps=8)


@pytest.mark.parametrize("size,cap,mixed", [(0, 0.0, True), (40, 2.0, True), (40, 2.0, False)])
def test_mix_needle(size, cap, mixed):
    K.case_mix_needle("cpu", F32, size=size, cap=cap, mixed=mixed, n=120)


def test_gla_strong_decay():
    K.case_gla_scan("cpu", F32, H=1, D=4, Dv=4, R=1, tau=1.0, T=60, bias=-6.0)


@pytest.mark.parametrize("cfg", CONFIGS, ids=lambda f: f.__name__)
def test_layers(cfg):
    K.case_layers("cpu", F32, cfg)


@pytest.mark.parametrize("cfg", [C.config_a, C.config_b], ids=lambda f: f.__name__)
def test_schedules(cfg):
    K.case_schedules("cpu", F32, cfg)


def test_long_decode():
    K.case_long_decode("cpu", F32)


def test_generate_through_engine():
    K.case_generate("cpu", F32)


def test_config_reader_and_registry():
    from enterprise_inference_amd.config import ModelConfig
    from enterprise_inference_amd.models import get_model_class
    from enterprise_inference_amd.models.mixers import GatedLinearMixer, MixAttentionMixer
    mc = ModelConfig.from_hf_dict(C.config_a())
    assert mc.architecture == "Borosun" and mc.extra["token_side"]["dim"] == 5
    assert mc.extra["logit_softcap"] == 6.0
    model = get_model_class("Borosun")(mc, dtype=F32)
    M, L = MixAttentionMixer, GatedLinearMixer
    assert [type(x.mix) for x in model.layers] == [M, L, M, M, L]
    assert [getattr(x.mix, "v_mix", None) for x in model.layers] == [None, None, "first", "later",
                                                                     None]
    assert model.layers[1].mlp is None and "rg2" not in model.layers[1].proj.offsets
    assert model.layers[3].mix.taps == 5 and model.layers[2].mix.taps == 1
    assert model.layers[2].mix.spec.window == 9 and model.layers[2].mix.spec.cap == 3.0
    plain = get_model_class("Borosun")(ModelConfig.from_hf_dict(C.config_b()), dtype=F32)
    assert plain.side_embed is None and plain.softcap == 0.0
    assert not any(".side." in n for n, _ in plain.named_parameters())


def test_decay_rank_comes_from_the_checkpoint(tmp_path):
    """The low-rank branch's size is a tensor shape, not a config key."""
    import json

    from safetensors.torch import save_file

    from enterprise_inference_amd.models.loader import resolve_model_config
    cfg = C.config_b()
    W = C.random_weights(cfg, 1)
    del cfg["layers"][0]["mixer"]["decay_rank"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in W.items()}, str(tmp_path / "model.safetensors"))
    mc = resolve_model_config(str(tmp_path))
    assert mc.extra["layers"][0]["mixer"]["decay_rank"] == 3


def test_every_tensor_has_a_place():
    """Every checkpoint name of a configuration lands in a parameter, every parameter is named
    by the checkpoint, and an unknown name is refused."""
    from enterprise_inference_amd.config import ModelConfig
    from enterprise_inference_amd.models import get_model_class
    for fn in CONFIGS:
        cfg = fn()
        model = get_model_class("Borosun")(ModelConfig.from_hf_dict(cfg), dtype=F32)
        W = C.random_weights(cfg, 1)
        loaded = set(model.load_weights(W.items()))
        assert loaded == {n for n, _ in model.named_parameters()}
        for bad in ("l0.mix.nothing", "l0.mix.rg1", "l99.norm1", "head"):
            with pytest.raises(ValueError):
                model.load_weights([(bad, torch.zeros(1))])
