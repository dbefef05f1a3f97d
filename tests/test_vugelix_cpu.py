"""Vugelix on the framework's CPU path (PyTorch ops, fp32) against the plain oracle in
tests/oracles: every mechanism alone, then the whole model through the engine."""

import copy

import pytest
import torch

import vugelix_cases as K
import vugelix_common as C

F32 = torch.float32
CONFIGS = [C.config_a, C.config_b, C.config_c]


@pytest.mark.parametrize("case", [K.case_relu2, K.case_hyper_step, K.case_delta_prep],
                         ids=lambda f: f.__name__)
def test_mechanism(case):
    case("cpu", F32)


def test_frequencies():
    K.case_frequencies()


@pytest.mark.parametrize("size", [0, 40])
def test_needle(size):
    K.case_needle("cpu", F32, size=size, n=100)


@pytest.mark.parametrize("taps", [1, 2, 6])
def test_delta_prep_taps(taps):
    K.case_delta_prep("cpu", F32, H=3, G=3, D=4, Dv=8, taps=taps, aH=3, aG=3, aD=6, aDv=4, dims=0, T=20)


@pytest.mark.parametrize("kind", ["needle", "same", "forget"])
def test_delta_scan(kind):
    K.case_delta_scan("cpu", F32, kind=kind, T=50)


@pytest.mark.parametrize("cfg", CONFIGS, ids=lambda f: f.__name__)
def test_layers(cfg):
    K.case_layers("cpu", F32, cfg, n=30)


@pytest.mark.parametrize("cfg", [C.config_a, C.config_b], ids=lambda f: f.__name__)
def test_schedules(cfg):
    K.case_schedules("cpu", F32, cfg)


def test_long_decode():
    K.case_long_decode("cpu", F32)


def test_generate_through_engine():
    K.case_generate("cpu", F32)


def _model(cfg):
    from enterprise_inference_amd.config import ModelConfig
    from enterprise_inference_amd.models import get_model_class
    mc = ModelConfig.from_hf_dict(copy.deepcopy(cfg))
    return get_model_class(mc.architecture)(mc, dtype=F32)


def test_config_reader_and_registry():
    m = _model(C.config_a())
    assert m.streams == 3 and m.embed_scale == 2.5 and m.logit_scale == 0.7 and m.head is None
    assert m.layers[2] is m.layers[0] and m.layers[3] is not m.layers[0]
    assert m.layers[1].mlp is None and m.layers[3].mix.right.spec.taps == 5
    assert m.layers[0].mix.left.spec.window == 24 and m.layers[1].mix.left.spec.window == 17
    b = _model(C.config_b())
    assert b.layers[3] is b.layers[1] and b.embed_scale == 1.0 and b.logit_scale == 1.0
    assert b.layers[1].mix.left.spec.window == 0 and b.layers[1].mix.left.spec.cap == 0.0
    c = _model(C.config_c())
    assert c.layers[0] is c.layers[2] and c.layers[3] is c.layers[1]
    for wrong in (7, 0):                                # no such layer; a layer of its own
        bad = C.config_a()
        bad["layers"][0]["weights_of"] = wrong
        with pytest.raises(ValueError):
            _model(bad)


def test_layers_that_share_weights_have_caches_of_their_own():
    m = _model(C.config_a())
    caches = m.allocate_cache(4, 16, 2, F32, torch.device("cpu"))
    kv0, st0 = caches[0]
    kv2, st2 = caches[2]
    assert kv0.k.data_ptr() != kv2.k.data_ptr() and st0.S.data_ptr() != st2.S.data_ptr()
    assert st0.hist.data_ptr() != st2.hist.data_ptr() and caches[4] is None
    per = sum(c[1].S[0].numel() * 4 + (c[1].hist[0].numel() * 4 if c[1].hist is not None else 0)
              for c in caches[:4])
    assert m.state_slot_bytes() == per
    assert m.cache_block_bytes(16, F32) == sum((c[0].k[0].numel() + c[0].v[0].numel()) * 4
                                               for c in caches[:4])


def test_every_tensor_has_a_place():
    """Every checkpoint name of a configuration lands in a parameter, every parameter is named by the
    checkpoint, and unknown names (a sharing layer's too) are refused."""
    for cfg in (C.config_a(), C.config_b(), C.config_c()):
        m = _model(cfg)
        loaded = set(m.load_weights(C.random_weights(cfg, 1).items()))
        params = {n: p for n, p in m.named_parameters(remove_duplicate=False)}
        assert {id(params[n]) for n in loaded} == {id(p) for p in m.parameters()}
        shared = [i for i, L in enumerate(cfg["layers"]) if L.get("weights_of") is not None]
        for name in ("l0.mix.nothing", "l9.norm1", f"l{shared[0]}.norm1", "l1.mix.left.norm"):
            with pytest.raises(ValueError):
                m.load_weights([(name, torch.zeros(1))])


def test_random_initialisation_keeps_pads_zero():
    m = _model(C.config_a())
    m.init_random(3)
    m.post_load()
    for L in m.layers:
        o, mix = L.mix.o.data, L.mix
        assert not o[:, mix.lw:mix.lw_pad].any() and not o[:, mix.lw_pad + mix.rw:].any()
        assert o[:, :mix.lw].any() and bool(torch.isfinite(mix.right.spec.exp_a).all())


def test_kernel_source_subset_has_a_library_of_its_own():
    import importlib.util
    import os
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    spec = importlib.util.spec_from_file_location("eia_build", os.path.join(root, "csrc", "build.py"))
    b = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(b)
    from enterprise_inference_amd.models.vugelix import VugelixForCausalLM
    stems = [os.path.basename(p)[:-4] for p in b.kernel_sources()]
    src = VugelixForCausalLM.kernel_sources
    assert set(src) < set(stems)
    assert b.partial_so(src) == b.partial_so(tuple(reversed(src))) != b.KERNELS_SO
    assert b.partial_so(src[:-1]) != b.partial_so(src)
    with pytest.raises(ValueError):
        b.build_kernels(only=("no_such_file",))
