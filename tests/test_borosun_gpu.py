"""Borosun on the MI355X path (HIP kernels; fp32 and bf16 activations) against the plain oracle
in tests/oracles: every kernel alone, then the whole model through the engine."""

import pytest
import torch

import borosun_cases as K
import borosun_common as C

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
IDS = ["fp32", "bf16"]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("case", [K.case_gated_residual, K.case_side_output, K.case_act_mul_embed],
                         ids=lambda f: f.__name__)
def test_kernel(case, dtype):
    case("cuda", dtype)


@pytest.mark.parametrize("shape", [(288, 28, 300, 2, True), (64, 128, 257, 1, False),
                                   (1056, 130, 256, 2, True), (2048, 256, 270, 2, True),
                                   (480, 500, 256, 1, True)], ids=lambda s: "-".join(map(str, s)))
def test_token_side(shape):
    K.case_token_side(*shape)


@pytest.mark.parametrize("cfg", [C.config_c, C.config_d], ids=lambda f: f.__name__)
def test_long_prompt_mixed_with_decoding(cfg):
    K.case_long_prompt("cuda", torch.bfloat16, cfg)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("shape", [
    # H, G, D, Dv, rotated entries, taps, head norm, page, split-K partials
    (4, 2, 10, 6, 6, 3, False, 16, False),
    (3, 3, 8, 12, 8, 0, True, 16, False),
    (4, 2, 32, 16, 8, 1, False, 16, True),
    (8, 2, 64, 32, 32, 4, False, 32, True),
    (5, 1, 16, 9, 0, 8, False, 16, False),
    (2, 1, 160, 200, 100, 2, True, 32, False),
    (6, 2, 128, 128, 128, 5, True, 64, True),
    (2, 2, 48, 16, 20, 6, False, 16, False),
    (2, 2, 32, 16, 32, 7, False, 16, True),
], ids=lambda s: "-".join(map(str, s)))
def test_prep(shape, dtype):
    H, G, D, Dv, dims, taps, normed, bs, split = shape
    K.case_prep("cuda", dtype, H, G, D, Dv, dims, taps, normed, 45, bs, split)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("shape", [
    # H, G, D, Dv, window, cap, tokens, page
    (4, 2, 16, 8, 0, 0.0, 150, 16),
    (3, 3, 10, 6, 40, 2.0, 120, 16),
    # bf16: the matrix-core form's variants (all heads on one kv head, groups of two, three, four
    # and five, one head per kv head, more than sixteen heads, values wider and narrower than
    # keys, key sizes that are no multiple of 32, 32- to 128-token pages, key partitions)
    (8, 2, 64, 64, 0, 0.0, 300, 64),
    (4, 1, 128, 128, 0, 0.0, 260, 32),
    (4, 2, 80, 112, 70, 3.0, 200, 32),
    (6, 2, 32, 80, 0, 0.0, 180, 32),
    (4, 4, 24, 16, 0, 0.0, 150, 32),
    (20, 4, 40, 32, 0, 5.0, 220, 64),
    (16, 4, 128, 128, 0, 0.0, 420, 128),
    (1, 1, 64, 96, 33, 0.0, 140, 32),
    (24, 6, 16, 128, 0, 0.0, 700, 64),
    (7, 1, 128, 48, 0, 0.0, 1100, 64),
], ids=lambda s: "-".join(map(str, s)))
def test_mix_needle(shape, dtype):
    H, G, D, Dv, size, cap, n, bs = shape
    K.case_mix_needle("cuda", dtype, H, G, D, Dv, n, bs, size, cap)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("shape", [
    (4, 2, 16, 8, 9, 2.0, 100, 16),
    (6, 2, 64, 80, 75, 5.0, 200, 64),
    (4, 1, 128, 128, 50, 20.0, 220, 32),
    (6, 3, 48, 96, 0, 1.5, 150, 32),
], ids=lambda s: "-".join(map(str, s)))
def test_softcap_needle(shape, dtype):
    H, G, D, Dv, size, cap, n, bs = shape
    K.case_mix_needle("cuda", dtype, H, G, D, Dv, n, bs, size, cap, mixed=False)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("shape", [
    # H, D, Dv, rank, tau, tokens, decay bias
    (3, 10, 6, 5, 4.0, 75, 1.0),
    (2, 32, 40, 12, 12.0, 60, 0.0),
    (1, 64, 48, 3, 1.0, 70, -6.0),
    (2, 24, 128, 16, 8.0, 40, 2.0),
    (1, 160, 96, 33, 2.0, 30, 1.0),
], ids=lambda s: "-".join(map(str, s)))
def test_gla_scan(shape, dtype):
    H, D, Dv, R, tau, T, bias = shape
    K.case_gla_scan("cuda", dtype, H, D, Dv, R, tau, T, False, bias)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("shape", [(3, 10, 6, 5, 4.0, 150, 1.0), (2, 64, 48, 16, 16.0, 140, 0.0),
                                   (2, 128, 128, 16, 8.0, 135, 2.0), (1, 24, 128, 2, 1.0, 200, -8.0),
                                   (1, 33, 16, 7, 1.0, 170, 0.5)],
                         ids=lambda s: "-".join(map(str, s)))
def test_gla_scan_chunk_parallel(shape, dtype):
    H, D, Dv, R, tau, T, bias = shape
    K.case_gla_scan("cuda", dtype, H, D, Dv, R, tau, T, True, bias)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("cfg", [C.config_a, C.config_b, C.config_c, C.config_d],
                         ids=lambda f: f.__name__)
def test_layers(cfg, dtype):
    K.case_layers("cuda", dtype, cfg)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("cfg,seed,bs", [(C.config_a, 7, 16), (C.config_b, 7, 16),
                                         (C.config_c, 7, 16), (C.config_c, 3, 32),
                                         (C.config_d, 5, 32)],
                         ids=lambda v: getattr(v, "__name__", str(v)))
def test_schedules(cfg, seed, bs, dtype):
    K.case_schedules("cuda", dtype, cfg, seed, bs)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
def test_long_decode(dtype):
    K.case_long_decode("cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
def test_generate_through_engine(dtype):
    K.case_generate("cuda", dtype, C.config_a)


@pytest.mark.parametrize("cfg", [C.config_c, C.config_d], ids=lambda f: f.__name__)
def test_generate_graph_decode(cfg):
    K.case_generate("cuda", torch.bfloat16, cfg, expect_graphs=True, block_size=32)


def test_native_library_loaded():
    from enterprise_inference_amd import _native
    lib = _native.kernels()
    assert hasattr(lib, "eia_head_mix_attn") and hasattr(lib, "eia_qkv_prep")
    assert any("libeia_kernels" in p for p in _native.loaded_native_libraries())
