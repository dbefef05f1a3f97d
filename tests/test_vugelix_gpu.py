"""Vugelix on the MI355X path (HIP kernels; fp32 and bf16 activations) against the plain oracle in
tests/oracles: every kernel alone, then the whole model through the engine."""

import pytest
import torch

import vugelix_cases as K
import vugelix_common as C

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
IDS = ["fp32", "bf16"]
CONFIGS = [C.config_a, C.config_b, C.config_c]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("case", [K.case_relu2, K.case_hyper_step], ids=lambda f: f.__name__)
def test_kernel(case, dtype):
    case("cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("shape", [
    # H, G, D, Dv, window, tokens, page, cap
    (4, 2, 16, 8, 40, 120, 16, 12.0),
    (3, 3, 10, 6, 17, 90, 16, 0.0),
    # bf16: the matrix-core form's variants (values wider and narrower than keys, a partial last
    # workgroup of heads, 32- and 64-token pages, key partitions, no window)
    (8, 2, 64, 64, 64, 200, 64, 20.0),
    (6, 1, 80, 112, 0, 150, 64, 9.0),
    (5, 5, 32, 80, 100, 200, 32, 15.0),
    (4, 4, 48, 16, 300, 420, 32, 30.0),
], ids=lambda s: "-".join(map(str, s)))
def test_needle(shape, dtype):
    H, G, D, Dv, size, n, bs, cap = shape
    K.case_needle("cuda", dtype, H, G, D, Dv, size, n, bs, cap)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("shape", [
    # H, G, D, Dv, taps, attention heads, kv heads, key / value sizes, rotated entries, tokens, page
    (4, 2, 10, 6, 3, 2, 1, 12, 8, 6, 45, 16),
    (3, 3, 4, 9, 1, 3, 3, 6, 4, 0, 20, 16),
    (2, 1, 64, 48, 4, 4, 2, 32, 64, 16, 45, 32),
    (4, 1, 33, 17, 8, 1, 1, 16, 16, 16, 44, 8),
    (2, 2, 136, 24, 2, 1, 1, 160, 24, 40, 26, 16),
    (6, 3, 128, 128, 6, 8, 1, 128, 128, 128, 30, 64),
], ids=lambda s: "-".join(map(str, s)))
def test_delta_prep(shape, dtype):
    K.case_delta_prep("cuda", dtype, *shape)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("kind", ["needle", "same", "forget"])
@pytest.mark.parametrize("shape", [
    # H, G, D, Dv, tokens
    (3, 1, 10, 6, 75), (2, 2, 64, 64, 70), (4, 2, 48, 112, 40), (2, 1, 160, 33, 30),
    (1, 1, 24, 200, 20), (2, 2, 5, 3, 40),
], ids=lambda s: "-".join(map(str, s)))
def test_delta_scan(shape, kind, dtype):
    K.case_delta_scan("cuda", dtype, *shape, kind=kind)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("kind", ["needle", "same", "forget"])
@pytest.mark.parametrize("shape", [
    (3, 1, 10, 6, 150), (2, 2, 64, 64, 140), (4, 2, 48, 112, 131), (2, 1, 128, 128, 200),
    (1, 1, 96, 17, 64), (2, 2, 5, 80, 66),
], ids=lambda s: "-".join(map(str, s)))
def test_delta_scan_chunk_parallel(shape, kind, dtype):
    K.case_delta_scan("cuda", dtype, *shape, kind=kind, chunked=True)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("cfg", CONFIGS, ids=lambda f: f.__name__)
def test_layers(cfg, dtype):
    K.case_layers("cuda", dtype, cfg)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("cfg", CONFIGS, ids=lambda f: f.__name__)
def test_schedules(cfg, dtype):
    K.case_schedules("cuda", dtype, cfg, seed=7)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
def test_schedules_pages_of_32(dtype):
    """Pages of 32 tokens: the bf16 run takes the matrix-core attention form end to end."""
    K.case_schedules("cuda", dtype, C.config_c, seed=3, block_size=32)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
def test_long_decode(dtype):
    K.case_long_decode("cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("cfg", CONFIGS, ids=lambda f: f.__name__)
def test_generate_through_engine(cfg, dtype):
    """(bf16 and fp32 decode steps replay HIP graphs)"""
    K.case_generate("cuda", dtype, cfg)


def test_generate_graph_decode():
    K.case_generate("cuda", torch.bfloat16, C.config_c, expect_graphs=True)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
def test_declared_kernel_sources_cover_a_step(dtype):
    """Every kernel that a replayed step launches comes from the source files the model declares (a
    fresh checkout compiles those alone)."""
    import os
    import re

    from enterprise_inference_amd import _native
    from enterprise_inference_amd.models.vugelix import VugelixForCausalLM
    kdir = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "csrc", "kernels")
    declared = set()
    for stem in VugelixForCausalLM.kernel_sources:
        with open(os.path.join(kdir, stem + ".hip")) as f:
            declared |= set(re.findall(r"EIA_API int (eia_\w+)", f.read()))
    real, used = _native.kernels(), set()

    class Recorder:
        def __getattr__(self, name):
            used.add(name)
            return getattr(real, name)

    _native._kernels = Recorder()
    try:
        for cfg in (C.config_a, C.config_c):
            K.case_schedules("cuda", dtype, cfg, seed=7, block_size=32)
    finally:
        _native._kernels = real
    assert "eia_delta_prep" in used and used <= declared, used - declared


def test_native_library_loaded():
    from enterprise_inference_amd import _native
    lib = _native.kernels()
    assert hasattr(lib, "eia_delta_prep") and hasattr(lib, "eia_delta_scan_chunked")
    assert any("libeia_kernels" in p for p in _native.loaded_native_libraries())
