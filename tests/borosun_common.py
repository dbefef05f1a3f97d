"""Shared pieces of the Borosun tests: small configurations, random checkpoints under the design's
tensor names and a session that drives the engine (scheduler bookkeeping, model runner, kernels)
step by step.  The expected values come from tests/oracles/borosun_oracle.py only."""

from __future__ import annotations

import copy

import torch

from oracles import borosun_oracle as O


def att(heads=4, kv=2, dim=10, vdim=6, dims=6, base=900.0, scaling=None, conv=3, scale=0.4,
        v_mix=True, ff=20):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if conv:
        m["conv"] = conv
    if v_mix:
        m["v_mix"] = True
    if dims:
        m["rot"] = {"base": base, "dims": dims}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def att2(heads=4, kv=2, dim=12, vdim=6, dims=4, base=5000.0, size=9, cap=3.0, scale=0.7,
         v_mix=True, ff=20):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
         "softcap": cap, "mask": {"size": size}}
    if v_mix:
        m["v_mix"] = True
    if dims:
        m["rot"] = {"base": base, "dims": dims}
    return {"type": "attention_2", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def gla(heads=3, dim=6, vdim=10, tau=4.0, rank=5, ff=20):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau,
                                     "decay_rank": rank},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config_a():
    """Odd sizes: a width that is no multiple of four, rotation on part of a head with banded
    frequency scaling, key / value sizes that differ, an odd side width, layers without
    feed-forward, one attention layer without value mixing ahead of the first that has it."""
    return {"architecture": "Borosun", "vocab": 90, "width": 46, "norm": {"eps": 1e-5},
            "token_side": {"dim": 5}, "logit_softcap": 6.0,
            "layers": [att(scaling=(4.0, 1.0, 4.0, 64), v_mix=False), gla(ff=0),
                       att2(heads=2, kv=1, dim=12, vdim=12, size=9),
                       att(heads=6, kv=2, dim=8, vdim=6, dims=8, base=70.0, conv=5, ff=0,
                           scaling=(2.0, 0.5, 3.0, 40)),
                       gla(heads=1, dim=9, vdim=7, tau=1.0, rank=2, ff=16)]}


def config_b():
    """A recurrent layer first, two taps, one kv head, no frequency scaling, no rotation in one
    layer, a window of one page and a bit, no token side, no logit cap, one head."""
    return {"architecture": "Borosun", "vocab": 70, "width": 40, "norm": {"eps": 1e-6},
            "layers": [gla(heads=2, dim=8, vdim=4, tau=16.0, rank=3, ff=24),
                       att2(heads=3, kv=3, dim=6, vdim=4, dims=6, size=21, cap=20.0, ff=0),
                       att(heads=3, kv=1, dim=8, vdim=12, dims=0, conv=2, ff=12),
                       att(heads=1, kv=1, dim=4, vdim=12, dims=2, conv=0, ff=8),
                       att(heads=2, kv=2, dim=4, vdim=6, dims=4, conv=1, ff=0)]}


def config_c():
    """Sizes in multiples of the matrix-core tiles; eight heads on two kv heads, value sizes above
    and below the key sizes, a window of 40, a side width of 16."""
    return {"architecture": "Borosun", "vocab": 160, "width": 128, "norm": {"eps": 1e-5},
            "token_side": {"dim": 16}, "logit_softcap": 9.0,
            "layers": [att(heads=8, kv=2, dim=32, vdim=64, dims=32, base=20000.0, conv=4, scale=0.2,
                           scaling=(4.0, 1.0, 4.0, 32), ff=128),
                       gla(heads=2, dim=64, vdim=32, tau=8.0, rank=16, ff=64),
                       att2(heads=4, kv=4, dim=64, vdim=32, dims=16, size=40, cap=10.0, scale=0.3,
                            ff=128),
                       att(heads=4, kv=2, dim=24, vdim=64, dims=24, conv=4, scale=0.25, ff=0),
                       gla(heads=4, dim=16, vdim=16, tau=2.0, rank=16, ff=128)]}


def config_d():
    """More than sixteen mixed heads, groups of five, wide heads, eight taps, a strong decay."""
    return {"architecture": "Borosun", "vocab": 80, "width": 64, "norm": {"eps": 1e-5},
            "token_side": {"dim": 130}, "logit_softcap": 20.0,
            "layers": [att(heads=20, kv=4, dim=16, vdim=16, dims=8, base=300.0, conv=8, scale=0.3,
                           ff=32),
                       att2(heads=2, kv=1, dim=104, vdim=64, dims=104, size=33, cap=5.0, scale=0.1,
                            ff=32),
                       gla(heads=1, dim=128, vdim=16, tau=1.0, rank=4, ff=0)]}


def random_weights(cfg: dict, seed: int = 0, dtype=torch.float32, tie_qk: bool = False) -> dict:
    """A checkpoint for ``cfg`` under the design's tensor names (values rounded to ``dtype``).
    ``tie_qk``: W_k = W_q in the recurrent layers, so a first token's q . k is a square and the
    sign of its normed output survives 16-bit rounding."""
    g = torch.Generator().manual_seed(seed)
    W = {}

    def mat(n, k, s=1.0):
        return torch.randn(n, k, generator=g) * (s / k ** 0.5)

    def vec(n, mean=0.0, s=0.2):
        return mean + torch.randn(n, generator=g) * s

    Wd, V = cfg["width"], cfg["vocab"]
    side = (cfg.get("token_side") or {}).get("dim", 0)
    W["embed"] = torch.randn(V, Wd, generator=g)
    if side:
        W["side.embed"] = torch.randn(V, len(cfg["layers"]) * side, generator=g)
    W["final.norm"] = vec(Wd, 0.4, 0.1)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        W[p + "norm1"] = vec(Wd, 1.0)
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        if L["type"] == "gla":
            W[p + "mix.q"], W[p + "mix.k"] = mat(H * D, Wd, 1.5), mat(H * D, Wd, 1.5)
            if tie_qk:
                W[p + "mix.k"] = W[p + "mix.q"].clone()
            W[p + "mix.v"], W[p + "mix.g"] = mat(H * Dv, Wd), mat(H * Dv, Wd, 2.0)
            R = m["decay_rank"]
            W[p + "mix.a1"], W[p + "mix.a2"] = mat(R, Wd, 1.5), mat(H * D, R, 2.0)
            W[p + "mix.a2.b"] = vec(H * D, 1.0, 1.5)
            W[p + "mix.norm"] = vec(Dv, 1.0)
        else:
            G = m["kv_heads"]
            W[p + "mix.q"], W[p + "mix.k"] = mat(H * D, Wd, 1.5), mat(G * D, Wd, 1.5)
            W[p + "mix.v"] = mat(G * Dv, Wd)
            if m.get("conv"):
                for n, c in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                    W[p + f"mix.{n}.conv"] = torch.randn(c, m["conv"], generator=g) * 0.5
            if m.get("v_mix"):
                W[p + "mix.vmix"] = torch.tensor(0.2 + 0.1 * i)
            if L["type"] == "attention":
                W[p + "mix.talk"] = torch.eye(H) + torch.randn(H, H, generator=g) * 0.4
        W[p + "mix.o"] = mat(Wd, H * Dv, 0.9)
        W[p + "rg1"], W[p + "rg1.b"] = mat(Wd, Wd, 1.5), vec(Wd, 0.3, 0.5)
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            W[p + "mlp.gate"], W[p + "mlp.up"] = mat(ff, Wd, 1.5), mat(ff, Wd, 1.5)
            W[p + "mlp.down"] = mat(Wd, ff, 0.9)
            W[p + "rg2"], W[p + "rg2.b"] = mat(Wd, Wd, 1.5), vec(Wd, -0.2, 0.5)
        if side:
            W[p + "side.gate"], W[p + "side.proj"] = mat(side, Wd), mat(Wd, side)
            W[p + "side.norm"] = vec(Wd, 0.3, 0.1)
    return {k: v.to(dtype).float() for k, v in W.items()}


def as_numpy(W: dict) -> dict:
    return {k: v.double().numpy() for k, v in W.items()}


def oracle_logits(cfg, W, tokens, collect=None):
    return torch.from_numpy(O.forward(cfg, as_numpy(W), list(tokens), collect)).float()


def make_session(cfg: dict, W: dict, device: str, dtype=torch.float32, max_tokens: int = 512,
                 block_size: int = 16, max_live: int = 4):
    """A replay session of the engine holding the checkpoint W."""
    from enterprise_inference_amd.config import ModelConfig
    from enterprise_inference_amd.entrypoints.trace_run import TraceSession, replay_config

    mc = ModelConfig.from_hf_dict(copy.deepcopy(cfg))
    ec = replay_config(mc, None, dtype, device, max_tokens, block_size, max_live,
                       load_format="dummy")
    sess = TraceSession(ec)
    model = sess.runner.model
    model.load_weights(W.items())
    model.post_load()
    return sess


def rel_err(got: torch.Tensor, want: torch.Tensor) -> float:
    """Row-wise error as the mean-free RMS difference over the RMS of the expected logits."""
    d = got.double().cpu() - want.double()
    d = d - d.mean(-1, keepdim=True)
    w = want.double() - want.double().mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt().clamp_min(1e-9)).max())
