"""Borosun: a decoder whose config.json lists its layers one by one.  A layer reads ONE RMS norm of
the fp32 residual stream; both of its sublayers join it through element-wise gates of the same
normed input, and a per-layer token embedding follows:

    h = norm1(x)
    x <- x + mixer(h) * sigmoid(W_rg1 h + b1) + ff(h) * sigmoid(W_rg2 h + b2)
    y = W_proj (gelu_tanh(W_gate x) * e_i[token]);    x <- x + rms(y) * w_side

The mixer is ``attention`` (MixAttentionMixer: short convolutions on q, k and v, rotation with
wavelength-banded frequency scaling, full causal softmax, softmax weights mixed across the heads),
``attention_2`` (MixAttentionMixer: rotation, weightless per-head RMS norm of q and k, soft-capped
scores, sliding window) or ``gla`` (GatedLinearMixer), models/mixers.py.  Attention layers with
``v_mix`` add the first such layer's values to theirs.  The feed-forward, where a layer has one, is
``W_down (gelu_tanh(W_gate h) * (W_up h))``.  The LM head is the embedding table behind the model's
norm; logits are soft-capped.

config.json keys: architecture, vocab, width, norm{eps}, token_side{dim}, logit_softcap and
layers[i] = {type, mixer{heads, kv_heads, dim, vdim, scale, rot{base, dims, scaling{factor, low,
high, original}}, conv, mask{size}, softcap, v_mix, tau}, mlp{kind: dense, ff} | null}.  Checkpoint
names: embed, side.embed, final.norm, l<i>.norm1, l<i>.mix.*, l<i>.mlp.*, l<i>.rg1|rg2[.b],
l<i>.side.gate|proj|norm.

Residual stream, norms, angles, scores, softmax weights and their mixing, decays and the recurrent
state are fp32 whatever the activation dtype; with dtype float32 the matrix products are fp32 too.
Everything that reads h rides in one fused projection (mixer inputs and both gates) and one gated
feed-forward GEMM.  A layer's end is one launch for prompt-sized batches (ops/norm.py
token_side_step); decode-sized ones take five (gated residual sum, side gate GEMM, activation
times token embedding, side projection GEMM, and the normed side output with the next layer's
input norm).
"""

from __future__ import annotations

import re
from typing import Iterable, List, Optional, Tuple

import torch
import torch.nn as nn

from ..config import ModelConfig
from ..ops import activation as act_ops
from ..ops import embedding as emb_ops
from ..ops import gemm, norm as norm_ops
from ..ops.attention import AttentionMetadata
from .layers import _param, default_loader
from .llama import LlamaMLP
from .mixers import (FusedProjection, GatedLinearMixer, MixAttentionMixer, PagedKVRows, ValueCarry)


def _plain(shape, dtype, device):
    p = _param(shape, dtype, device)
    p.weight_loader = default_loader
    return p


class TokenSide(nn.Module):
    """A layer's token input: y = W_proj (gelu_tanh(W_gate x) * table[token, col0:col0 + dim]),
    x <- x + rms(y) * norm.  The inner width is padded with zeros to a multiple of 128, the
    reduction unit of the decode GEMMs."""

    def __init__(self, width: int, dim: int, index: int, dtype, device):
        super().__init__()
        self.dim, self.col0, self.pad = dim, index * dim, -(-dim // 128) * 128
        self.gate = _param((self.pad, width), dtype, device)
        self.proj = _param((width, self.pad), dtype, device)
        for p in (self.gate, self.proj):
            p.data.zero_()
        self.gate.weight_loader = lambda p, t, sid=None: p.data[:dim].copy_(t)
        self.proj.weight_loader = lambda p, t, sid=None: p.data[:, :dim].copy_(t)
        self.norm = _plain((width,), dtype, device)
        # copies in matrix-core operand order for the prompt-sized form (refreshed IN PLACE)
        self.packed = None
        if dtype == torch.bfloat16 and width % 32 == 0:
            self.packed = [torch.zeros_like(p.data) for p in (self.gate, self.proj)]

    def refresh(self) -> None:
        if self.packed is not None:
            for dst, w in zip(self.packed, (self.gate, self.proj)):
                dst.copy_(norm_ops.pack_operand(w.data))

    def forward(self, xb: torch.Tensor, ids: torch.Tensor, table: torch.Tensor):
        """xb: the residual in the activation dtype -> y (a tensor or gemm.SplitK)."""
        u = gemm.linear(xb, self.gate, defer_reduce=True)
        g = act_ops.act_mul_embed(u, "gelu_tanh", ids, table, self.col0, self.dim, self.pad)
        return gemm.linear(g, self.proj, defer_reduce=True)


class BorosunLayer(nn.Module):
    def __init__(self, spec: dict, index: int, width: int, eps: float, side_dim: int, v_mix,
                 dtype, device):
        super().__init__()
        m = spec["mixer"]
        self.kind, self.eps = spec["type"], eps
        mlp = spec.get("mlp")
        if mlp is not None and mlp.get("kind", "dense") != "dense":
            raise ValueError(f"unknown Borosun feed-forward kind {mlp.get('kind')!r}")
        H = int(m["heads"])
        D = int(m["dim"])
        Dv = int(m.get("vdim", D))
        gates = [("rg1", width)] + ([("rg2", width)] if mlp is not None else [])
        if self.kind == "gla":
            parts = GatedLinearMixer.parts(H, D, Dv, int(m["decay_rank"]))
        elif self.kind in ("attention", "attention_2"):
            G = int(m.get("kv_heads", H))
            parts = MixAttentionMixer.parts(H, G, D, Dv)
        else:
            raise ValueError(f"unknown Borosun layer type {self.kind!r}")
        self.proj = FusedProjection(width, parts + gates, dtype, device, [n for n, _ in gates])
        if self.kind == "gla":
            self.mix = GatedLinearMixer(H, D, Dv, int(m["decay_rank"]), float(m.get("tau", 1.0)),
                                        eps, dtype, device, proj=self.proj)
        else:
            rot = m.get("rot") or {}
            second = self.kind == "attention_2"
            self.mix = MixAttentionMixer(
                H, G, D, Dv, float(m.get("scale", D ** -0.5)),
                int(rot.get("dims", D if rot else 0)), float(rot.get("base", 10000.0)),
                rot.get("scaling"), eps, dtype, device, offsets=self.proj.offsets,
                taps=int(m.get("conv") or 0), qk_norm=second,
                softcap=float(m.get("softcap") or 0.0),
                window=int((m.get("mask") or {}).get("size", 0)), head_mix=not second,
                v_mix=v_mix)
        self.o = _plain((width, H * Dv), dtype, device)
        self.norm1 = _plain((width,), dtype, device)
        self.mlp = None
        if mlp is not None:
            self.mlp = LlamaMLP(width, int(mlp["ff"]), "gelu_tanh", dtype, device)
        self.side = TokenSide(width, side_dim, index, dtype, device) if side_dim else None

    def forward(self, x, h, md: AttentionMetadata, cache, carry: ValueCarry, ids, table,
                w_next: Optional[torch.Tensor]):
        """x: fp32 residual [T, width], updated in place; h = norm1(x) in the activation dtype.
        Returns the next layer's input norm of the new x, or None when ``w_next`` is None."""
        fused = self.proj(h, defer_reduce=True)
        if self.kind == "gla":
            if isinstance(fused, gemm.SplitK):
                fused = fused.materialize()
            a = self.mix.attend(fused, md, cache)
        else:
            a = self.mix.attend(fused, md, cache, carry)
        ys = [gemm.linear(a, self.o, defer_reduce=True)]
        gates = [gemm.columns(fused, *self.proj.offsets["rg1"])]
        if self.mlp is not None:
            ys.append(self.mlp(h))
            gates.append(gemm.columns(fused, *self.proj.offsets["rg2"]))
        if self.side is None:
            return norm_ops.residual_rms_step(x, self.eps, ys, w_next, gates)
        s = self.side
        if s.packed is not None and norm_ops.token_side_ok(x, ys, gates, s.pad, h.dtype):
            return norm_ops.token_side_step(x, self.eps, ys, gates, ids, table, s.col0, s.dim,
                                            *s.packed, s.norm, w_next)       # prompt-sized
        xb = norm_ops.residual_rms_step(x, self.eps, ys, None, gates, copy_dtype=h.dtype)
        y = s(xb, ids, table)
        return norm_ops.group_norm_step(x, 1, self.eps, y, s.norm, None, w_next)


class BorosunForCausalLM(nn.Module):
    supports_pp = False
    supports_float32 = True        # every kernel of this model has an fp32 form
    needs_state_slots = True       # recurrent layers and convolution histories
    supports_graphs = True         # no step reads anything back to the host

    def __init__(self, cfg: ModelConfig, dtype=torch.bfloat16, device=None):
        super().__init__()
        self.cfg = cfg
        self.dtype = dtype
        device = torch.device(device) if device is not None else torch.device("cpu")
        ex = cfg.extra
        specs = ex["layers"]
        W = cfg.hidden_size
        self.eps = float((ex.get("norm") or {}).get("eps", cfg.rms_norm_eps))
        self.side_dim = int((ex.get("token_side") or {}).get("dim", 0))
        self.softcap = float(ex.get("logit_softcap") or 0.0)
        self.embed = _plain((cfg.vocab_size, W), dtype, device)
        self.side_embed = None
        if self.side_dim:
            self.side_embed = _plain((cfg.vocab_size, len(specs) * self.side_dim), dtype, device)
        layers, seen = [], False
        for i, s in enumerate(specs):
            mixes = s["type"] != "gla" and bool(s["mixer"].get("v_mix"))
            layers.append(BorosunLayer(s, i, W, self.eps, self.side_dim,
                                       ("later" if seen else "first") if mixes else None, dtype,
                                       device))
            seen = seen or mixes
        self.layers = nn.ModuleList(layers)
        self.final_norm = _plain((W,), dtype, device)

    # ------------------------------------------------------------------ cache geometry
    def kv_heads_per_rank(self) -> int:
        return 1

    def cache_block_bytes(self, block_size: int, dtype: torch.dtype) -> int:
        e = torch.tensor([], dtype=dtype).element_size()
        return sum(block_size * sum(L.mix.cache_widths()) * e for L in self.layers
                   if L.kind != "gla") or 1

    def state_slot_bytes(self) -> int:
        e = torch.tensor([], dtype=self.dtype).element_size()
        return sum(L.mix.state_bytes() if L.kind == "gla" else L.mix.state_bytes(e)
                   for L in self.layers)

    def allocate_cache(self, num_blocks: int, block_size: int, num_slots: int,
                       dtype: torch.dtype, device) -> list:
        """Per-layer cache objects: recurrent state slots for a gla layer, (paged K / V rows,
        convolution history slots or None) for an attention layer.  Zero filled: never-written
        rows stay finite under a zero softmax weight."""
        out: list = []
        for L in self.layers:
            if L.kind == "gla":
                out.append(L.mix.allocate_state(num_slots, device))
            else:
                kw, vw = L.mix.cache_widths()
                out.append((PagedKVRows.allocate(num_blocks, block_size, kw, vw, dtype, device),
                            L.mix.allocate_state(num_slots, dtype, device)))
        return out

    def prefill_query_block(self, block_size: int) -> int:
        """The step's work list is built for the first attention layer's query block; layers with
        another one get theirs from AttentionMetadata.prefill_work_for."""
        for L in self.layers:
            if L.kind != "gla":
                return L.mix.query_block(block_size)
        return 16

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, md: AttentionMetadata, caches: list,
                intermediate=None, collect: Optional[list] = None):
        """Returns the fp32 residual stream [T, width].  ``collect`` (a list) receives a copy of
        the stream after every layer."""
        T = input_ids.shape[0]
        x = emb_ops.bigram_embed(input_ids, self.embed, 1.0, None, 1, 0, 0, None, None, None, T,
                                 md.positions, 1).view(T, -1)
        n = len(self.layers)
        if n == 0:
            return x
        carry = ValueCarry()
        h = norm_ops.residual_rms_step(x, self.eps, (), self.layers[0].norm1)
        for i, L in enumerate(self.layers):
            h = L(x, h, md, caches[i], carry, input_ids, self.side_embed,
                  self.layers[i + 1].norm1 if i + 1 < n else None)
            if collect is not None:
                collect.append(x.clone())
        return x

    def compute_logits(self, x: torch.Tensor) -> torch.Tensor:
        """x: rows of the fp32 residual stream -> fp32 logits (tied head, soft cap)."""
        h = norm_ops.residual_rms_step(x.contiguous(), self.eps, (), self.final_norm)
        out = gemm.linear_f32(h, self.embed) if h.dtype == torch.bfloat16 and h.is_cuda else None
        if out is None:
            out = gemm.linear(h, self.embed).float()
        return act_ops.softcap_(out, self.softcap)

    # ------------------------------------------------------------------ weights
    _LAYER = re.compile(r"^l(\d+)\.(.+)$")
    _MLP = {"gate": ("gate_up_proj.weight", 0), "up": ("gate_up_proj.weight", 1),
            "down": ("down_proj.weight", None)}
    _ATTN = {"q.conv": "q_conv", "k.conv": "k_conv", "v.conv": "v_conv", "talk": "talk",
             "vmix": "vmix"}
    _GLA = {"a2": "a2", "a2.b": "a2_bias", "norm": "norm"}

    def _target(self, name: str):
        """checkpoint name -> (parameter name, shard id)."""
        top = {"embed": "embed", "side.embed": "side_embed", "final.norm": "final_norm"}
        if name in top:
            return top[name], None
        m = self._LAYER.match(name)
        if not m or int(m.group(1)) >= len(self.layers):
            return None, None
        i, rest = int(m.group(1)), m.group(2)
        pre, L = f"layers.{i}.", self.layers[i]
        if rest == "norm1":
            return pre + rest, None
        if rest in ("side.gate", "side.proj", "side.norm"):
            return pre + rest, None
        if rest in ("rg1", "rg2") and rest in L.proj.offsets:
            return pre + "proj.weight", rest
        if rest in ("rg1.b", "rg2.b") and rest[:3] in L.proj.offsets:
            return pre + "proj.bias", rest[:3]
        if rest.startswith("mix."):
            k = rest[4:]
            if k == "o":
                return pre + "o", None
            if k in L.proj.offsets and not k.startswith("rg"):
                return pre + "proj.weight", k
            p = (self._GLA if L.kind == "gla" else self._ATTN).get(k)
            return (pre + "mix." + p, None) if p else (None, None)
        if rest.startswith("mlp.") and rest[4:] in self._MLP:
            p, sid = self._MLP[rest[4:]]
            return pre + "mlp." + p, sid
        return None, None

    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]) -> List[str]:
        params = dict(self.named_parameters())
        loaded = []
        for name, t in weights:
            pname, sid = self._target(name)
            if pname is None or pname not in params:
                raise ValueError(f"unexpected tensor {name!r} for this Borosun configuration")
            p = params[pname]
            t = t.to(p.dtype)
            if sid is None:
                p.weight_loader(p, t)
            else:
                p.weight_loader(p, t, sid)
            loaded.append(pname)
        return loaded

    def init_random(self, seed: int = 0) -> None:
        """Random weights of a plausible scale (no checkpoint): unit norm weights, matrices
        N(0, 1/fan_in), convolutions near the identity, a mixing matrix near the identity, decay
        biases that keep most of the state."""
        import zlib
        for mname, mod in self.named_modules():
            if isinstance(mod, FusedProjection):
                g = torch.Generator(device=mod.weight.device)
                g.manual_seed(seed * 1000003 + zlib.crc32(mname.encode()))
                mod.init_random(g)
        for name, p in self.named_parameters():
            if name.endswith(("proj.weight", "proj.bias")) and ".mlp." not in name:
                continue
            g = torch.Generator(device=p.device)
            g.manual_seed(seed * 1000003 + zlib.crc32(name.encode()))
            leaf = name.rsplit(".", 1)[-1]
            rnd = lambda s: torch.randn(p.shape, generator=g, device=p.device,
                                        dtype=torch.float32) * s
            if leaf in ("norm1", "final_norm", "norm"):
                p.data.copy_(1.0 + rnd(0.02))
            elif leaf in ("q_conv", "k_conv", "v_conv"):
                p.data.copy_(rnd(0.1))
                p.data[:, -1] += 1.0
            elif leaf == "talk":
                p.data.copy_(torch.eye(p.shape[0], device=p.device) + rnd(0.1))
            elif leaf == "vmix":
                p.data.fill_(0.3)
            elif leaf == "a2_bias":
                p.data.copy_(2.0 + rnd(0.5))
            elif leaf == "side_embed":
                p.data.copy_(rnd(1.0))
            elif leaf in ("gate", "proj") and ".side." in name:
                side = self.get_submodule(name.rsplit(".", 1)[0])
                p.data.zero_()                      # pad rows / columns stay zero
                if leaf == "gate":
                    p.data[:side.dim].copy_(rnd(p.shape[1] ** -0.5)[:side.dim])
                else:
                    p.data[:, :side.dim].copy_(rnd(side.dim ** -0.5)[:, :side.dim])
            else:
                p.data.copy_(rnd(p.shape[-1] ** -0.5))

    def post_load(self) -> None:
        for L in self.layers:
            L.mix.refresh()
            if L.side is not None:
                L.side.refresh()
