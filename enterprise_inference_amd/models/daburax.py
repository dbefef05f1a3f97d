"""Daburax: a decoder whose config.json lists its layers one by one.  The token embedding is
scaled and joined by a row of a hashed bigram table (ops/embedding.py); the residual is kept as
``streams`` fp32 copies joined by hyper-connections (models/hyper_connected.py; norm weights are
stored around zero, every sublayer output is multiplied by ``residual_mult``).  Mixers
(models/mixers.py): ``retention`` (RetentionMixer: rotated q / k, a fixed decay per head, matrix
state on state slots, head RMS norm, SiLU gate) and ``parallel``
(ParallelMixer: a grouped-query softmax attention with biases, partial interleaved rotation with
position interpolation and a per-head sink in the denominator, beside a gated matrix memory with
a stabilised exponential input gate; one fused input projection, one output projection).  The
optional feed-forward is a mixture of SiLU-gated experts behind a group-limited softmax router
with a selection-only correction, identity experts and a sigmoid-gated shared expert
(models/mixtral.py GroupLimitedMoE).  The model's norm with ``final.norm`` on the sum of the
streams precedes the LM head.

config.json keys: architecture, vocab, width, norm{eps}, residual_mult, streams,
embedding{scale, bigram{buckets, mul_prev, mul_cur}} and layers[i] = {type, mixer{...},
mlp{kind: moe, expert{ff}, router{experts, top, identity, groups{count, keep}}, shared{ff}} |
null}.  Checkpoint names: embed, bigram, head, final.norm, l<i>.norm1|norm2, l<i>.hc1|hc2.in|
out|mix, l<i>.mix.*, l<i>.mlp.*.

Residual streams, norms, angles, scores and softmax weights, routing, gates, decays and the
recurrent states are fp32 whatever the activation dtype; with dtype float32 the matrix products
are fp32 too.
"""

from __future__ import annotations

import re

import torch

from ..config import ModelConfig
from .hyper_connected import HyperConnectedDecoder, HyperConnectedLayer, HyperConnection
from .mixers import FusedProjection, PagedKVRows, ParallelMixer, RetentionMixer
from .mixtral import GroupLimitedMoE


class DaburaxLayer(HyperConnectedLayer):
    def __init__(self, spec: dict, width: int, eps: float, streams: int, dtype, device):
        super().__init__()
        m = spec["mixer"]
        self.kind = spec["type"]
        if self.kind == "retention":
            rot = m.get("rot") or {}
            # (a rot entry without dims rotates the whole head)
            self.mix = RetentionMixer(width, m["heads"], m["dim"], m.get("vdim", m["dim"]),
                                      m["decay"], int(rot.get("dims", m["dim"] if rot else 0)),
                                      float(rot.get("base", 10000.0)), rot.get("scaling"), eps,
                                      dtype, device)
        elif self.kind == "parallel":
            left, right = dict(m["left"]), dict(m["right"])
            left.setdefault("kv_heads", left["heads"])
            left.setdefault("vdim", left["dim"])
            left.setdefault("scale", float(left["dim"]) ** -0.5)
            right.setdefault("gate_cap", 0.0)           # (no cap)
            right.setdefault("vdim", right["dim"])
            self.mix = ParallelMixer(width, left, right, float(m.get("left_scale", 1.0)),
                                     float(m.get("right_scale", 1.0)), eps, dtype, device)
        else:
            raise ValueError(f"unknown Daburax layer type {self.kind!r}")
        mlp = spec.get("mlp")
        self.mlp = None
        if mlp is not None:
            if mlp.get("kind", "moe") != "moe":
                raise ValueError(f"unknown Daburax feed-forward kind {mlp.get('kind')!r}")
            r = mlp["router"]
            g = r.get("groups") or {"count": 1, "keep": 1}
            self.mlp = GroupLimitedMoE(width, int(mlp["expert"]["ff"]), int(r["experts"]),
                                       int(r["top"]), int(g.get("count", 1)), int(g.get("keep", 1)),
                                       int(r.get("identity", 0)),
                                       int((mlp.get("shared") or {}).get("ff", 0)),
                                       dtype=dtype, device=device)
        self._setup(width, streams, dtype, device)

    def block_bytes(self, block_size: int, elem: int) -> int:
        if self.kind != "parallel":
            return 0
        return block_size * sum(self.mix.left.cache_widths()) * elem

    def state_bytes(self, elem: int) -> int:
        return (self.mix if self.kind == "retention" else self.mix.right).state_bytes()

    def allocate_cache(self, num_blocks: int, block_size: int, num_slots: int, dtype, device):
        """State slots for a retention layer, (paged K / V rows, state slots) for a parallel one."""
        if self.kind == "retention":
            return self.mix.allocate_state(num_slots, device)
        kw, vw = self.mix.left.cache_widths()
        return (PagedKVRows.allocate(num_blocks, block_size, kw, vw, dtype, device),
                self.mix.right.allocate_state(num_slots, device))

    def query_block(self, block_size: int):
        return self.mix.left.query_block(block_size) if self.kind == "parallel" else None


class DaburaxForCausalLM(HyperConnectedDecoder):
    # (state slots: recurrent layers and the previous token of the bigram term)
    norm_offset = 1.0              # norm weights are stored around zero

    def __init__(self, cfg: ModelConfig, dtype=torch.bfloat16, device=None):
        super().__init__()
        device = torch.device(device) if device is not None else torch.device("cpu")
        W = cfg.hidden_size
        self.eps, self.streams = self.read_basics(cfg)
        self._setup(cfg, [DaburaxLayer(s, W, self.eps, self.streams, dtype, device)
                          for s in cfg.extra["layers"]], dtype, device)
        # decode steps replay HIP graphs when every expert block has a device-side grouped form
        # (bf16, width a multiple of 128 and expert ff a multiple of 64); else they read row
        # offsets back per layer
        self.supports_graphs = dtype == torch.bfloat16 and all(
            L.mlp is None or (W % 128 == 0 and L.mlp.I % 64 == 0) for L in self.layers)

    # ------------------------------------------------------------------ weights
    _LAYER = re.compile(r"^l(\d+)\.(.+)$")

    def _target(self, name: str):
        """checkpoint name -> (parameter name, shard id)."""
        if name in ("embed", "head", "bigram"):
            return name, None
        if name == "final.norm":
            return "final_norm", None
        m = self._LAYER.match(name)
        if not m or int(m.group(1)) >= len(self.layers):
            return None, None
        i, rest = int(m.group(1)), m.group(2)
        pre = f"layers.{i}."
        L = self.layers[i]
        if rest in ("norm1", "norm2"):
            return pre + rest, None
        hc = re.match(r"^(hc[12])\.(in|out|mix)$", rest)
        if hc:
            return pre + hc.group(1) + "." + HyperConnection.NAMES[hc.group(2)], None
        if rest.startswith("mix."):
            k = rest[4:]
            if L.kind == "retention":
                if k in ("q", "k", "v", "g"):
                    return pre + "mix.proj.weight", k
                return pre + "mix." + k, None
            side, _, leaf = k.partition(".")
            if side not in ("left", "right"):
                return None, None
            if leaf == "o":
                return pre + "mix.o", side
            if leaf.endswith(".b") and leaf[:-2] in ("q", "k", "v", "i", "f"):
                return pre + "mix.proj.bias", side + "." + leaf[:-2]
            if leaf in ("q", "k", "v", "g", "i", "f") and not (side == "left" and leaf in ("g", "i", "f")):
                return pre + "mix.proj.weight", side + "." + leaf
            return pre + f"mix.{side}.{leaf}", None
        if rest.startswith("mlp.") and L.mlp is not None:
            k = rest[4:]
            e = re.match(r"^e(\d+)\.(gate|up|down)$", k)
            if e:
                if e.group(2) == "down":
                    return pre + "mlp.w2", int(e.group(1))
                return pre + "mlp.w13", (int(e.group(1)), e.group(2))
            table = {"router": ("router", None), "correction": ("correction", None),
                     "shared.gate": ("shared.gate_up_proj.weight", 0),
                     "shared.up": ("shared.gate_up_proj.weight", 1),
                     "shared.down": ("shared.down_proj.weight", None),
                     "shared.sg": ("shared_gate", None)}
            if k in table:
                return pre + "mlp." + table[k][0], table[k][1]
        return None, None

    def init_random(self, seed: int = 0) -> None:
        """Random weights of a plausible scale (no checkpoint): norm weights and corrections
        around zero, matrices N(0, 1/fan_in), stream constants near the plain residual sum,
        small sinks and gate biases."""
        import zlib
        for mname, mod in self.named_modules():
            if isinstance(mod, FusedProjection):
                g = torch.Generator(device=mod.weight.device)
                g.manual_seed(seed * 1000003 + zlib.crc32(mname.encode()))
                mod.init_random(g)
            if isinstance(mod, HyperConnection):
                g = torch.Generator(device=mod.in_f32.device)
                g.manual_seed(seed * 1000003 + zlib.crc32(mname.encode()))
                mod.init_random(lambda p, s: torch.randn(p.shape, generator=g, device=p.device,
                                                         dtype=torch.float32) * s)
        for name, p in self.named_parameters():
            if name.endswith(("proj.weight", "proj.bias")) and ".mix." in name or ".hc" in name:
                continue
            g = torch.Generator(device=p.device)
            g.manual_seed(seed * 1000003 + zlib.crc32(name.encode()))
            leaf = name.rsplit(".", 1)[-1]
            rnd = lambda s: torch.randn(p.shape, generator=g, device=p.device,
                                        dtype=torch.float32) * s
            if leaf in ("norm1", "norm2", "final_norm", "correction"):
                p.data.copy_(rnd(0.02))
            elif leaf == "norm":
                p.data.copy_(1.0 + rnd(0.05))
            elif leaf == "sink":
                p.data.copy_(rnd(0.3))
            elif leaf == "bigram":
                p.data.copy_(rnd(0.5))
            elif leaf == "o" and p.dim() == 2 and name.endswith("mix.o"):
                p.data.copy_(rnd(p.shape[-1] ** -0.5))
                mix = self.get_submodule(name.rsplit(".", 1)[0])
                if isinstance(mix, ParallelMixer):
                    mix.zero_pads()
            else:
                p.data.copy_(rnd(p.shape[-1] ** -0.5))
