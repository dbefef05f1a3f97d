"""Vugelix: a decoder whose config.json lists its layers one by one.  The scaled token embedding
starts ``streams`` fp32 residual streams joined by hyper-connections (models/hyper_connected.py).
Every layer is a ``parallel`` mixer (models/mixers.py WindowDeltaMixer) and an optional ungated
squared-ReLU feed-forward:

* left: grouped-query sliding-window attention -- partial half-split rotation, soft-capped scores, one
  unit added to the softmax denominator, a sigmoid gate per head
* right: gated delta rule -- short convolutions on q, k and v, unit-length queries and keys, a decay
  and a step size per head and token, head RMS norm, SiLU gate
* one fused input projection for both sides, one output projection over both sides' scaled heads.

A layer with ``weights_of: j`` runs layer j's tensors on a cache and state of its own.  The LM head is
the embedding table behind the model's norm; logits are multiplied by ``logit_scale``.

config.json keys: architecture, vocab, width, norm{eps}, streams, embedding{scale}, logit_scale and
layers[i] = {type: parallel, mixer{left{heads, kv_heads, dim, vdim, scale, softcap, rot{base, dims},
mask{size}}, left_scale, right{heads, kv_heads, dim, vdim, conv}, right_scale}, mlp{kind: dense, ff} |
null, weights_of}.  Checkpoint names: embed, final.norm, l<i>.norm1|norm2, l<i>.hc1|hc2.in|out|mix,
l<i>.mix.left.q|k|v|g|o, l<i>.mix.right.q|k|v[.conv], l<i>.mix.right.b|a|g|o|A_log|dt_bias|norm,
l<i>.mlp.up|down.

Residual streams, norms, angles, scores and softmax weights, everything in the recurrence past the
convolutions and the recurrent state are fp32 whatever the activation dtype; with dtype float32 the
matrix products are fp32 too.
"""

from __future__ import annotations

import re

import torch

from ..config import ModelConfig
from .hyper_connected import HyperConnectedDecoder, HyperConnectedLayer, HyperConnection
from .mixers import FusedProjection, PagedKVRows, WindowDeltaMixer
from .mixtral import UngatedMLP


class VugelixLayer(HyperConnectedLayer):
    def __init__(self, spec: dict, width: int, eps: float, streams: int, dtype, device):
        super().__init__()
        m = spec["mixer"]
        self.kind = spec["type"]
        if self.kind != "parallel":
            raise ValueError(f"unknown Vugelix layer type {self.kind!r}")
        left, right = dict(m["left"]), dict(m["right"])
        left.setdefault("scale", float(left["dim"]) ** -0.5)
        for side in (left, right):
            side.setdefault("kv_heads", side["heads"])
            side.setdefault("vdim", side["dim"])
        self.mix = WindowDeltaMixer(width, left, right, float(m.get("left_scale", 1.0)),
                                    float(m.get("right_scale", 1.0)), eps, dtype, device)
        mlp = spec.get("mlp")
        self.mlp = None
        if mlp is not None:
            if mlp.get("kind", "dense") != "dense":
                raise ValueError(f"unknown Vugelix feed-forward kind {mlp.get('kind')!r}")
            self.mlp = UngatedMLP(width, int(mlp["ff"]), dtype, device, act="relu2", defer=True)
        self._setup(width, streams, dtype, device)

    def apply_mlp(self, h, md):
        return self.mlp(h)         # may return gemm.SplitK: the boundary step reduces it

    def block_bytes(self, block_size: int, elem: int) -> int:
        return block_size * sum(self.mix.left.cache_widths()) * elem

    def state_bytes(self, elem: int) -> int:
        return self.mix.right.state_bytes(elem)

    def allocate_cache(self, num_blocks: int, block_size: int, num_slots: int, dtype, device):
        """(paged K / V rows, state slots)."""
        kw, vw = self.mix.left.cache_widths()
        return (PagedKVRows.allocate(num_blocks, block_size, kw, vw, dtype, device),
                self.mix.right.allocate_state(num_slots, dtype, device))

    def query_block(self, block_size: int):
        return self.mix.left.query_block(block_size)


def weight_owners(specs) -> list:
    """For every layer of a layer list the index of the layer whose tensors it runs on."""
    out = []
    for i, s in enumerate(specs):
        j, seen = i, set()
        while specs[j].get("weights_of") is not None:
            seen.add(j)
            j = int(specs[j]["weights_of"])
            if not 0 <= j < len(specs) or j in seen:
                raise ValueError(f"layer {i}: weights_of names no layer with tensors")
        out.append(j)
    return out


class VugelixForCausalLM(HyperConnectedDecoder):
    supports_graphs = True         # no step reads anything back to the host
    # csrc/kernels files of a step without sampling
    kernel_sources = ("activation", "delta_prep", "delta_scan", "embed", "gemm_skinny", "norm",
                      "window_attention")

    def __init__(self, cfg: ModelConfig, dtype=torch.bfloat16, device=None):
        super().__init__()
        device = torch.device(device) if device is not None else torch.device("cpu")
        specs = cfg.extra["layers"]
        self.eps, self.streams = self.read_basics(cfg)
        self.owners = weight_owners(specs)
        own = {j: VugelixLayer(specs[j], cfg.hidden_size, self.eps, self.streams, dtype, device)
               for j in sorted(set(self.owners))}
        self._setup(cfg, [own[j] for j in self.owners], dtype, device, tied_head=True)

    # ------------------------------------------------------------------ weights
    _LAYER = re.compile(r"^l(\d+)\.(.+)$")
    _RIGHT = {"q.conv": "q_conv", "k.conv": "k_conv", "v.conv": "v_conv", "A_log": "A_log",
              "dt_bias": "dt_bias", "norm": "norm"}

    def _target(self, name: str):
        """checkpoint name -> (parameter name, shard id)."""
        if name == "embed":
            return name, None
        if name == "final.norm":
            return "final_norm", None
        m = self._LAYER.match(name)
        i = int(m.group(1)) if m else -1
        if not 0 <= i < len(self.layers) or self.owners[i] != i:
            return None, None
        rest, pre = m.group(2), f"layers.{i}."
        if rest in ("norm1", "norm2"):
            return pre + rest, None
        hc = re.match(r"^(hc[12])\.(in|out|mix)$", rest)
        if hc:
            return pre + hc.group(1) + "." + HyperConnection.NAMES[hc.group(2)], None
        if rest in ("mlp.up", "mlp.down"):
            return pre + rest + ".weight", None
        mix = re.match(r"^mix\.(left|right)\.(.+)$", rest)
        if not mix:
            return None, None
        side, leaf = mix.groups()
        if leaf == "o":
            return pre + "mix.o", side
        if f"{side}.{leaf}" in self.layers[i].mix.proj.offsets:
            return pre + "mix.proj.weight", f"{side}.{leaf}"
        if side == "right" and leaf in self._RIGHT:
            return pre + "mix.right." + self._RIGHT[leaf], None
        return None, None

    def init_random(self, seed: int = 0) -> None:
        """Random weights of a plausible scale (no checkpoint): unit norm weights, matrices
        N(0, 1/fan_in), stream constants near the plain residual sum, convolutions near the
        identity, decays between about 0.5 and 0.999."""
        import zlib

        def draw(name, p, s):
            g = torch.Generator(device=p.device)
            g.manual_seed(seed * 1000003 + zlib.crc32(name.encode()))
            return torch.randn(p.shape, generator=g, device=p.device, dtype=torch.float32) * s

        for mname, mod in self.named_modules():
            if isinstance(mod, FusedProjection):
                g = torch.Generator(device=mod.weight.device)
                g.manual_seed(seed * 1000003 + zlib.crc32(mname.encode()))
                mod.init_random(g)
            elif isinstance(mod, HyperConnection):
                n = iter(range(3))
                mod.init_random(lambda p, s: draw(f"{mname}.{next(n)}", p, s))
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if name.endswith("proj.weight") or ".hc" in name:
                continue
            if leaf in ("norm1", "norm2", "final_norm", "norm"):
                p.data.copy_(1.0 + draw(name, p, 0.02))
            elif leaf in ("q_conv", "k_conv", "v_conv"):
                p.data.copy_(draw(name, p, 0.1))
                p.data[:, -1] += 1.0
            elif leaf == "A_log":
                p.data.copy_(draw(name, p, 0.7))
            elif leaf == "dt_bias":
                p.data.copy_(draw(name, p, 1.0) - 3.0)
            elif leaf == "o":
                p.data.copy_(draw(name, p, p.shape[-1] ** -0.5))
                self.get_submodule(name.rsplit(".", 1)[0]).zero_pads()
            else:
                p.data.copy_(draw(name, p, p.shape[-1] ** -0.5))
