"""Decoders whose residual is kept as several fp32 streams joined by hyper-connections.

Every sublayer q of a layer reads u = sum_s in_q[s] x_s through an RMS norm, and all streams are
rewritten at once from the old ones,

    x_t <- sum_s mix_q[s, t] x_s + mult * out_q[t] * sublayer(norm_q(u)),

(ops/norm.py hyper_step: one launch per sublayer boundary; without ``streams`` it is the plain
pre-norm residual sum).  The model's norm with ``final.norm`` on the sum of the streams precedes the
LM head.  ``HyperConnectedDecoder`` is the stack; a design derives from it with its own layers
(``HyperConnectedLayer``), weight names and random initialisation.
"""

from __future__ import annotations

from typing import Iterable, List, Optional, Tuple

import torch
import torch.nn as nn

from ..config import ModelConfig
from ..ops import embedding as emb_ops
from ..ops import gemm, norm as norm_ops
from ..ops.attention import AttentionMetadata
from .layers import _param, default_loader


def _plain(shape, dtype, device):
    p = _param(shape, dtype, device)
    p.weight_loader = default_loader
    return p


class HyperConnection(nn.Module):
    """The three learned pieces of one sublayer's hyper-connection over ``streams`` residual
    streams: read weights ``inw`` [s], write weights ``outw`` [s] and the stream-mixing matrix
    ``mix`` [s, s] (from, to), with fp32 copies for the boundary launches (refreshed IN PLACE
    after a weight load: captured decode graphs hold their addresses).  ``streams`` 0: the plain
    residual sum, one stream with unit constants and no parameters."""

    NAMES = {"in": "inw", "out": "outw", "mix": "mix"}      # checkpoint leaf -> parameter

    def __init__(self, streams: int, dtype, device):
        super().__init__()
        self.learned = streams > 0
        n = max(1, streams)
        if self.learned:
            self.inw = _plain((n,), dtype, device)
            self.outw = _plain((n,), dtype, device)
            self.mix = _plain((n, n), dtype, device)
        self.in_f32 = torch.ones(n, dtype=torch.float32, device=device)
        self.out_f32 = torch.ones(n, dtype=torch.float32, device=device)
        self.mix_f32 = torch.eye(n, dtype=torch.float32, device=device)

    def refresh(self) -> None:
        if self.learned:
            self.in_f32.copy_(self.inw.float())
            self.out_f32.copy_(self.outw.float())
            self.mix_f32.copy_(self.mix.float())

    def init_random(self, rnd) -> None:
        """Constants near the plain residual sum; ``rnd(parameter, scale)`` draws N(0, scale^2)."""
        if self.learned:
            n = self.inw.shape[0]
            self.inw.data.copy_(1.0 / n + rnd(self.inw, 0.05))
            self.outw.data.copy_(1.0 + rnd(self.outw, 0.05))
            self.mix.data.copy_(torch.eye(n, device=self.mix.device) + rnd(self.mix, 0.05))


class HyperConnectedLayer(nn.Module):
    """A layer: ``mix`` behind (hc1, norm1) and an optional ``mlp`` behind (hc2, norm2).  A design's
    layer sets ``kind``, ``mix`` and ``mlp`` and calls ``_setup``; its mixer's caches are described
    by the four cache methods."""

    def _setup(self, width: int, streams: int, dtype, device) -> None:
        self.norm1 = _plain((width,), dtype, device)
        self.hc1 = HyperConnection(streams, dtype, device)
        if self.mlp is not None:
            self.norm2 = _plain((width,), dtype, device)
            self.hc2 = HyperConnection(streams, dtype, device)

    def boundaries(self):
        """(hyper-connection, norm weight) of this layer's sublayers, in order."""
        out = [(self.hc1, self.norm1)]
        if self.mlp is not None:
            out.append((self.hc2, self.norm2))
        return out

    def refresh(self) -> None:
        self.mix.refresh()
        self.hc1.refresh()
        if self.mlp is not None:
            if hasattr(self.mlp, "refresh"):
                self.mlp.refresh()
            self.hc2.refresh()

    def apply_mlp(self, h, md):
        return self.mlp(h, md)

    # cache geometry of the mixer
    def block_bytes(self, block_size: int, elem: int) -> int:
        return 0

    def state_bytes(self, elem: int) -> int:
        return 0

    def allocate_cache(self, num_blocks: int, block_size: int, num_slots: int, dtype, device):
        raise NotImplementedError

    def query_block(self, block_size: int) -> Optional[int]:
        """Queries per prefill work item of the layer's attention kernel; None: no attention."""
        return None


class HyperConnectedDecoder(nn.Module):
    supports_pp = False
    supports_float32 = True        # every kernel of these models has an fp32 form
    needs_state_slots = True
    norm_offset = 0.0              # norm weights are stored around this distance from their value

    def _setup(self, cfg: ModelConfig, layers, dtype, device, tied_head: bool = False) -> None:
        """``layers``: the design's layers in running order (one object may run several times, with
        a cache entry each).  ``tied_head``: the LM head is the embedding table."""
        self.cfg, self.dtype = cfg, dtype
        ex, W = cfg.extra, cfg.hidden_size
        emb = ex.get("embedding") or {}
        self.embed_scale = float(emb.get("scale", 1.0))
        self.bigram_cfg = dict(emb["bigram"]) if emb.get("bigram") else None
        mult = ex.get("residual_mult")
        self.mult = 1.0 if mult is None else float(mult)
        scale = ex.get("logit_scale")
        self.logit_scale = 1.0 if scale is None else float(scale)
        self.embed = _plain((cfg.vocab_size, W), dtype, device)
        self.bigram = None
        if self.bigram_cfg:
            self.bigram = _plain((int(self.bigram_cfg["buckets"]) + 1, W), dtype, device)
        self.layers = nn.ModuleList(layers)
        self.final_norm = _plain((W,), dtype, device)
        self.head = None if tied_head else _plain((cfg.vocab_size, W), dtype, device)
        self.ones = torch.ones(max(1, self.streams), dtype=torch.float32, device=device)
        # the sublayer boundaries in order: (layer, hyper-connection, norm weight)
        self.steps = [(i, hc, w) for i, L in enumerate(self.layers) for hc, w in L.boundaries()]

    @staticmethod
    def read_basics(cfg: ModelConfig):
        """(norm eps, streams) of a configuration; streams 0: plain residual (one stream)."""
        ex = cfg.extra
        return (float((ex.get("norm") or {}).get("eps", cfg.rms_norm_eps)),
                int(ex.get("streams") or 0))

    # ------------------------------------------------------------------ cache geometry
    def kv_heads_per_rank(self) -> int:
        return 1

    def cache_block_bytes(self, block_size: int, dtype: torch.dtype) -> int:
        e = torch.tensor([], dtype=dtype).element_size()
        return sum(L.block_bytes(block_size, e) for L in self.layers) or 1

    def state_slot_bytes(self) -> int:
        e = torch.tensor([], dtype=self.dtype).element_size()
        return (4 if self.bigram_cfg else 0) + sum(L.state_bytes(e) for L in self.layers)

    def allocate_cache(self, num_blocks: int, block_size: int, num_slots: int,
                       dtype: torch.dtype, device) -> list:
        """Per-layer cache objects, then one more entry for the embedding: the previous token per
        slot (int32) for the bigram term, or None.  Zero filled: never-written rows stay finite
        under a zero softmax weight."""
        out = [L.allocate_cache(num_blocks, block_size, num_slots, dtype, device)
               for L in self.layers]
        out.append(torch.zeros(max(1, num_slots), dtype=torch.int32, device=device)
                   if self.bigram_cfg else None)
        return out

    def prefill_query_block(self, block_size: int) -> int:
        """The step's work list is built for the first attention layer's query block; layers
        with another one get theirs from AttentionMetadata.prefill_work_for."""
        for L in self.layers:
            qb = L.query_block(block_size)
            if qb:
                return qb
        return 16

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, md: AttentionMetadata, caches: list,
                intermediate=None, collect: Optional[list] = None):
        """Returns the fp32 residual streams [T, streams, width].  ``collect`` (a list) receives
        the sum of the streams after every layer."""
        bg = self.bigram_cfg or {}
        T = input_ids.shape[0]
        nseq = md.num_seqs if md.num_seqs else T
        last = caches[len(self.layers)]
        X = emb_ops.bigram_embed(input_ids, self.embed, self.embed_scale, self.bigram,
                                 int(bg.get("buckets", 1)), int(bg.get("mul_prev", 0)),
                                 int(bg.get("mul_cur", 0)), last,
                                 md.seq_slots if last is not None else None,
                                 md.seq_cu if last is not None else None,
                                 nseq if last is not None else T, md.positions,
                                 max(1, self.streams))
        steps = self.steps
        if not steps:
            return X
        off = self.norm_offset
        h = norm_ops.hyper_step(X, self.eps, None, in_next=steps[0][1].in_f32,
                                w_next=steps[0][2], w_offset=off)
        for n, (i, hc, _) in enumerate(steps):
            L = self.layers[i]
            y = L.mix(h, md, caches[i]) if hc is L.hc1 else L.apply_mlp(h, md)
            nxt = steps[n + 1] if n + 1 < len(steps) else None
            h = norm_ops.hyper_step(X, self.eps, y, hc.mix_f32, hc.out_f32, self.mult,
                                    nxt[1].in_f32 if nxt else None, nxt[2] if nxt else None, off)
            if collect is not None and (nxt is None or nxt[0] != i):
                collect.append(X.sum(1))
        return X

    def compute_logits(self, X: torch.Tensor) -> torch.Tensor:
        """X: rows of the fp32 residual streams [n, streams, width] -> fp32 logits."""
        h = norm_ops.hyper_step(X.contiguous(), self.eps, None, in_next=self.ones,
                                w_next=self.final_norm, w_offset=self.norm_offset)
        head = self.embed if self.head is None else self.head
        out = gemm.linear_f32(h, head) if h.dtype == torch.bfloat16 and h.is_cuda else None
        if out is None:
            out = gemm.linear(h, head).float()
        return out if self.logit_scale == 1.0 else out.mul_(self.logit_scale)

    # ------------------------------------------------------------------ weights
    def _target(self, name: str):
        """checkpoint name -> (parameter name, shard id), (None, None) for an unknown name."""
        raise NotImplementedError

    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]) -> List[str]:
        # (a layer that runs several times keeps all its names)
        params = dict(self.named_parameters(remove_duplicate=False))
        loaded = []
        for name, t in weights:
            pname, sid = self._target(name)
            if pname is None or pname not in params:
                raise ValueError(f"unexpected tensor {name!r} for this "
                                 f"{self.cfg.architecture} configuration")
            p = params[pname]
            t = t.to(p.dtype)
            if sid is None:
                p.weight_loader(p, t)
            else:
                p.weight_loader(p, t, sid)
            loaded.append(pname)
        return loaded

    def post_load(self) -> None:
        for L in self.layers:
            L.refresh()
