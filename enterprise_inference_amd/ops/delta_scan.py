"""Gated delta rule on per-sequence state slots -> csrc/kernels/delta_prep.hip, delta_scan.hip.

Per head a matrix state S [dk, dv] (fp32, slot-resident) whose answer to the token's key moves
towards its value:

    S <- a_t S_(t-1);    u_t = b_t (v_t - S^T k_t);    S_t = S + k_t u_t^T;    o_t = S_t^T q_t

a_t = exp(-exp(A_log[h]) softplus(x_a + dt_bias[h])) and b_t = sigmoid(x_b) are one number per head
and token.  The q and k projections (``kv_heads`` heads) and the v projection (``heads`` heads) pass a
short causal convolution over time and silu; q and k become unit vectors per head, x / sqrt(sum x^2
+ 1e-6), q times ``qscale``; head h reads q / k head h // (heads // kv_heads).  Every head's o is
divided by its root mean square, multiplied by a weight [dv] shared by the heads, by silu of the
gate columns and by ``out_scale``.

``delta_prep`` turns fused projection rows into fp32 rows (``DeltaRows``); with ``attn`` the same
launch also rotates an attention mixer's queries and keys from the same projection rows and writes
its cache.  ``delta_scan`` runs the recurrence: token by token (decode rows, short portions, heads
up to 256 wide), or -- prompt portions on the GPU, heads up to 128 wide -- chunk by chunk of 64
tokens: every chunk's triangular system is solved in parallel, a scan over a sequence's chunks
carries the state, and all outputs are formed in parallel.

A sequence whose first row of the step is position 0 starts from zeros whatever its slot held.
Batch layout: [decode rows (one per sequence) | prefill portions]; ``md.seq_slots`` names the slots
(< 0: padding row, skipped).
"""

from __future__ import annotations

import dataclasses
import os
from typing import Optional

import torch

from ._dispatch import check, lib, ptr, require, stream, use_hip
from .linear_scan import ChunkPlan, chunk_plan, _seq_bounds
from .window_attention import PREP_MAX_TAPS, PREP_ROWS, PrepSpec, _prep_ref, build_work

CHUNK = 64                 # tokens per chunk of the chunk-parallel form (delta_scan.hip DC)
CHUNK_MAX_DIM = 128        # ... and its largest dk / dv
CHUNK_MIN_ROWS = 48        # a portion with at least this many rows selects it
# tests and measurements: take the chunk-parallel form for every step that has prompt portions (1),
# or never (0)
FORCE_CHUNKED = {"0": False, "1": True}.get(os.environ.get("EIA_DELTA_FORCE_CHUNKED", ""))


@dataclasses.dataclass
class DeltaSpec:
    """Constants of one gated-delta layer (convolution weights in the activation dtype; the other
    device tensors fp32)."""
    heads: int
    kv_heads: int
    dim: int                        # dk
    vdim: int                       # dv
    taps: int
    cw_q: Optional[torch.Tensor] = None     # [kv_heads*dk, taps], newest token last
    cw_k: Optional[torch.Tensor] = None
    cw_v: Optional[torch.Tensor] = None     # [heads*dv, taps]
    exp_a: Optional[torch.Tensor] = None    # [heads], exp(A_log)
    dt_bias: Optional[torch.Tensor] = None  # [heads]
    qscale: float = 1.0
    out_scale: float = 1.0
    eps: float = 0.0

    def channels(self) -> int:
        """Channels of the convolution history: q, k, v columns in this order."""
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim


class DeltaState:
    """Per-sequence slots of one layer: S fp32 [slots, H, dk, dv] and the projected values of the
    last taps - 1 tokens, [slots, taps - 1, channels] in the activation dtype (None: one tap)."""

    __slots__ = ("S", "hist")

    def __init__(self, S: torch.Tensor, hist: Optional[torch.Tensor]):
        self.S, self.hist = S, hist

    @classmethod
    def allocate(cls, num_slots: int, spec: DeltaSpec, dtype, device):
        n = max(1, num_slots)
        S = torch.zeros(n, spec.heads, spec.dim, spec.vdim, dtype=torch.float32, device=device)
        hist = torch.zeros(n, spec.taps - 1, spec.channels(), dtype=dtype, device=device) \
            if spec.taps > 1 else None
        return cls(S, hist)

    @staticmethod
    def slot_bytes(spec: DeltaSpec, elem: int) -> int:
        return 4 * spec.heads * spec.dim * spec.vdim + elem * (spec.taps - 1) * spec.channels()


@dataclasses.dataclass
class AttnPrep:
    """An attention mixer's share of the projection rows: column offsets of q, k, v, its PrepSpec
    (rotation only), its caches, and the columns of a gate with one number per head."""
    q_off: int
    k_off: int
    v_off: int
    spec: PrepSpec
    k_cache: torch.Tensor
    v_cache: torch.Tensor
    gate_off: int = 0
    gate_heads: int = 0


@dataclasses.dataclass
class DeltaRows:
    """What delta_prep leaves: fp32 q, k [T, G, DP], v [T, H, VP] (zero past dk / dv), log decays
    and step sizes [T, H], the gate columns, and with an attention mixer its rotated queries and
    head gates."""
    q: torch.Tensor
    k: torch.Tensor
    v: torch.Tensor
    la: torch.Tensor
    beta: torch.Tensor
    gate: torch.Tensor
    attn_q: Optional[torch.Tensor] = None
    attn_gate: Optional[torch.Tensor] = None


def _pad16(n: int) -> int:
    return -(-n // 16) * 16


def _ref_prep(f, offs, spec: DeltaSpec, state: DeltaState, md, dtype):
    """Plain form of the delta rule's part of delta_prep (CPU path); f: fused rows."""
    T = f.shape[0]
    H, G, D, Dv, K = spec.heads, spec.kv_heads, spec.dim, spec.vdim, spec.taps
    u = torch.cat([f[:, offs["q"]:offs["q"] + G * D], f[:, offs["k"]:offs["k"] + G * D],
                   f[:, offs["v"]:offs["v"] + H * Dv]], 1).to(dtype).float()
    w = torch.cat([spec.cw_q, spec.cw_k, spec.cw_v], 0).float()            # [C, taps]
    y = torch.zeros_like(u)
    for s, (lo, hi) in enumerate(_seq_bounds(md.seq_cu, md.num_seqs or T)):
        sl = int(md.seq_slots[s])
        if hi <= lo or sl < 0:
            continue
        ext = u[lo:hi]
        if K > 1:
            hist = state.hist[sl].float().clone()
            p0 = int(md.positions[lo])
            if p0 < K - 1:                                                 # before the sequence
                hist[:K - 1 - p0] = 0
            ext = torch.cat([hist, ext], 0)
            state.hist[sl] = ext[-(K - 1):].to(state.hist.dtype)
        for j in range(K):
            y[lo:hi] += ext[j:j + hi - lo] * w[:, j]
    y = torch.nn.functional.silu(y)
    q, k, v = torch.split(y, [G * D, G * D, H * Dv], 1)

    def unit(x, scale):
        x = x.reshape(T, G, D)
        x = x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6) * scale
        return torch.nn.functional.pad(x, (0, _pad16(D) - D))

    za = f[:, offs["a"]:offs["a"] + H].float() + spec.dt_bias
    la = -spec.exp_a * torch.nn.functional.softplus(za)
    beta = torch.sigmoid(f[:, offs["b"]:offs["b"] + H].float())
    v = torch.nn.functional.pad(v.reshape(T, H, Dv), (0, _pad16(Dv) - Dv))
    return DeltaRows(unit(q, spec.qscale), unit(k, 1.0), v, la, beta,
                     f[:, offs["g"]:offs["g"] + H * Dv].to(dtype))


def delta_prep(fused, offs: dict, spec: DeltaSpec, state: DeltaState, md,
               attn: Optional[AttnPrep] = None) -> DeltaRows:
    """``fused``: projection rows [T, *] or a ``gemm.SplitK``; ``offs``: first columns of q, k, v, g
    (gate), b (step size) and a (decay).  Updates the sequences' convolution histories (and with
    ``attn`` that mixer's paged cache)."""
    from .gemm import SplitK
    split = isinstance(fused, SplitK)
    if split and not fused.part.is_cuda:
        fused = fused.part.sum(0)
        split = False
    H, G, D, Dv = spec.heads, spec.kv_heads, spec.dim, spec.vdim
    dt = spec.cw_q.dtype
    if not split and not use_hip(fused):
        r = _ref_prep(fused, offs, spec, state, md, dt)
        if attn is not None:
            r.attn_q = _prep_ref(fused, (attn.q_off, attn.k_off, attn.v_off), attn.spec, md,
                                 attn.k_cache, attn.v_cache, None, None, None, 0)
            if attn.gate_heads:
                r.attn_gate = fused[:, attn.gate_off:attn.gate_off + attn.gate_heads].to(dt)
        return r
    bf = dt == torch.bfloat16
    require(bf or dt == torch.float32, "delta_prep: bf16 or fp32")
    if split:
        T, width, dev = fused.M, fused.N, fused.part.device
        require(fused.part.dtype == torch.float32 and fused.part.is_contiguous() and
                fused.bias is None, "delta_prep: partials")
    else:
        T, width, dev = fused.shape[0], fused.shape[1], fused.device
        require(fused.stride(1) == 1 and fused.dtype == dt, "delta_prep: fused row layout")
    cols = [offs["q"] + G * D, offs["k"] + G * D, offs["v"] + H * Dv, offs["g"] + H * Dv,
            offs["b"] + H, offs["a"] + H]
    require(max(cols) <= width and min(offs[n] for n in ("q", "k", "v", "g", "b", "a")) >= 0,
            "delta_prep: columns outside the row")
    require(1 <= spec.taps <= PREP_MAX_TAPS, f"delta_prep: 1 .. {PREP_MAX_TAPS} taps")
    for w, rows in ((spec.cw_q, G * D), (spec.cw_k, G * D), (spec.cw_v, H * Dv)):
        require(w is not None and w.dtype == dt and w.is_contiguous() and
                w.shape == (rows, spec.taps), "delta_prep: convolution weights")
    for t in (spec.exp_a, spec.dt_bias):
        require(t is not None and t.dtype == torch.float32 and t.is_cuda and t.numel() == H,
                "delta_prep: fp32 numbers per head")
    hist = state.hist
    if spec.taps > 1:
        require(hist is not None and hist.dtype == dt and hist.is_contiguous() and
                hist.shape[1:] == (spec.taps - 1, spec.channels()) and md.seq_slots is not None and
                md.seq_slots.dtype == torch.int32, "delta_prep: convolution history")
    require(md.positions.dtype == torch.int32 and md.positions.numel() >= T, "int32 positions")
    require(md.num_decode + md.num_prefill_tokens == T, "delta_prep: rows of the step")
    DP, VP = _pad16(D), _pad16(Dv)
    f32 = lambda *s: torch.empty(*s, dtype=torch.float32, device=dev)
    q, k, v, la, beta = f32(T, G, DP), f32(T, G, DP), f32(T, H, VP), f32(T, H), f32(T, H)
    gate = torch.empty(T, H * Dv, dtype=dt, device=dev) if split else \
        fused[:, offs["g"]:offs["g"] + H * Dv]
    r = DeltaRows(q, k, v, la, beta, gate)
    hg = None
    wargs = [0, 0, 0, 0, 0, 0, 0, None, 0, 0, 1.0, None, None, 0, None, None, 1]
    if attn is not None:
        w, kc, vc = attn.spec, attn.k_cache, attn.v_cache
        require(w.taps == 1 and w.cw_q is None and not w.norm, "delta_prep: rotation only")
        require(max(attn.q_off + w.heads * w.dim, attn.k_off + w.kv_heads * w.dim,
                    attn.v_off + w.kv_heads * w.vdim, attn.gate_off + attn.gate_heads) <= width,
                "delta_prep: columns outside the row")
        require(kc.dtype == dt and vc.dtype == dt and kc.is_contiguous() and vc.is_contiguous() and
                kc.shape[-1] == w.kv_heads * w.dim and vc.shape[1] == w.kv_heads * w.vdim and
                vc.shape[2] == kc.shape[1], "delta_prep: cache layout")
        require(0 <= w.rot_dims <= w.dim and w.rot_dims % 2 == 0 and
                w.inv_freq.dtype == torch.float32 and w.inv_freq.numel() >= w.rot_dims // 2 and
                md.slot_mapping.dtype == torch.int32 and md.slot_mapping.numel() >= T,
                "delta_prep: rotation and cache slots")
        r.attn_q = torch.empty(T, w.heads * w.dim, dtype=dt, device=dev)
        wargs = [attn.q_off, attn.k_off, attn.v_off, w.heads, w.kv_heads, w.dim, w.vdim,
                 ptr(w.inv_freq), w.rot_dims, 1 if w.rot_half else 0, float(w.rot_amp),
                 ptr(md.slot_mapping), ptr(r.attn_q), r.attn_q.stride(0), ptr(kc), ptr(vc),
                 kc.shape[1]]
        if attn.gate_heads and split:
            hg = r.attn_gate = torch.empty(T, attn.gate_heads, dtype=dt, device=dev)
        elif attn.gate_heads:
            r.attn_gate = fused[:, attn.gate_off:attn.gate_off + attn.gate_heads]

    def launch(base, n_items, cu, work):
        sl = md.seq_slots[base:] if md.seq_slots is not None else None
        check(lib().eia_delta_prep(
            None if split else ptr(fused), width if split else fused.stride(0),
            ptr(fused.part) if split else None, fused.sk if split else 0, T * width if split else 0,
            offs["q"], offs["k"], offs["v"], offs["g"], offs["b"], offs["a"], H, G, D, Dv,
            ptr(spec.cw_q), ptr(spec.cw_k), ptr(spec.cw_v), spec.taps, ptr(hist), ptr(spec.exp_a),
            ptr(spec.dt_bias), float(spec.qscale), ptr(md.positions), ptr(sl), ptr(cu), ptr(work),
            base, n_items, ptr(q), ptr(k), ptr(v), DP, VP, ptr(la), ptr(beta),
            ptr(gate) if split else None, H * Dv, attn.gate_off if attn else 0,
            attn.gate_heads if attn else 0, ptr(hg), *wargs, 1 if bf else 0, stream(q)),
            "delta_prep")

    nd = md.num_decode
    if nd:
        launch(0, nd, None, None)
    if md.num_prefill_tokens:
        work, n_work = md.prefill_work_for(PREP_ROWS, build_work)
        launch(nd, n_work, md.prefill_cu_q, work)
    return r


def prefill_plan(md, device) -> Optional[ChunkPlan]:
    """The 64-token chunk list of a step's prompt portions (sequence numbers of the portions alone,
    row numbers of the step), built once per step and shared by its layers; None when no portion is
    long enough."""
    if "delta_chunks" not in md.work_cache:
        plan = None
        lens = list(md.prefill_q_lens or [])
        if md.seq_cu is not None and lens and len(lens) == md.num_seqs - md.num_decode:
            plan = chunk_plan(lens, device, CHUNK, 1 if FORCE_CHUNKED else CHUNK_MIN_ROWS,
                              md.num_decode)
        md.work_cache["delta_chunks"] = plan
    return md.work_cache["delta_chunks"]


def delta_scan(rows: DeltaRows, spec: DeltaSpec, state: DeltaState, md, norm_w: torch.Tensor,
               out: Optional[torch.Tensor] = None, plan: Optional[ChunkPlan] = None) -> torch.Tensor:
    """-> y [T, H*dv] in the gate's dtype (``out``: a view to write into).  ``norm_w`` [dv].  Updates
    the sequences' states.  ``plan``: the step's ``prefill_plan``."""
    T = rows.q.shape[0]
    H, G, D, Dv = spec.heads, spec.kv_heads, spec.dim, spec.vdim
    gate = rows.gate
    if out is None:
        out = torch.empty(T, H * Dv, dtype=gate.dtype, device=gate.device)
    require(out.shape == (T, H * Dv) and out.dtype == gate.dtype and out.stride(1) == 1,
            "delta_scan: out layout")
    if not use_hip(rows.q):
        rep = H // G
        q = rows.q[..., :D].repeat_interleave(rep, 1)
        k = rows.k[..., :D].repeat_interleave(rep, 1)
        v, a = rows.v[..., :Dv], torch.exp(rows.la)
        y = torch.zeros(T, H, Dv)
        for s, (lo, hi) in enumerate(_seq_bounds(md.seq_cu, md.num_seqs or T)):
            sl = int(md.seq_slots[s])
            if hi <= lo or sl < 0:
                continue
            S = torch.zeros(H, D, Dv) if int(md.positions[lo]) == 0 else state.S[sl].clone()
            for t in range(lo, hi):
                S = a[t][:, None, None] * S
                u = rows.beta[t][:, None] * (v[t] - torch.einsum("hi,hij->hj", k[t], S))
                S = S + k[t][:, :, None] * u[:, None, :]
                o = torch.einsum("hi,hij->hj", q[t], S)
                y[t] = o / torch.sqrt((o * o).mean(-1, keepdim=True) + spec.eps)
            state.S[sl] = S
        y = (y * norm_w.float()).reshape(T, H * Dv) * torch.nn.functional.silu(gate.float())
        out.copy_((y * spec.out_scale).to(out.dtype))
        return out
    bf = gate.dtype == torch.bfloat16
    DP, VP = rows.q.shape[2], rows.v.shape[2]
    require((bf or gate.dtype == torch.float32) and gate.stride(1) == 1 and
            gate.shape == (T, H * Dv), "delta_scan: gate rows")
    for t, shp in ((rows.q, (T, G, DP)), (rows.k, (T, G, DP)), (rows.v, (T, H, VP)),
                   (rows.la, (T, H)), (rows.beta, (T, H))):
        require(t.dtype == torch.float32 and t.is_contiguous() and t.shape == shp,
                "delta_scan: fp32 rows")
    require(DP == _pad16(D) and VP == _pad16(Dv), "delta_scan: padded heads")
    require(state.S.dtype == torch.float32 and state.S.is_contiguous() and
            state.S.shape[1:] == (H, D, Dv), "delta_scan: state layout")
    require(norm_w.dtype == gate.dtype and norm_w.is_contiguous() and norm_w.numel() == Dv,
            "delta_scan: norm weight")
    require(md.seq_slots.dtype == torch.int32 and md.positions.dtype == torch.int32 and
            (md.seq_cu is None or md.seq_cu.dtype == torch.int32), "delta_scan: int32 metadata")
    common = (ptr(rows.q), ptr(rows.k), ptr(rows.v), ptr(rows.la), ptr(rows.beta), H, G, D, Dv, DP,
              VP, ptr(gate), gate.stride(0), ptr(norm_w), float(spec.out_scale), float(spec.eps),
              ptr(state.S))

    def step(first, nseq):
        """Sequences [first, first + nseq) token by token."""
        if nseq:
            cu, lens = md.seq_cu, md.decode_seq_lens if md.seq_cu is None else None
            check(lib().eia_delta_scan(
                *common, ptr(md.seq_slots[first:]), ptr(cu[first:]) if cu is not None else None,
                ptr(md.positions), ptr(lens), ptr(out), out.stride(0), nseq, 1 if bf else 0,
                stream(out)), "delta_scan")

    nseq = md.num_seqs if md.num_seqs else T
    if (plan is None or not plan.n or max(D, Dv) > CHUNK_MAX_DIM or md.seq_cu is None or
            plan.rows != T or FORCE_CHUNKED is False or torch.cuda.is_current_stream_capturing()):
        step(0, nseq)
        return out
    nd = nseq - plan.nseq                       # decode rows stay token by token
    step(0, nd)
    dev = out.device
    f32 = lambda *s: torch.empty(*s, dtype=torch.float32, device=dev)
    Y, X, wsS = f32(T, H, DP), f32(T, H, VP), f32(plan.n, H, DP, VP)
    cA, wsG = f32(T, H), f32(plan.n, H)
    check(lib().eia_delta_scan_chunked(
        *common, ptr(md.seq_slots[nd:]), ptr(md.positions), ptr(out), out.stride(0), plan.nseq,
        ptr(plan.chunks), ptr(plan.seq_first), plan.n, ptr(Y), ptr(X), ptr(wsS), ptr(cA), ptr(wsG),
        1 if bf else 0, stream(out)), "delta_scan_chunked")
    return out
