"""RMSNorm / LayerNorm ops (K5, K5b) -> csrc/kernels/norm.hip on the GPU."""

from __future__ import annotations

from typing import Optional, Tuple

import torch

from . import reference as ref
from ._dispatch import check, lib, ptr, require, stream, use_hip


def _rows(x: torch.Tensor) -> torch.Tensor:
    return x.reshape(-1, x.shape[-1])


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float,
             out: Optional[torch.Tensor] = None) -> torch.Tensor:
    if not (use_hip(x) and x.dtype == torch.bfloat16):
        r = ref.rms_norm(x, weight, eps)
        if out is not None:
            out.copy_(r)
            return out
        return r
    x2 = _rows(x)
    require(x2.stride(-1) == 1, "rms_norm: last dim must be contiguous")
    o = torch.empty(x.shape, dtype=x.dtype, device=x.device) if out is None else out
    o2 = _rows(o)
    T, H = x2.shape
    check(lib().eia_rms_norm(ptr(o2), ptr(x2), None, ptr(weight), float(eps), T, H,
                             x2.stride(0), o2.stride(0), stream(x)), "rms_norm")
    return o


def fused_add_rms_norm(x: torch.Tensor, residual: torch.Tensor, weight: torch.Tensor,
                       eps: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """residual <- x + residual (in place); returns (rms_norm(residual), residual)."""
    if not (use_hip(x, residual) and x.dtype == torch.bfloat16):
        out, r = ref.fused_add_rms_norm(x, residual, weight, eps)
        residual.copy_(r)
        return out, residual
    x2, r2 = _rows(x), _rows(residual)
    require(r2.is_contiguous() and x2.stride(-1) == 1, "fused_add_rms_norm: layout")
    T, H = x2.shape
    o = torch.empty_like(r2)
    check(lib().eia_rms_norm(ptr(o), ptr(x2), ptr(r2), ptr(weight), float(eps), T, H,
                             x2.stride(0), o.stride(0), stream(x)), "fused_add_rms_norm")
    return o.view(residual.shape), residual


def layer_norm(x: torch.Tensor, weight: torch.Tensor, bias: Optional[torch.Tensor], eps: float,
               residual: Optional[torch.Tensor] = None) -> torch.Tensor:
    """LayerNorm; with ``residual`` computes residual <- x + residual first (in place)."""
    if not (use_hip(x) and x.dtype == torch.bfloat16):
        if residual is not None:
            out, r = ref.fused_add_layer_norm(x, residual, weight, bias, eps)
            residual.copy_(r)
            return out
        return ref.layer_norm(x, weight, bias, eps)
    x2 = _rows(x).contiguous()
    T, H = x2.shape
    o = torch.empty_like(x2)
    r2 = None if residual is None else _rows(residual)
    check(lib().eia_layer_norm(ptr(o), ptr(x2), ptr(r2), ptr(weight), ptr(bias), float(eps), T, H,
                               stream(x)), "layer_norm")
    return o.view(x.shape)


def post_norm_residual(y: torch.Tensor, weight: torch.Tensor, eps: float, x: torch.Tensor,
                       copy: bool = True) -> Optional[torch.Tensor]:
    """Sublayer-output norm with an fp32 residual stream: x += layernorm(y) * weight in place
    (no bias, variance = mean of squared deviations, all fp32); returns the new x in y's dtype
    for the next GEMMs (``copy``; an fp32 model reads x itself)."""
    if not use_hip(y, x):
        yf = y.float()
        d = yf - yf.mean(-1, keepdim=True)
        x += d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight.float()
        return x.to(y.dtype) if copy and y.dtype != torch.float32 else (x if copy else None)
    require(x.dtype == torch.float32 and x.is_contiguous() and y.stride(-1) == 1 and
            y.shape == x.shape and weight.dtype == y.dtype, "post_norm_residual: layout")
    bf = y.dtype == torch.bfloat16
    require(bf or y.dtype == torch.float32, "post_norm_residual: bf16 or fp32")
    T, W = x.shape
    xb = torch.empty(T, W, dtype=y.dtype, device=y.device) if (copy and bf) else None
    check(lib().eia_ln_residual(ptr(y), y.stride(0), ptr(weight), ptr(x), ptr(xb),
                                W, float(eps), T, W, 1 if bf else 0, stream(y)), "ln_residual")
    return xb if bf else (x if copy else None)


def layer_norm_f32(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """layernorm(x fp32 [T, W]) * weight (no bias) -> [T, W] in the weight's dtype."""
    if not use_hip(x):
        d = x - x.mean(-1, keepdim=True)
        return (d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight.float()).to(weight.dtype)
    require(x.dtype == torch.float32 and x.stride(-1) == 1, "layer_norm_f32: fp32 rows")
    bf = weight.dtype == torch.bfloat16
    require(bf or weight.dtype == torch.float32, "layer_norm_f32: bf16 or fp32 weight")
    T, W = x.shape
    out = torch.empty(T, W, dtype=weight.dtype, device=x.device)
    check(lib().eia_ln_f32in(ptr(x), x.stride(0), ptr(weight), ptr(out), W, float(eps), T, W,
                             1 if bf else 0, stream(x)), "ln_f32in")
    return out


def _group_rms(v: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    p = v.reshape(*v.shape[:-1], groups, v.shape[-1] // groups)
    return (p / torch.sqrt((p * p).mean(-1, keepdim=True) + eps)).reshape(v.shape)


def group_norm_step(x: torch.Tensor, groups: int, eps: float, y=None,
                    w_post: Optional[torch.Tensor] = None, add: Optional[torch.Tensor] = None,
                    w_next: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """One sublayer boundary of a model whose norms are RMS norms in ``groups`` equal consecutive
    parts (each part divided by its own root mean square, the row times a weight) around an fp32
    residual stream x [T, W], in one pass over the row:

        x += gnorm(y) * w_post      (y given: a sublayer's output joins the stream, in place)
        x += add                    (add given: fp32 rows, in place)
        h  = gnorm(x) * w_next      (w_next given: returned in the weights' dtype)

    All arithmetic is fp32; y and the weights are in the activation dtype.  y may also be a
    ``gemm.SplitK`` (the fp32 partial sums of the GEMM that produced it, plus its bias): the
    reduction then happens here, on fp32 values that were never rounded."""
    from .gemm import SplitK
    T, W = x.shape
    require(W % groups == 0, "group_norm_step: width not divisible by the group count")
    split = isinstance(y, SplitK)
    if split and use_hip(x) and W % 4:
        # the kernel sums partials in 16-byte units: other widths (no GEMM of the framework
        # produces them) take the unfused fp32 sum
        ys = y.part.sum(0) + (y.bias.float() if y.bias is not None else 0.0)
        x += _group_rms(ys, groups, eps) * w_post.float()
        y, split = None, False
        if add is None and w_next is None:
            return None
    if not use_hip(x):
        if split:
            y = y.part.sum(0) + (y.bias.float() if y.bias is not None else 0.0)
        if y is not None:
            x += _group_rms(y.float(), groups, eps) * w_post.float()
        if add is not None:
            x += add
        if w_next is None:
            return None
        return (_group_rms(x, groups, eps) * w_next.float()).to(w_next.dtype)
    ref_w = w_next if w_next is not None else w_post
    require(x.dtype == torch.float32 and x.is_contiguous(), "group_norm_step: fp32 stream")
    require(ref_w is not None and ref_w.dtype in (torch.bfloat16, torch.float32),
            "group_norm_step: bf16 or fp32 weights")
    bf = ref_w.dtype == torch.bfloat16
    part = ybias = yt = None
    sk = 0
    if split:
        require(y.M == T and y.N == W and y.part.is_contiguous() and y.part.dtype == torch.float32
                and w_post is not None and w_post.dtype == ref_w.dtype and w_post.numel() == W
                and (y.bias is None or y.bias.dtype == ref_w.dtype), "group_norm_step: partials")
        part, sk, ybias = y.part, y.sk, y.bias
    elif y is not None:
        require(y.shape == x.shape and y.stride(-1) == 1 and y.dtype == ref_w.dtype and
                w_post.dtype == ref_w.dtype and w_post.numel() == W, "group_norm_step: y layout")
        yt = y
    if add is not None:
        require(add.dtype == torch.float32 and add.is_contiguous() and add.shape == x.shape,
                "group_norm_step: add layout")
    h = None
    if w_next is not None:
        require(w_next.numel() == W, "group_norm_step: weight size")
        h = torch.empty(T, W, dtype=w_next.dtype, device=x.device)
    if groups == 1 and add is None and (yt is not None or part is not None) and W % 4 == 0 and \
            (yt is None or yt.stride(0) % 4 == 0) and W <= 16384:
        # one group: a whole workgroup per row
        check(lib().eia_post_rms(ptr(yt), yt.stride(0) if yt is not None else 0, ptr(part), sk,
                                 ptr(ybias), ptr(w_post), ptr(x), ptr(w_next), ptr(h), W,
                                 float(eps), T, W, 1 if bf else 0, stream(x)), "post_rms")
        return h
    check(lib().eia_gnorm(ptr(yt), yt.stride(0) if yt is not None else 0, ptr(part), sk,
                          ptr(ybias), ptr(w_post), ptr(x), ptr(add), ptr(w_next), ptr(h), W,
                          float(eps), T, W, groups, 1 if bf else 0, stream(x)), "gnorm")
    return h


def residual_rms_step(x: torch.Tensor, eps: float, ys=(), w_next: Optional[torch.Tensor] = None,
                      gates=(), copy_dtype: Optional[torch.dtype] = None) -> Optional[torch.Tensor]:
    """Boundary of a layer whose sublayers run side by side on one normed input, around an fp32
    residual stream x [T, W], in one pass over the row:

        x += y            for every y in ``ys`` (at most two sublayer outputs, un-normed, in place)
        x += y * sigmoid(g)     where ``gates`` holds a g for that y
        h  = x / sqrt(mean(x^2) + eps) * w_next      (w_next given: returned in its dtype)
        h  = x                                       (else copy_dtype given: returned in it)

    All arithmetic is fp32.  A y is a tensor in the activation dtype or a ``gemm.SplitK`` (the
    fp32 partial sums of the GEMM that produced it, plus its bias), reduced here; a g is a tensor
    (W columns, possibly of a wider row) or a ``gemm.SplitKSlice`` of a fused projection."""
    from .gemm import SplitK, SplitKSlice
    T, W = x.shape
    gates = list(gates) + [None] * (len(ys) - len(gates))
    pairs = [(y, g) for y, g in zip(ys, gates) if y is not None]
    require(len(pairs) <= 2, "residual_rms_step: at most two sublayer outputs")

    def dense(y):
        if isinstance(y, SplitK):
            return y.part.sum(0) + (y.bias.float() if y.bias is not None else 0.0)
        if isinstance(y, SplitKSlice):
            return y.dense(torch.float32)
        return y.float()

    def joined(y, g):
        return dense(y) * torch.sigmoid(dense(g)) if g is not None else dense(y)

    if use_hip(x) and W % 4:
        # the kernel sums partials in 16-byte units; other widths (no GEMM of the framework
        # produces them) join the stream through the unfused fp32 sum
        odd = lambda y, g: isinstance(y, SplitK) or isinstance(g, SplitKSlice)
        for y, g in pairs:
            if odd(y, g):
                x += joined(y, g)
        pairs = [(y, g) for y, g in pairs if not odd(y, g)]
    if not use_hip(x):
        for y, g in pairs:
            x += joined(y, g)
        if w_next is None:
            return x.to(copy_dtype, copy=True) if copy_dtype is not None else None
        return (x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w_next.float()).to(w_next.dtype)
    require(x.dtype == torch.float32 and x.is_contiguous(), "residual_rms_step: fp32 stream")
    dt = w_next.dtype if w_next is not None else copy_dtype
    args = []
    for y, g in pairs:
        if isinstance(y, SplitK):
            require(y.M == T and y.N == W and y.part.is_contiguous() and
                    y.part.dtype == torch.float32, "residual_rms_step: partials")
            dt = dt or (y.bias.dtype if y.bias is not None else None)
            a = (None, 0, ptr(y.part), y.sk, ptr(y.bias))
            own = [y.bias]
        else:
            require(y.shape == x.shape and y.stride(-1) == 1, "residual_rms_step: y layout")
            dt = dt or y.dtype
            a = (ptr(y), y.stride(0), None, 0, None)
            own = [y]
        if g is None:
            a += (None, 0, None, 0, 0, None)
        elif isinstance(g, SplitKSlice):
            src = g.src
            require(src.M == T and g.n == W and g.off % 4 == 0 and src.N % 4 == 0 and
                    src.part.is_contiguous(), "residual_rms_step: gate partials")
            b = src.bias[g.off:g.off + W] if src.bias is not None else None
            a += (None, 0, src.part.data_ptr() + 4 * g.off, src.sk, src.N, ptr(b))
            own.append(b)
        else:
            require(g.shape == x.shape and g.stride(-1) == 1, "residual_rms_step: gate layout")
            dt = dt or g.dtype
            a += (ptr(g), g.stride(0), None, 0, 0, None)
            own.append(g)
        args.append((a, own))
    for _, own in args:
        require(all(t is None or t.dtype == dt for t in own),
                "residual_rms_step: one activation dtype")
    dt = dt or torch.float32
    require(dt in (torch.bfloat16, torch.float32), "residual_rms_step: bf16 or fp32")
    while len(args) < 2:
        args.append(((None, 0, None, 0, None, None, 0, None, 0, 0, None), []))
    h = None
    if w_next is not None or copy_dtype is not None:
        require(w_next is None or w_next.numel() == W, "residual_rms_step: weight size")
        h = torch.empty(T, W, dtype=dt, device=x.device)
    check(lib().eia_add_rms(*args[0][0], *args[1][0], ptr(x), ptr(w_next), ptr(h), W, float(eps), T,
                            W, 1 if dt == torch.bfloat16 else 0, stream(x)), "add_rms")
    return h


TOKEN_SIDE_MIN_ROWS = 256     # below it the unfused launches fill the chip better


def token_side_ok(x: torch.Tensor, ys, gates, pad: int, dtype) -> bool:
    """Whether ``token_side_step`` takes this layer end: bf16 on the GPU, a prompt-sized batch of
    stored (not split-K) rows, a supported width."""
    T, W = x.shape
    return (use_hip(x) and dtype == torch.bfloat16 and T >= TOKEN_SIDE_MIN_ROWS and
            1 <= len(ys) <= 2 and
            all(isinstance(t, torch.Tensor) and t.stride(-1) == 1 and t.stride(0) % 4 == 0 and
                t.data_ptr() % 8 == 0 for t in list(ys) + list(gates)) and
            bool(lib().eia_token_side_ok(W, pad)))


def pack_operand(w: torch.Tensor) -> torch.Tensor:
    """[N, K] row-major -> matrix-core operand order, same shape: [16-row tile][32-column step]
    [lane r + 16 g][8] (row r of the tile, columns 8 g .. 8 g + 7 of the step)."""
    N, K = w.shape
    return w.reshape(N // 16, 16, K // 32, 4, 8).permute(0, 2, 3, 1, 4).contiguous().view(N, K)


def token_side_step(x: torch.Tensor, eps: float, ys, gates, ids: torch.Tensor,
                    table: torch.Tensor, col0: int, n: int, gate_w: torch.Tensor,
                    proj_w: torch.Tensor, w_side: torch.Tensor,
                    w_next: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """A whole layer end in one launch (csrc/kernels/token_side.hip), x fp32 [T, W] in place:

        x += sum_q y_q * sigmoid(g_q)
        y  = W_proj (gelu_tanh(W_gate x) * table[ids, col0:col0 + n])
        x += y / sqrt(mean(y^2) + eps) * w_side
        h  = x / sqrt(mean(x^2) + eps) * w_next      (w_next given: returned)

    ``gate_w`` [pad, W] and ``proj_w`` [W, pad] are zero past ``n`` and packed by
    ``pack_operand``.  See ``token_side_ok``."""
    T, W = x.shape
    bf = torch.bfloat16
    pad = gate_w.shape[0]
    require(x.dtype == torch.float32 and x.is_contiguous() and len(ys) == len(gates) and
            all(t.shape == (T, W) and t.dtype == bf for t in list(ys) + list(gates)),
            "token_side_step: rows")
    require(gate_w.shape == (pad, W) and proj_w.shape == (W, pad) and gate_w.is_contiguous() and
            proj_w.is_contiguous() and w_side.numel() == W and
            all(t is None or t.dtype == bf for t in (gate_w, proj_w, w_side, w_next, table)) and
            table.stride(1) == 1 and 0 < n <= pad and col0 + n <= table.shape[1] and
            (w_next is None or w_next.numel() == W) and ids.dtype == torch.int32 and
            ids.numel() >= T, "token_side_step: weights")
    h = torch.empty(T, W, dtype=bf, device=x.device) if w_next is not None else None
    y2, g2 = (ys[1], gates[1]) if len(ys) > 1 else (None, None)
    check(lib().eia_token_side(
        ptr(x), ptr(ys[0]), ys[0].stride(0), ptr(gates[0]), gates[0].stride(0), ptr(y2),
        y2.stride(0) if y2 is not None else 0, ptr(g2), g2.stride(0) if g2 is not None else 0,
        ptr(ids), ptr(table), table.stride(0), col0, table.shape[0], ptr(gate_w), ptr(proj_w),
        ptr(w_side), ptr(w_next), ptr(h), W, float(eps), T, W, n, pad, stream(x)), "token_side")
    return h


def hyper_step(X: torch.Tensor, eps: float, y=None, mix: Optional[torch.Tensor] = None,
               outw: Optional[torch.Tensor] = None, ymult: float = 1.0,
               in_next: Optional[torch.Tensor] = None, w_next: Optional[torch.Tensor] = None,
               w_offset: float = 0.0) -> Optional[torch.Tensor]:
    """Boundary of a sublayer whose residual is kept as several streams joined by
    hyper-connections, X fp32 [T, NS, W] updated in place, in one pass over the row:

        X_j <- sum_s mix[s, j] X_s + ymult * outw[j] * y        (y given; all streams at once)
        u    = sum_j in_next[j] X_j
        h    = u / sqrt(mean(u^2) + eps) * (w_offset + w_next)   (w_next given: returned)

    ``mix`` [NS, NS] (from, to), ``outw`` [NS] and ``in_next`` [NS] are fp32.  y is a tensor in the
    activation dtype or a ``gemm.SplitK`` (fp32 partial sums of the GEMM that produced it, plus
    its bias), reduced here.  NS = 1 with unit constants is the plain residual sum."""
    from .gemm import SplitK
    T, NS, W = X.shape
    split = isinstance(y, SplitK)
    if split and (not use_hip(X)):
        y = y.part.sum(0) + (y.bias.float() if y.bias is not None else 0.0)
        split = False
    if not use_hip(X):
        if y is not None:
            X.copy_(torch.einsum("sj,tsw->tjw", mix.float(), X)
                    + ymult * outw.float()[None, :, None] * y.float()[:, None, :])
        if w_next is None:
            return None
        u = torch.einsum("j,tjw->tw", in_next.float(), X)
        return (u / torch.sqrt((u * u).mean(-1, keepdim=True) + eps)
                * (w_offset + w_next.float())).to(w_next.dtype)
    require(X.dtype == torch.float32 and X.is_contiguous() and NS <= 8, "hyper_step: fp32 streams")
    dt = w_next.dtype if w_next is not None else (
        (y.bias.dtype if y.bias is not None else torch.bfloat16) if split else
        (y.dtype if y is not None else torch.float32))
    require(dt in (torch.bfloat16, torch.float32), "hyper_step: bf16 or fp32")
    for t in (mix, outw, in_next):
        require(t is None or (t.dtype == torch.float32 and t.is_cuda and t.is_contiguous()),
                "hyper_step: fp32 device constants")
    yt = part = ybias = None
    sk = 0
    if split:
        require(y.M == T and y.N == W and y.part.is_contiguous() and
                y.part.dtype == torch.float32 and (y.bias is None or y.bias.dtype == dt),
                "hyper_step: partials")
        part, sk, ybias = y.part, y.sk, y.bias
    elif y is not None:
        require(y.shape == (T, W) and y.stride(-1) == 1 and y.dtype == dt, "hyper_step: y layout")
        yt = y
    if y is not None:
        require(mix is not None and outw is not None and mix.numel() == NS * NS and
                outw.numel() == NS, "hyper_step: stream constants")
    h = None
    if w_next is not None:
        require(w_next.numel() == W and in_next is not None and in_next.numel() == NS,
                "hyper_step: next norm")
        h = torch.empty(T, W, dtype=dt, device=X.device)
    check(lib().eia_hyper_step(ptr(X), NS, W, ptr(yt), yt.stride(0) if yt is not None else 0,
                               ptr(part), sk, ptr(ybias), ptr(mix), ptr(outw), float(ymult),
                               ptr(in_next), ptr(w_next), float(w_offset), ptr(h),
                               h.stride(0) if h is not None else 0, float(eps), T,
                               1 if dt == torch.bfloat16 else 0, stream(X)), "hyper_step")
    return h
