"""Borosun test bodies, parametrised by device and dtype: the CPU file runs them on the
framework's PyTorch ops in fp32, the GPU file on the HIP kernels in fp32 and bf16."""

from __future__ import annotations

import math

import numpy as np
import torch

import borosun_common as C
from gapidra_cases import _metadata, _paged
from oracles import borosun_oracle as O


def tol(dtype):
    # fp32 is the sharp check; bf16 activations round at every product of these tiny models
    return 2e-4 if dtype == torch.float32 else 0.12


def ktol(dtype):
    """Kernel-level checks: inputs are already rounded to the dtype, so only the kernel's own
    roundings (bf16 outputs) remain."""
    return 2e-4 if dtype == torch.float32 else 1.5e-2


def _tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def _check(got, want, dtype, what):
    e = C.rel_err(got, want)
    assert e < tol(dtype), (what, e)


def _np(t):
    return t.double().cpu().numpy()


def _i32(v, device):
    return torch.tensor(v, dtype=torch.int32, device=device)


def _weights(cfg, seed, dtype):
    return C.random_weights(cfg, seed, dtype, tie_qk=dtype != torch.float32)


# ------------------------------------------------------------------ mechanisms alone
def case_frequencies():
    """Wavelength-banded scaling against the plain rule, with pairs in all three bands."""
    from enterprise_inference_amd.ops.rotary import rotary_frequencies
    for dims, base, sc in ((16, 5000.0, (4.0, 1.0, 4.0, 256)), (48, 1e5, (8.0, 0.5, 2.0, 4096)),
                           (6, 70.0, (2.0, 0.5, 3.0, 40))):
        scaling = dict(zip(("factor", "low", "high", "original"), sc))
        rot = {"base": base, "dims": dims, "scaling": scaling}
        f, amp = rotary_frequencies(dims, base, scaling)
        want = np.array(O.frequencies(rot))
        plain = np.array(O.frequencies({"base": base, "dims": dims}))
        kept, slow = np.isclose(want, plain), np.isclose(want, plain / sc[0])
        assert kept.any() and slow.any() and (~kept & ~slow).any()
        assert amp == 1.0 and np.allclose(_np(f), want, rtol=1e-6)


def case_gated_residual(device, dtype):
    """The gated boundary: outputs and gates as stored rows (a gate being columns of a wider row)
    or split-K partial sums with and without a bias, one or two sublayers, one of them without a
    gate; followed by the next norm, by a copy in the activation dtype, or by nothing."""
    from enterprise_inference_amd.ops import norm
    from enterprise_inference_amd.ops.gemm import SplitK, columns
    g = torch.Generator().manual_seed(1)
    T = 5
    for W in (46, 40, 256, 1028):
        for kinds in (((1, 1),), ((1, 2), (1, 1)), ((2, 2), (2, 2)), ((3, 3), (2, 1)),
                      ((1, 1), (2, 3)), ((1, 0), (1, 1))):
            for end in ("norm", "copy", None):
                x = torch.randn(T, W, generator=g) * 2
                want = _np(x).copy()
                ys, gates = [], []

                def src(kind, width, off, n):
                    """(device value, float64 columns off .. off + n)"""
                    if kind == 1:
                        v = (torch.randn(T, width, generator=g) * 1.5).to(dtype)
                        return v.to(device), _np(v)[:, off:off + n]
                    part = torch.randn(3, T, width, generator=g)
                    bias = torch.randn(width, generator=g).to(dtype) if kind == 3 else None
                    ref = _np(part).sum(0) + (_np(bias) if bias is not None else 0.0)
                    return SplitK(part.to(device), 3, T, width,
                                  bias.to(device) if bias is not None else None), ref[:, off:off + n]
                for ky, kg in kinds:
                    y, yr = src(ky, W, 0, W)
                    ys.append(y)
                    if kg:
                        f, gr = src(kg, 2 * W + 8, W // 4 * 4, W)
                        gates.append(columns(f, W // 4 * 4, W))
                        yr = yr * O.sigmoid(gr)
                    else:
                        gates.append(None)
                    want += yr
                w = torch.randn(W, generator=g).to(dtype)
                xd = x.clone().to(device)
                h = norm.residual_rms_step(xd, 1e-5, ys, w.to(device) if end == "norm" else None,
                                           gates, dtype if end == "copy" else None)
                assert np.allclose(_np(xd), want, atol=5e-5, rtol=1e-5), (W, kinds, end)
                if end is None:
                    assert h is None
                    continue
                hw = np.stack([O.rms(r, 1e-5) * _np(w) for r in want]) if end == "norm" else want
                assert h.dtype == dtype
                assert np.allclose(_np(h), hw, atol=ktol(dtype), rtol=ktol(dtype)), (W, kinds, end)


def case_side_output(device, dtype):
    """x += rms(y) w, then the next norm: y as stored rows or split-K partial sums (with and
    without a bias); widths of one and of several passes of a workgroup, and no multiple of four."""
    from enterprise_inference_amd.ops import norm
    from enterprise_inference_amd.ops.gemm import SplitK
    g = torch.Generator().manual_seed(2)
    T = 4
    for W in (46, 40, 512, 2052):
        for kind in (1, 2, 3):
            for nxt in (True, False):
                x = torch.randn(T, W, generator=g) * 2
                wp, wn = (torch.randn(W, generator=g).to(dtype) for _ in range(2))
                if kind == 1:
                    y = (torch.randn(T, W, generator=g) * 0.1).to(dtype)
                    yr, yd = _np(y), y.to(device)
                else:
                    part = torch.randn(2, T, W, generator=g)
                    bias = torch.randn(W, generator=g).to(dtype) if kind == 3 else None
                    yr = _np(part).sum(0) + (_np(bias) if bias is not None else 0.0)
                    yd = SplitK(part.to(device), 2, T, W,
                                bias.to(device) if bias is not None else None)
                want = _np(x) + np.stack([O.rms(r, 1e-5) * _np(wp) for r in yr])
                xd = x.clone().to(device)
                h = norm.group_norm_step(xd, 1, 1e-5, yd, wp.to(device), None,
                                         wn.to(device) if nxt else None)
                assert np.allclose(_np(xd), want, atol=5e-5, rtol=1e-5), (W, kind)
                if nxt:
                    hw = np.stack([O.rms(r, 1e-5) * _np(wn) for r in want])
                    assert np.allclose(_np(h), hw, atol=ktol(dtype), rtol=ktol(dtype)), (W, kind)


def case_act_mul_embed(device, dtype):
    """The gated token embedding at several layers' columns, with pad columns; the soft cap."""
    from enterprise_inference_amd.ops import activation as act
    from enterprise_inference_amd.ops.gemm import SplitK
    g = torch.Generator().manual_seed(3)
    for n, pad, layers, T in ((5, 128, 3, 7), (28, 28, 2, 1), (130, 256, 2, 9), (128, 128, 1, 3)):
        table = torch.randn(31, layers * n, generator=g).to(dtype)
        ids = torch.randint(0, 31, (T,), generator=g).to(torch.int32)
        u = (torch.randn(T, pad, generator=g) * 2).to(dtype)
        part = torch.randn(3, T, pad, generator=g)
        for i in range(layers):
            e = _np(table)[ids.long().numpy(), i * n:(i + 1) * n]
            for src, ref in ((u.to(device), _np(u)),
                             (SplitK(part.to(device), 3, T, pad), _np(part).sum(0))):
                got = act.act_mul_embed(src, "gelu_tanh", ids.to(device), table.to(device), i * n, n,
                                        pad)
                assert got.shape == (T, pad) and got.dtype == dtype
                assert np.allclose(_np(got[:, :n]), O.gelu_tanh(ref[:, :n]) * e, atol=ktol(dtype),
                                   rtol=ktol(dtype))
                assert not bool(got[:, n:].float().abs().max() > 0) if pad > n else True
    x = torch.randn(3, 50, generator=g) * 20
    got = act.softcap_(x.clone().to(device), 7.0)
    assert np.allclose(_np(got), O.softcap(_np(x), 7.0), atol=1e-5)
    assert torch.equal(act.softcap_(x.clone().to(device), 0.0).cpu(), x)


def case_token_side(W=288, n=28, T=300, sublayers=2, nxt=True):
    """The whole layer end in one launch (bf16, prompt-sized): a last workgroup that is partly
    empty, one or two sublayers, gates as columns of a wider row, side widths below, at and above
    the padding unit, widths that do not fill the last wave's tiles, with and without a next norm."""
    from enterprise_inference_amd.ops import norm
    g = torch.Generator().manual_seed(31)
    bf = torch.bfloat16
    rnd = lambda *s, k=1.0: (torch.randn(*s, generator=g) * k)
    x = rnd(T, W, k=2.0)
    ys = [rnd(T, W).to(bf) for _ in range(sublayers)]
    wide = rnd(T, 2 * W + 8).to(bf)
    pad = -(-n // 128) * 128
    gw, pw = torch.zeros(pad, W), torch.zeros(W, pad)
    gw[:n], pw[:, :n] = rnd(n, W, k=W ** -0.5), rnd(W, n, k=n ** -0.5)
    gw, pw = gw.to(bf), pw.to(bf)
    table = rnd(40, 3 * n).to(bf)
    ids = torch.randint(0, 40, (T,), generator=g).to(torch.int32)
    ws, wn = (1 + rnd(W, k=0.2)).to(bf), (1 + rnd(W, k=0.2)).to(bf)
    xd, wd = x.clone().cuda(), wide.cuda()
    ysd = [y.cuda() for y in ys]
    gates = [wd[:, q * W + 8 * q:q * W + 8 * q + W] for q in range(sublayers)]
    assert norm.token_side_ok(xd, ysd, gates, pad, bf)
    h = norm.token_side_step(xd, 1e-5, ysd, gates, ids.cuda(), table.cuda(), n, n,
                             norm.pack_operand(gw.cuda()), norm.pack_operand(pw.cuda()), ws.cuda(), wn.cuda() if nxt else None)
    want = _np(x)
    for q in range(sublayers):
        want = want + _np(ys[q]) * O.sigmoid(_np(wide)[:, q * W + 8 * q:q * W + 8 * q + W])
    e = _np(table)[ids.long().numpy(), n:2 * n]
    z = O.gelu_tanh(want @ _np(gw)[:n].T) * e
    y = z @ _np(pw)[:, :n].T
    want = want + np.stack([O.rms(r, 1e-5) for r in y]) * _np(ws)
    # (the products read the residual and the side values in bf16)
    assert np.allclose(_np(xd), want, atol=5e-2, rtol=1e-2), np.abs(_np(xd) - want).max()
    d = _np(xd) - want
    assert math.sqrt(float((d * d).mean())) < 6e-3
    if nxt:
        hw = np.stack([O.rms(r, 1e-5) for r in want]) * _np(wn)
        assert np.allclose(_np(h), hw, atol=3e-2, rtol=2e-2)
    else:
        assert h is None


def case_prep(device, dtype, H=4, G=2, D=10, Dv=6, dims=6, taps=3, normed=False, T=45, bs=16,
              split=False):
    """Convolution, rotation, head norm, value mixing and the cache write against the plain
    functions: one sequence whole, and in portions (down to one token, shorter than the taps)
    beside decoding and prefilling neighbours, on slots and pages that held something else; the
    portion edges fall inside and on the borders of pages and of the kernel's runs."""
    from enterprise_inference_amd.ops import window_attention as wa
    from enterprise_inference_amd.ops.attention import AttentionMetadata
    from enterprise_inference_amd.ops.gemm import SplitK
    from enterprise_inference_amd.ops.rotary import rotary_frequencies
    g = torch.Generator().manual_seed(21)
    rot = {"base": 200.0, "dims": dims}
    inv, _ = rotary_frequencies(dims, 200.0, None, device)
    conv = lambda c: (torch.randn(c, taps, generator=g) * 0.5).to(dtype)
    ws = [conv(H * D), conv(G * D), conv(G * Dv)]
    if not taps:                                       # no convolution at all
        ws, taps = [None] * 3, 1
    dev = lambda t: t.to(device).contiguous() if t is not None else None
    sp = wa.PrepSpec(H, G, D, Dv, inv, dims, True, 1.0, normed, 1e-5, taps,
                     *[dev(w) for w in ws])
    qo, ko, vo = 4, 4 + H * D, 4 + (H + G) * D + 4
    width = -(-(vo + G * Dv + 3) // 4) * 4
    fused = torch.randn(T, width, generator=g).to(dtype)
    vfirst = torch.randn(T, G * Dv, generator=g).to(dtype)
    lam = 0.35
    f64 = _np(fused)
    cols = {"q": f64[:, qo:qo + H * D], "k": f64[:, ko:ko + G * D], "v": f64[:, vo:vo + G * Dv]}
    u = {n: O.short_conv(list(cols[n]), _np(w)) if w is not None else list(cols[n])
         for n, w in zip("qkv", ws)}

    def side(x, m, t):
        x = [O.rotate(r, t, rot) for r in x.reshape(m, D)]
        return np.concatenate([O.rms(r, 1e-5) for r in x] if normed else x)

    want_q = np.stack([side(u["q"][t], H, t) for t in range(T)])
    want_k = np.stack([side(u["k"][t], G, t) for t in range(T)])
    raw_v = np.stack(u["v"])
    want_v = {0: raw_v, 1: raw_v, 2: O.mix_values(raw_v, _np(vfirst), lam)}
    table, slots, nblk = _paged(T, bs, 9)
    ntable, nslots, _ = _paged(T, bs, 10)
    lam_d = torch.tensor([lam], device=device)
    tk = ktol(dtype) * 2

    def run(cuts, mode):
        # page pool: the sequence's pages, then as many for the neighbours
        kc = torch.full((2 * nblk, bs, G * D), 7.0, dtype=dtype, device=device)
        vc = torch.full((2 * nblk, G * Dv, bs), 7.0, dtype=dtype, device=device)
        state = torch.full((3, max(1, taps - 1), sp.channels()), 9.0, dtype=dtype, device=device)
        q_out, first_out = [], []
        for lo, hi in cuts:
            n = hi - lo
            # rows: [a decoding row that is a padding row | a neighbour's portion of two from its
            # start | this portion]; a lone token runs as a decode row instead
            alone = n == 1 and lo > 0
            nd = 2 if alone else 1
            nb = 2
            if alone:
                rows = torch.cat([fused[:1], fused[lo:hi], fused[:nb]])
                sl, pos = [-1, 1, 2], [0, lo] + list(range(nb))
                cu = [0, 1, 2, 2 + nb]
                sm = [-1, int(slots[lo])] + [int(nslots[j]) + nblk * bs for j in range(nb)]
                mine = slice(1, 2)
                lens, vf = [nb], torch.cat([vfirst[:1], vfirst[lo:hi], vfirst[:nb]])
            else:
                rows = torch.cat([fused[:1], fused[:nb], fused[lo:hi]])
                sl, pos = [-1, 2, 1], [0] + list(range(nb)) + list(range(lo, hi))
                cu = [0, 1, 1 + nb, 1 + nb + n]
                sm = [-1] + [int(nslots[j]) + nblk * bs for j in range(nb)] + \
                    [int(slots[j]) for j in range(lo, hi)]
                mine = slice(1 + nb, 1 + nb + n)
                lens, vf = [nb, n], torch.cat([vfirst[:1], vfirst[:nb], vfirst[lo:hi]])
            cup = [0]
            for x in lens:
                cup.append(cup[-1] + x)
            md = AttentionMetadata(
                num_decode=nd, num_prefill_tokens=cup[-1], slot_mapping=_i32(sm, device),
                positions=_i32(pos, device), prefill_cu_q=_i32(cup, device), prefill_q_lens=lens,
                num_seqs=len(sl), seq_slots=_i32(sl, device), seq_cu=_i32(cu, device))
            src = dev(rows)
            if split:
                half = (rows.float() * 0.25)
                src = SplitK(torch.stack([half, rows.float() - half]).to(device), 2, rows.shape[0],
                             width)
            vfd = dev(vf) if mode == 2 else torch.zeros_like(dev(vf)) if mode == 1 else None
            q = wa.qkv_prep_cache(src, qo, ko, vo, sp, md, kc, vc, state if taps > 1 else None,
                                  lam_d, vfd, mode)
            q_out.append(q[mine])
            if mode == 1:
                first_out.append(vfd[mine])
        rows_k = kc.view(-1, G * D)[slots.to(device)]
        rows_v = vc[(slots // bs).to(device), :, (slots % bs).to(device)]
        assert np.allclose(_np(torch.cat(q_out)), want_q, atol=tk, rtol=tk)
        assert np.allclose(_np(rows_k), want_k, atol=tk, rtol=tk)
        assert np.allclose(_np(rows_v), want_v[mode], atol=tk, rtol=tk)
        if mode == 1:
            assert np.allclose(_np(torch.cat(first_out)), raw_v, atol=tk, rtol=tk)
        # the neighbours' rows, written again at every step from their own start
        nk = kc.view(-1, G * D)[(nslots[:2] + nblk * bs).to(device)]
        assert np.allclose(_np(nk), want_k[:2], atol=tk, rtol=tk)

    run([(0, T)], 0)
    pts = [c for c in (0, 1, 3, 4, 6, 16, 17, 25, 27, 32, 40, 42) if c < T] + [T]
    run(list(zip(pts[:-1], pts[1:])), 1)
    run(list(zip(pts[:-1], pts[1:])), 2)
    run([(0, 2)] + [(t, t + 1) for t in range(2, T)], 2)


def case_mix_needle(device, dtype, H=4, G=2, D=16, Dv=8, n=150, bs=16, size=0, cap=0.0,
                    mixed=True):
    """One key made to stand out for ONE head: through the mixing matrix every head's output is
    about that key's value, each in its own kv head's values.  j runs over far keys, page borders,
    the first tokens, the query itself and a window's edges; i is read as prefill rows and as
    decode rows.  ``cap``: soft-capped scores (the needle's score is far above the cap)."""
    from enterprise_inference_amd.ops import window_attention as wa
    g = torch.Generator().manual_seed(5)
    table, slots, nblk = _paged(n, bs, 6)
    i = n - 7
    T = torch.eye(H) * 0.5 + torch.randn(H, H, generator=g) * 0.4
    spec = wa.WindowSpec(H, G, 1, D, Dv, size, 0, mult=torch.full((H,), 0.3).to(device), cap=cap,
                         talk=T.to(device) if mixed else None, talk_post=mixed)
    edge = i - size + 1 if size else 0
    cand = {0, 1, n // 3, i, i - 1, (i // bs) * bs, (i // bs) * bs - 1, bs, edge, edge - 1, edge + 1}
    for j in sorted(c for c in cand if 0 <= c <= i):
        q = torch.randn(n, H, D, generator=g) * 0.5
        k = torch.randn(n, G, D, generator=g) * 0.5
        v = torch.randn(n, G, Dv, generator=g)
        u = torch.zeros(D)
        u[j % D] = 1.0
        q[i, j % H] += 8.0 * u
        k[j] += 8.0 * u
        q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
        kc = torch.zeros(nblk, bs, G * D, dtype=dtype)
        vc = torch.zeros(nblk, G * Dv, bs, dtype=dtype)
        kc.view(-1, G * D)[slots] = k.reshape(n, -1)
        vc[slots // bs, :, slots % bs] = v.reshape(n, -1)
        rows = [i, min(i + 3, n - 1), j]
        chunk = (max(0, i - 35), 40 if i >= 35 else 9)
        chunk = (chunk[0], min(chunk[1], n - chunk[0]))
        md = _metadata(device, table, rows, chunk)
        pos = rows + list(range(chunk[0], chunk[0] + chunk[1]))
        qs = torch.stack([q[p].reshape(-1) for p in pos])
        got = wa.window_attention(qs.to(device), kc.to(device), vc.to(device), md, spec, None)
        for r, p in enumerate(pos):
            if r >= len(rows) and p not in (i, i - 1, chunk[0], chunk[0] + chunk[1] - 1):
                continue
            lo = max(0, p - size + 1) if size else 0
            want = O.attend(_np(q[p]), [_np(k[t]) for t in range(lo, p + 1)],
                            [_np(v[t]) for t in range(lo, p + 1)], 0.3, cap,
                            _np(T) if mixed else None)
            d = np.abs(_np(got[r]) - want).max()
            assert d < (2e-4 if dtype == torch.float32 else 4e-2), (j, p, d)


def case_gla_scan(device, dtype, H=3, D=10, Dv=6, R=5, tau=4.0, T=75, chunked=False, bias=1.0):
    """The recurrence with a decay per key channel alone: a sequence run whole, and in portions
    (down to one token) beside another sequence on slots that held something else; one early
    key stands out and one channel hardly decays, so the state still shows it at the end; a
    strong bias towards forgetting makes whole-chunk decays underflow.  ``chunked``: long portions
    take the chunk-parallel form, short ones the token-by-token form, on the same slots."""
    from enterprise_inference_amd.ops import linear_scan as ls
    g = torch.Generator().manual_seed(11)
    a2 = torch.randn(H * D, R, generator=g) * (2.0 / R ** 0.5)
    a2b = bias + torch.randn(H * D, generator=g)
    a2[0], a2b[0] = 0.0, 9.0                          # channel 0 of head 0 keeps almost everything
    a2, a2b = a2.to(dtype).float(), a2b.to(dtype).float()
    spec = ls.ScanSpec(H, D, Dv, "channel", qscale=D ** -0.5, gate_act="silu", eps=1e-5, tau=tau,
                       a2t=a2.t().contiguous().to(device), a2b=a2b.to(device), norm_shared=True)
    width = 2 * H * D + 2 * H * Dv + R + 3
    qo, ko, vo = 0, H * D, 2 * H * D
    go, ro = vo + H * Dv, vo + 2 * H * Dv
    fused = torch.randn(T, width, generator=g)
    fused[3, ko] *= 30.0
    fused[3, vo:vo + Dv] += 4.0
    fused = fused.to(dtype)
    nw = (1 + 0.2 * torch.randn(Dv, generator=g)).to(dtype)
    f64 = _np(fused)
    want = np.zeros((T, H * Dv))
    S = [np.zeros((D, Dv)) for _ in range(H)]
    for t in range(T):
        z = _np(a2) @ f64[t, ro:ro + R] + _np(a2b)
        al = np.exp(O.logsigmoid(z) / tau).reshape(H, D)
        for a in range(H):
            sl = lambda o, w: f64[t, o + a * w:o + (a + 1) * w]
            o, S[a] = O.gla_core(sl(qo, D) * D ** -0.5, sl(ko, D), sl(vo, Dv), al[a], S[a])
            want[t, a * Dv:(a + 1) * Dv] = O.rms(o, 1e-5) * _np(nw)
        want[t] *= O.silu(f64[t, go:go + H * Dv])
    state = ls.ScanState.allocate(3, spec, device)
    state.S.fill_(5.0)                                 # stale slots
    fd = fused.to(device)
    ls.FORCE_CHUNKED = bool(chunked)

    def run(chunks):
        out = []
        for sl, lo, hi in chunks:
            rows = torch.cat([fd[:2] * 0.5, fd[lo:hi]])        # a second sequence beside it, slot 0
            pos = _i32([0, 1] + list(range(lo, hi)), device)
            plan = ls.chunk_plan([2, hi - lo], device) if chunked else None
            y = ls.linear_scan(rows, qo, ko, vo, go, spec, state, _i32([0, sl], device),
                               _i32([0, 2, 2 + hi - lo], device), 2, pos, None, nw.to(device),
                               plan=plan, lo_off=ro)
            out.append(y[2:])
        return torch.cat(out)

    try:
        tk = ktol(dtype) * 4
        got = run([(1, 0, T)])
        assert np.allclose(_np(got), want, atol=tk, rtol=tk), np.abs(_np(got) - want).max()
        cuts = [c for c in (0, 2, 3, 19, 20, 36, 37, 39, 70) if c < T] + [T]
        got = run([(2, a, b) for a, b in zip(cuts[:-1], cuts[1:])])
        assert np.allclose(_np(got), want, atol=tk, rtol=tk), np.abs(_np(got) - want).max()
        if chunked and T > 130:                        # long portions that start from a held state
            got = run([(2, 0, 65), (2, 65, 66), (2, 66, T)])
            assert np.allclose(_np(got), want, atol=tk, rtol=tk), np.abs(_np(got) - want).max()
    finally:
        ls.FORCE_CHUNKED = False
    # pure decode rows (no row ranges), a padding row between: slot 1 at position T - 1 again
    # after the tokens before it
    run([(1, 0, T - 1)])
    rows = torch.stack([fd[0], fd[T - 1]])
    y = ls.linear_scan(rows, qo, ko, vo, go, spec, state, _i32([-1, 1], device), None, 2,
                       _i32([0, T - 1], device), _i32([0, T], device), nw.to(device), lo_off=ro)
    assert np.allclose(_np(y[1]), want[T - 1], atol=tk, rtol=tk)


# ------------------------------------------------------------------ whole models
def case_layers(device, dtype, cfg_fn=C.config_a):
    """The residual after every layer."""
    cfg = cfg_fn()
    W = _weights(cfg, 9, dtype)
    t = _tokens(21, cfg["vocab"], 5)
    want = []
    C.oracle_logits(cfg, W, t, want)
    sess = C.make_session(cfg, W, device, dtype, max_tokens=64, block_size=16, max_live=1)
    try:
        from enterprise_inference_amd.engine.sequence import Sequence
        seq = Sequence("s", list(t), sess._params)
        plan = sess.scheduler.plan_given([(seq, len(t))])
        r = sess.runner
        r._flip_staging()
        sp = r._prepare_eager(sess.scheduler.bm, plan, logit_rows=[])
        r.d_e_buf[:sp["off"]].copy_(r.e_buf[:sp["off"]])
        ids, md, _ = r._eager_inputs(sp)
        got = []
        with torch.no_grad():
            r.model(ids, md, r.kv_caches, collect=got)
        r.finish_step()
        assert len(got) == len(want) == len(cfg["layers"])
        for k, (a, b) in enumerate(zip(got, want)):
            e = np.abs(_np(a) - b).max() / np.abs(b).max()
            assert e < (1e-4 if dtype == torch.float32 else 0.08), (k, e)
    finally:
        sess.close()


def case_schedules(device, dtype, cfg_fn=C.config_a, seed=0, block_size=16):
    """Whole prompts, prompt + one-by-one decoding, portions of several sizes down to two tokens
    and mixed batches with reuse of pages and state slots all give the oracle's logits."""
    cfg = cfg_fn()
    W = _weights(cfg, seed, dtype)
    V = cfg["vocab"]
    reqs = {"a": _tokens(70, V, 11), "b": _tokens(37, V, 12), "c": _tokens(5, V, 13),
            "d": _tokens(1, V, 14), "e": _tokens(49, V, 15)}
    want = {k: C.oracle_logits(cfg, W, t) for k, t in reqs.items()}
    # pool of 8 pages (of 16 tokens: "a" alone needs 5) and two slots: both are used again
    sess = C.make_session(cfg, W, device, dtype, max_tokens=8 * block_size, block_size=block_size,
                          max_live=2)
    try:
        for k, t in reqs.items():
            got = sess.step([{"id": k, "tokens": t, "want": list(range(len(t)))}], end=[k])
            _check(got, want[k], dtype, ("whole", k))
        # a prompt portion, then token by token
        for k in ("a", "b"):
            t = reqs[k]
            n0 = len(t) - 34
            got = [sess.step([{"id": k, "tokens": t[:n0], "want": [n0 - 1]}])]
            for i in range(n0, len(t)):
                got.append(sess.step([{"id": k, "tokens": [t[i]], "want": [0]}],
                                     end=[k] if i == len(t) - 1 else []))
            _check(torch.cat(got), want[k][n0 - 1:], dtype, ("decode", k))
        # portions: sizes cross page borders (16) and scan chunks and go down to two tokens
        t, at, got = reqs["a"], 0, []
        for n in (2, 13, 2, 16, 1, 17, 2, 15, 2):
            got.append(sess.step([{"id": "a", "tokens": t[at:at + n], "want": list(range(n))}],
                                 end=["a"] if at + n == len(t) else []))
            at += n
        assert at == len(t)
        _check(torch.cat(got), want["a"], dtype, "portions")
    finally:
        sess.close()
    # mixed batches on 4 sequences / 10 pages: unequal requests side by side, decode rows beside
    # prompt portions, requests that pause, pages and slots freed and taken again
    sess = C.make_session(cfg, W, device, dtype, max_tokens=10 * block_size, block_size=block_size,
                          max_live=4)
    try:
        got = {k: [] for k in reqs}
        at = {k: 0 for k in reqs}

        def run(plan, end=()):
            entries = []
            for k, n in plan:
                entries.append({"id": k, "tokens": reqs[k][at[k]:at[k] + n], "want": list(range(n))})
            out = sess.step(entries, end)
            r = 0
            for k, n in plan:
                got[k].append(out[r:r + n])
                r += n
                at[k] += n
        run([("d", 1), ("b", 3), ("c", 2)], end=["d"])
        run([("b", 1), ("c", 3), ("a", 20)], end=["c"])           # c finishes: page and slot free
        run([("a", 1), ("e", 30), ("b", 17)])                     # e takes them
        run([("e", 1), ("b", 16), ("a", 2)], end=["b"])
        run([("a", 47)], end=["a"])                               # e pauses
        run([("e", 18)], end=["e"])
        for k in reqs:
            assert at[k] == len(reqs[k])
            _check(torch.cat(got[k]), want[k], dtype, ("mixed", k))
        # a second life for a finished request's name, on reused pages and slots
        got2 = sess.step([{"id": "b", "tokens": reqs["b"], "want": list(range(len(reqs["b"])))},
                          {"id": "c", "tokens": reqs["c"], "want": [4]}], end=["b", "c"])
        _check(got2[:-1], want["b"], dtype, "again b")
        _check(got2[-1:], want["c"][4:], dtype, "again c")
        bm = sess.scheduler.bm
        assert bm.num_free_blocks() == bm.num_blocks and bm.slots.num_free() == 4
    finally:
        sess.close()


def case_long_prompt(device, dtype, cfg_fn=C.config_c, n=330, block_size=32):
    """A prompt long enough for the prompt-sized forms, its first portion beside a decoding
    request, then a second portion and single tokens: the logits do not depend on which form a
    row takes."""
    cfg = cfg_fn()
    W = _weights(cfg, 4, dtype)
    t, o = _tokens(n, cfg["vocab"], 41), _tokens(9, cfg["vocab"], 42)
    want, want_o = C.oracle_logits(cfg, W, t), C.oracle_logits(cfg, W, o)
    sess = C.make_session(cfg, W, device, dtype, max_tokens=384, block_size=block_size, max_live=2)
    try:
        e = lambda k, s, lo, hi: {"id": k, "tokens": s[lo:hi], "want": list(range(hi - lo))}
        got, got_o = [], [sess.step([e("o", o, 0, 8)])]
        out = sess.step([e("o", o, 8, 9), e("x", t, 0, 300)], end=["o"])
        got_o.append(out[:1])
        got.append(out[1:])
        got.append(sess.step([e("x", t, 300, 325)]))
        for i in range(325, n):
            got.append(sess.step([e("x", t, i, i + 1)]))
        _check(torch.cat(got), want, dtype, "long prompt")
        _check(torch.cat(got_o), want_o, dtype, "beside it")
    finally:
        sess.close()


def case_long_decode(device, dtype, cfg_fn=C.config_b):
    """140 tokens decoded one by one after a 3-token prompt, over many page borders."""
    cfg = cfg_fn()
    W = _weights(cfg, 3, dtype)
    t = _tokens(143, cfg["vocab"], 21)
    want = C.oracle_logits(cfg, W, t)
    sess = C.make_session(cfg, W, device, dtype, max_tokens=160, block_size=16, max_live=1)
    try:
        got = [sess.step([{"id": "x", "tokens": t[:3], "want": [0, 1, 2]}])]
        for i in range(3, len(t)):
            got.append(sess.step([{"id": "x", "tokens": [t[i]], "want": [0]}]))
        _check(torch.cat(got), want, dtype, "long decode")
    finally:
        sess.close()


def case_generate(device, dtype, cfg_fn=C.config_a, expect_graphs=None, block_size=16):
    """Greedy generation through LLMEngine (its scheduler, batching and sampler): every emitted
    token is the oracle's argmax given the tokens before it, for unequal prompts in one batch."""
    import copy

    from enterprise_inference_amd.config import (CacheConfig, EngineConfig, ModelConfig,
                                                 SchedulerConfig)
    from enterprise_inference_amd.engine.llm_engine import LLMEngine
    from enterprise_inference_amd.engine.sampling_params import SamplingParams
    cfg = cfg_fn()
    W = _weights(cfg, 5, dtype)
    ec = EngineConfig(model=ModelConfig.from_hf_dict(copy.deepcopy(cfg)), dtype=dtype, device=device,
                      load_format="dummy",
                      cache=CacheConfig(block_size=block_size, num_gpu_blocks=24),
                      scheduler=SchedulerConfig(max_num_seqs=3, max_num_batched_tokens=32,
                                                max_model_len=128))
    eng = LLMEngine(ec)
    model = eng.executor.runner.model
    model.load_weights(W.items())
    model.post_load()
    if expect_graphs is not None:
        assert bool(eng.executor.runner.graphs) == expect_graphs
    prompts = [_tokens(n, cfg["vocab"], 30 + n) for n in (40, 7, 1, 19)]     # 4 prompts, 3 seats
    outs = eng.generate(prompt_token_ids=prompts,
                        params=SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    for p, o in zip(prompts, outs):
        toks = list(o.outputs[0].token_ids)
        assert len(toks) == 12
        lg = C.oracle_logits(cfg, W, p + toks[:-1])
        scale = 1.0 if dtype == torch.float32 else float(lg.std())
        for i, tk in enumerate(toks):
            row = lg[len(p) - 1 + i]
            # the chosen token is the oracle's best, or within rounding of it
            assert float(row.max() - row[tk]) <= (1e-3 if dtype == torch.float32 else 0.15 * scale), \
                (i, tk)
    eng.shutdown()
