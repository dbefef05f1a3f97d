"""Vugelix test bodies, parametrised by device and dtype: the CPU file runs them on the framework's
PyTorch ops in fp32, the GPU file on the HIP kernels in fp32 and bf16."""

from __future__ import annotations

import math

import numpy as np
import torch

import vugelix_common as C
from gapidra_cases import _metadata, _paged
from oracles import vugelix_oracle as O


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


def _batch(device, portions, pos=None):
    """Step metadata: portions = (slot, first position, tokens) per sequence; one-token portions with
    a position above 0 that come first are decode rows."""
    from enterprise_inference_amd.ops.attention import AttentionMetadata
    nd = 0
    while nd < len(portions) and portions[nd][2] == 1 and portions[nd][1] != 0:
        nd += 1
    plist, cu, pl = [], [0], []
    for sl, p0, n in portions:
        plist += list(range(p0, p0 + n))
        cu.append(cu[-1] + n)
    for sl, p0, n in portions[nd:]:
        pl.append(n)
    T = cu[-1]
    pcu = [c - nd for c in cu[nd:]]
    return AttentionMetadata(
        num_decode=nd, num_prefill_tokens=T - nd, slot_mapping=_i32([-1] * T, device),
        positions=_i32(plist, device), decode_seq_lens=_i32([p + 1 for _, p, _ in portions[:nd]], device)
        if nd else None, prefill_cu_q=_i32(pcu, device) if pl else None, prefill_q_lens=pl or None,
        num_seqs=len(portions), seq_slots=_i32([s for s, _, _ in portions], device),
        seq_cu=_i32(cu, device) if pl else None)


# ------------------------------------------------------------------ mechanisms alone
def case_frequencies():
    from enterprise_inference_amd.ops.rotary import rotary_frequencies
    for dims, base in ((6, 3000.0), (48, 5e5), (2, 7.0)):
        f, amp = rotary_frequencies(dims, base, None)
        assert amp == 1.0 and np.allclose(_np(f), O.frequencies({"dims": dims, "base": base}), rtol=1e-6)


def case_relu2(device, dtype):
    """The squared ReLU of stored rows (odd widths, column slices) and of split-K partial sums."""
    from enterprise_inference_amd.ops import activation, gemm
    g = torch.Generator().manual_seed(4)
    for T, F in ((3, 20), (7, 33), (64, 256), (1, 4)):
        x = torch.randn(T, 2 * F, generator=g).to(dtype)
        for v in (x[:, :F], x[:, F:], x[:, :F].contiguous()):
            got = activation.relu2(v.to(device) if v.is_contiguous() else x.to(device)[
                :, v.storage_offset():v.storage_offset() + F])
            assert np.allclose(_np(got), np.maximum(_np(v), 0) ** 2, rtol=ktol(dtype), atol=1e-6)
        for sk in (1, 3, 9):
            part = torch.randn(sk, T, F, generator=g)
            got = activation.relu2(gemm.SplitK(part.to(device), sk, T, F), dtype)
            want = np.maximum(_np(part).sum(0), 0) ** 2
            assert got.dtype == dtype and np.allclose(_np(got), want, rtol=ktol(dtype), atol=1e-5)


def case_hyper_step(device, dtype):
    """The sublayer boundary with plain norm weights: 1 .. 5 streams; no output (only the next input),
    a stored one, split-K partial sums (1 to 19 of them); widths that are no multiple of four and wide
    rows."""
    from enterprise_inference_amd.ops import norm
    from enterprise_inference_amd.ops.gemm import SplitK
    g = torch.Generator().manual_seed(1)
    for W in (42, 300, 2056):
        for NS in (1, 2, 3, 5):
            for sk in (None, 0, 1, 8, 19):
                T = 3
                X = torch.randn(T, NS, W, generator=g) * 2
                mix = torch.eye(NS) + torch.randn(NS, NS, generator=g) * 0.3
                outw, inw = torch.randn(NS, generator=g), torch.randn(NS, generator=g)
                wn = (1 + torch.randn(W, generator=g) * 0.2).to(dtype)
                want = _np(X).copy()
                y = None
                if sk == 0:
                    y = torch.randn(T, W, generator=g).to(dtype)
                    yd, y = _np(y), y.to(device)
                elif sk:
                    part = torch.randn(sk, T, W, generator=g)
                    yd, y = _np(part).sum(0), SplitK(part.to(device), sk, T, W)
                if sk is not None:
                    want = np.einsum("sj,tsw->tjw", _np(mix), want) \
                        + _np(outw)[None, :, None] * yd[:, None, :]
                Xd = X.to(device)
                h = norm.hyper_step(Xd, 1e-5, y, mix.to(device), outw.to(device), 1.0,
                                    inw.to(device), wn.to(device), 0.0)
                assert np.allclose(_np(Xd), want, atol=1e-4, rtol=1e-5), (W, NS, sk)
                u = np.einsum("j,tjw->tw", _np(inw), want)
                hw = np.stack([O.rms(u[t], 1e-5) * _np(wn) for t in range(T)])
                assert np.allclose(_np(h), hw, atol=ktol(dtype) * 3, rtol=ktol(dtype)), (W, NS, sk)


def case_needle(device, dtype, H=4, G=2, D=16, Dv=8, size=40, n=150, bs=16, cap=12.0):
    """Windowed attention with soft-capped scores, the unit in the denominator and a gate per head;
    ONE key made to stand out (the query at position i and the key at position j share a large
    component, above the cap before capping).  j runs over the window's inside and outside edge, page
    borders, the first tokens and far keys; i is read as a prefill row and as a decode row.  Every
    other query row is turned against its keys, so that the unit takes most of its weight."""
    from enterprise_inference_amd.ops import window_attention as wa
    g = torch.Generator().manual_seed(5)
    table, slots, nblk = _paged(n, bs, 6)
    i = n - 7
    scale = 0.5
    spec = wa.WindowSpec(H, G, 1, D, Dv, size, 0, mult=torch.full((H,), scale).to(device), cap=cap,
                         sink=torch.zeros(H).to(device), post=0.8, gate_heads=True)
    edge = i - size + 1 if size else 0
    cand = {0, 1, 2, n // 3, i, i - 1, (i // bs) * bs, (i // bs) * bs - 1, bs - 1, bs, edge, edge - 1,
            edge + 1}
    for j in sorted(c for c in cand if 0 <= c <= i):
        q = torch.randn(n, H, D, generator=g) * 0.5
        k = torch.randn(n, G, D, generator=g) * 0.5 + 0.4
        q[1::2] -= 1.2
        q[i] += 1.2 * (i & 1)
        v = torch.randn(n, G, Dv, generator=g)
        gate = torch.randn(n, H, generator=g) * 2
        u = torch.zeros(D)
        u[j % D] = 1.0
        q[i] += 6.0 * u
        k[j] += 6.0 * u
        q, k, v, gate = (x.to(dtype) for x in (q, k, v, gate))
        kc = torch.zeros(nblk, bs, G * D, dtype=dtype)
        vc = torch.zeros(nblk, G * Dv, bs, dtype=dtype)
        kc.view(-1, G * D)[slots] = k.reshape(n, -1)
        vc[slots // bs, :, slots % bs] = v.reshape(n, -1)
        rows = [i, min(i + 3, n - 1), j]
        chunk = (i - 5, 9)
        md = _metadata(device, table, rows, chunk)
        pos = rows + list(range(chunk[0], chunk[0] + chunk[1]))
        qs = torch.stack([q[p].reshape(-1) for p in pos])
        # (the gate as columns of a wider row)
        gw = torch.cat([torch.zeros(len(pos), 8, dtype=dtype), gate[pos]], 1).to(device)
        got = wa.window_attention(qs.to(device), kc.to(device), vc.to(device), md, spec, gw[:, 8:])
        for r, p in enumerate(pos):
            lo = max(0, p - size + 1) if size else 0
            for a in range(H):
                kv = a // (H // G)
                want = 0.8 * O.sigmoid(float(gate[p, a])) * O.off_by_one_attention(
                    _np(q[p, a]), [_np(k[t, kv]) for t in range(lo, p + 1)],
                    [_np(v[t, kv]) for t in range(lo, p + 1)], scale, cap)
                d = np.abs(_np(got[r, a * Dv:(a + 1) * Dv]) - want).max()
                assert d < (2e-4 if dtype == torch.float32 else 4e-2), (j, p, a, d)


def _delta_spec(device, dtype, g, H, G, D, Dv, taps, slow=True):
    from enterprise_inference_amd.ops import delta_scan as ds
    cw = lambda n: (torch.randn(n, taps, generator=g) * 0.5 + (torch.arange(taps) == taps - 1)).to(dtype)
    w = {"q": cw(G * D), "k": cw(G * D), "v": cw(H * Dv)}
    A = torch.randn(H, generator=g) * 0.5
    dt = torch.randn(H, generator=g)
    if slow:
        A[0], dt[0] = -3.0, -4.0                       # one head that hardly decays
    spec = ds.DeltaSpec(H, G, D, Dv, taps, *(w[n].to(device) for n in "qkv"), torch.exp(A).to(device),
                        dt.to(device), D ** -0.5, 0.9, 1e-5)
    return spec, w, _np(torch.exp(A)), _np(dt)


def _offsets(H, G, D, Dv, lead=0):
    offs, n = {}, lead
    for name, c in (("q", G * D), ("k", G * D), ("v", H * Dv), ("g", H * Dv), ("b", H), ("a", H)):
        n = -(-n // 8) * 8
        offs[name] = n
        n += c
    return offs, -(-n // 4) * 4


def case_delta_prep(device, dtype, H=4, G=2, D=10, Dv=6, taps=3, aH=2, aG=1, aD=12, aDv=8, dims=6,
                    T=45, bs=16):
    """From projection rows to the inputs of both mixers: convolution, silu, unit norms, decays and step
    sizes of the delta side, rotation and cache write of the attention side.  One sequence run whole and
    in portions down to one token (decode rows included) beside a decoding and a prefilling neighbour and
    a padding row, on stale slots; stored rows and split-K partials."""
    from enterprise_inference_amd.ops import delta_scan as ds
    from enterprise_inference_amd.ops import gemm
    from enterprise_inference_amd.ops import window_attention as wa
    from enterprise_inference_amd.ops.rotary import rotary_frequencies
    g = torch.Generator().manual_seed(21)
    spec, w, expA, dt = _delta_spec(device, dtype, g, H, G, D, Dv, taps)
    aw = (aH + 2 * aG) * max(aD, aDv) + aH
    offs, width = _offsets(H, G, D, Dv, aw)
    qo, ko, vo, go = 0, aH * aD, (aH + aG) * aD, (aH + aG) * aD + aG * aDv
    seq = torch.randn(T, width, generator=g).to(dtype)
    other = torch.randn(12, width, generator=g).to(dtype)
    f = _np(seq)
    conv = {n: O.short_conv([f[t, offs[n]:offs[n] + r] for t in range(T)], _np(w[n]))
            for n, r in (("q", G * D), ("k", G * D), ("v", H * Dv))}
    rot = {"base": 500.0, "dims": dims}
    inv, _ = rotary_frequencies(dims, 500.0, None)
    prep = wa.PrepSpec(aH, aG, aD, aDv, inv.to(device), dims, True)
    tk = ktol(dtype)

    def run(cuts, split, slot):
        st = ds.DeltaState.allocate(4, spec, dtype, device)
        if st.hist is not None:
            st.hist.fill_(3.0)                          # stale slots
        nblk = -(-T // bs) + 2
        kc = torch.full((nblk, bs, aG * aD), 9.0, dtype=dtype).to(device)
        vc = torch.full((nblk, aG * aDv, bs), 9.0, dtype=dtype).to(device)
        attn = ds.AttnPrep(qo, ko, vo, prep, kc, vc, go, aH)
        for lo, hi in zip(cuts[:-1], cuts[1:]):
            n = hi - lo
            own_decode = n == 1 and lo > 0
            # neighbours: a decode row (slot 0), a padding row, a prefilling sequence (slot 3)
            parts = [(0, 40, 1, other[:1])]
            if own_decode:
                parts += [(slot, lo, 1, seq[lo:hi]), (-1, 1, 1, other[1:2])]
            else:
                parts += [(-1, 1, 1, other[1:2]), (3, 0, 5, other[2:7]), (slot, lo, n, seq[lo:hi])]
            md = _batch(device, [p[:3] for p in parts])
            rows = torch.cat([p[3] for p in parts])
            r0 = 1 if own_decode else 7
            slots = [-1] * rows.shape[0]
            for t in range(n):
                slots[r0 + t] = bs + lo + t             # (the sequence's pages start at block 1)
            md.slot_mapping = _i32(slots, device)
            x = rows.to(device)
            if split:
                a1 = torch.randn(2, *rows.shape, generator=g)
                part = torch.cat([a1, (rows.float() - a1.sum(0))[None]], 0).contiguous()
                x = gemm.SplitK(part.to(device), 3, *rows.shape)
            out = ds.delta_prep(x, offs, spec, st, md, attn)
            for t in range(n):
                r, p = r0 + t, lo + t
                for name, got, hd, cnt in (("q", out.q, D, G), ("k", out.k, D, G), ("v", out.v, Dv, H)):
                    want = conv[name][p].reshape(cnt, hd)
                    if name != "v":
                        want = np.stack([O.unit(z) for z in want]) * (D ** -0.5 if name == "q" else 1.0)
                    gv = _np(got[r])
                    assert np.allclose(gv[:, :hd], want, atol=2 * tk, rtol=2 * tk), (name, p, split)
                    assert not gv[:, hd:].any()
                za = f[p, offs["a"]:offs["a"] + H] + dt
                la = [-e * O.softplus(float(z)) for e, z in zip(expA, za)]
                assert np.allclose(_np(out.la[r]), la, atol=tk, rtol=tk)
                assert np.allclose(_np(out.beta[r]), O.sigmoid(f[p, offs["b"]:offs["b"] + H]), atol=tk)
                assert np.allclose(_np(out.gate[r]), f[p, offs["g"]:offs["g"] + H * Dv], atol=2 * tk,
                                   rtol=tk)
                assert np.allclose(_np(out.attn_gate[r]), f[p, go:go + aH], atol=2 * tk, rtol=tk)
                for a in range(aH):
                    want = O.rotate(f[p, qo + a * aD:qo + (a + 1) * aD], p, rot if dims else None)
                    assert np.allclose(_np(out.attn_q[r, a * aD:(a + 1) * aD]), want, atol=3 * tk,
                                       rtol=3 * tk), (p, a)
        for p in range(T):
            blk, off = 1 + p // bs, p % bs
            for a in range(aG):
                want = O.rotate(f[p, ko + a * aD:ko + (a + 1) * aD], p, rot if dims else None)
                assert np.allclose(_np(kc[blk, off, a * aD:(a + 1) * aD]), want, atol=3 * tk, rtol=3 * tk)
            assert np.allclose(_np(vc[blk, :, off]), f[p, vo:vo + aG * aDv], atol=2 * tk, rtol=tk)
        assert float(kc[0].float().min()) == 9.0        # no row of a neighbour was written

    for split in (False, True):
        run([0, T], split, 2)
        run([c for c in (0, 1, 2, 3, 5, 6, 14, 22, 23, 25, 41, 42, 43) if c < T] + [T], split, 1)


def _scan_rows(device, g, T, H, G, D, Dv, kind):
    """fp32 rows of delta_prep's form: unit queries and keys; ``kind`` "needle": one early key and value
    that stand out and whose key is asked for again from time to time; "same": all keys of a head equal
    (the strongest coupling inside a chunk), step sizes near 1; "forget": decays that underflow over a
    few tokens."""
    from enterprise_inference_amd.ops.delta_scan import _pad16
    unit = lambda x: x / x.norm(dim=-1, keepdim=True)
    q, k = unit(torch.randn(T, G, D, generator=g)), unit(torch.randn(T, G, D, generator=g))
    v = torch.randn(T, H, Dv, generator=g)
    la = -torch.rand(T, H, generator=g) * 0.15
    la[:, 0] *= 0.02                                   # one slow head
    beta = torch.sigmoid(torch.randn(T, H, generator=g) * 2)
    if kind == "needle":
        e = unit(torch.randn(G, D, generator=g))
        keep = torch.ones(T, dtype=torch.bool)
        keep[3] = False
        kk = k[keep] - (k[keep] * e).sum(-1, keepdim=True) * e
        if D > 2:
            k[keep] = unit(kk)                         # no other key writes over it
        k[3], beta[3] = e, 0.98
        v[3] *= 6.0
        q[5::9] = e
    elif kind == "same":
        k[:] = k[:1]
        q[::2] = k[:1]
        beta = 1.0 - 0.05 * torch.rand(T, H, generator=g)
        la *= 0.01
    elif kind == "forget":
        la[:, 1:] = -torch.rand(T, max(0, H - 1), generator=g) * 60.0
        la[:, 0] = -20.0 * (torch.arange(T) % 7 == 3)
    pad = lambda x: torch.nn.functional.pad(x, (0, _pad16(x.shape[-1]) - x.shape[-1])).contiguous()
    return pad(q), pad(k), pad(v), la, beta


def case_delta_scan(device, dtype, H=3, G=1, D=10, Dv=6, T=75, kind="needle", chunked=False):
    """The recurrence alone: a sequence run whole and in portions (down to one token) beside a decode
    row, another sequence and a padding row, on slots that held something else; the chunk-parallel form
    for portions (``chunked``) or the token-by-token form; portions that start from a held state; the
    states both forms leave."""
    from enterprise_inference_amd.ops import delta_scan as ds
    g = torch.Generator().manual_seed(13)
    spec, _, _, _ = _delta_spec(device, dtype, g, H, G, D, Dv, 2)
    q, k, v, la, beta = _scan_rows(device, g, T, H, G, D, Dv, kind)
    gate = torch.randn(T, H * Dv, generator=g).to(dtype)
    nw = (1 + 0.2 * torch.randn(Dv, generator=g)).to(dtype)
    want = np.zeros((T, H * Dv))
    S = [np.zeros((D, Dv)) for _ in range(H)]
    for t in range(T):
        for a in range(H):
            kh = a // (H // G)
            o, S[a] = O.delta_core(_np(q[t, kh, :D]), _np(k[t, kh, :D]), _np(v[t, a, :Dv]),
                                   math.exp(float(la[t, a])), float(beta[t, a]), S[a])
            want[t, a * Dv:(a + 1) * Dv] = O.rms(o, 1e-5) * _np(nw)
        want[t] *= O.silu(_np(gate[t])) * 0.9
    S = np.stack(S)
    extra = [torch.randn(8, *x.shape[1:], generator=g) * 0.3 for x in (q, k, v)]
    ex_la, ex_b = -torch.rand(8, H, generator=g), torch.rand(8, H, generator=g)
    ex_g = torch.randn(8, H * Dv, generator=g).to(dtype)
    tk = ktol(dtype) * 4
    ds.FORCE_CHUNKED = chunked
    try:
        def run(cuts, slot):
            st = ds.DeltaState.allocate(4, spec, dtype, device)
            st.S.fill_(5.0)                             # stale slots
            out = []
            for lo, hi in zip(cuts[:-1], cuts[1:]):
                n = hi - lo
                portions = [(0, 30, 1), (-1, 1, 1), (3, 0, 6), (slot, lo, n)]
                md = _batch(device, portions)
                cat = lambda e, x: torch.cat([e, x[lo:hi]]).contiguous().to(device)
                rows = ds.DeltaRows(cat(extra[0], q), cat(extra[1], k), cat(extra[2], v),
                                    cat(ex_la, la), cat(ex_b, beta), cat(ex_g, gate))
                plan = ds.prefill_plan(md, torch.device(device)) if chunked else None
                wide = torch.full((8 + n, H * Dv + 8), 7.0, dtype=dtype).to(device)
                ds.delta_scan(rows, spec, st, md, nw.to(device), wide[:, 8:], plan)
                assert float(wide[:, :8].float().min()) == 7.0      # the shared row's other columns
                out.append(wide[8:, 8:])
            assert np.allclose(_np(st.S[slot]), S, atol=2e-4 * max(1.0, np.abs(S).max())), \
                np.abs(_np(st.S[slot]) - S).max()
            assert float(st.S[2 if slot == 1 else 1].min()) == 5.0  # untouched slots
            return torch.cat(out), st

        for cuts, slot in (([0, T], 1), ([0] + [c for c in (2, 3, 19, 20, 36, 63, 64, 65, 127, 129, 130)
                                                if c < T] + [T], 2)):
            got, st = run(cuts, slot)
            e = np.abs(_np(got) - want)
            assert np.allclose(_np(got), want, atol=tk, rtol=tk), (cuts, e.max(), e.max(1).argmax())
        # a pure decode step (no row ranges), with a padding row
        md = _batch(device, [(slot, T, 1), (-1, 5, 1)])
        assert md.seq_cu is None
        rows = ds.DeltaRows(*(x[:2].contiguous().to(device) for x in (q, k, v, la, beta, gate)))
        y = ds.delta_scan(rows, spec, st, md, nw.to(device))
        for a in range(H):
            o, _ = O.delta_core(_np(q[0, a // (H // G), :D]), _np(k[0, a // (H // G), :D]),
                                _np(v[0, a, :Dv]), math.exp(float(la[0, a])), float(beta[0, a]), S[a])
            w1 = O.rms(o, 1e-5) * _np(nw) * O.silu(_np(gate[0, a * Dv:(a + 1) * Dv])) * 0.9
            assert np.allclose(_np(y[0, a * Dv:(a + 1) * Dv]), w1, atol=tk, rtol=tk), a
    finally:
        ds.FORCE_CHUNKED = None


# ------------------------------------------------------------------ whole models
def case_layers(device, dtype, cfg_fn=C.config_a, n=70):
    """The sum of the residual streams after every layer run."""
    from enterprise_inference_amd.engine.sequence import Sequence
    cfg = cfg_fn()
    W = _weights(cfg, 9, dtype)
    t = _tokens(n, cfg["vocab"], 5)
    want = []
    C.oracle_logits(cfg, W, t, want)
    sess = C.make_session(cfg, W, device, dtype, max_tokens=96, block_size=16, max_live=1)
    try:
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
    """Whole prompts, prompt + one-by-one decoding, portions of several sizes down to two tokens and
    mixed batches with reuse of pages and state slots all give the oracle's logits."""
    cfg = cfg_fn()
    W = _weights(cfg, seed, dtype)
    V = cfg["vocab"]
    reqs = {"a": _tokens(83, V, 11), "b": _tokens(37, V, 12), "c": _tokens(5, V, 13),
            "d": _tokens(1, V, 14), "e": _tokens(71, V, 15)}
    want = {k: C.oracle_logits(cfg, W, t) for k, t in reqs.items()}
    # pool of 8 pages (of 16 tokens: "a" alone needs 6) and two slots: both are used again
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
        # portions: sizes cross page borders, windows and scan chunks and go down to two tokens
        for sizes in ((2, 13, 2, 16, 1, 17, 2, 15, 2, 13), (65, 2, 16), (2, 66, 15), (17, 49, 17)):
            t, at, got = reqs["a"], 0, []
            for n in sizes:
                got.append(sess.step([{"id": "a", "tokens": t[at:at + n], "want": list(range(n))}],
                                     end=["a"] if at + n == len(t) else []))
                at += n
            assert at == len(t)
            _check(torch.cat(got), want["a"], dtype, ("portions", sizes))
    finally:
        sess.close()
    # mixed batches on 4 sequences / 12 pages: unequal requests side by side, decode rows beside
    # prompt portions, requests that pause, pages and slots freed and taken again
    sess = C.make_session(cfg, W, device, dtype, max_tokens=12 * block_size, block_size=block_size,
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
        run([("a", 1), ("e", 50), ("b", 17)])                     # e takes them
        run([("e", 1), ("b", 16), ("a", 2)], end=["b"])
        run([("a", 60)], end=["a"])                               # e pauses
        run([("e", 20)], end=["e"])
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


def case_generate(device, dtype, cfg_fn=C.config_a, expect_graphs=None):
    """Greedy generation through LLMEngine (its scheduler, batching and sampler): every emitted token
    is the oracle's argmax given the tokens before it, for unequal prompts in one batch."""
    import copy

    from enterprise_inference_amd.config import (CacheConfig, EngineConfig, ModelConfig,
                                                 SchedulerConfig)
    from enterprise_inference_amd.engine.llm_engine import LLMEngine
    from enterprise_inference_amd.engine.sampling_params import SamplingParams
    cfg = cfg_fn()
    W = _weights(cfg, 5, dtype)
    eng = LLMEngine(EngineConfig(
        model=ModelConfig.from_hf_dict(copy.deepcopy(cfg)), dtype=dtype, device=device,
        load_format="dummy", cache=CacheConfig(block_size=16, num_gpu_blocks=24),
        scheduler=SchedulerConfig(max_num_seqs=3, max_num_batched_tokens=32, max_model_len=128)))
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
        spread = float(lg.std())
        for i, tk in enumerate(toks):
            row = lg[len(p) - 1 + i]
            # the chosen token is the oracle's best, or within rounding of it
            slack = (1e-3 if dtype == torch.float32 else 0.15) * max(1.0, spread)
            assert float(row.max() - row[tk]) <= slack, (i, tk)
    eng.shutdown()
