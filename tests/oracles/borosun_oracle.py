"""Plain float64 implementation of the Borosun design, written from its equations: loops over
tokens, heads and keys, one function per mechanism, no code shared with the framework.

A layer reads one RMS norm of the residual and adds both sublayers to it, each scaled by an
element-wise sigmoid gate computed from the same normed input; a per-layer token embedding then
joins through a gated low-width projection whose output is RMS-normed.  Mixers: ``attention`` (short
causal convolutions on q, k and v, rotation with banded frequency scaling, softmax weights mixed
across the heads, value mixing with the first such layer's values), ``attention_2`` (rotation,
weightless RMS norm of q and k per head, soft-capped scores, sliding window, value mixing) and
``gla`` (linear attention whose state decays per key channel, gated and normed per head).  ``W``
maps the checkpoint's tensor names to float64 arrays.
"""

from __future__ import annotations

import math

import numpy as np


def rms(x, eps):
    return x / math.sqrt(float(np.mean(x * x)) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def logsigmoid(z):
    return -(np.log1p(np.exp(-np.abs(z))) + np.maximum(-z, 0.0))


def softcap(z, cap):
    return cap * np.tanh(z / cap) if cap else z


def frequencies(rot):
    """Wavelengths below original/high keep their frequency, those above original/low are slowed
    by factor, the ones between blend linearly in original/wavelength."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = []
    sc = rot.get("scaling")
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            length = 2.0 * math.pi / f
            n, lo, hi = float(sc["original"]), float(sc["low"]), float(sc["high"])
            slow = f / float(sc["factor"])
            if length > n / lo:
                f = slow
            elif length >= n / hi:
                s = (n / length - lo) / (hi - lo)
                f = (1.0 - s) * slow + s * f
        out.append(f)
    return out


def rotate(v, pos, rot):
    """Turns entries (i, i + dims/2) of one head by pos * f_i."""
    if not rot or not int(rot.get("dims", 0)):
        return v
    half = int(rot["dims"]) // 2
    out = v.copy()
    for i, f in enumerate(frequencies(rot)):
        c, s = math.cos(pos * f), math.sin(pos * f)
        out[i] = v[i] * c - v[i + half] * s
        out[i + half] = v[i + half] * c + v[i] * s
    return out


def short_conv(u, w):
    """u: projected rows [T][C] of one sequence; w [C, taps], newest token last."""
    taps = w.shape[1]
    out = []
    for t in range(len(u)):
        y = np.zeros(w.shape[0])
        for j in range(taps):
            p = t - taps + 1 + j
            if p >= 0:
                y = y + w[:, j] * u[p]
        out.append(y)
    return out


def mix_values(v, v_first, lam):
    return (1.0 - lam) * v + lam * v_first


def softmax_weights(q, keys, scale, cap=0.0):
    s = softcap(np.array([float(q @ k) for k in keys]) * scale, cap)
    e = np.exp(s - s.max())
    return e / e.sum()


def talk(weights, T):
    """weights [H][keys] -> mixed across the heads."""
    H = len(weights)
    return [sum(T[h, g] * weights[g] for g in range(H)) for h in range(H)]


def attend(q, keys, values, scale, cap=0.0, T=None):
    """One query row: q [H][D]; keys [n][G][D], values [n][G][Dv] of the visible positions ->
    [H * Dv]."""
    H, G = len(q), len(keys[0])
    w = [softmax_weights(q[h], [k[h // (H // G)] for k in keys], scale, cap) for h in range(H)]
    if T is not None:
        w = talk(w, T)
    out = []
    for h in range(H):
        V = np.stack([v[h // (H // G)] for v in values])
        out.append(w[h] @ V)
    return np.concatenate(out)


def attention(h, W, p, m, eps, first, is_first, normed):
    """h: the mixer inputs of one sequence, [T][width] -> ([T][width], the layer's values)."""
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rot, cap = m.get("rot"), float(m.get("softcap") or 0.0)
    window = int((m.get("mask") or {}).get("size", 0))
    u = {n: [W[p + n] @ x for x in h] for n in ("q", "k", "v")}
    if m.get("conv"):
        for n in u:
            u[n] = short_conv(u[n], W[p + n + ".conv"])
    q, k, v = [], [], []
    for t in range(len(h)):
        qt = [rotate(x, t, rot) for x in u["q"][t].reshape(H, D)]
        kt = [rotate(x, t, rot) for x in u["k"][t].reshape(G, D)]
        if normed:
            qt, kt = [rms(x, eps) for x in qt], [rms(x, eps) for x in kt]
        vt = u["v"][t]
        if m.get("v_mix") and not is_first:
            vt = mix_values(vt, first[t], float(W[p + "vmix"]))
        q.append(qt)
        k.append(kt)
        v.append(vt.reshape(G, Dv))
    out = []
    for t in range(len(h)):
        lo = max(0, t - window + 1) if window else 0
        a = attend(q[t], k[lo:t + 1], v[lo:t + 1], float(m["scale"]), cap, W.get(p + "talk"))
        out.append(W[p + "o"] @ a)
    return out, [x.reshape(-1) for x in v]


def gla_core(q, k, v, alpha, S):
    """One token of one head: (output [vdim], new state [dim, vdim])."""
    S = alpha[:, None] * S + np.outer(k, v)
    return S.T @ q, S


def gla(h, W, p, m, eps):
    H, D, Dv, tau = m["heads"], m["dim"], m["vdim"], float(m["tau"])
    S = [np.zeros((D, Dv)) for _ in range(H)]
    out = []
    for x in h:
        q = (W[p + "q"] @ x * D ** -0.5).reshape(H, D)
        k, v = (W[p + "k"] @ x).reshape(H, D), (W[p + "v"] @ x).reshape(H, Dv)
        z = W[p + "a2"] @ (W[p + "a1"] @ x) + W[p + "a2.b"]
        alpha = np.exp(logsigmoid(z) / tau).reshape(H, D)
        o = []
        for a in range(H):
            r, S[a] = gla_core(q[a], k[a], v[a], alpha[a], S[a])
            o.append(rms(r, eps) * W[p + "norm"])
        out.append(W[p + "o"] @ (np.concatenate(o) * silu(W[p + "g"] @ x)))
    return out


def dense_ff(x, W, p):
    return W[p + "down"] @ (gelu_tanh(W[p + "gate"] @ x) * (W[p + "up"] @ x))


def token_side(x, e, W, p, eps):
    g = gelu_tanh(W[p + "gate"] @ x) * e
    return x + rms(W[p + "proj"] @ g, eps) * W[p + "norm"]


def forward(cfg, W, tokens, collect=None):
    """Logits [T, vocab] of one sequence; ``collect`` receives the residual after every layer."""
    eps = float((cfg.get("norm") or {}).get("eps", 1e-6))
    side = int((cfg.get("token_side") or {}).get("dim", 0))
    x = [W["embed"][t].copy() for t in tokens]
    first, seen = None, False
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = [rms(r, eps) * W[p + "norm1"] for r in x]
        if L["type"] == "gla":
            y = gla(h, W, p + "mix.", m, eps)
        else:
            is_first = bool(m.get("v_mix")) and not seen
            y, v = attention(h, W, p + "mix.", m, eps, first, is_first, L["type"] == "attention_2")
            if is_first:
                first, seen = v, True
        for t in range(len(x)):
            d = y[t] * sigmoid(W[p + "rg1"] @ h[t] + W[p + "rg1.b"])
            if L.get("mlp"):
                d = d + dense_ff(h[t], W, p + "mlp.") * sigmoid(W[p + "rg2"] @ h[t] + W[p + "rg2.b"])
            x[t] = x[t] + d
            if side:
                e = W["side.embed"][tokens[t], i * side:(i + 1) * side]
                x[t] = token_side(x[t], e, W, p + "side.", eps)
        if collect is not None:
            collect.append(np.stack(x))
    return np.stack([softcap(W["embed"] @ (rms(r, eps) * W["final.norm"]),
                             float(cfg.get("logit_softcap") or 0.0)) for r in x])
