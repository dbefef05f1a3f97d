"""Plain float64 implementation of the Vugelix design, written from its equations: loops over
tokens, heads and keys, one function per mechanism, no code shared with the framework.

Every layer is a mixer and an optional feed-forward joined to several residual streams by
hyper-connections.  The mixer runs two cores on the same input and adds their outputs with fixed
factors: a windowed grouped-query attention (partial half-split rotation, soft-capped scores, one
extra unit in the softmax denominator, a sigmoid gate per head) and a gated delta rule (short
convolutions over time, unit-length queries and keys, a decay and a step size per head, head RMS
norm, SiLU gate).  The feed-forward is an ungated squared-ReLU block.  A layer may run on the
tensors of another one.  ``W`` maps the checkpoint's tensor names to float64 arrays.
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


def softplus(z):
    return math.log1p(math.exp(-abs(z))) + max(z, 0.0)


def frequencies(rot):
    n, base = int(rot["dims"]), float(rot["base"])
    return [base ** (-2.0 * i / n) for i in range(n // 2)]


def rotate(v, pos, rot):
    """Turns entries (i, i + dims/2) of one head by pos * f_i; entries past dims stay."""
    if not rot or not int(rot.get("dims", 0)):
        return v
    half = int(rot["dims"]) // 2
    out = v.copy()
    for i, f in enumerate(frequencies(rot)):
        c, s = math.cos(pos * f), math.sin(pos * f)
        out[i] = v[i] * c - v[i + half] * s
        out[i + half] = v[i + half] * c + v[i] * s
    return out


# ------------------------------------------------------------------ left: windowed attention

def soft_cap(s, cap):
    return cap * math.tanh(s / cap) if cap else s


def off_by_one_attention(q, keys, vals, scale, cap):
    """One query of one head over its visible keys; the denominator holds 1 + sum exp(s)."""
    s = [soft_cap(float(q @ k) * scale, cap) for k in keys]
    top = max(s + [0.0])
    den = math.exp(-top) + sum(math.exp(x - top) for x in s)
    return sum(math.exp(x - top) * v for x, v in zip(s, vals)) / den


def window_mixer(hs, W, pre, m):
    H, G, D, Dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    size = int((m.get("mask") or {}).get("size", 0))
    ks, vs, out = [], [], []
    for t, h in enumerate(hs):
        q = (W[pre + "q"] @ h).reshape(H, D)
        k = (W[pre + "k"] @ h).reshape(G, D)
        ks.append([rotate(k[g], t, m.get("rot")) for g in range(G)])
        vs.append((W[pre + "v"] @ h).reshape(G, Dv))
        gate = sigmoid(W[pre + "g"] @ h)
        first = max(0, t - size + 1) if size else 0
        o = np.zeros((H, Dv))
        for a in range(H):
            g = a // (H // G)
            o[a] = gate[a] * off_by_one_attention(
                rotate(q[a], t, m.get("rot")), [ks[j][g] for j in range(first, t + 1)],
                [vs[j][g] for j in range(first, t + 1)], float(m["scale"]),
                float(m.get("softcap") or 0.0))
        out.append(W[pre + "o"] @ o.reshape(-1))
    return out


# ------------------------------------------------------------------ right: gated delta rule

def short_conv(us, w):
    """us: projected vectors token by token; w [channels, taps], newest token last -> silu of the
    filtered vectors (zeros ahead of the sequence)."""
    n = w.shape[1]
    out = []
    for t in range(len(us)):
        y = np.zeros_like(us[t])
        for lag in range(n):
            if t - lag >= 0:
                y = y + w[:, n - 1 - lag] * us[t - lag]
        out.append(silu(y))
    return out


def unit(x):
    return x / math.sqrt(float(np.sum(x * x)) + 1e-6)


def delta_core(q, k, v, decay, beta, S):
    """One token of one head: the decayed state's answer to k moves towards v by beta."""
    S = decay * S
    S = S + np.outer(k, beta * (v - S.T @ k))
    return S.T @ q, S


def delta_mixer(hs, W, pre, m, eps):
    H, G, D, Dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    qs = short_conv([W[pre + "q"] @ h for h in hs], W[pre + "q.conv"])
    ks = short_conv([W[pre + "k"] @ h for h in hs], W[pre + "k.conv"])
    vs = short_conv([W[pre + "v"] @ h for h in hs], W[pre + "v.conv"])
    S = [np.zeros((D, Dv)) for _ in range(H)]
    out = []
    for t, h in enumerate(hs):
        q, k, v = qs[t].reshape(G, D), ks[t].reshape(G, D), vs[t].reshape(H, Dv)
        beta = sigmoid(W[pre + "b"] @ h)
        z = W[pre + "a"] @ h + W[pre + "dt_bias"]
        o = np.zeros((H, Dv))
        for a in range(H):
            g = a // (H // G)
            decay = math.exp(-math.exp(float(W[pre + "A_log"][a])) * softplus(float(z[a])))
            y, S[a] = delta_core(unit(q[g]) * D ** -0.5, unit(k[g]), v[a], decay, float(beta[a]),
                                 S[a])
            o[a] = rms(y, eps) * W[pre + "norm"]
        out.append(W[pre + "o"] @ (o.reshape(-1) * silu(W[pre + "g"] @ h)))
    return out


def parallel_mixer(hs, W, pre, m, eps):
    a = window_mixer(hs, W, pre + "left.", m["left"])
    b = delta_mixer(hs, W, pre + "right.", m["right"], eps)
    return [float(m["left_scale"]) * x + float(m["right_scale"]) * y for x, y in zip(a, b)]


# ------------------------------------------------------------------ layers

def relu2_block(h, W, pre):
    return W[pre + "down"] @ (np.maximum(W[pre + "up"] @ h, 0.0) ** 2)


def owner(layers, i):
    """The layer whose tensors layer i runs on."""
    while layers[i].get("weights_of") is not None:
        i = int(layers[i]["weights_of"])
    return i


def forward(cfg, W, tokens, collect=None):
    """Logits [tokens, vocab] of one sequence.  ``collect`` receives the sum of the streams after
    every layer, [tokens, width] each."""
    eps, ns, T = float(cfg["norm"]["eps"]), int(cfg["streams"]), len(tokens)
    scale = float((cfg.get("embedding") or {}).get("scale", 1.0))
    X = [[W["embed"][tok] * scale for _ in range(ns)] for tok in tokens]

    def sublayer(q, p, fn):
        read, write, mix = (W[f"{p}hc{q}.{n}"] for n in ("in", "out", "mix"))
        ys = fn([rms(sum(read[s] * X[t][s] for s in range(ns)), eps) * W[f"{p}norm{q}"]
                 for t in range(T)])
        for t in range(T):
            X[t] = [sum(mix[s, j] * X[t][s] for s in range(ns)) + write[j] * ys[t]
                    for j in range(ns)]

    for i, L in enumerate(cfg["layers"]):
        p = f"l{owner(cfg['layers'], i)}."
        sublayer(1, p, lambda hs: parallel_mixer(hs, W, p + "mix.", L["mixer"], eps))
        if L.get("mlp"):
            sublayer(2, p, lambda hs: [relu2_block(h, W, p + "mlp.") for h in hs])
        if collect is not None:
            collect.append(np.stack([sum(X[t]) for t in range(T)]))
    return np.stack([W["embed"] @ (rms(sum(X[t]), eps) * W["final.norm"])
                     for t in range(T)]) * float(cfg.get("logit_scale", 1.0))
