"""A plain, slow float64 implementation of the Felavik design, written from its equations: one function
per mechanism, whole sequences, loops over tokens and heads, numpy only.  It shares no code with the
package: the tests compare the framework's kernels, cache and scheduler against it.

A model is (``cfg``: the design's ``config.json`` dict, ``w``: checkpoint name -> float64 array).

Notation: h [T, W] a sublayer's input, i / j query / key positions, n = i - j.
"""
import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, -1, keepdims=True) + eps)


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def softmax(z):
    e = np.exp(z - np.max(z, -1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


# --------------------------------------------------------------------------- attention
def bucket(n, rows, far):
    """The bias row of distance n: one row per distance up to rows / 2, then rows that widen with the logarithm of
    the distance until ``far``; everything behind shares the last one."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half) + 1e-12))


def temperature(p, t):
    return 1.0 + t["coef"] * math.log((p + 1) // t["every"] + 1)


def attention_heads(h, w, p, m, eps):
    """The gated heads side by side [T, H vdim], before the output projection."""
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, D), eps) * w[p + "q.norm"]
    k = rms((h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, D), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, Dv)
    rel = w[p + "rel"]
    bias = np.stack([rel[bucket(n, rel.shape[0], m["bias_max"])] for n in range(T)])       # [distance, head]
    out = np.zeros((T, H, Dv))
    for i in range(T):
        for hh in range(H):
            g = hh // (H // G)
            s = (k[:i + 1, g] @ (q[i, hh] * temperature(i, m["q_temp"]))) * m["scale"]
            out[i, hh] = softmax(s + bias[i::-1, hh]) @ v[:i + 1, g]
    return out.reshape(T, H * Dv) * sigmoid(h @ w[p + "g"].T)


def attention(h, w, p, m, eps):
    return attention_heads(h, w, p, m, eps) @ w[p + "o"].T


# --------------------------------------------------------------------------- linear attention with fixed decays
def turn_halves(x, pos, dims, base):
    """coordinates (i, i + dims / 2), i < dims / 2, of the vector x turned by pos * base^(-2 i / dims)."""
    y = np.array(x, dtype=np.float64)
    half = dims // 2
    for i in range(half):
        a = pos * base ** (-2.0 * i / dims)
        u, v = x[i], x[i + half]
        y[i] = u * math.cos(a) - v * math.sin(a)
        y[i + half] = v * math.cos(a) + u * math.sin(a)
    return y


def recurrence(q, k, v, decay, S=None):
    """q / k [T, H, N], v [T, H, P], decay [H] -> (o [T, H, P], the state after the last token [H, N, P])."""
    T, H, N = q.shape
    S = np.zeros((H, N, v.shape[2])) if S is None else np.array(S)
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for hh in range(H):
            S[hh] = decay[hh] * S[hh] + np.outer(k[t, hh], v[t, hh])
            o[t, hh] = S[hh].T @ q[t, hh]
    return o, S


def retention_inputs(h, w, p, m):
    T, H, N, P = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = (h @ w[p + "q"].T).reshape(T, H, N), (h @ w[p + "k"].T).reshape(T, H, N)
    r = m["rot"]
    turn = lambda x: np.stack([[turn_halves(x[t, hh], t, r["dims"], r["base"]) for hh in range(H)] for t in range(T)])
    return turn(q), turn(k) * N ** -0.5, (h @ w[p + "v"].T).reshape(T, H, P)


def retention(h, w, p, m, eps):
    o, _ = recurrence(*retention_inputs(h, w, p, m), m["decay"])
    return (rms(o, eps).reshape(h.shape[0], -1) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def lightning_inputs(h, w, p, m):
    T, H, N, P = h.shape[0], m["heads"], m["dim"], m["vdim"]
    return (silu(h @ w[p + "q"].T).reshape(T, H, N), silu(h @ w[p + "k"].T).reshape(T, H, N), silu(h @ w[p + "v"].T).reshape(T, H, P))


def lightning(h, w, p, m, eps):
    o, _ = recurrence(*lightning_inputs(h, w, p, m), m["decay"])
    o = rms(o.reshape(h.shape[0], -1), eps) * w[p + "norm"]
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h, w, p, m, eps):
    return m["left_scale"] * attention(h, w, p + "left.", m["left"], eps) + m["right_scale"] * retention(h, w, p + "right.", m["right"], eps)


# --------------------------------------------------------------------------- experts
def choose(s, top, count=1, keep=1):
    """The experts one token uses, best first: the ``top`` largest scores among the experts of the ``keep`` best
    of ``count`` equal groups of neighbours (a group is as good as its best expert)."""
    E = len(s)
    size = E // count
    best = sorted(range(count), key=lambda g: (-max(s[g * size:(g + 1) * size]), g))[:keep]
    open_ = [e for e in range(E) if e // size in best]
    return sorted(open_, key=lambda e: (-s[e], e))[:top]


def route(h, w, p, r):
    s = softmax(h @ w[p + "router"].T)
    g = r.get("groups") or {"count": 1, "keep": 1}
    idx = np.array([choose(row, r["top"], g["count"], g["keep"]) for row in s])
    wt = np.take_along_axis(s, idx, -1)
    return idx, wt / (wt.sum(-1, keepdims=True) + 1e-20)


def experts(h, w, p, mlp):
    idx, wt = route(h, w, p, mlp["router"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(idx[t], wt[t]):
            out[t] += g * ((silu(h[t] @ w[f"{p}e{e}.gate"].T) * (h[t] @ w[f"{p}e{e}.up"].T)) @ w[f"{p}e{e}.down"].T)
    return out


# --------------------------------------------------------------------------- the model
def owner(cfg, i):
    """The layer whose tensors layer i runs on."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def layer(x, w, cfg, i):
    l, p, eps = cfg["layers"][i], f"l{owner(cfg, i)}.", cfg["norm"]["eps"]
    mixer = {"parallel": parallel, "lightning": lightning}[l["type"]]
    x = x + mixer(rms(x, eps) * w[p + "norm1"], w, p + "mix.", l["mixer"], eps)
    if l.get("mlp"):
        x = x + experts(rms(x, eps) * w[p + "norm2"], w, p + "mlp.", l["mlp"])
    return x


def forward(cfg, w, tokens):
    """-> (logits [T, vocab], the stream after every layer [layers, T, W])."""
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    taps = []
    for i in range(len(cfg["layers"])):
        x = layer(x, w, cfg, i)
        taps.append(x)
    z = (rms(x, cfg["norm"]["eps"]) * w["final.norm"]) @ w["head"].T
    cap = cfg["logit_softcap"]
    return cap * np.tanh(z / cap), np.stack(taps)
