"""A plain, slow float64 implementation of the Numizen design, written from its equations: one
function per mechanism, whole sequences, loops over tokens and heads, numpy only.  It shares no code
with the package: the tests compare the framework's kernels, cache and scheduler against it.

A model is (``cfg``: the design's ``config.json`` dict, ``w``: checkpoint name -> float64 array).

Notation: h [T, W] a sublayer's input, i / j query / key positions.
"""
import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, -1, keepdims=True) + eps)


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def softmax(z):
    e = np.exp(z - np.max(z, -1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu2(z):
    return np.maximum(z, 0.0) ** 2


def dynamic_tanh(x, w, name):
    """tanh(alpha x) weight + bias: no statistics."""
    return np.tanh(float(w[name + ".alpha"]) * x) * w[name] + w[name + ".b"]


# --------------------------------------------------------------------------- latent attention
def turn_pairs(x, pos, dims, base):
    """coordinates (2 m, 2 m + 1), m < dims / 2, of the vector x turned by pos * base^(-2 m / dims)."""
    y = np.array(x, dtype=np.float64)
    for m in range(dims // 2):
        a = pos * base ** (-2.0 * m / dims)
        u, v = x[2 * m], x[2 * m + 1]
        y[2 * m] = u * math.cos(a) - v * math.sin(a)
        y[2 * m + 1] = v * math.cos(a) + u * math.sin(a)
    return y


def latent_attention(h, w, p, m, eps):
    """``p``: tensor prefix ('l3.mix.'), ``m``: the mixer's config entry."""
    T = h.shape[0]
    H, D, R, Dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    q = ((rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]) @ w[p + "uq"].T).reshape(T, H, D + R)
    d = h @ w[p + "dkv"].T
    c = rms(d[:, :rank], eps) * w[p + "dkv.norm"]
    shared = np.stack([turn_pairs(d[t, rank:], t, rot["dims"], rot["base"]) for t in range(T)])
    k = (c @ w[p + "uk"].T).reshape(T, H, D)
    v = (c @ w[p + "uv"].T).reshape(T, H, Dv)
    out = np.zeros((T, H, Dv))
    for i in range(T):
        for hh in range(H):
            qr = turn_pairs(q[i, hh, D:], i, rot["dims"], rot["base"])
            s = (k[:i + 1, hh] @ q[i, hh, :D] + shared[:i + 1] @ qr) * m["scale"]
            out[i, hh] = softmax(s) @ v[:i + 1, hh]
    out = out.reshape(T, H * Dv)
    if p + "g" in w:
        out = out * sigmoid(h @ w[p + "g"].T)
    return out @ w[p + "o"].T


# --------------------------------------------------------------------------- gated linear attention
def gla_decays(h, w, p, m):
    """alpha [T, H, dim] = sigmoid(W_a2 W_a1 h + b)^(1 / tau)."""
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    return (sigmoid(z) ** (1.0 / m["tau"])).reshape(h.shape[0], m["heads"], m["dim"])


def gla_recurrence(q, k, v, alpha, S=None):
    """q / k / alpha [T, H, N], v [T, H, P] -> (o [T, H, P], the state after the last token [H, N, P])."""
    T, H, N = q.shape
    S = np.zeros((H, N, v.shape[2])) if S is None else np.array(S)
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for hh in range(H):
            S[hh] = alpha[t, hh][:, None] * S[hh] + np.outer(k[t, hh], v[t, hh])
            o[t, hh] = S[hh].T @ q[t, hh]
    return o, S


def gla(h, w, p, m, eps):
    T, H, N, P = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, N) * N ** -0.5
    k = (h @ w[p + "k"].T).reshape(T, H, N)
    v = (h @ w[p + "v"].T).reshape(T, H, P)
    o, _ = gla_recurrence(q, k, v, gla_decays(h, w, p, m))
    o = (rms(o, eps) * w[p + "norm"]).reshape(T, H * P)
    g = h @ w[p + "g"].T
    return (o * (g * sigmoid(g))) @ w[p + "o"].T


# --------------------------------------------------------------------------- feed-forwards
def dense_ff(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def choose(s, correction, top, count=1, keep=1):
    """The experts one token uses, best first: the ``top`` largest of s + correction among the experts of
    the ``keep`` best of ``count`` equal groups of neighbours (a group is as good as its best expert)."""
    c = s + correction
    E = len(s)
    size = E // count
    best = sorted(range(count), key=lambda g: (-max(c[g * size:(g + 1) * size]), g))[:keep]
    open_ = [e for e in range(E) if e // size in best]
    return sorted(open_, key=lambda e: (-c[e], e))[:top]


def route(h, w, p, r):
    """(chosen experts [T, top], their weights): scores softmax(W h); chosen by score + correction, weighted
    by the scores alone, over their sum."""
    s = softmax(h @ w[p + "router"].T)
    corr = w.get(p + "correction", np.zeros(s.shape[1]))
    g = r.get("groups") or {"count": 1, "keep": 1}
    idx = np.array([choose(row, corr, r["top"], g["count"], g["keep"]) for row in s])
    wt = np.take_along_axis(s, idx, -1)
    return idx, wt / (wt.sum(-1, keepdims=True) + 1e-20)


def moe_ff(h, w, p, mlp):
    idx, wt = route(h, w, p, mlp["router"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(idx[t], wt[t]):
            out[t] += g * (relu2(h[t] @ w[f"{p}e{e}.up"].T) @ w[f"{p}e{e}.down"].T)
    if mlp.get("shared"):
        y = relu2(h @ w[p + "shared.up"].T) @ w[p + "shared.down"].T
        if p + "shared.sg" in w:
            y = y * sigmoid(h @ w[p + "shared.sg"].T)
        out = out + y
    return out


# --------------------------------------------------------------------------- the model
def layer(x, w, cfg, i):
    l, p, eps = cfg["layers"][i], f"l{i}.", cfg["norm"]["eps"]
    mixer = {"latent_attention": latent_attention, "gla": gla}[l["type"]]
    y = mixer(dynamic_tanh(x, w, p + "norm1"), w, p + "mix.", l["mixer"], eps) * w[p + "ls1"]
    mlp = l.get("mlp")
    if mlp:
        h = dynamic_tanh(x, w, p + "norm2")
        f = dense_ff(h, w, p + "mlp.") if mlp["kind"] == "dense" else moe_ff(h, w, p + "mlp.", mlp)
        y = y + f * w[p + "ls2"]
    return x + y


def run_order(cfg):
    n, lp = len(cfg["layers"]), cfg.get("loop") or {"start": 0, "stop": 0, "times": 0}
    return list(range(lp["start"])) + list(range(lp["start"], lp["stop"])) * lp["times"] + list(range(lp["stop"], n))


def forward(cfg, w, tokens):
    """-> (logits [T, vocab], the stream after every layer run [runs, T, W])."""
    x = w["embed"][np.asarray(tokens)] + w["pos"][:len(tokens)]
    taps = []
    for i in run_order(cfg):
        x = layer(x, w, cfg, i)
        taps.append(x)
    return dynamic_tanh(x, w, "final.norm") @ w["head"].T, np.stack(taps)
