"""Plain float64 statement of the Fumotar layers, one function per mechanism, token by token where the mechanism is a
recurrence.  Test infrastructure only: it shares no code with the product path and is written for reading, not speed.

Weights are a dict name -> float64 array in the checkpoint's names; `cfg` is the parsed config.json.
"""
from __future__ import annotations

import numpy as np

from .pusavik import causal_conv, layer_runs, rms_norm, silu, softplus


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def relu2(z):
    return np.maximum(z, 0.0) ** 2


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * w + b


def bigram_rows(tokens, mul_prev, mul_cur, buckets):
    """Row of the second table per token: a hash of the token and the one before it, the last row for the first token."""
    return [buckets] + [(int(a) * mul_prev + int(b) * mul_cur) % buckets for a, b in zip(tokens, tokens[1:])]


def embedding(cfg, w, tokens):
    x = w["embed"][np.asarray(tokens)]
    g = (cfg.get("embedding") or {}).get("bigram")
    if g:
        x = x + w["bigram"][bigram_rows(list(tokens), g["mul_prev"], g["mul_cur"], g["buckets"])]
    return x


# ---- attention ----

def rot_frequencies(rot):
    """(radians per position of every pair, factor of cos and sin), with the frequencies stretched where `scaling` says so."""
    dims, base = rot["dims"], rot["base"]
    f = base ** (-2.0 * np.arange(dims // 2) / dims)
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def dim(turns):
        return dims * np.log(s["original"] / (2.0 * np.pi * turns)) / (2.0 * np.log(base))

    lo, hi = max(np.floor(dim(s["fast"])), 0.0), min(np.ceil(dim(s["slow"])), dims - 1.0)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * np.log(s["factor"]) + 1.0


def rotate(x, rot):
    """x [T, heads, dim] from position 0: pairs (i, i + dims / 2) of the first `dims` elements."""
    f, mag = rot_frequencies(rot)
    half, dims = rot["dims"] // 2, rot["dims"]
    a = np.arange(x.shape[0], dtype=np.float64)[:, None, None] * f
    c, s = np.cos(a) * mag, np.sin(a) * mag
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def attention(h, w, p, m, eps):
    """h [T, width] from position 0: causal attention whose values are the unnormalised, unrotated keys."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = h @ w[p + "q"].T, h @ w[p + "k"].T
    v = k.reshape(T, G, D)
    q = rotate(rms_norm(q, w[p + "q.norm"], eps).reshape(T, H, D), m["rot"])
    k = rotate(rms_norm(k, w[p + "k.norm"], eps).reshape(T, G, D), m["rot"])
    out = np.zeros((T, H, D))
    for n in range(H):
        g = n // (H // G)
        s = q[:, n] @ k[:, g].T * m["scale"]
        s[np.triu_indices(T, 1)] = -np.inf
        e = np.exp(s - s.max(-1, keepdims=True))
        out[:, n] = e / e.sum(-1, keepdims=True) @ v[:, g]
    return out.reshape(T, H * D) @ w[p + "o"].T


# ---- gated delta rule, one decay per key channel ----

def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def delta_decay(h, w, p, heads, dim):
    """log of the decay [T, heads, dim]."""
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    return -np.exp(w[p + "A_log"])[:, None] * softplus(z).reshape(-1, heads, dim)


def delta_recurrence(q, k, v, beta, log_g):
    """q, k, log_g [T, H, K], v [T, H, V], beta [T, H] -> o [T, H, V]; one state [K, V] per head, from zero."""
    T, H, K = k.shape
    S = np.zeros((H, K, v.shape[2]))
    o = np.zeros_like(v)
    for t in range(T):
        S = np.exp(log_g[t])[:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hkv,hk->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hkv,hk->hv", S, q[t])
    return o


def channel_delta(h, w, p, m, eps):
    T, H, G, K, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"], 0.0)) for n in "qkv")
    of = np.arange(H) // (H // G)
    q = unit(q.reshape(T, G, K))[:, of] * K ** -0.5
    k = unit(k.reshape(T, G, K))[:, of]
    o = delta_recurrence(q, k, v.reshape(T, H, V), sigmoid(h @ w[p + "b"].T), delta_decay(h, w, p, H, K))
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).reshape(T, H, V)
    return (rms_norm(o, w[p + "norm"], eps) * gate).reshape(T, H * V) @ w[p + "o"].T


# ---- real-gated linear recurrent unit ----

def block_product(u, a, b):
    """u [T, blocks * n], a [blocks, n, n] (out, in), b [blocks, n]."""
    T, B, n = u.shape[0], a.shape[0], a.shape[1]
    return np.stack([u.reshape(T, B, n)[:, i] @ a[i].T + b[i] for i in range(B)], 1).reshape(T, B * n)


def gated_recurrence(u, r, i, lam):
    """u, r, i [T, width], lam [width] -> the state after every token, from zero."""
    log_a = -8.0 * r * softplus(lam)
    S, out = np.zeros(u.shape[1]), np.zeros_like(u)
    for t in range(u.shape[0]):
        S = np.exp(log_a[t]) * S + np.sqrt(-np.expm1(2.0 * log_a[t])) * i[t] * u[t]
        out[t] = S
    return out


def rglru(h, w, p, m, eps):
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u = causal_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"], w[p + "conv.b"])
    r, i = (sigmoid(block_product(u, w[p + n], w[p + n + ".b"])) for n in ("ra", "ri"))
    return (gated_recurrence(u, r, i, w[p + "lam"]) * y) @ w[p + "o"].T


MIXERS = {"attention": attention, "channel_delta": channel_delta, "rglru": rglru}


def forward(cfg, w, tokens):
    """(logits [T, vocab], residual stream after every layer run) of one sequence."""
    eps = cfg["norm"]["eps"]
    x0 = x = embedding(cfg, w, tokens)
    after = []
    for i, first in layer_runs(cfg):
        if first is not None:
            x = np.concatenate([x, x0], -1) @ w["loop.in"].T
        ly, p = cfg["layers"][i], f"l{i}."
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        y = MIXERS[ly["type"]](h, w, p + "mix.", ly["mixer"], eps)
        if ly.get("mlp"):
            y = y + relu2(h @ w[p + "mlp.up"].T) @ w[p + "mlp.down"].T
        x = x + y
        after.append(x)
    return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["embed"].T, after
