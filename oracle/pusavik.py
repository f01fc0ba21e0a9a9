"""Plain float64 statement of the Pusavik layers, one function per mechanism, token by token where the mechanism is a
recurrence.  Test infrastructure only: it shares no code with the product path and is written for reading, not speed.

Weights are a dict name -> float64 array in the checkpoint's names; `cfg` is the parsed config.json.
"""
from __future__ import annotations

import numpy as np


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def silu(z):
    return z / (1.0 + np.exp(-z))


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def rotate_half(v, positions, base, dims):
    """v [..., T, d]: the first `dims` of the last axis rotated, element i paired with i + dims / 2."""
    half = dims // 2
    f = base ** (-2.0 * np.arange(half) / dims)
    a = np.asarray(positions, np.float64)[:, None] * f[None, :]
    out = v.copy()
    u, w = v[..., :half], v[..., half:dims]
    out[..., :half] = u * np.cos(a) - w * np.sin(a)
    out[..., half:dims] = w * np.cos(a) + u * np.sin(a)
    return out


def window_sees(i, j, size):
    return 0 <= i - j < size


def sink_softmax(scores, sink):
    """Weights of one query over its visible keys; the sink enters the denominator only."""
    top = max(float(np.max(scores)), float(sink))
    e = np.exp(scores - top)
    return e / (e.sum() + np.exp(sink - top))


def latent_attention(h, w, p, m, eps):
    """h [T, width] of one sequence from position 0 -> [T, width]."""
    T, H = h.shape[0], m["heads"]
    dim, rd, vd, rank, size = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["mask"]["size"]
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (cq @ w[p + "uq"].T).reshape(T, H, dim + rd)
    kv = h @ w[p + "dkv"].T
    c, kr = rms_norm(kv[:, :rank], w[p + "dkv.norm"], eps), kv[:, rank:]
    pos = np.arange(T)
    kr = rotate_half(kr, pos, m["rot"]["base"], m["rot"]["dims"])
    k = (c @ w[p + "uk"].T).reshape(T, H, dim)
    v = (c @ w[p + "uv"].T).reshape(T, H, vd)
    out = np.zeros((T, H, vd))
    for n in range(H):
        qn, qr = q[:, n, :dim], rotate_half(q[:, n, dim:], pos, m["rot"]["base"], m["rot"]["dims"])
        for i in range(T):
            j0 = max(0, i - size + 1)
            s = (k[j0:i + 1, n] @ qn[i] + kr[j0:i + 1] @ qr[i]) * m["scale"]
            out[i, n] = sink_softmax(s, w[p + "sink"][n]) @ v[j0:i + 1, n]
    return out.reshape(T, H * vd) @ w[p + "o"].T


def causal_conv(x, w, b):
    """x [T, channels], w [channels, taps]: the last tap meets the current row, zeros before the first."""
    T, taps = x.shape[0], w.shape[1]
    y = np.zeros_like(x)
    for t in range(T):
        for k in range(taps):
            s = t - (taps - 1) + k
            if s >= 0:
                y[t] += w[:, k] * x[s]
    return y + b


def ssd_recurrence(x, B, C, dt, A_log, D):
    """x [T, H, P], B / C [T, H, N] (already per head), dt [T, H] -> y [T, H, P]; one state [N, P] per head."""
    T, H, P = x.shape
    S = np.zeros((H, B.shape[2], P))
    y = np.zeros_like(x)
    for t in range(T):
        decay = np.exp(-np.exp(A_log) * dt[t])
        for n in range(H):
            S[n] = decay[n] * S[n] + dt[t, n] * np.outer(B[t, n], x[t, n])
            y[t, n] = S[n].T @ C[t, n] + D[n] * x[t, n]
    return y


def gated_group_norm(y, z, w, groups, eps):
    g = (y * silu(z)).reshape(y.shape[0], groups, -1)
    g = g / np.sqrt(np.mean(g * g, axis=-1, keepdims=True) + eps)
    return g.reshape(y.shape) * w


def mamba2(h, w, p, m, eps):
    T, H, P, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    u = h @ w[p + "in"].T
    z, xbc, dt = u[:, :inner], u[:, inner:2 * inner + 2 * G * N], u[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x = xbc[:, :inner].reshape(T, H, P)
    group_of = np.arange(H) // (H // G)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)[:, group_of]
    C = xbc[:, inner + G * N:].reshape(T, G, N)[:, group_of]
    y = ssd_recurrence(x, B, C, softplus(dt + w[p + "dt_bias"]), w[p + "A_log"], w[p + "D"])
    return gated_group_norm(y.reshape(T, inner), z, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


def route(z, correction, top):
    """(indices, weights) of one token: chosen by corrected softmax score, weighted by the uncorrected one."""
    s = np.exp(z - z.max())
    s /= s.sum()
    idx = np.argsort(-(s + correction), kind="stable")[:top]
    wt = s[idx]
    return idx, wt / (wt.sum() + 1e-20)


def moe(h, w, p, m):
    experts, top = m["router"]["experts"], m["router"]["top"]
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        idx, wt = route(w[p + "router"] @ h[t], w[p + "correction"], top)
        for e, g in zip(idx, wt):
            if e >= experts:
                out[t] += g * h[t]           # identity expert
            else:
                q = f"{p}e{e}."
                out[t] += g * (w[q + "down"] @ (silu(w[q + "gate"] @ h[t]) * (w[q + "up"] @ h[t])))
    return out


def layer_runs(cfg):
    """(layer, first-of-pass number or None) in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, w, tokens):
    """(logits [T, vocab], residual stream after every layer run) of one sequence."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    after = []
    for i, step in layer_runs(cfg):
        if step is not None:
            x = x + w["loop.step"][step]
        ly, p = cfg["layers"][i], f"l{i}."
        mixer = {"latent_attention": latent_attention, "mamba2": mamba2}[ly["type"]]
        y = mixer(rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", ly["mixer"], eps)
        if ly.get("mlp"):
            y = y + moe(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", ly["mlp"])
        x = x + y
        after.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T, after
