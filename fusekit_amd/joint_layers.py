"""Layers of the layer-list decoder whose mixer and dense feed-forward read ONE norm: everything that reads it is one
product, everything that leaves the layer another.

A joint layer's input projection writes a row `u` = [parts of the mixer .. | up], its epilogue applying biases and
activations per range of columns.  The mixer leaves its result in the place of its last part, directly ahead of `up`, so
the output projection and the down projection are one product over adjacent columns.  Heads and blocks are padded with
zero rows of the matrices, so padding columns are zeros in every row and no kernel has a tail.

Mixers: causal attention with grouped queries whose values are the unnormalised keys, a gated delta rule with one decay
per key channel, and a real-gated linear recurrent unit.  The design that uses them today is Fumotar.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Callable, Dict, List, Optional, Tuple

import numpy as np

from . import native
from .native import DeviceBuffer
from .runtime import Dispatch, arg

FN_RELU2, FN_GELU = 1, 2     # column functions of a product
LRU_CHUNK = 32
DELTA_ROWS = 16              # the recurrence goes in chunks from this many rows


def pad(n: int, to: int = 64) -> int:
    """Padded length of a row (kernels walk rows in whole blocks; the padding holds zeros)."""
    return -(-n // to) * to


# ---------------------------------------------------------------- configuration

@dataclass
class RotaryScaling:
    """Stretched rotation: frequencies of fewer than `slow` turns within `original` positions are divided by `factor`, those
    of more than `fast` turns stay, with a ramp between."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass
class CausalAttention:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    rot_base: float
    rot_dims: int
    rot_scaling: Optional[RotaryScaling] = None

    kind = "attention"
    out_part = "q"

    @property
    def vdim(self) -> int:
        return self.dim

    @property
    def dim_ld(self) -> int:
        return pad(self.dim) if self.dim <= 128 else pad(self.dim, 128)

    def parts(self) -> List[Tuple[str, int]]:
        return [("k", self.kv_heads * self.dim_ld), ("q", self.heads * self.dim_ld)]

    def rotation(self) -> Tuple[np.ndarray, float]:
        """Radians per position of every rotated pair, and the factor of cos and sin."""
        n, b = self.rot_dims, self.rot_base
        i = np.arange(n // 2, dtype=np.float64)
        f = np.float64(b) ** (-2.0 * i / max(n, 1))
        s = self.rot_scaling
        if s is None:
            return f, 1.0
        turns_at = lambda turns: n * math.log(s.original / (turns * 2.0 * math.pi)) / (2.0 * math.log(b))
        first, last = max(math.floor(turns_at(s.fast)), 0), min(math.ceil(turns_at(s.slow)), n - 1)
        ramp = np.clip((i - first) / max(last - first, 0.001), 0.0, 1.0)
        return f * (1.0 - ramp) + f / s.factor * ramp, 1.0 + 0.1 * math.log(s.factor)


@dataclass
class ChannelDelta:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int
    gate_rank: int

    kind = "channel_delta"
    out_part = "v"

    @property
    def dim_ld(self) -> int:
        return pad(self.dim, 32)

    @property
    def vdim_ld(self) -> int:
        return pad(self.vdim, 32)

    @property
    def state_ld(self) -> int:
        return pad(self.dim)

    @property
    def channels(self) -> int:
        """Convolved columns: queries | keys | values."""
        return 2 * self.kv_heads * self.dim_ld + self.heads * self.vdim_ld

    def parts(self) -> List[Tuple[str, int]]:
        qk = self.kv_heads * self.dim_ld
        return [("a1", pad(self.decay_rank)), ("g1", pad(self.gate_rank)), ("q", qk), ("k", qk), ("v", pad(self.heads * self.vdim_ld))]


@dataclass
class RgLru:
    width: int
    blocks: int
    conv: int

    kind = "rglru"
    out_part = "y"

    @property
    def heads(self) -> int:
        return self.blocks

    @property
    def vdim(self) -> int:
        return self.block

    @property
    def block(self) -> int:
        return self.width // self.blocks

    @property
    def block_ld(self) -> int:
        return pad(self.block)

    @property
    def inner(self) -> int:
        return self.blocks * self.block_ld

    def parts(self) -> List[Tuple[str, int]]:
        return [("x", self.inner), ("y", self.inner)]


@dataclass
class DenseMlp:
    ff: int


JOINT = ("attention", "channel_delta", "rglru")


class Columns:
    """Where the parts of a joint layer's row `u` lie."""

    def __init__(self, m, f: Optional[DenseMlp]):
        self.at: Dict[str, int] = {}
        self.width = 0
        for name, n in m.parts() + [("up", pad(f.ff) if f else 0)]:
            self.at[name] = self.width
            self.width += n
        self.tail = m.heads if m.kind == "channel_delta" else 0   # fp32 columns behind the row: step sizes
        self.rows = self.width + self.tail                         # rows of the joint input matrix
        self.out = self.at[m.out_part]
        self.ko = self.width - self.out                            # mixer's result and `up`
        self.up = self.at["up"]
        self.fns: Dict[str, int] = {}
        if f:
            self.fns = dict(fn=FN_RELU2, fn_begin=self.up, fn_end=self.width)
        if m.kind == "rglru":
            self.fns.update(fn2=FN_GELU, fn2_begin=self.out)
            if f:   # gelu up to `up`, relu^2 behind it
                self.fns = dict(fn=FN_GELU, fn_begin=self.out, fn_end=self.up, fn2=FN_RELU2, fn2_begin=self.up)


def out_parts(rows: int, n: int, k: int) -> int:
    """Parts of the sum that the product [rows, k] . [n, k] is formed in, side by side: a long sum over few output tiles would
    leave most compute units without work.  The rows form (8 rows or fewer) has a wave per column and needs none."""
    if rows <= 8:
        return 1
    tiles = -(-n // 64) * (1 if rows <= 32 else -(-rows // 64))
    want = 8 if rows <= 32 or tiles <= 64 else 4 if tiles <= 128 else 2 if tiles <= 256 else max(1, 2048 // tiles)
    return next(p for p in (8, 4, 2, 1) if p <= want and (p == 1 or (k % (64 * p) == 0 and k >= 512 * p)))


# ---------------------------------------------------------------- checkpoint

def mixer_shapes(m, p: str, D: int) -> Dict[str, Tuple[int, ...]]:
    if m.kind == "attention":
        nq, nk = m.heads * m.dim, m.kv_heads * m.dim
        return {p + "q": (nq, D), p + "k": (nk, D), p + "q.norm": (nq,), p + "k.norm": (nk,), p + "o": (D, nq)}
    if m.kind == "channel_delta":
        nk, nd, nv = m.kv_heads * m.dim, m.heads * m.dim, m.heads * m.vdim
        s = {}
        for n, c in (("q", nk), ("k", nk), ("v", nv)):
            s[p + n], s[p + n + ".conv"] = (c, D), (c, m.conv)
        s.update({p + "b": (m.heads, D), p + "A_log": (m.heads,), p + "norm": (m.vdim,), p + "a1": (m.decay_rank, D), p + "a2": (nd, m.decay_rank),
                  p + "dt_bias": (nd,), p + "g1": (m.gate_rank, D), p + "g2": (nv, m.gate_rank), p + "o": (D, nv)})
        return s
    s = {}
    for n in ("y", "x"):
        s[p + n], s[p + n + ".b"] = (m.width, D), (m.width,)
    s[p + "conv"], s[p + "conv.b"] = (m.width, m.conv), (m.width,)
    for n in ("ra", "ri"):
        s[p + n], s[p + n + ".b"] = (m.blocks, m.block, m.block), (m.blocks, m.block)
    s[p + "lam"], s[p + "o"] = (m.width,), (D, m.width)
    return s


def mlp_shapes(f: DenseMlp, p: str, D: int) -> Dict[str, Tuple[int, ...]]:
    return {p + "up": (f.ff, D), p + "down": (D, f.ff)}


def spread(a: np.ndarray, groups: int, ld: int) -> np.ndarray:
    """Rows in `groups` equal parts, each padded with zeros to `ld` rows."""
    a = a.reshape((groups, a.shape[0] // groups) + a.shape[1:])
    out = np.zeros((groups, ld) + a.shape[2:], a.dtype)
    out[:, :a.shape[1]] = a
    return out.reshape((groups * ld,) + a.shape[2:])


def load_layer(w, p: str, layer, D: int, get: Callable[[str], np.ndarray]) -> None:
    """The weights of one joint layer in the kernels' layouts."""
    m, f = layer.mixer, layer.mlp
    c, q = Columns(m, f), p + "mix."
    rows = np.zeros((c.rows, D), np.uint16)
    bias = np.zeros(c.rows, np.uint16)

    def put(name: str, a: np.ndarray) -> None:
        rows[c.at[name]:c.at[name] + a.shape[0]] = a

    if m.kind == "attention":
        put("q", spread(get(q + "q"), m.heads, m.dim_ld))
        put("k", spread(get(q + "k"), m.kv_heads, m.dim_ld))
        w._vector(q + "q.norm", spread(get(q + "q.norm"), m.heads, m.dim_ld))
        w._vector(q + "k.norm", spread(get(q + "k.norm"), m.kv_heads, m.dim_ld))
        w._vector(q + "rot_freq", m.rotation()[0] if m.rot_dims else np.zeros(1))
        out = spread(np.ascontiguousarray(get(q + "o").T), m.heads, m.dim_ld)
    elif m.kind == "channel_delta":
        G, H, K, V = m.kv_heads, m.heads, m.dim_ld, m.vdim_ld
        put("a1", get(q + "a1"))
        put("g1", get(q + "g1"))
        for n, heads, ld in (("q", G, K), ("k", G, K), ("v", H, V)):
            put(n, spread(get(q + n), heads, ld))
        rows[c.width:] = get(q + "b")
        w._vector(q + "conv", np.concatenate([spread(get(q + n + ".conv"), heads, ld) for n, heads, ld in (("q", G, K), ("k", G, K), ("v", H, V))]))
        w._matrix(q + "a2", spread(get(q + "a2"), H, K))
        w._matrix(q + "g2", spread(get(q + "g2"), H, V))
        w._vector(q + "dt_bias", spread(get(q + "dt_bias"), H, K))
        w._vector(q + "A_log", get(q + "A_log"))
        w._vector(q + "norm", spread(get(q + "norm"), 1, V))
        out = spread(np.ascontiguousarray(get(q + "o").T), H, V)
    else:
        B, n = m.blocks, m.block_ld
        for name in ("x", "y"):
            put(name, spread(get(q + name), B, n))
            bias[c.at[name]:c.at[name] + m.inner] = spread(get(q + name + ".b"), B, n)
        w._vector(q + "in.b", bias)
        w._vector(q + "conv", spread(get(q + "conv"), B, n))
        w._vector(q + "conv.b", spread(get(q + "conv.b"), B, n))
        gates = np.zeros((B, 2, n, n), np.uint16)
        for k, name in enumerate(("ra", "ri")):
            gates[:, k, :m.block, :m.block] = get(q + name)
            w._vector(q + name + ".b", spread(get(q + name + ".b").reshape(-1), B, n))
        w._matrix(q + "gates", gates.reshape(B * 2 * n, n))
        w._vector(q + "lam", spread(get(q + "lam"), B, n))
        out = spread(np.ascontiguousarray(get(q + "o").T), B, n)
    both = np.zeros((c.ko, D), np.uint16)
    both[:out.shape[0]] = out
    if f:
        put("up", get(p + "mlp.up"))
        both[c.up - c.out:c.up - c.out + f.ff] = get(p + "mlp.down").T
    w._matrix(q + "in", rows)
    w._matrix(p + "out", np.ascontiguousarray(both.T))


def random_layer(w, p: str, layer, D: int, fill: Callable, matrix: Callable) -> None:
    """The same generated in HBM, for measurements (widths that need no padding)."""
    m, f = layer.mixer, layer.mlp
    c, q = Columns(m, f), p + "mix."
    v = w.vecs
    if m.kind == "attention":
        if m.dim != m.dim_ld:
            raise ValueError("random_init takes head widths that need no padding")
        v[q + "q.norm"], v[q + "k.norm"] = fill(m.heads * m.dim, 1.0, 0.1), fill(m.kv_heads * m.dim, 1.0, 0.1)
        w._vector(q + "rot_freq", m.rotation()[0] if m.rot_dims else np.zeros(1))
    elif m.kind == "channel_delta":
        if m.dim != m.dim_ld or m.vdim != m.vdim_ld:
            raise ValueError("random_init takes head widths that need no padding")
        v[q + "conv"] = fill(m.channels * m.conv, 0.0, 0.4)
        matrix(q + "a2", m.heads * m.dim, m.decay_rank)
        matrix(q + "g2", m.heads * m.vdim, m.gate_rank)
        v[q + "dt_bias"], v[q + "A_log"], v[q + "norm"] = fill(m.heads * m.dim, -3.0, 0.5), fill(m.heads, 0.5, 0.5), fill(m.vdim, 1.0, 0.1)
    else:
        if m.block != m.block_ld:
            raise ValueError("random_init takes block widths that need no padding")
        v[q + "in.b"], v[q + "conv"], v[q + "conv.b"] = fill(c.rows, 0.0, 0.1), fill(m.inner * m.conv, 0.0, 0.4), fill(m.inner, 0.0, 0.1)
        v[q + "ra.b"], v[q + "ri.b"], v[q + "lam"] = fill(m.inner, 0.0, 0.1), fill(m.inner, 0.0, 0.1), fill(m.inner, -4.0, 0.5)
        matrix(q + "gates", m.blocks * 2 * m.block, m.block)
    matrix(q + "in", c.rows, D)
    matrix(p + "out", D, c.ko)


# ---------------------------------------------------------------- state, scratch, tasks

def state_entry(m, act: int, capacity: int) -> Dict[str, DeviceBuffer]:
    """What one run of a mixer leaves behind."""
    e = act // 8
    if m.kind == "attention":
        n = m.kv_heads * capacity * m.dim_ld * e
        return dict(k=native.zeros(n), v=native.zeros(n))
    if m.kind == "channel_delta":
        return dict(state=native.zeros(m.heads * m.vdim_ld * m.state_ld * 4), hist=native.zeros(m.conv * pad(m.channels) * e))
    return dict(state=native.zeros(m.inner * 4), hist=native.zeros(m.conv * m.inner * e))


def scratch(m, f, R: int, act: int, capacity: int, want: Callable[[str, int], None]) -> None:
    e = act // 8
    c = Columns(m, f)
    want("u", R * c.width * e)
    if m.kind == "attention":
        want("q", R * m.heads * m.dim_ld * e)
        if act == 16:
            part, count = native.sdpa_workspace_bytes(m.heads, m.kv_heads, m.dim_ld, m.dim_ld, capacity)
            want("part", part)
            want("counters", count)
    elif m.kind == "channel_delta":
        want("beta", R * m.heads * 4)
        want("xbc", R * pad(m.channels) * e)
        want("decays", R * m.heads * m.dim_ld * 4)
        want("qk", R * 2 * m.kv_heads * m.dim_ld * 4)
        want("o", pad(R) * m.heads * m.vdim_ld * 4)
        want("gate", R * m.heads * m.vdim_ld * e)
        if act == 16 and native.delta_chunk_supported(m.dim_ld, m.vdim_ld):
            want("work", native.delta_chunk_work_bytes(R, m.heads, m.dim_ld, m.vdim_ld))
    else:
        want("xbc", R * m.inner * e)
        want("gates", R * 2 * m.inner * 4)
        want("carry", -(-R // LRU_CHUNK) * 2 * m.inner * 4)


def fusable(m) -> bool:
    """Whether the mixer has the fused launches of one token."""
    if m.kind == "attention":
        return m.dim_ld <= 512
    if m.kind == "channel_delta":
        return m.state_ld <= 256
    return m.block_ld <= 30720


class JointTasks:
    """Task lists of joint layers (a part of LayerRuntime)."""

    def _joint_tasks(self, t, run: int, rows: int, off, kv_len) -> None:
        """One layer of a pass, from its norm in h1 to what it adds to the residual stream in mix."""
        c, w, b = self.cfg, self.w, self.buf
        i = self.runs[run][0]
        l, p = c.layers[i], f"l{i}."
        m, q = l.mixer, p + "mix."
        col = Columns(m, l.mlp)
        D, e = pad(c.width), c.act // 8
        more = dict(col.fns)
        base, tail = [], []
        if m.kind == "rglru":
            more["has_bias"], base = 1, [arg(w.vecs[q + "in.b"])]
        if col.tail:
            more.update(tail_begin=col.width, ldt=col.tail)
            tail = [arg(b["beta"])]
        self._dense(t, arg(b["h1"]), w.mats[q + "in"], arg(b["u"]), rows, D, col.width, base=base, tail=tail, **more)
        u = lambda name: arg(b["u"], None, col.at[name] * e)
        {"attention": self._attention_tasks, "channel_delta": self._delta_tasks, "rglru": self._lru_tasks}[m.kind](t, m, q, col, run, rows, off, kv_len, u)
        W, parts = w.mats[p + "out"], self._out_parts(i, rows)
        k = W.k // parts
        self._dense(t, arg(b["u"], None, col.out * e), W, arg(b["mix"]), rows, col.width, D, y32=True, **(dict(batch=parts, k=k, xb=k, wb=k, yb=rows * D) if parts > 1 else {}))

    def _out_parts(self, layer: int, rows: int) -> int:
        c = self.cfg
        l = c.layers[layer]
        return out_parts(rows, c.width, Columns(l.mixer, l.mlp).ko) if l.joint and c.act == 16 and c.tiled else 1

    def _qk_store(self, m, q: str, col: Columns, run: int, rows: int, off) -> Dispatch:
        c, w, b, st = self.cfg, self.w, self.buf, self.state.entries[run]
        return Dispatch(self._name("qk_store"),
                        [arg(b["u"]), arg(w.vecs[q + "q.norm"]), arg(w.vecs[q + "k.norm"]), arg(w.vecs[q + "rot_freq"]), off, arg(b["q"]), arg(st["k"]), arg(st["v"])],
                        dict(rows=rows, heads=m.heads, kv_heads=m.kv_heads, dim=m.dim, dim_ld=m.dim_ld, rot_dims=m.rot_dims, ldu=col.width,
                             k0=col.at["k"], q0=col.at["q"], capacity=c.capacity, mag=m.rotation()[1], eps=c.eps, act=c.act))

    def _attention_tasks(self, t, m, q: str, col: Columns, run: int, rows: int, off, kv_len, u) -> None:
        c, b, st = self.cfg, self.buf, self.state.entries[run]
        t.append(self._qk_store(m, q, col, run, rows, off))
        if c.act == 16 and rows == 1 and m.dim_ld <= 512:
            t.append(Dispatch(self._name("sdpa_decode"), [arg(b["q"]), arg(st["k"]), arg(st["v"]), kv_len, u("q"), arg(b["part"]), arg(b["counters"])],
                              dict(n_heads=m.heads, n_kv=m.kv_heads, head_dim=m.dim_ld, capacity=c.capacity, scale=m.scale)))
        elif c.act == 16 and c.tiled and m.dim_ld in (64, 128):
            t.append(Dispatch(self._name("sdpa_prefill"), [arg(b["q"]), arg(st["k"]), arg(st["v"]), kv_len, u("q")],
                              dict(rows=rows, n_heads=m.heads, n_kv=m.kv_heads, head_dim=m.dim_ld, capacity=c.capacity, scale=m.scale, ldo=col.width)))
        else:
            t.append(Dispatch(self._name("gqa_rows"), [arg(b["q"]), arg(st["k"]), arg(st["v"]), off, u("q")],
                              dict(rows=rows, heads=m.heads, kv_heads=m.kv_heads, dim_ld=m.dim_ld, capacity=c.capacity, scale=m.scale, ldo=col.width, act=c.act)))

    def _conv(self, m, q: str, x, run: int, rows: int, off, channels: int, ldu: int, bias: bool, linear: bool) -> Dispatch:
        c, w, b, st = self.cfg, self.w, self.buf, self.state.entries[run]
        a = [x, arg(w.vecs[q + "conv"])] + ([arg(w.vecs[q + "conv.b"])] if bias else []) + [arg(st["hist"]), off, arg(b["xbc"])]
        return Dispatch(self._name("ssm_conv"), a, dict(rows=rows, channels=channels, taps=m.conv, ldu=ldu, ldy=pad(channels), ldh=pad(channels),
                                                        has_bias=int(bias), linear=int(linear), update=1, act=c.act))

    def _delta_tasks(self, t, m, q: str, col: Columns, run: int, rows: int, off, kv_len, u) -> None:
        c, w, b, st = self.cfg, self.w, self.buf, self.state.entries[run]
        X, e = pad(m.channels), c.act // 8
        nd, nv, nk = m.heads * m.dim_ld, m.heads * m.vdim_ld, m.kv_heads * m.dim_ld
        t.append(self._conv(m, q, u("q"), run, rows, off, m.channels, col.width, bias=False, linear=False))
        self._dense(t, u("a1"), w.mats[q + "a2"], arg(b["decays"]), rows, col.width, nd, y32=True)
        self._dense(t, u("g1"), w.mats[q + "g2"], arg(b["gate"]), rows, col.width, nv)
        shape = dict(rows=rows, heads=m.heads, kv_heads=m.kv_heads, dim_ld=m.dim_ld, ldx=X, ldb=m.heads, act=c.act)
        t.append(Dispatch(self._name("delta_prep"),
                          [arg(b["xbc"]), arg(w.vecs[q + "dt_bias"]), arg(w.vecs[q + "A_log"]), arg(b["decays"]), arg(b["beta"]), arg(b["qk"])], dict(shape, dim=m.dim)))
        long = c.act == 16 and c.tiled and rows >= DELTA_ROWS and native.delta_chunk_supported(m.dim_ld, m.vdim_ld)
        t.append(Dispatch(self._name("delta_chunk" if long else "delta_scan"),
                          [arg(b["qk"]), arg(b["decays"]), arg(b["beta"]), arg(b["xbc"], None, 2 * nk * e), arg(st["state"]), arg(b["o"])] + ([arg(b["work"])] if long else []),
                          dict(shape, vdim_ld=m.vdim_ld, state_ld=m.state_ld)))
        t.append(Dispatch(self._name("head_norm"), [arg(b["o"]), arg(b["gate"]), arg(w.vecs[q + "norm"]), u("v")],
                          dict(rows=rows, heads=m.heads, dim=m.vdim, ld=m.vdim_ld, ldx=nv, ldz=nv, ldy=col.width, eps=c.eps, act=c.act)))

    def _lru_tasks(self, t, m, q: str, col: Columns, run: int, rows: int, off, kv_len, u) -> None:
        c, w, b, st = self.cfg, self.w, self.buf, self.state.entries[run]
        n, G = m.block_ld, w.mats[q + "gates"]
        t.append(self._conv(m, q, u("x"), run, rows, off, m.inner, col.width, bias=True, linear=True))
        self._dense(t, arg(b["xbc"]), G, arg(b["gates"]), rows, m.inner, 2 * m.inner, n=2 * n, y32=True, batch=m.blocks, xb=n, wb=2 * n * n, yb=2 * n)
        t.append(Dispatch(self._name("lru_scan"),
                          [arg(b["xbc"]), arg(b["gates"]), arg(w.vecs[q + "ra.b"]), arg(w.vecs[q + "ri.b"]), arg(w.vecs[q + "lam"]), arg(st["state"]), u("y"), arg(b["carry"])],
                          dict(rows=rows, width=m.inner, block=n, ldx=m.inner, ldy=col.width, act=c.act)))

    # -- one decoded token in fused launches
    def _fused_joint_tasks(self, t, run: int, x, step) -> None:
        """Norm and joint input projection | the recurrence's step (or cache rows | attention) | joint output projection."""
        c, w, b, st = self.cfg, self.w, self.buf, self.state.entries[run]
        i = self.runs[run][0]
        l, p, off = c.layers[i], f"l{i}.", arg(self.offset)
        m, q = l.mixer, p + "mix."
        col = Columns(m, l.mlp)
        u = lambda name: arg(b["u"], None, col.at[name] * 2)
        more = dict(col.fns, mode=1, width=c.width, eps=c.eps, step=len(step), layer_norm=int(c.layer_norm), has_bias=int(m.kind == "rglru"))
        norm = [arg(w.vecs[p + "norm1"])] + ([arg(w.vecs[p + "norm1.b"])] if c.layer_norm else [])
        W = w.mats[q + "in"]
        self._jobs(t, [x] + step + norm + [arg(W.w)] + ([arg(w.vecs[q + "in.b"])] if m.kind == "rglru" else []) + [arg(b["u"])] + ([arg(b["beta"])] if col.tail else []),
                   **self._product(0, W, col.width, **more))
        a, prm = [x, u(m.out_part), arg(w.mats[p + "out"].w)], dict(n=c.width, ko=col.ko, ldo=w.mats[p + "out"].k)
        after = []
        if m.kind == "attention":
            t.append(self._qk_store(m, q, col, run, 1, off))
            t.append(Dispatch(self._name("sdpa_decode"), [arg(b["q"]), arg(st["k"]), arg(st["v"]), arg(self.kv_len), u("q"), arg(b["part"]), arg(b["counters"])],
                              dict(n_heads=m.heads, n_kv=m.kv_heads, head_dim=m.dim_ld, capacity=c.capacity, scale=m.scale)))
        elif m.kind == "channel_delta":
            A, G = w.mats[q + "a2"], w.mats[q + "g2"]
            self._jobs(t, [u("g1"), arg(G.w), arg(b["gate"]), u("q"), u("a1"), arg(b["beta"]), arg(w.vecs[q + "conv"]), arg(A.w), arg(w.vecs[q + "dt_bias"]),
                           arg(w.vecs[q + "A_log"]), off, arg(st["state"]), arg(st["hist"]), arg(b["o"])],
                       **self._product(0, G, G.n, mode=0), delta_heads=m.heads, delta_kv_heads=m.kv_heads, delta_dim=m.dim, delta_dim_ld=m.dim_ld,
                       delta_vdim_ld=m.vdim_ld, delta_state_ld=m.state_ld, delta_rank_ld=A.k, delta_ldh=pad(m.channels), delta_taps=m.conv)
            after = [arg(b["o"]), arg(b["gate"]), arg(w.vecs[q + "norm"])]
            prm.update(norm_heads=m.heads, norm_dim=m.vdim, norm_ld=m.vdim_ld, norm_eps=c.eps)
        else:
            self._jobs(t, [u("x"), arg(w.vecs[q + "conv"]), arg(w.vecs[q + "conv.b"]), arg(w.mats[q + "gates"].w), arg(w.vecs[q + "ra.b"]), arg(w.vecs[q + "ri.b"]),
                           arg(w.vecs[q + "lam"]), off, arg(st["state"]), arg(st["hist"]), u("y")],
                       lru_width=m.inner, lru_block=m.block_ld, lru_ldh=m.inner, lru_taps=m.conv)
        if step:
            a, prm["has_step"] = a + step, 1
        t.append(Dispatch(self._name("layer_out"), a + after, prm))
