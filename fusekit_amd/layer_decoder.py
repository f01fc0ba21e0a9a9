"""Layer-list decoder on the MI355X backend: a model whose layers are described one by one.

Every layer has a mixer and optionally a feed-forward.  The two run side by side and their outputs join a 32-bit residual
stream together.  Either each reads its own norm of the layer's input (latent attention over a sliding window, Mamba-2
state-space mixers, mixtures of experts: this module; the design is Pusavik), or both read one norm (joint layers with
causal attention, gated delta rules, gated linear recurrences and dense feed-forwards: joint_layers.py; the design is
Fumotar).
A range of layers may run several times in a row with the same weights (`loop`), each pass with its own cache or state.
Ahead of a pass a learned vector is added, or the stream is projected together with the embedding output (`join`).

What a sequence leaves behind is held by `LayerState`: per layer RUN (a looped layer has several) a ring of latent rows
just long enough for the window, a key / value cache of `capacity` positions, or a recurrent state and the convolution's
last inputs.

Two task lists share the kernels' families: the decode list (one token, captured as one hipGraph and replayed) and the
rows list (a portion of a prompt of any length).  `act` 32 runs everything in fp32 through the same families.
"""
from __future__ import annotations

import ctypes as C
from collections import OrderedDict
from dataclasses import dataclass, field
from typing import Callable, Dict, List, Optional, Sequence, Tuple

import numpy as np

from . import joint_layers, native
from .decoder import _synth
from .joint_layers import JOINT, CausalAttention, ChannelDelta, DenseMlp, JointTasks, RgLru, RotaryScaling, pad
from .native import DeviceBuffer, DeviceWeight
from .runtime import FK_CHUNK, Dispatch, Dispatcher, arg, make_uniforms


# ---------------------------------------------------------------- configuration

@dataclass
class LatentAttention:
    heads: int
    dim: int          # unrotated query / key dimensions per head
    rot_dim: int      # rotated ones; one key part shared by all heads
    vdim: int
    kv_rank: int
    q_rank: int
    window: int
    scale: float
    rot_base: float
    rot_dims: int

    kind = "latent_attention"

    # padded widths: a query head is [dim_ld | rot_ld], a cache row [rank_ld | rot_ld]
    @property
    def dim_ld(self) -> int:
        return pad(self.dim, 32)

    @property
    def rot_ld(self) -> int:
        return pad(self.rot_dim, 32)

    @property
    def vdim_ld(self) -> int:
        return pad(self.vdim, 32)

    @property
    def hs(self) -> int:
        return self.dim_ld + self.rot_ld

    @property
    def rank_ld(self) -> int:
        return pad(self.kv_rank)

    @property
    def ldc(self) -> int:
        return self.rank_ld + self.rot_ld

    @property
    def low_rows(self) -> int:
        """Rows of the joint down projection [query latent | key / value latent | rotated key part]."""
        return self.q_rank + self.kv_rank + self.rot_dim


@dataclass
class Mamba2:
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    kind = "mamba2"

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.state

    @property
    def state_ld(self) -> int:
        return pad(self.state)


@dataclass
class Experts:
    experts: int
    identity: int
    top: int
    ff: int

    @property
    def outputs(self) -> int:
        return self.experts + self.identity


@dataclass
class Layer:
    mixer: object
    mlp: object = None           # Experts, DenseMlp (joint layers) or None

    @property
    def joint(self) -> bool:
        return self.mixer.kind in JOINT

    @property
    def experts(self) -> Optional[Experts]:
        return self.mlp if isinstance(self.mlp, Experts) else None

    def __post_init__(self):
        if self.mlp is not None and isinstance(self.mlp, DenseMlp) != self.joint:
            raise ValueError("dense feed-forwards go with joint mixers, experts with the others")


@dataclass
class PairTable:
    """A second embedding table, its rows chosen by a hash of a token and the one before it (row `buckets`: no token before)."""
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass
class LayerConfig:
    width: int
    vocab: int
    layers: List[Layer]
    eps: float = 1e-6
    embed_scale: float = 1.0
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1
    design: str = "Pusavik"
    layer_norm: bool = False     # norms: x - mean over the standard deviation, with a bias; else RMS norms
    tied: bool = False           # the embedding table is the head
    pairs: Optional[PairTable] = None
    join: bool = False           # ahead of a loop pass: x <- W [x; embedding output]; else a learned vector is added
    capacity: int = 4096         # positions of a key / value cache
    act: int = 16                # 16: bf16 matrices and activations, 32-bit residual, norms, router, softmax and state; 32: all fp32
    rows_per_pass: int = 2048    # most tokens of one rows pass
    artifact_type = "layer-list-decoder"
    tiled: bool = True           # the matrix-core forms of attention, recurrence and experts for portions (False: the row forms)
    fuse: bool = True            # the decode list's fused launches (False: the rows list at one row)

    @property
    def hidden(self) -> int:
        return self.width

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @property
    def n_heads(self) -> int:
        return max((l.mixer.heads for l in self.layers), default=0)

    @property
    def head_dim(self) -> int:
        return max((l.mixer.vdim for l in self.layers), default=0)

    @property
    def max_positions(self) -> Optional[int]:
        """Longest sequence the state holds, None without a limit."""
        return self.capacity if any(l.mixer.kind == "attention" for l in self.layers) else None

    @property
    def padded_lookup(self) -> bool:
        """Whether token rows come from tables in padded rows (those of a tied head, pairs, copies for a join)."""
        return bool(self.pairs or self.tied or (self.looped and self.join))

    @property
    def looped(self) -> bool:
        return self.loop_stop > self.loop_start

    def runs(self) -> List[Tuple[int, Optional[int]]]:
        """(layer, number of the pass that starts here or None) in the order the layers run."""
        n = self.n_layers
        if not self.looped:
            return [(i, None) for i in range(n)]
        out: List[Tuple[int, Optional[int]]] = [(i, None) for i in range(self.loop_start)]
        for t in range(self.loop_times):
            out += [(i, t if i == self.loop_start else None) for i in range(self.loop_start, self.loop_stop)]
        return out + [(i, None) for i in range(self.loop_stop, n)]


def small_config(width: int = 256, vocab: int = 1000, heads: int = 4, ff: int = 96, window: int = 48, **more) -> LayerConfig:
    """A four-layer model of both mixers with a loop, for examples and tests."""
    lat = LatentAttention(heads=heads, dim=40, rot_dim=16, vdim=48, kv_rank=72, q_rank=80, window=window, scale=56 ** -0.5,
                          rot_base=10000.0, rot_dims=16)
    ssm = Mamba2(heads=2 * heads, vdim=24, state=40, groups=2, conv=3, norm_groups=4)
    moe = Experts(experts=6, identity=1, top=3, ff=ff)
    return LayerConfig(width=width, vocab=vocab, layers=[Layer(lat, moe), Layer(ssm, moe), Layer(lat), Layer(ssm, moe)], embed_scale=0.7,
                       loop_start=1, loop_stop=3, loop_times=2, **more)


def small_joint_config(width: int = 256, vocab: int = 1000, heads: int = 4, ff: int = 96, **more) -> LayerConfig:
    """A four-layer model of the three joint mixers with a loop, for examples and tests."""
    att = CausalAttention(heads=heads, kv_heads=max(1, heads // 2), dim=40, scale=40 ** -0.5, rot_base=5000.0, rot_dims=24,
                          rot_scaling=RotaryScaling(factor=3.0, original=512, fast=16.0, slow=1.5))
    dlt = ChannelDelta(heads=heads, kv_heads=max(1, heads // 2), dim=24, vdim=40, conv=3, decay_rank=20, gate_rank=28)
    lru = RgLru(width=3 * 40, blocks=3, conv=4)
    mlp = DenseMlp(ff)
    return LayerConfig(width=width, vocab=vocab, layers=[Layer(lru, mlp), Layer(att, mlp), Layer(dlt), Layer(att, mlp)], loop_start=1, loop_stop=3,
                       loop_times=2, design="Fumotar", layer_norm=True, tied=True, pairs=PairTable(buckets=211, mul_prev=13, mul_cur=7), join=True, **more)


def tensor_shapes(cfg: LayerConfig) -> Dict[str, Tuple[int, ...]]:
    """Names and shapes of a checkpoint's tensors."""
    D = cfg.width
    s: Dict[str, Tuple[int, ...]] = {"embed": (cfg.vocab, D)}
    if cfg.pairs:
        s["bigram"] = (cfg.pairs.buckets + 1, D)
    if cfg.looped and cfg.join:
        s["loop.in"] = (D, 2 * D)
    elif cfg.looped:
        s["loop.step"] = (cfg.loop_times, D)

    def norm(name: str) -> None:
        s[name] = (D,)
        if cfg.layer_norm:
            s[name + ".b"] = (D,)

    for i, l in enumerate(cfg.layers):
        p, m, f = f"l{i}.", l.mixer, l.experts
        norm(p + "norm1")
        if l.joint:
            s.update(joint_layers.mixer_shapes(m, p + "mix.", D))
            if l.mlp:
                s.update(joint_layers.mlp_shapes(l.mlp, p + "mlp.", D))
        elif m.kind == "latent_attention":
            s[p + "mix.dq"], s[p + "mix.dq.norm"] = (m.q_rank, D), (m.q_rank,)
            s[p + "mix.uq"] = (m.heads * (m.dim + m.rot_dim), m.q_rank)
            s[p + "mix.dkv"], s[p + "mix.dkv.norm"] = (m.kv_rank + m.rot_dim, D), (m.kv_rank,)
            s[p + "mix.uk"], s[p + "mix.uv"] = (m.heads * m.dim, m.kv_rank), (m.heads * m.vdim, m.kv_rank)
            s[p + "mix.sink"], s[p + "mix.o"] = (m.heads,), (D, m.heads * m.vdim)
        else:
            s[p + "mix.in"] = (2 * m.inner + 2 * m.groups * m.state + m.heads, D)
            s[p + "mix.conv"], s[p + "mix.conv.b"] = (m.channels, m.conv), (m.channels,)
            for n in ("dt_bias", "A_log", "D"):
                s[p + "mix." + n] = (m.heads,)
            s[p + "mix.norm"], s[p + "mix.o"] = (m.inner,), (D, m.inner)
        if f:
            s[p + "norm2"] = (D,)
            for e in range(f.experts):
                s[p + f"mlp.e{e}.gate"], s[p + f"mlp.e{e}.up"], s[p + f"mlp.e{e}.down"] = (f.ff, D), (f.ff, D), (D, f.ff)
            s[p + "mlp.router"], s[p + "mlp.correction"] = (f.outputs, D), (f.outputs,)
    norm("final.norm")
    if not cfg.tied:
        s["head"] = (cfg.vocab, D)
    return s


def random_tensors(cfg: LayerConfig, seed: int = 0, std: float = 0.05) -> Dict[str, np.ndarray]:
    """Random bf16 bit patterns for every tensor of a small model: matrices N(0, std^2), norms around one, decays and
    step sizes in their usual ranges."""
    rng = np.random.Generator(np.random.PCG64(seed))
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        v = rng.standard_normal(shape)
        if leaf == "lam":
            v = -3.0 + v
        elif leaf in ("norm1", "norm2", "norm"):
            v = 1.0 + 0.1 * v
        elif leaf == "A_log":
            v = np.log(1.0 + 7.0 * rng.random(shape))
        elif leaf == "dt_bias":
            v = -2.0 + 0.5 * v
        elif leaf in ("D", "sink"):
            v = 1.0 + 0.5 * v
        elif leaf in ("embed", "head", "bigram"):
            v = v * 0.5
        elif leaf == "router":
            v = v * 0.3
        elif leaf == "correction":
            v = 0.02 * v
        elif leaf == "conv":
            v = 0.4 * v
        elif leaf in ("b", "step"):
            v = 0.1 * v
        else:
            v = v * max(std, 0.7 / np.sqrt(shape[-1]))
        out[name] = f32_to_bf16(v)
    return out


def f32_to_bf16(a) -> np.ndarray:
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_to_f32(a: np.ndarray) -> np.ndarray:
    return (np.asarray(a, np.uint16).astype(np.uint32) << 16).view(np.float32)


# ---------------------------------------------------------------- weights

class LayerWeights:
    """Weights of one model in HBM in the layouts the kernels walk: rows padded with zeros, the down projections of a
    latent mixer joined, head parts padded to whole matrix-instruction steps, experts stacked."""

    def __init__(self, cfg: LayerConfig):
        self.cfg = cfg
        self.mats: Dict[str, DeviceWeight] = {}
        self.vecs: Dict[str, DeviceBuffer] = {}
        self.vec_dtype: Dict[str, str] = {}

    def _dense(self, name: str, buf: DeviceBuffer, n: int, ld: int, experts: int = 0) -> None:
        W = DeviceWeight.__new__(DeviceWeight)
        W.n, W.k, W.bits, W.group, W.w, W.scales, W.biases = n, ld, 16, 0, buf, None, None
        if experts:
            W.n_experts = experts
        self.mats[name] = W

    def _matrix(self, name: str, a: np.ndarray, experts: int = 0) -> None:
        n, k = a.shape[-2:]
        ld = pad(k)
        p = np.zeros(a.shape[:-1] + (ld,), np.uint16)
        p[..., :k] = a
        self._dense(name, DeviceBuffer.from_numpy(p), n, ld, experts)

    def _vector(self, name: str, a: np.ndarray, padded: bool = False) -> None:
        a = np.asarray(a)
        if padded:
            p = np.zeros(a.shape[:-1] + (pad(a.shape[-1]),), a.dtype)
            p[..., :a.shape[-1]] = a
            a = p
        self.vecs[name] = DeviceBuffer.from_numpy(a)
        if a.dtype == np.float64:
            self.vec_dtype[name] = "float64"

    @staticmethod
    def rot_freq(m: LatentAttention) -> np.ndarray:
        return np.asarray(m.rot_base, np.float64) ** (-2.0 * np.arange(m.rot_dims // 2) / max(m.rot_dims, 1))

    @classmethod
    def from_tensors(cls, cfg: LayerConfig, get: Callable[[str], np.ndarray]) -> "LayerWeights":
        """`get(name)` returns a tensor's bf16 bit patterns in its own shape."""
        self, c = cls(cfg), cfg
        if c.tied:
            self._matrix("head", get("embed"))
            self.mats["embed"] = self.mats["head"]
        else:
            if c.padded_lookup:
                self._matrix("embed", get("embed"))
            else:
                self._dense("embed", DeviceBuffer.from_numpy(get("embed")), c.vocab, c.width)
            self._matrix("head", get("head"))
        if c.pairs:
            self._matrix("bigram", get("bigram"))

        def norm(name: str) -> None:
            self._vector(name, get(name), True)
            if c.layer_norm:
                self._vector(name + ".b", get(name + ".b"), True)

        norm("final.norm")
        if c.looped and c.join:
            W, D = get("loop.in"), pad(c.width)
            both = np.zeros((c.width, 2 * D), np.uint16)
            both[:, :c.width], both[:, D:D + c.width] = W[:, :c.width], W[:, c.width:]
            self._matrix("loop.in", both)
        elif c.looped:
            self._vector("loop.step", get("loop.step"), True)
        for i, l in enumerate(c.layers):
            p, m, f = f"l{i}.", l.mixer, l.experts
            norm(p + "norm1")
            q = p + "mix."
            if l.joint:
                joint_layers.load_layer(self, p, l, c.width, get)
            elif m.kind == "latent_attention":
                self._matrix(q + "down", np.concatenate([get(q + "dq"), get(q + "dkv")], 0))
                self._vector(q + "dq.norm", get(q + "dq.norm"), True)
                self._vector(q + "dkv.norm", get(q + "dkv.norm"), True)
                uq = np.zeros((m.heads, m.hs, m.q_rank), np.uint16)
                src = get(q + "uq").reshape(m.heads, m.dim + m.rot_dim, m.q_rank)
                uq[:, :m.dim], uq[:, m.dim_ld:m.dim_ld + m.rot_dim] = src[:, :m.dim], src[:, m.dim:]
                self._matrix(q + "uq", uq.reshape(-1, m.q_rank))
                uk = np.zeros((m.heads, m.dim_ld, m.kv_rank), np.uint16)
                uk[:, :m.dim] = get(q + "uk").reshape(m.heads, m.dim, m.kv_rank)
                self._matrix(q + "uk", uk.reshape(-1, m.kv_rank))
                # W_uk per head with the latent along the rows: carries a query into the latent space
                self._matrix(q + "uk_t", np.ascontiguousarray(uk[:, :m.dim].transpose(0, 2, 1)).reshape(-1, m.dim))
                uv = np.zeros((m.heads, m.vdim_ld, m.kv_rank), np.uint16)
                uv[:, :m.vdim] = get(q + "uv").reshape(m.heads, m.vdim, m.kv_rank)
                self._matrix(q + "uv", uv.reshape(-1, m.kv_rank))
                o = np.zeros((c.width, m.heads, m.vdim_ld), np.uint16)
                o[:, :, :m.vdim] = get(q + "o").reshape(c.width, m.heads, m.vdim)
                self._matrix(q + "o", o.reshape(c.width, -1))
                self._vector(q + "sink", get(q + "sink"))
                self._vector(q + "rot_freq", self.rot_freq(m))
            else:
                self._matrix(q + "in", get(q + "in"))
                for n in ("conv", "conv.b", "dt_bias", "A_log", "D"):
                    self._vector(q + n, get(q + n))
                self._vector(q + "norm", get(q + "norm"), True)
                self._matrix(q + "o", get(q + "o"))
            if f:
                q = p + "mlp."
                self._vector(p + "norm2", get(p + "norm2"), True)
                for n in ("gate", "up", "down"):
                    self._matrix(q + n, np.stack([get(q + f"e{e}.{n}") for e in range(f.experts)]), f.experts)
                self._matrix(q + "router", get(q + "router"))
                self._vector(q + "correction", get(q + "correction"))
        native.sync()
        return self

    @classmethod
    def random_init(cls, cfg: LayerConfig, seed: int = 0, std: float = 0.02) -> "LayerWeights":
        """A model of any size generated in HBM, for measurements: every padded width must equal the width itself."""
        self, c = cls(cfg), cfg
        count = [seed * 100003 + 11]

        def fill(n: int, mean: float, sd: float) -> DeviceBuffer:
            count[0] += 1
            b = DeviceBuffer(n * 2)
            _synth(b, n, count[0], mean, sd, 1)
            return b

        def matrix(name: str, n: int, k: int, experts: int = 0, sd: float = std) -> None:
            if k % 64:
                raise ValueError(f"{name}: random_init takes widths that need no padding")
            self._dense(name, fill(n * k * max(experts, 1), 0.0, sd), n, k, experts)

        matrix("embed", c.vocab, c.width, sd=std if c.tied else 0.5)
        if c.tied:
            self.mats["head"] = self.mats["embed"]
        else:
            matrix("head", c.vocab, c.width)
        if c.pairs:
            matrix("bigram", c.pairs.buckets + 1, c.width, sd=0.5)

        def norm(name: str) -> None:
            self.vecs[name] = fill(pad(c.width), 1.0, 0.1)
            if c.layer_norm:
                self.vecs[name + ".b"] = fill(pad(c.width), 0.0, 0.1)

        norm("final.norm")
        if c.looped and c.join:
            matrix("loop.in", c.width, 2 * c.width)
        elif c.looped:
            self.vecs["loop.step"] = fill(c.loop_times * pad(c.width), 0.0, 0.1)
        for i, l in enumerate(c.layers):
            p, m, f = f"l{i}.", l.mixer, l.experts
            norm(p + "norm1")
            q = p + "mix."
            if l.joint:
                joint_layers.random_layer(self, p, l, c.width, fill, matrix)
            elif m.kind == "latent_attention":
                if m.dim % 32 or m.rot_dim % 32 or m.vdim % 32:
                    raise ValueError("random_init takes head widths that need no padding")
                matrix(q + "down", m.low_rows, c.width)
                self.vecs[q + "dq.norm"], self.vecs[q + "dkv.norm"] = fill(pad(m.q_rank), 1.0, 0.1), fill(m.rank_ld, 1.0, 0.1)
                matrix(q + "uq", m.heads * m.hs, m.q_rank)
                matrix(q + "uk", m.heads * m.dim_ld, m.kv_rank)
                matrix(q + "uk_t", m.heads * m.kv_rank, m.dim)
                matrix(q + "uv", m.heads * m.vdim_ld, m.kv_rank)
                matrix(q + "o", c.width, m.heads * m.vdim_ld)
                self.vecs[q + "sink"] = fill(m.heads, 1.0, 0.5)
                self._vector(q + "rot_freq", self.rot_freq(m))
            else:
                matrix(q + "in", 2 * m.inner + 2 * m.groups * m.state + m.heads, c.width)
                self.vecs[q + "conv"], self.vecs[q + "conv.b"] = fill(m.channels * m.conv, 0.0, 0.4), fill(m.channels, 0.0, 0.1)
                self.vecs[q + "dt_bias"], self.vecs[q + "A_log"], self.vecs[q + "D"] = fill(m.heads, -2.0, 0.5), fill(m.heads, 1.0, 0.5), fill(m.heads, 1.0, 0.3)
                self.vecs[q + "norm"] = fill(m.inner, 1.0, 0.1)
                matrix(q + "o", c.width, m.inner)
            if f:
                q = p + "mlp."
                self.vecs[p + "norm2"] = fill(c.width, 1.0, 0.1)
                matrix(q + "gate", f.ff, c.width, f.experts)
                matrix(q + "up", f.ff, c.width, f.experts)
                matrix(q + "down", c.width, f.ff, f.experts)
                matrix(q + "router", f.outputs, c.width, sd=0.05)
                self.vecs[q + "correction"] = fill(f.outputs, 0.0, 0.01)
        native.sync()
        return self

    def nbytes(self) -> int:
        mats = {id(m): m for m in self.mats.values()}   # a tied head is one matrix under two names
        return sum(m.nbytes for m in mats.values()) + sum(v.nbytes for v in self.vecs.values())


# ---------------------------------------------------------------- what a sequence leaves behind

class LayerState:
    """Caches and states of one sequence, one entry per layer run.  Position p of a windowed attention run lies in row
    p % ring of its ring of latent rows (rows a window can no longer see are overwritten), of a causal one in row p of its
    key and value caches; a recurrent run holds its fp32 state and the last convolution inputs (position p in row
    p % taps).  `prev` is the last token, where a table of token pairs needs it."""

    def __init__(self, cfg: LayerConfig, rows: int):
        e = cfg.act // 8
        self.entries: List[Dict[str, DeviceBuffer]] = []
        self.rings: List[int] = []
        self.prev = native.zeros(4)
        for i, _ in cfg.runs():
            m = cfg.layers[i].mixer
            if cfg.layers[i].joint:
                self.rings.append(0)
                self.entries.append(joint_layers.state_entry(m, cfg.act, cfg.capacity))
            elif m.kind == "latent_attention":
                ring = 1 << (m.window + rows - 2).bit_length()
                self.rings.append(ring)
                # a product that walks padded rows may read up to one padding block past the last row
                self.entries.append(dict(cache=native.zeros(ring * m.ldc * e + 256)))
            else:
                self.rings.append(0)
                self.entries.append(dict(state=native.zeros(m.heads * m.vdim * m.state_ld * 4),
                                         hist=native.zeros(m.conv * pad(m.channels) * e)))

    def reset(self) -> None:
        """A new sequence: recurrent states start at zero.  Cache rows need no clearing: a position sees only rows that the
        sequence itself has written, and the first one looks at no token before it."""
        for e in self.entries:
            for name in ("state", "hist"):
                if name in e:
                    native.fill_u32(e[name], 0, e[name].nbytes // 4)
        native.sync()

    def nbytes(self) -> int:
        return sum(b.nbytes for e in self.entries for b in e.values())


# ---------------------------------------------------------------- runtime

class LayerRuntime(JointTasks):
    """Scratch arena, sequence state, decode graph and rows passes of one model."""

    HEAD_ROWS = 64      # logits rows formed at once for a portion that asks for them

    def __init__(self, cfg: LayerConfig, weights: LayerWeights, dispatcher: Optional[Dispatcher] = None, hist_capacity: int = 4096):
        c = cfg
        self.cfg, self.w = cfg, weights
        self.d = dispatcher or Dispatcher()
        self.runs = c.runs()
        tops = [l.experts.top for l in c.layers if l.experts]
        self.R = max(1, min(c.rows_per_pass, 65535 // max(tops, default=1), c.max_positions or c.rows_per_pass))
        self.position = 0
        self.state = LayerState(c, self.R)
        z = native.zeros
        self.token, self.step_counter, self.offset, self.kv_len, self.hist_counter = (z(4) for _ in range(5))
        self.history = z(4 * hist_capacity)
        self.row_offset, self.row_kv, self.tokens = z(4), z(4), z(4 * self.R)
        self.argmax_ws = z(native.ARGMAX_WORKSPACE_BYTES)
        self.buf: Dict[str, DeviceBuffer] = {}
        self._alloc_rows()
        self.logits = z(self.HEAD_ROWS * pad(c.vocab) * 4)
        self.head_x = z(self.HEAD_ROWS * pad(c.width) * (c.act // 8) + 256)
        self.uniforms = make_uniforms(self.token, self.step_counter, self.hist_counter, self.history)
        self._passes: "OrderedDict[int, object]" = OrderedDict()
        self._full_pass: Optional[int] = None
        self.tasks = self.build_tasks()
        self.graph = self.d.build_decode_graph(self.tasks, False)

    # -- scratch
    def _alloc_rows(self) -> None:
        c, R, e = self.cfg, self.R, self.cfg.act // 8
        need: Dict[str, int] = {}

        def want(name: str, nbytes: int) -> None:
            need[name] = max(need.get(name, 0), nbytes + 256)   # slack: padded walks may read past the last row

        D = pad(c.width)
        for n, b in (("x", 4), ("h1", e), ("h2", e)):
            want(n, R * D * b)
        most = {rows: max(self._out_parts(i, rows) for i in range(c.n_layers)) for rows in {R, *range(1, min(R, 2048) + 1)}}
        want("mix", max(rows * p for rows, p in most.items()) * D * 4)
        if c.looped and c.join:
            want("cat", R * 2 * D * e)
            want("x2", D * 4)
        for l in c.layers:
            m, f = l.mixer, l.experts
            if l.joint:
                joint_layers.scratch(m, l.mlp, R, c.act, c.capacity, want)
            elif m.kind == "latent_attention":
                want("low", R * pad(m.low_rows) * 4)
                want("cq", R * pad(m.q_rank) * e)
                want("q", R * pad(m.heads * m.hs) * e)
                want("qa", R * m.heads * m.rank_ld * e)
                want("ol", R * m.heads * m.rank_ld * e)
                want("att", R * pad(m.heads * m.vdim_ld) * e)
                want("rot", m.rot_dims * 4)
                if self._split_latent(m):
                    most = max(rows * self._splits(m, rows)[0] for rows in range(1, R + 1) if not self._long_latent(m, rows))
                    want("part", most * m.heads * (m.rank_ld + 2) * 4)
                if self._long_latent(m, R):
                    want("kx", (m.window - 1 + R) * m.heads * m.dim_ld * e)
                    want("vx", m.heads * m.vdim_ld * self._ldv(m) * e)
            else:
                want("u", R * pad(m.inner + m.channels) * e)
                want("dt", R * pad(m.heads) * 4)
                want("xbc", R * pad(m.channels) * e)
                want("y", R * pad(m.inner) * e)
                want("g", R * pad(m.inner) * e)
                if self._long_ssm(m, R):
                    want("chunks", -(-R // 64) * m.heads * m.vdim * m.state_ld * 4)
                    want("decay", -(-R // 64) * m.heads * 4)
            if f:
                want("rl", R * pad(f.outputs) * 4)
                want("ridx", R * f.top * 4)
                want("rwt", R * f.top * 4)
                want("eh", R * f.top * pad(f.ff) * e)
                want("eo", R * f.top * D * e)
                want("perm", R * f.top * 4)
                want("tiles", (R * f.top // 32 + f.experts) * 16)
                want("tile_count", 4)
        for name, nbytes in need.items():
            self.buf[name] = native.zeros(nbytes)

    # -- which form a portion takes
    def _long_latent(self, m: LatentAttention, rows: int) -> bool:
        """Keys and values formed once for the pass (instead of queries carried into the latent space)."""
        return self.cfg.act == 16 and self.cfg.tiled and rows >= 64 and native.latent_prefill_supported(m.dim_ld, m.rot_ld, m.vdim_ld)

    def _split_latent(self, m: LatentAttention) -> bool:
        """The window of a few query rows split over workgroups on the matrix cores (instead of a workgroup per head)."""
        return self.cfg.act == 16 and self.cfg.tiled and native.latent_split_supported(m.rank_ld, m.ldc)

    def _splits(self, m: LatentAttention, rows: int) -> Tuple[int, int]:
        """(splits, positions per split): whole 64-position tiles, fewer and longer splits as rows fill the device."""
        tiles = -(-m.window // 64)
        groups = rows * -(-m.heads // 16)
        span = 64 * max(1, -(-tiles // 32), min(tiles, tiles * groups // 1024))
        return -(-m.window // span), span

    def _ldv(self, m: LatentAttention) -> int:
        return pad(m.window - 1 + self.R + 64)

    def _long_ssm(self, m: Mamba2, rows: int) -> bool:
        """The recurrence in chunks (instead of token after token)."""
        return self.cfg.act == 16 and self.cfg.tiled and rows >= 64 and native.ssm_chunk_supported(m.heads, m.vdim, m.state)

    def _grouped(self, f: Experts, rows: int) -> int:
        """Routes per tile of the grouped expert products, 0: route by route."""
        if self.cfg.act != 16 or not self.cfg.tiled or rows <= 8:
            return 0
        per = rows * f.top / f.outputs
        return 32 if per <= 32 else 64 if per <= 96 else 128

    # -- task lists
    def _name(self, kind: str) -> str:
        self._fid += 1
        return f"fusekit_{kind}_f{self._fid}"

    def _dense(self, t: List[Dispatch], x, W: DeviceWeight, y, rows: int, ldx: int, ldy: int, n0: int = 0, n: Optional[int] = None,
               y32: bool = False, **more) -> None:
        """y = x . W[n0 : n0 + n]^T."""
        n = W.n - n0 if n is None else n
        k = more.pop("k", W.k)      # a part of the sum
        t.append(Dispatch(self._name("dense"), [x, arg(W.w, (W.w.nbytes // (2 * W.k) - n0) * W.k * 2, n0 * W.k * 2)] + more.pop("base", []) + [y] + more.pop("tail", []),
                          dict(rows=rows, n=n, k=k, ldx=ldx, ldw=W.k, ldy=ldy, y32=int(y32), act=self.cfg.act, **more)))

    def _norm_tasks(self, t, run: int, rows: int, first: bool) -> None:
        """The residual sum behind run - 1 (nothing yet when `first`), the vector ahead of a loop pass and the norms
        that run `run` (or the head) reads."""
        c, w, b = self.cfg, self.w, self.buf
        D = pad(c.width)
        shape = dict(rows=rows, width=c.width, ld=D, act=c.act, eps=c.eps)
        p, a = dict(shape), [arg(b["x"])]

        def norm(name: str) -> None:
            a.append(arg(w.vecs[name]))
            if c.layer_norm:
                a.append(arg(w.vecs[name + ".b"]))
                p["layer_norm"] = 1
            a.append(arg(b["h1"]))
            p["has_h1"] = 1

        if not first:
            a.append(arg(b["mix"]))
            p.update(has_mix=1, mix_parts=self._out_parts(self.runs[run - 1][0], rows))
            f = c.layers[self.runs[run - 1][0]].experts
            if f:
                a += [arg(b["eo"]), arg(b["rwt"]), arg(b["ridx"]), arg(b["h2"])]
                p.update(top=f.top, experts=f.experts)
        if run == len(self.runs):
            norm("final.norm")
        else:
            i, step = self.runs[run]
            if step is not None and c.join:   # the stream beside the embedding output, their product is the new stream
                a.append(arg(b["cat"]))
                p["ldcopy"] = 2 * D
                t.append(Dispatch(self._name("residual_norm"), list(a), dict(p)))
                self._dense(t, arg(b["cat"]), w.mats["loop.in"], arg(b["x"]), rows, 2 * D, D, y32=True)
                a[:], p = [arg(b["x"])], dict(shape)
            elif step is not None:
                a.append(arg(w.vecs["loop.step"], D * 2, step * D * 2))
                p["has_step"] = 1
            norm(f"l{i}.norm1")
            if c.layers[i].experts:
                a += [arg(w.vecs[f"l{i}.norm2"]), arg(b["h2"])]
                p["has_h2"] = 1
        t.append(Dispatch(self._name("residual_norm"), a, p))

    def _latent_tasks(self, t, run: int, rows: int, off) -> None:
        c, w, b = self.cfg, self.w, self.buf
        i = self.runs[run][0]
        m, p, act, e = c.layers[i].mixer, f"l{i}.mix.", c.act, c.act // 8
        cache, ring = self.state.entries[run]["cache"], self.state.rings[run]
        D, L, Q, A = pad(c.width), pad(m.low_rows), pad(m.heads * m.hs), pad(m.heads * m.vdim_ld)
        self._dense(t, arg(b["h1"]), w.mats[p + "down"], arg(b["low"]), rows, D, L, y32=True)
        t.append(Dispatch(self._name("group_norm"), [arg(b["low"]), arg(w.vecs[p + "dq.norm"]), arg(b["cq"])],
                          dict(rows=rows, width=m.q_rank, ldx=L, ldy=pad(m.q_rank), x32=1, act=act, eps=c.eps)))
        self._dense(t, arg(b["cq"]), w.mats[p + "uq"], arg(b["q"]), rows, pad(m.q_rank), Q)
        t.append(Dispatch(self._name("latent_store"),
                          [arg(b["low"], None, m.q_rank * 4), arg(w.vecs[p + "dkv.norm"]), arg(w.vecs[p + "rot_freq"]), arg(cache), arg(b["q"]), off],
                          dict(rows=rows, rank=m.kv_rank, rank_ld=m.rank_ld, ldkv=L, ldc=m.ldc, ring=ring, heads=m.heads, hs=m.hs,
                               dim_ld=m.dim_ld, rot=m.rot_dim, rot_dims=m.rot_dims, ldq=Q, eps=c.eps, act=act)))
        if self._long_latent(m, rows):
            ldk, ldv, seen = m.heads * m.dim_ld, self._ldv(m), m.window - 1 + rows
            back = dict(ring=ring, row_back=m.window - 1)
            self._dense(t, arg(cache), w.mats[p + "uk"], arg(b["kx"]), seen, m.ldc, ldk, base=[off], **back)
            self._dense(t, arg(cache), w.mats[p + "uv"], arg(b["vx"]), seen, m.ldc, ldv, base=[off], transposed=1, **back)
            t.append(Dispatch(self._name("latent_prefill"),
                              [arg(b["q"]), arg(b["kx"]), arg(b["vx"]), arg(cache), arg(w.vecs[p + "sink"]), off, arg(b["att"])],
                              dict(rows=rows, heads=m.heads, dim_ld=m.dim_ld, rot_ld=m.rot_ld, vdim_ld=m.vdim_ld, rank_ld=m.rank_ld, ldq=Q,
                                   ldk=ldk, ldv=ldv, ldo=A, ldc=m.ldc, ring=ring, window=m.window, scale=m.scale)))
            self._dense(t, arg(b["att"]), w.mats[p + "o"], arg(b["mix"]), rows, A, D, y32=True)
            return
        lat = m.heads * m.rank_ld
        self._dense(t, arg(b["q"]), w.mats[p + "uk_t"], arg(b["qa"]), rows, Q, lat, n=m.kv_rank, batch=m.heads, xb=m.hs,
                    wb=m.kv_rank * w.mats[p + "uk_t"].k, yb=m.rank_ld)
        if self._split_latent(m):
            t.append(self._split_task(m, p, run, rows, off, rotate=False))
        else:
            t.append(Dispatch(self._name("latent_attn"),
                              [arg(b["qa"]), arg(b["q"]), arg(cache), arg(w.vecs[p + "sink"]), off, arg(b["ol"])],
                              dict(rows=rows, heads=m.heads, hs=m.hs, dim_ld=m.dim_ld, rot=m.rot_dim, rank=m.kv_rank, rank_ld=m.rank_ld,
                                   ldc=m.ldc, ldq=Q, ring=ring, window=m.window, scale=m.scale, act=act)))
        self._dense(t, arg(b["ol"]), w.mats[p + "uv"], arg(b["att"]), rows, lat, A, n=m.vdim_ld, batch=m.heads, xb=m.rank_ld,
                    wb=m.vdim_ld * w.mats[p + "uv"].k, yb=m.vdim_ld)
        self._dense(t, arg(b["att"]), w.mats[p + "o"], arg(b["mix"]), rows, A, D, y32=True)

    def _split_task(self, m: LatentAttention, p: str, run: int, rows: int, off, rotate: bool) -> Dispatch:
        """Split attention; `rotate`: q is not rotated yet and the partial rows are left to the product with W_uv."""
        w, b = self.w, self.buf
        splits, span = self._splits(m, rows)
        cache = self.state.entries[run]["cache"]
        a = [arg(b["qa"]), arg(b["q"]), arg(cache), off] + ([arg(b["rot"])] if rotate else []) + [arg(b["part"])]
        a += [] if rotate else [arg(w.vecs[p + "sink"]), arg(b["ol"])]
        return Dispatch(self._name("latent_split"), a,
                        dict(rows=rows, heads=m.heads, hs=m.hs, dim_ld=m.dim_ld, rot=m.rot_dim, rot_dims=m.rot_dims, rank_ld=m.rank_ld,
                             ldc=m.ldc, ldq=pad(m.heads * m.hs), ring=self.state.rings[run], window=m.window, splits=splits, span=span,
                             scale=m.scale, rotate=int(rotate), combine=int(not rotate)))

    # -- one decoded token in fused launches
    def _fused(self) -> bool:
        """Whether every layer has the fused decode launches."""
        c = self.cfg
        if c.act != 16 or not c.fuse or not c.tiled or pad(c.width) * (2 if c.looped and c.join else 1) > 30720:
            return False
        for l in c.layers:
            m, f = l.mixer, l.experts
            ko = 0
            if l.joint:
                ko = joint_layers.Columns(m, l.mlp).ko
                if not joint_layers.fusable(m):
                    return False
            elif m.kind == "latent_attention":
                ko = pad(m.heads * m.vdim_ld)
                if not self._split_latent(m) or max(pad(m.q_rank), m.rank_ld) > 30720:
                    return False
            elif m.norm_groups > 64 or pad(m.inner) > 30720 or m.state > 256:
                return False
            kf = f.top * pad(f.ff) if f else 0
            items = -(-ko // 512) + (f.top * -(-pad(f.ff) // 512) if f else 0) + 2
            if (ko + kf) * 2 + items * 24 + 16 > 60 * 1024:
                return False
        return True

    def _jobs(self, t: List[Dispatch], args: list, **params) -> None:
        t.append(Dispatch(self._name("layer_jobs"), args, params))

    def _product(self, i: int, W: DeviceWeight, n_act: int, **more) -> Dict[str, float]:
        return {f"g{i}_{k}": v for k, v in dict(more, n=W.n, k=W.k, ldw=W.k, n_act=n_act).items()}

    def _fused_tasks(self, t: List[Dispatch]) -> None:
        c, w, b = self.cfg, self.w, self.buf
        off, D = arg(self.offset), pad(c.width)
        t.append(self._embed_task(arg(self.token), off, 1))
        x, other = arg(b["x"]), arg(b["x2"]) if "x2" in b else None
        for run, (i, first) in enumerate(self.runs):
            m, f, p = c.layers[i].mixer, c.layers[i].experts, f"l{i}."
            q = p + "mix."
            st = self.state.entries[run]
            step = []
            if first is not None and c.join:   # a product of the whole row: into the other of two rows
                W = w.mats["loop.in"]
                self._jobs(t, [x, arg(b["cat"], None, D * 2), arg(W.w), other], **self._product(0, W, 0, mode=4, width=c.width))
                x, other = other, x
            elif first is not None:
                step = [arg(w.vecs["loop.step"], D * 2, first * D * 2)]
            if c.layers[i].joint:
                self._fused_joint_tasks(t, run, x, step)
                continue
            norm = dict(mode=1, width=c.width, eps=c.eps, step=len(step), layer_norm=int(c.layer_norm))
            norm1 = [arg(w.vecs[p + "norm1"])] + ([arg(w.vecs[p + "norm1.b"])] if c.layer_norm else [])
            latent = m.kind == "latent_attention"
            # 1: norms; the mixer's joint down / input projection and the router
            Win = w.mats[q + ("down" if latent else "in")]
            n_act = 0 if latent else m.inner + m.channels
            a = [x] + step + norm1 + [arg(Win.w)]
            a += [arg(b["low"])] if latent else [arg(b["u"]), arg(b["dt"])]
            prm = self._product(0, Win, n_act, **norm)
            if f:
                Wr = w.mats[p + "mlp.router"]
                a += [x] + step + [arg(w.vecs[p + "norm2"]), arg(b["h2"]), arg(Wr.w), arg(b["rl"])]
                prm.update(self._product(1, Wr, 0, keep=1, **dict(norm, layer_norm=0)))
            self._jobs(t, a, **prm)
            route = [arg(b["rl"]), arg(w.vecs[p + "mlp.correction"]), arg(b["ridx"]), arg(b["rwt"])] if f else []
            prm_route = dict(route_outputs=f.outputs, route_top=f.top) if f else {}
            pair, prm_pair = [], {}
            if f:
                F = pad(f.ff)
                pair = [arg(b["h2"]), arg(w.mats[p + "mlp.gate"].w), arg(w.mats[p + "mlp.up"].w), arg(b["ridx"]), arg(b["eh"])]
                prm_pair = dict(pair_n=f.ff, pair_k=D, pair_ldw=D, pair_ldy=F, pair_top=f.top, pair_experts=f.experts)
            if latent:
                # 2: queries, the cache row, the choice of experts
                Wq, Wk, Wv = w.mats[q + "uq"], w.mats[q + "uk_t"], w.mats[q + "uv"]
                a = [arg(b["low"]), arg(w.vecs[q + "dq.norm"]), arg(Wq.w), arg(b["q"])] + route
                a += [arg(b["low"], None, m.q_rank * 4), arg(w.vecs[q + "dkv.norm"]), arg(w.vecs[q + "rot_freq"]), off, arg(st["cache"]), arg(b["rot"])]
                self._jobs(t, a, **self._product(0, Wq, Wq.n, mode=1, width=m.q_rank, eps=c.eps), **prm_route, store_rank=m.kv_rank,
                           store_rank_ld=m.rank_ld, store_ldc=m.ldc, store_ring=self.state.rings[run], store_rot=m.rot_dim,
                           store_rot_dims=m.rot_dims, store_eps=c.eps)
                # 3: queries into the latent space, gate / up
                self._jobs(t, [arg(b["q"]), arg(Wk.w), arg(b["qa"])] + pair,
                           **self._product(0, Wk, Wk.n, mode=0, rows_per_head=m.kv_rank, x_head=m.hs, y_head=m.rank_ld), **prm_pair)
                # 4, 5: attention over the window, its combination and W_uv
                t.append(self._split_task(m, q, run, 1, off, rotate=True))
                self._jobs(t, [arg(b["part"]), arg(w.vecs[q + "sink"]), arg(Wv.w), arg(b["att"])],
                           **self._product(0, Wv, Wv.n, mode=3, rows_per_head=m.vdim_ld, y_head=m.vdim_ld, heads=m.heads,
                                           splits=self._splits(m, 1)[0]))
            else:
                # 2: convolution and state, the choice of experts
                a = route + [arg(b["u"], None, m.inner * 2), arg(b["dt"]), arg(w.vecs[q + "conv"]), arg(w.vecs[q + "conv.b"]), arg(w.vecs[q + "dt_bias"]),
                             arg(w.vecs[q + "A_log"]), arg(w.vecs[q + "D"]), off, arg(st["state"]), arg(st["hist"]), arg(b["y"])]
                self._jobs(t, a, **prm_route, scan_heads=m.heads, scan_groups=m.groups, scan_n=m.state, scan_p=m.vdim, scan_state_ld=m.state_ld,
                           scan_ldh=pad(m.channels), scan_taps=m.conv)
                # 3: gated norm and output projection, gate / up
                Wo = w.mats[q + "o"]
                self._jobs(t, [arg(b["y"]), arg(b["u"]), arg(w.vecs[q + "norm"]), arg(Wo.w), arg(b["mix"])] + pair,
                           **self._product(0, Wo, 0, mode=2, width=m.inner, groups=m.norm_groups, eps=c.eps), **prm_pair)
            # last: everything into the residual row
            a, prm = [x], dict(n=c.width)
            if latent:
                A = pad(m.heads * m.vdim_ld)
                a += [arg(b["att"]), arg(w.mats[q + "o"].w)]
                prm.update(ko=A, ldo=A)
            else:
                a.append(arg(b["mix"]))
                prm["has_mix"] = 1
            if f:
                a += [arg(b["eh"]), arg(w.mats[p + "mlp.down"].w), arg(b["ridx"]), arg(b["rwt"]), arg(b["h2"])]
                prm.update(kf=pad(f.ff), top=f.top, experts=f.experts)
            if step:
                a += step
                prm["has_step"] = 1
            t.append(Dispatch(self._name("layer_out"), a, prm))
        head = w.mats["head"]
        norm = [arg(w.vecs["final.norm"])] + ([arg(w.vecs["final.norm.b"])] if c.layer_norm else [])
        self._jobs(t, [x] + norm + [arg(head.w), arg(self.logits)],
                   **self._product(0, head, 0, mode=1, width=c.width, eps=c.eps, layer_norm=int(c.layer_norm)))

    def _ssm_tasks(self, t, run: int, rows: int, off) -> None:
        c, w, b = self.cfg, self.w, self.buf
        i = self.runs[run][0]
        m, p, act, e = c.layers[i].mixer, f"l{i}.mix.", c.act, c.act // 8
        st = self.state.entries[run]
        D, U, X, Y, T, H = pad(c.width), pad(m.inner + m.channels), pad(m.channels), pad(m.inner), pad(m.heads), pad(m.channels)
        Win = w.mats[p + "in"]
        self._dense(t, arg(b["h1"]), Win, arg(b["u"]), rows, D, U, n=m.inner + m.channels)
        self._dense(t, arg(b["h1"]), Win, arg(b["dt"]), rows, D, T, n0=m.inner + m.channels, y32=True)
        u = arg(b["u"], None, m.inner * e)
        t.append(Dispatch(self._name("ssm_conv"),
                          [u, arg(w.vecs[p + "conv"]), arg(w.vecs[p + "conv.b"]), arg(st["hist"]), off, arg(b["xbc"])],
                          dict(rows=rows, channels=m.channels, taps=m.conv, ldu=U, ldy=X, ldh=H, act=act)))
        long = self._long_ssm(m, rows)
        t.append(Dispatch(self._name("ssm_chunk" if long else "ssm_scan"),
                          [arg(b["xbc"]), arg(b["dt"]), arg(w.vecs[p + "dt_bias"]), arg(w.vecs[p + "A_log"]), arg(w.vecs[p + "D"]), u, off,
                           arg(st["state"]), arg(st["hist"]), arg(b["y"])] + ([arg(b["chunks"]), arg(b["decay"])] if long else []),
                          dict(rows=rows, heads=m.heads, groups=m.groups, n=m.state, p=m.vdim, state_ld=m.state_ld, ldx=X, lddt=T, ldy=Y,
                               ldu=U, ldh=H, channels=m.channels, taps=m.conv, act=act)))
        t.append(Dispatch(self._name("group_norm"), [arg(b["y"]), arg(b["u"]), arg(w.vecs[p + "norm"]), arg(b["g"])],
                          dict(rows=rows, width=m.inner, groups=m.norm_groups, ldx=Y, ldz=U, ldy=Y, has_z=1, act=act, eps=c.eps)))
        self._dense(t, arg(b["g"]), w.mats[p + "o"], arg(b["mix"]), rows, Y, D, y32=True)

    def _expert_tasks(self, t, run: int, rows: int) -> None:
        c, w, b = self.cfg, self.w, self.buf
        i = self.runs[run][0]
        f, p, act = c.layers[i].mlp, f"l{i}.mlp.", c.act
        D, O, F = pad(c.width), pad(f.outputs), pad(f.ff)
        self._dense(t, arg(b["h2"]), w.mats[p + "router"], arg(b["rl"]), rows, D, O, y32=True)
        t.append(Dispatch(self._name("route_rows"), [arg(b["rl"]), arg(w.vecs[p + "correction"]), arg(b["ridx"]), arg(b["rwt"])],
                          dict(rows=rows, outputs=f.outputs, top=f.top, ld=O)))
        q = dict(routes=rows * f.top, experts=f.experts, act=act)
        tile, groups = self._grouped(f, rows), []
        if tile:
            groups = [arg(b["perm"]), arg(b["tiles"]), arg(b["tile_count"])]
            t.append(Dispatch(self._name("route_group"), [arg(b["ridx"])] + groups, dict(routes=rows * f.top, experts=f.experts, tile_rows=tile)))
            q.update(grouped=1, tile_rows=tile)
        t.append(Dispatch(self._name("experts"),
                          [arg(b["h2"]), arg(w.mats[p + "gate"].w), arg(w.mats[p + "up"].w), arg(b["ridx"])] + groups + [arg(b["eh"])],
                          dict(q, n=f.ff, k=D, ldx=D, ldw=D, ldy=F, x_div=f.top, pair=1)))
        t.append(Dispatch(self._name("experts"), [arg(b["eh"]), arg(w.mats[p + "down"].w), arg(b["ridx"])] + groups + [arg(b["eo"])],
                          dict(q, n=c.width, k=F, ldx=F, ldw=F, ldy=D, x_div=1)))

    def _embed_task(self, tokens, off, rows: int) -> Dispatch:
        """Embedding rows; with a join their copies beside the place of the stream."""
        c, b, W, D = self.cfg, self.buf, self.w.mats["embed"], pad(self.cfg.width)
        if not c.padded_lookup:
            return Dispatch(self._name("embed_lookup_decode"), [tokens, arg(W.w), arg(b["x"])],
                            dict(bits=16, hidden=c.width, vocab=c.vocab, output_scale=c.embed_scale, rows=rows, out_bits=32, x_row_stride=D))
        a, p = [tokens, arg(W.w)], dict(rows=rows, width=c.width, vocab=c.vocab, ldw=W.k, ld=D, scale=c.embed_scale, act=c.act)
        if c.pairs:
            n = c.pairs.buckets
            a += [arg(self.w.mats["bigram"].w), arg(self.state.prev), off]
            p.update(buckets=n, mul_prev=c.pairs.mul_prev % n, mul_cur=c.pairs.mul_cur % n)
        a.append(arg(b["x"]))
        if c.looped and c.join:
            a.append(arg(b["cat"], None, D * (c.act // 8)))
            p["ldcopy"] = 2 * D
        return Dispatch(self._name("embed_rows"), a, p)

    def _body_tasks(self, t, tokens, off, kv_len, rows: int) -> None:
        """Embedding to the final norm of `rows` tokens; h1 holds the head's input rows."""
        c, b = self.cfg, self.buf
        t.append(self._embed_task(tokens, off, rows))
        self._norm_tasks(t, 0, rows, True)
        for run, (i, _) in enumerate(self.runs):
            if c.layers[i].joint:
                self._joint_tasks(t, run, rows, off, kv_len)
            elif c.layers[i].mixer.kind == "latent_attention":
                self._latent_tasks(t, run, rows, off)
            else:
                self._ssm_tasks(t, run, rows, off)
            if c.layers[i].experts:
                self._expert_tasks(t, run, rows)
            self._norm_tasks(t, run + 1, rows, False)

    def _argmax_task(self) -> Dispatch:
        return Dispatch(self._name("argmax_logits_decode"),
                        [arg(self.logits, pad(self.cfg.vocab) * 4), arg(self.token), arg(self.argmax_ws), arg(self.history), arg(self.hist_counter)],
                        dict(vocab=self.cfg.vocab, logits_bits=32))

    def build_tasks(self) -> List[Dispatch]:
        self._fid = 0
        c = self.cfg
        t = [Dispatch("fusekit_step_init", [arg(self.step_counter), arg(self.offset), arg(self.kv_len)])]
        self.fused = self._fused()
        if self.fused:
            self._fused_tasks(t)
        else:
            self._body_tasks(t, arg(self.token), arg(self.offset), arg(self.kv_len), 1)
            self._dense(t, arg(self.buf["h1"]), self.w.mats["head"], arg(self.logits), 1, pad(c.width), pad(c.vocab), y32=True)
        t.append(self._argmax_task())
        return t

    def rows_tasks(self, rows: int) -> List[Dispatch]:
        """The task list of a portion of `rows` tokens at positions *row_offset .. *row_kv - 1 (device words, as are the tokens)."""
        self._fid = 0
        t: List[Dispatch] = []
        self._body_tasks(t, arg(self.tokens, rows * 4), arg(self.row_offset), arg(self.row_kv), rows)
        return t

    # -- running
    def reset(self) -> None:
        self.position = 0
        for b in (self.step_counter, self.offset, self.kv_len, self.hist_counter):
            b.upload(np.zeros(1, np.uint32))
        self.state.reset()

    def _run_rows(self, tokens: np.ndarray) -> None:
        m = len(tokens)
        self.tokens.upload(tokens)
        self.row_offset.upload(np.array([self.position], np.uint32))
        self.row_kv.upload(np.array([self.position + m], np.uint32))
        if m == self.R:                      # whole passes are replayed; odd portions are launched as they come
            if self._full_pass is None:
                self._full_pass = self.d.build_decode_graph(self.rows_tasks(m), False)
            self.d.execute_graph(self._full_pass)
        else:
            tasks = self._passes.pop(m, None) or self.d.prepare(self.rows_tasks(m))
            self._passes[m] = tasks
            if len(self._passes) > 16:
                self._passes.popitem(last=False)
            self.d.dispatch_prepared(tasks)
        self.position += m

    def _head_rows(self, rows: Sequence[int], argmax: bool = False) -> None:
        """Logits of the given rows of the last pass (at most HEAD_ROWS) into `logits`."""
        c, ld = self.cfg, pad(self.cfg.width)
        nb = ld * (c.act // 8)
        for k, r in enumerate(rows):
            native.copy(self.head_x.ptr + k * nb, self.buf["h1"].ptr + r * nb, nb)
        native.sync()
        self._fid = 0
        t: List[Dispatch] = []
        self._dense(t, arg(self.head_x), self.w.mats["head"], arg(self.logits), len(rows), ld, pad(c.vocab), y32=True)
        if argmax:
            t.append(self._argmax_task())
        self.d.dispatch_batch(t)

    def _logits(self, rows: int) -> np.ndarray:
        return self.logits.to_numpy(np.float32, (rows, pad(self.cfg.vocab)))[:, :self.cfg.vocab]

    def _check_tokens(self, tokens: Sequence[int]) -> np.ndarray:
        t = np.asarray(tokens, np.int64)
        if t.ndim != 1 or t.size == 0 or t.min() < 0 or t.max() >= self.cfg.vocab:
            raise ValueError("token ids must lie in 0 .. vocab - 1, at least one")
        self._check_room(t.size)
        return t.astype(np.uint32)

    def _check_room(self, n: int) -> None:
        limit = self.cfg.max_positions
        if limit is not None and self.position + n > limit:
            raise ValueError(f"the sequence would exceed the cache's {limit} positions")

    def step(self, tokens: Sequence[int], want: Sequence[int] = ()) -> np.ndarray:
        """Runs the sequence's next tokens from the state earlier calls left; logits [len(want), vocab] at the wanted
        places among them.  One token goes through the decode graph, more through rows passes."""
        t, want = self._check_tokens(tokens), list(want)
        out = np.empty((len(want), self.cfg.vocab), np.float32)
        if len(t) == 1:
            self.d.decode_host_loop(self.graph, self.uniforms, self.position, t.tolist())
            self.position += 1
            if want:
                out[:] = self._logits(1)
            return out
        for p0 in range(0, len(t), self.R):
            part = t[p0:p0 + self.R]
            self._run_rows(part)
            here = [(k, r - p0) for k, r in enumerate(want) if p0 <= r < p0 + len(part)]
            for g0 in range(0, len(here), self.HEAD_ROWS):
                group = here[g0:g0 + self.HEAD_ROWS]
                self._head_rows([r for _, r in group])
                out[[k for k, _ in group]] = self._logits(len(group))
        return out

    def prefill(self, prompt: Sequence[int], start_offset: int = 0) -> int:
        """Runs the prompt behind what the state holds (start_offset must be that position) and returns the greedy
        token after it."""
        if start_offset != self.position:
            raise ValueError(f"the state ends at position {self.position}, not {start_offset}")
        t = self._check_tokens(prompt)
        if len(t) == 1:
            nxt, _ = self.d.decode_host_loop(self.graph, self.uniforms, self.position, t.tolist())
            self.position += 1
            return nxt[-1]
        for p0 in range(0, len(t), self.R):
            self._run_rows(t[p0:p0 + self.R])
        self._head_rows([(len(t) - 1) % self.R], argmax=True)
        return int(self.token.to_numpy(np.uint32)[0])

    def generate(self, prompt: Sequence[int], max_tokens: int):
        """Greedy decode of a new sequence: (tokens, seconds on the GPU for the decode chunks, decode steps)."""
        self.reset()
        out = [self.prefill(prompt)]
        gpu_s, steps = 0.0, 0
        while len(out) < max_tokens:
            n = min(FK_CHUNK, max_tokens - len(out), self.uniforms.hist_capacity)
            self._check_room(n)
            toks, sec = self.d.decode_chunk(self.graph, self.uniforms, self.position, out[-1], n)
            self.position += n
            out += toks
            gpu_s += sec
            steps += n
        return out, gpu_s, steps

    def scratch_symbols(self):
        """name -> (buffer, dtype, zero-initialised) of every arena buffer, as the artifact describes them."""
        act = "float32" if self.cfg.act == 32 else "bfloat16"
        out = {n: (getattr(self, n), "uint32", True) for n in ("token", "step_counter", "offset", "kv_len", "hist_counter", "history", "argmax_ws")}
        out["logits"] = (self.logits, "float32", True)
        words = ("ridx", "perm", "tiles", "tile_count", "counters")
        floats = ("x", "x2", "mix", "low", "dt", "rl", "rwt", "rot", "part", "chunks", "decay", "beta", "decays", "qk", "o", "gates", "carry")
        for n, b in self.buf.items():
            out[n] = (b, "uint32" if n in words else "float32" if n in floats else act, True)
        out["state.prev"] = (self.state.prev, "uint32", True)
        for r, e in enumerate(self.state.entries):
            for n, b in e.items():
                out[f"state.{n}.{r}"] = (b, "float32" if n == "state" else act, True)
        return out
