"""Prefill and decode throughput of the layer-list decoder at sizes that resemble a real model's layers, beside the closest
other model at equal size: Pusavik beside the mixture-of-experts decoder with low-rank keys (`python bench.py --workload
pusavik`), Fumotar beside Pusavik with one expert, which is a dense feed-forward (`--workload fumotar`).

Pusavik and the mixture-of-experts decoder have the same number of layers, width, heads, experts, active experts and vocabulary; the layer-list model
alternates latent attention and Mamba-2 mixers and keeps bf16 matrices, the other one has attention in every layer and
int4 matrices.  Fumotar and its Pusavik have the same layers, width, vocabulary and number of feed-forward weights, and bf16
matrices both.  Random weights, generated in HBM.  Per launch shape: algorithmic bytes or flops over the average launch
time in a chain of dependent launches with distinct weights (HIP events), as a fraction of the published peaks."""
from __future__ import annotations

import math
import time
from typing import Dict, List

import numpy as np

HBM_PEAK, MFMA_PEAK = 8.0e12, 2.5e15

# width, heads, kv rank, q rank, window, ssm heads, ssm groups, experts, identity, top, ff, vocab
SIZES = {
    "1k": dict(width=1024, heads=8, kv_rank=256, q_rank=512, window=512, ssm_heads=32, groups=4, experts=32, identity=4, top=6, ff=704, vocab=32768),
    "2k": dict(width=2048, heads=16, kv_rank=512, q_rank=1024, window=1024, ssm_heads=64, groups=8, experts=64, identity=8, top=8, ff=1408, vocab=102400),
    "4k": dict(width=4096, heads=32, kv_rank=512, q_rank=1536, window=1024, ssm_heads=128, groups=8, experts=64, identity=8, top=8, ff=2048, vocab=102400),
}
LAYERS = 8

# width, ff, attention heads / kv heads, delta heads, block and number of the linear recurrence, vocab; heads are 128 wide
JOINT_SIZES = {
    "1k": dict(width=1024, ff=4096, heads=8, kv_heads=2, delta_heads=8, blocks=8, rank=64, vocab=32768),
    "2k": dict(width=2048, ff=8192, heads=16, kv_heads=4, delta_heads=16, blocks=8, rank=128, vocab=102400),
    "4k": dict(width=4096, ff=16384, heads=32, kv_heads=8, delta_heads=32, blocks=16, rank=128, vocab=102400),
}


def joint_config(s: dict, rows_per_pass: int = 2048, capacity: int = 4096):
    from .joint_layers import CausalAttention, ChannelDelta, DenseMlp, RgLru, RotaryScaling
    from .layer_decoder import Layer, LayerConfig, PairTable
    att = CausalAttention(heads=s["heads"], kv_heads=s["kv_heads"], dim=128, scale=128 ** -0.5, rot_base=1e5, rot_dims=128,
                          rot_scaling=RotaryScaling(factor=4.0, original=4096, fast=24.0, slow=1.5))
    dlt = ChannelDelta(heads=s["delta_heads"], kv_heads=s["delta_heads"], dim=128, vdim=128, conv=4, decay_rank=s["rank"], gate_rank=s["rank"])
    lru = RgLru(width=s["width"], blocks=s["blocks"], conv=4)
    mlp = DenseMlp(s["ff"])
    return LayerConfig(width=s["width"], vocab=s["vocab"], layers=[Layer((dlt, lru, att)[i % 3], mlp) for i in range(LAYERS)], rows_per_pass=rows_per_pass,
                       capacity=capacity, design="Fumotar", layer_norm=True, tied=True, join=True, loop_start=0, loop_stop=LAYERS, loop_times=1,
                       pairs=PairTable(buckets=65535, mul_prev=8191, mul_cur=127))


def like_joint_config(s: dict, rows_per_pass: int = 2048):
    """The layer-list model of the other design with the same width, layers and feed-forward weights."""
    from .layer_decoder import Experts, LatentAttention, Layer, LayerConfig, Mamba2
    w = s["width"]
    lat = LatentAttention(heads=s["heads"], dim=128, rot_dim=64, vdim=128, kv_rank=min(512, w // 4), q_rank=w // 2, window=1024, scale=192 ** -0.5, rot_base=1e5, rot_dims=64)
    ssm = Mamba2(heads=w // 32, vdim=64, state=128, groups=max(4, w // 512), conv=4, norm_groups=max(4, w // 512))
    moe = Experts(experts=1, identity=0, top=1, ff=s["ff"] * 2 // 3 // 64 * 64)
    return LayerConfig(width=w, vocab=s["vocab"], layers=[Layer(lat if i % 3 == 2 else ssm, moe) for i in range(LAYERS)], rows_per_pass=rows_per_pass)


def layer_config(s: dict, rows_per_pass: int = 2048):
    from .layer_decoder import Experts, LatentAttention, Layer, LayerConfig, Mamba2
    lat = LatentAttention(heads=s["heads"], dim=128, rot_dim=64, vdim=128, kv_rank=s["kv_rank"], q_rank=s["q_rank"], window=s["window"],
                          scale=192 ** -0.5, rot_base=1e5, rot_dims=64)
    ssm = Mamba2(heads=s["ssm_heads"], vdim=64, state=128, groups=s["groups"], conv=4, norm_groups=s["groups"])
    moe = Experts(experts=s["experts"], identity=s["identity"], top=s["top"], ff=s["ff"])
    return LayerConfig(width=s["width"], vocab=s["vocab"], layers=[Layer(lat if i % 2 else ssm, moe) for i in range(LAYERS)],
                       rows_per_pass=rows_per_pass)


def moe_config(s: dict, capacity: int):
    from .moe_decoder import MoeConfig
    return MoeConfig(n_layers=LAYERS, hidden=s["width"], n_heads=s["heads"], kv_lora_rank=s["kv_rank"], rope_dim=64, nope_dim=128, v_dim=128,
                     n_experts=s["experts"], top_k=s["top"] - 2, moe_inter=s["ff"], n_shared=2, dense_inter=4 * s["width"], first_dense=0,
                     vocab=s["vocab"], capacity=capacity)


def _family(kernel: str) -> str:
    head, sep, tail = kernel[len("fusekit_"):].rpartition("_f")
    return head if sep and tail.isdigit() else kernel[len("fusekit_"):]


def label(t) -> str:
    p = t.params
    f = _family(t.kernel)
    if f == "layer_jobs":
        parts = [f"{int(p[f'g{i}_n'])}x{int(p[f'g{i}_k'])}" for i in (0, 1) if f"g{i}_n" in p]
        parts += [n for n, k in (("gate/up", "pair_n"), ("choice", "route_outputs"), ("cache row", "store_rank"), ("state step", "scan_heads"),
                                 ("delta step", "delta_heads"), ("lru step", "lru_width")) if p.get(k)]
        return "jobs: " + " | ".join(parts)
    if f == "layer_out":
        return "layer out" + (" %dx%d" % (p["n"], p["ko"]) if not p.get("top") else " (o + down)" if p.get("ko") else " (down)")
    if f in ("dense", "experts"):
        extra = " x%d heads" % p["batch"] if p.get("batch", 1) > 1 else ""
        return f"{f} {int(p['n'])}x{int(p['k'])}{extra}" + (" pair" if p.get("pair") else "")
    return f


def measure(rt, tasks, work, reps: int = 64) -> List[dict]:
    """Average launch time per launch shape; `work(task)` -> (bytes, flops)."""
    groups: Dict[str, list] = {}
    for t in tasks:
        if _family(t.kernel) != "step_init":
            groups.setdefault(label(t), []).append(t)
    out = []
    for name, ts in groups.items():
        chain = ts * max(1, min(32 // len(ts), 32))
        g = rt.d.build_graph(chain, barriers=[True] * len(chain))
        rt.d.execute_graph(g)
        n = max(2, reps // len(chain))
        us = rt.d.execute_graph(g, repeat=n) / (n * len(chain)) * 1e6
        b, fl = work(ts[0])
        e = dict(launch=name, count=len(ts), avg_us=round(us, 2))
        if b:
            e["hbm_frac"] = round(b / us / 1e-6 / HBM_PEAK, 4)
        if fl:
            e["mfma_frac"] = round(fl / us / 1e-6 / MFMA_PEAK, 4)
        out.append(e)
    return sorted(out, key=lambda e: -e["avg_us"] * e["count"])


def joint_work(c, rows: int, ctx: int):
    """Algorithmic bytes and flops of a task of a model of joint layers."""
    def work(t):
        p, f = t.params, _family(t.kernel)
        m = lambda *names: math.prod(p[n] for n in names)
        if rows == 1:
            w = {"layer_out": lambda: p["n"] * p["ko"] * 2,
                 "layer_jobs": lambda: (p["g0_n"] * p["g0_k"] * 2 if "g0_n" in p else 0)
                 + (m("delta_heads", "delta_vdim_ld", "delta_state_ld") * 8 + m("delta_heads", "delta_dim_ld", "delta_rank_ld") * 2 if p.get("delta_heads") else 0)
                 + (m("lru_width", "lru_block") * 4 + p["lru_width"] * 8 if p.get("lru_width") else 0),
                 "sdpa_decode": lambda: ctx * m("n_kv", "head_dim") * 4, "qk_store": lambda: (p["heads"] + 3 * p["kv_heads"]) * p["dim_ld"] * 4,
                 "embed_rows": lambda: p["width"] * 8}.get(f)
            return (w() if w else 0), 0
        fl = {"dense": lambda: 2.0 * m("rows", "n", "k") * p.get("batch", 1),
              "sdpa_prefill": lambda: 2.0 * rows * (rows + 1.0) * m("n_heads", "head_dim"),
              # per token and head: keys against keys and queries of the chunk, its triangular solve, three products with the state
              "delta_scan": lambda: 2.0 * rows * p["heads"] * 3 * m("dim_ld", "vdim_ld"),
              "delta_chunk": lambda: 2.0 * rows * p["heads"] * (3 * m("dim_ld", "vdim_ld") + 64 * (3 * p["dim_ld"] + 2 * p["vdim_ld"]) / 2)}.get(f)
        b = {"residual_norm": lambda: rows * c.width * (4 * 3 + 2), "ssm_conv": lambda: rows * p["channels"] * 4,
             "embed_rows": lambda: rows * c.width * (2 * 2 + 4 + 2), "qk_store": lambda: rows * (p["heads"] + 1.5 * p["kv_heads"]) * p["dim_ld"] * 4,
             "delta_prep": lambda: rows * (p["kv_heads"] * p["dim_ld"] * 12 + p["heads"] * p["dim_ld"] * 8),
             "head_norm": lambda: rows * m("heads", "ld") * 8, "lru_scan": lambda: rows * p["width"] * 14,
             "delta_scan": lambda: rows * (p["kv_heads"] * p["dim_ld"] * 8 + p["heads"] * (p["dim_ld"] * 4 + p["vdim_ld"] * 6)),
             # besides: per chunk the operands of its sequential part, written and read once
             "delta_chunk": lambda: rows * (p["kv_heads"] * p["dim_ld"] * 8 + p["heads"] * (p["dim_ld"] * 4 + p["vdim_ld"] * 6))
             + 2 * rows * p["heads"] * (p["dim_ld"] * 12 + p["vdim_ld"] * 4 + 64 * 4),
             "dense": lambda: rows * p["n"] * p["batch"] * 4 + m("n", "k", "batch") * 2 + m("rows", "k", "batch") * 2 if p.get("batch", 1) > 1 and p["n"] == 2 * p["k"] else 0}.get(f)
        return (b() if b else 0), (fl() if fl else 0)

    return work


def joint_token_bytes(c, ctx: int) -> int:
    """Algorithmic HBM bytes of one decoded token of a model of joint layers."""
    from .joint_layers import Columns
    n, state = c.vocab * c.width + (2 * c.width * c.width * c.loop_times if c.looped and c.join else 0), 0
    for i, _ in c.runs():
        m = c.layers[i].mixer
        col = Columns(m, c.layers[i].mlp)
        n += (col.rows + col.ko) * c.width
        if m.kind == "attention":
            state += ctx * m.kv_heads * m.dim_ld * 4
        elif m.kind == "channel_delta":
            n += m.heads * (m.dim_ld * m.decay_rank + m.vdim_ld * m.gate_rank)
            state += 2 * m.heads * m.vdim_ld * m.state_ld * 4
        else:
            n += 2 * m.inner * m.block_ld
            state += 2 * m.inner * 4
    return int(n * 2 + state)


def layer_work(c, rows: int, ctx: int):
    """Algorithmic bytes (decode) or flops (portions) of a task of the layer-list model."""
    if any(l.joint for l in c.layers):
        return joint_work(c, rows, ctx)
    lat = next(l.mixer for l in c.layers if l.mixer.kind == "latent_attention")
    ssm = next(l.mixer for l in c.layers if l.mixer.kind == "mamba2")
    moe = c.layers[0].mlp
    real = moe.top * moe.experts / moe.outputs      # matrices per token, identities aside

    def work(t):
        p, f = t.params, _family(t.kernel)
        if rows == 1:
            w = {"dense": lambda: p["n"] * p["k"] * p.get("batch", 1) * 2,
                 "experts": lambda: real * p["n"] * p["k"] * 2 * (2 if p.get("pair") else 1),
                 "latent_attn": lambda: min(ctx, lat.window) * lat.ldc * 2,
                 "latent_split": lambda: min(ctx, lat.window) * lat.ldc * 2,
                 "layer_out": lambda: p["n"] * (p.get("ko", 0) + real * p.get("kf", 0)) * 2,
                 "layer_jobs": lambda: sum(p[f"g{i}_n"] * p[f"g{i}_k"] * 2 for i in (0, 1) if f"g{i}_n" in p)
                 + (2 * real * p["pair_n"] * p["pair_k"] * 2 if p.get("pair_n") else 0)
                 + (2 * ssm.heads * ssm.vdim * ssm.state * 4 if p.get("scan_heads") else 0),
                 "ssm_scan": lambda: 2 * ssm.heads * ssm.vdim * ssm.state * 4}.get(f)
            return (w() if w else 0), 0
        seen = sum(min(i + 1, lat.window) for i in range(rows))
        fl = {"dense": lambda: 2.0 * p["rows"] * p["n"] * p["k"] * p.get("batch", 1),
              "experts": lambda: 2.0 * rows * real * p["n"] * p["k"] * (2 if p.get("pair") else 1),
              "latent_prefill": lambda: 2.0 * seen * lat.heads * (lat.dim + lat.rot_dim + lat.vdim),
              "ssm_chunk": lambda: 2.0 * rows * ssm.heads * ssm.vdim * (2 * ssm.state + 32) + 2.0 * rows * ssm.groups * 32 * ssm.state}.get(f)
        b = {"residual_norm": lambda: rows * c.width * (4 * 3 + 2 * 2 + 2 * moe.top),
             "group_norm": lambda: rows * p["width"] * 6, "ssm_conv": lambda: rows * p["channels"] * 4,
             "ssm_chunk": lambda: rows * ssm.channels * 2 * 2 + rows // 64 * ssm.heads * ssm.vdim * ssm.state * 4 * 4}.get(f)
        return (b() if b else 0), (fl() if fl else 0)

    return work


def token_bytes(c, ctx: int) -> int:
    """Algorithmic HBM bytes of one decoded token: the matrices it touches, the window's latents, the states."""
    if any(l.joint for l in c.layers):
        return joint_token_bytes(c, ctx)
    n = c.vocab * c.width
    state = 0
    for i, _ in c.runs():
        m, f = c.layers[i].mixer, c.layers[i].mlp
        if m.kind == "latent_attention":
            n += m.low_rows * c.width + m.heads * m.hs * m.q_rank + m.heads * (m.dim + m.vdim) * m.kv_rank + c.width * m.heads * m.vdim
            state += min(ctx, m.window) * m.ldc * 2
        else:
            n += (2 * m.inner + 2 * m.groups * m.state + m.heads) * c.width + c.width * m.inner
            state += 2 * m.heads * m.vdim * m.state * 4
        if f:
            n += f.outputs * c.width + 3 * f.top * f.experts / f.outputs * f.ff * c.width
    return int(n * 2 + state)


def bench_layer(size: str, ctx: int = 1024, steps: int = 128, kernels: bool = True, config=None) -> dict:
    from . import native as fk
    from .layer_decoder import LayerRuntime, LayerWeights
    c = config or layer_config(SIZES[size])
    w = LayerWeights.random_init(c, seed=1)
    rt = LayerRuntime(c, w)
    rng = np.random.Generator(np.random.PCG64(0))
    out: dict = dict(model="%s %s: %d layers, width %d, %.2f GB of bf16 weights" % (c.design, size, LAYERS, c.width, w.nbytes() / 1e9))
    for rows in (512, 2048):
        toks = rng.integers(0, c.vocab, rows).astype(np.uint32)
        rt.reset()
        rt.tokens.upload(toks)
        rt.row_offset.upload(np.zeros(1, np.uint32))
        rt.row_kv.upload(np.array([rows], np.uint32))
        tasks = rt.rows_tasks(rows)
        g = rt.d.build_decode_graph(tasks, False)
        rt.d.execute_graph(g)
        sec = min(rt.d.execute_graph(g) for _ in range(5))
        e = dict(rows=rows, tok_per_s=round(rows / sec, 1), ms=round(sec * 1e3, 3), launches=len(tasks))
        if kernels:
            e["by_launch"] = measure(rt, tasks, layer_work(c, rows, ctx), reps=16)
        out[f"prefill_{rows}"] = e
    rt.reset()
    rt.step(rng.integers(0, c.vocab, ctx - steps // 2).tolist())
    tok = 1
    rt.d.decode_chunk(rt.graph, rt.uniforms, rt.position, tok, 16)
    fk.sync()
    t0 = time.perf_counter()
    _, sec = rt.d.decode_chunk(rt.graph, rt.uniforms, rt.position, tok, steps)
    wall = time.perf_counter() - t0
    b = token_bytes(c, ctx)
    out["decode"] = dict(context=ctx, tok_per_s=round(steps / wall, 1), ms_per_token=round(wall / steps * 1e3, 4), launches=len(rt.tasks),
                         bytes_per_token=b, frac_of_roofline=round(b * steps / wall / HBM_PEAK, 4))
    if kernels:
        rt.offset.upload(np.array([ctx], np.uint32))
        rt.kv_len.upload(np.array([ctx + 1], np.uint32))
        out["decode"]["by_launch"] = measure(rt, rt.tasks, layer_work(c, 1, ctx))
    return out


def bench_moe(size: str, ctx: int = 1024, steps: int = 128) -> dict:
    from . import native as fk
    from .moe_decoder import MoeRuntime, MoeWeights
    s = SIZES[size]
    c = moe_config(s, capacity=2 * ctx)
    w = MoeWeights.random_init(c, seed=1)
    rt = MoeRuntime(c, w)
    rng = np.random.Generator(np.random.PCG64(0))
    out: dict = dict(model="mixture-of-experts decoder %s: %d layers, hidden %d, %.2f GB of int4 weights" % (size, LAYERS, c.hidden, w.nbytes() / 1e9))
    rows = 512
    rt.forward_rows(rng.integers(0, c.vocab, rows).tolist(), 0)
    g = rt._rows_variants[rows].graph
    sec = min(rt.d.execute_graph(g) for _ in range(3))
    v = rt._rows_variants[rows]
    out["prefill_512"] = dict(rows=rows, tok_per_s=round(rows / sec, 1), ms=round(sec * 1e3, 3), launches=len(v.tasks))
    us: Dict[str, list] = {}
    for t, x in zip(v.tasks, rt.d.profile_graph_nodes(g)):
        p, f = t.params, _family(t.kernel)
        fl = {"qgemm": lambda: 2.0 * rows * p["m"] * p["n"], "qgemm_swiglu": lambda: 4.0 * rows * p["hidden"] * p["inter"],
              "routed_qmv_swiglu": lambda: 4.0 * p["routes"] * p["k"] * p["o"],
              "routed_qmv_reduce": lambda: 2.0 * p["tokens"] * p["top_k"] * p["k"] * p["o"] + 2.0 * p["tokens"] * p.get("shared_k", 0) * p["o"],
              "sdpa_decode": lambda: rows * (rows + 1.0) * c.n_heads * (c.qk_dim + c.v_dim)}.get(f)
        a = us.setdefault(f, [0.0, 0, 0.0])
        a[0] += x * 1e6
        a[1] += 1
        a[2] += fl() if fl else 0.0
    out["prefill_512"]["by_family"] = [dict(family=f, us=round(a[0], 1), count=a[1], **({"mfma_frac": round(a[2] / (a[0] * 1e-6) / MFMA_PEAK, 4)} if a[2] else {}))
                                       for f, a in sorted(us.items(), key=lambda kv: -kv[1][0])]
    rt.reset()
    rt.d.decode_chunk(rt.graph, rt.uniforms, ctx - steps // 2, 1, 16)
    fk.sync()
    t0 = time.perf_counter()
    rt.d.decode_chunk(rt.graph, rt.uniforms, ctx - steps // 2, 1, steps)
    wall = time.perf_counter() - t0
    b = c.token_bytes(ctx)
    out["decode"] = dict(context=ctx, tok_per_s=round(steps / wall, 1), ms_per_token=round(wall / steps * 1e3, 4), launches=len(rt.tasks),
                         bytes_per_token=b, frac_of_roofline=round(b * steps / wall / HBM_PEAK, 4), xcd_launches=bool(rt.xcd))
    if not rt.xcd:
        return out
    # the per-dispatch list, the like-for-like of the layer-list model's launches
    c.xcd_moe = False
    rt2 = MoeRuntime(c, w)
    rt2.offset.upload(np.array([ctx - 1], np.uint32))
    rt2.kv_len.upload(np.array([ctx], np.uint32))
    per = c.bits / 8 + 4 / c.group

    def work(t):
        p, f = t.params, _family(t.kernel)
        w_ = {"rmsnorm_qkv": lambda: (p["n_q"] + 2 * p["n_kv"]) * p["hidden"] * per, "linear_residual": lambda: p["m"] * p["n"] * per,
              "split_store_sdpa_decode": lambda: ctx * c.n_heads * (c.qk_dim + c.v_dim) * 2, "moe_router": lambda: p["hidden"] * p["experts"] * 2,
              "routed_qmv_swiglu": lambda: 2 * (c.top_k + c.n_shared) * p["k"] * p["o"] * per,
              "routed_qmv_reduce": lambda: (c.top_k + c.n_shared) * p["k"] * p["o"] * per,
              "final_rmsnorm_lm_head": lambda: c.vocab * c.hidden * 2, "final_rmsnorm_lm_head_argmax": lambda: c.vocab * c.hidden * 2}.get(f)
        return (w_() if w_ else 0), 0

    fk.sync()
    t0 = time.perf_counter()
    rt2.d.decode_chunk(rt2.graph, rt2.uniforms, ctx - steps // 2, 1, steps)
    out["decode"]["per_dispatch_tok_per_s"] = round(steps / (time.perf_counter() - t0), 1)
    rt2.offset.upload(np.array([ctx - 1], np.uint32))
    rt2.kv_len.upload(np.array([ctx], np.uint32))
    out["decode"]["by_launch"] = measure(rt2, rt2.tasks, work)
    return out


def run_joint(sizes: List[str], kernels: bool = True) -> dict:
    return {s: dict(fumotar=bench_layer(s, kernels=kernels, config=joint_config(JOINT_SIZES[s])),
                    pusavik=bench_layer(s, kernels=kernels, config=like_joint_config(JOINT_SIZES[s]))) for s in sizes}


def run(sizes: List[str], kernels: bool = True) -> dict:
    return {s: dict(layer_list=bench_layer(s, kernels=kernels), moe=bench_moe(s)) for s in sizes}
