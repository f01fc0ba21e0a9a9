"""Every mechanism of the joint layers alone, through its dispatch family, against the plain implementation."""
import numpy as np
import pytest

from fumotar_helpers import stretch
from layer_rig import Rig, pad, padded
from oracle import fumotar as plain
from pusavik_helpers import bf16_round, rng

pytestmark = pytest.mark.gpu
ACTS = [32, 16]


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows,width", [(1, 40), (5, 192), (33, 1100)])
def test_layer_norm_and_copy(fk, act, rows, width):
    g, r = Rig(act), rng(rows)
    ld = pad(width)
    x, mix = (padded((3.0 + r.standard_normal((rows, width))).astype(np.float32), ld) for _ in range(2))
    (bw, w), (bb, b) = g.w16(padded(r.standard_normal(width), ld)), g.w16(padded(r.standard_normal(width), ld))
    bx, h, cat = g.raw(x), g.zeros(rows * ld), g.zeros(rows * 2 * ld)
    g.run("residual_norm", [bx, g.raw(mix), cat, bw, bb, h], rows=rows, width=width, ld=ld, eps=1e-3, has_mix=1, ldcopy=2 * ld, has_h1=1, layer_norm=1)
    y = x.astype(np.float64) + mix
    assert np.abs(bx.to_numpy(np.float32, (rows, ld)) - y).max() <= 1e-6 * np.abs(y).max()
    got = g.down(h, (rows, ld))
    g.close(got[:, :width], plain.layer_norm(y[:, :width], w[:width], b[:width], 1e-3))
    assert not got[:, width:].any()
    c = g.down(cat, (rows, 2 * ld))
    g.close(c[:, :ld], y, 4e-3 if act == 16 else 1e-6)
    assert not c[:, ld:].any()


@pytest.mark.parametrize("act", ACTS)
def test_embedding_with_a_table_of_pairs(fk, act):
    """Portions of one sequence: the token before a portion is remembered, the first token of a sequence has none."""
    g, r = Rig(act), rng(2)
    vocab, width, buckets = 50, 72, 31
    ld = pad(width)
    (bt, t), (bp, p) = g.w16(padded(r.standard_normal((vocab, width)), ld)), g.w16(padded(r.standard_normal((buckets + 1, width)), ld))
    tok = r.integers(0, vocab, 40).tolist()
    rows_of = plain.bigram_rows(tok, 1000003, 77, buckets)
    prev = g.raw(np.array([7], np.uint32))                      # left by another sequence
    at = 0
    for n in (1, 1, 2, 3, 17, 16):
        bx, cat = g.zeros(n * ld, 4), g.zeros(n * 2 * ld)
        ptr = (cat.ptr + ld * g.e, cat.nbytes - ld * g.e)
        g.run("embed_rows", [g.raw(np.array(tok[at:at + n], np.uint32)), bt, bp, prev, g.raw(np.array([at], np.uint32)), bx, ptr], rows=n, width=width, vocab=vocab,
              ldw=ld, ld=ld, ldcopy=2 * ld, buckets=buckets, mul_prev=1000003 % buckets, mul_cur=77 % buckets, scale=1.5)
        ref = 1.5 * t[tok[at:at + n]] + p[rows_of[at:at + n]]
        assert np.abs(bx.to_numpy(np.float32, (n, ld)) - ref).max() <= 1e-6
        g.close(g.down(cat, (n, 2 * ld))[:, ld:], ref, 4e-3 if act == 16 else 1e-6)
        at += n
    assert at == 40 and prev.to_numpy(np.uint32)[0] == tok[-1]
    bx = g.zeros(3 * ld, 4)
    g.run("embed_rows", [g.raw(np.array(tok[:3], np.uint32)), bt, bx], rows=3, width=width, vocab=vocab, ldw=ld, ld=ld)   # one table only
    assert np.array_equal(bx.to_numpy(np.float32, (3, ld)), t[tok[:3]])


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows,heads,dim", [(1, 3, 20), (7, 2, 128), (65, 5, 33), (3, 1, 300)])
def test_gated_head_norm(fk, act, rows, heads, dim):
    g, r = Rig(act), rng(dim)
    ld = pad(dim, 32)
    n = heads * ld
    x = padded(r.standard_normal((rows, heads, dim)).astype(np.float32), ld).reshape(rows, n)
    bz, z = g.up(r.standard_normal((rows, n)))
    bw, w = g.w16(padded(r.standard_normal(dim), ld))
    y = g.zeros(rows * 2 * n)
    g.run("head_norm", [g.raw(x), bz, bw, y], rows=rows, heads=heads, dim=dim, ld=ld, ldy=2 * n, eps=1e-4)
    ref = plain.rms_norm(x.reshape(rows, heads, ld)[..., :dim].astype(np.float64), w[:dim], 1e-4) * plain.sigmoid(z.reshape(rows, heads, ld)[..., :dim])
    got = g.down(y, (rows, 2 * n))[:, :n].reshape(rows, heads, ld)
    g.close(got[..., :dim], ref)
    assert not got[..., dim:].any()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows", [1, 7, 9, 33, 200])
@pytest.mark.parametrize("n,tail", [(192, 3), (448, 0), (1600, 17)])
def test_product_with_column_functions(fk, act, rows, n, tail):
    g, r = Rig(act), rng(rows + n)
    k, N = 128, n + tail
    (bx, x), (bw, w), (bb, b) = g.up(r.standard_normal((rows, k))), g.w16(r.standard_normal((N, k)) * 0.2), g.w16(r.standard_normal(N))
    y, t = g.zeros(rows * n), g.zeros(rows * max(tail, 1), 4)
    more = dict(tail_begin=n, ldt=tail, fn2_begin=pad(N, 4)) if tail else dict(has_bias=1, fn2_begin=n - 64)
    g.run("dense", [bx, bw] + ([y, t] if tail else [bb, y]), rows=rows, n=N, k=k, ldx=k, ldw=k, ldy=n, fn=2, fn_begin=64, fn_end=n - 64, fn2=1, **more)
    ref = x @ w.T + (0.0 if tail else b)
    got = g.down(y, (rows, n))
    g.close(got[:, :64], ref[:, :64])
    g.close(got[:, 64:n - 64], plain.gelu_tanh(ref[:, 64:n - 64]))
    g.close(got[:, n - 64:], ref[:, n - 64:n] if tail else plain.relu2(ref[:, n - 64:n]))
    if tail:
        assert np.abs(t.to_numpy(np.float32, (rows, tail)) - ref[:, n:]).max() <= 2e-6 * np.abs(ref).max()


@pytest.mark.parametrize("rows,parts", [(9, 8), (33, 4), (130, 2)])
def test_product_in_parts_of_its_sum(fk, rows, parts):
    """One product as `parts` products over a share of k each, added where the residual takes them."""
    g, r = Rig(16), rng(rows)
    n, k = 100, 1024
    ld, kp = pad(n), k // parts
    (bx, x), (bw, w) = g.up(r.standard_normal((rows, k))), g.w16(r.standard_normal((n, k)))
    mix, h = g.zeros(parts * rows * ld, 4), g.zeros(rows * ld)
    g.run("dense", [bx, bw, mix], rows=rows, n=n, k=kp, ldx=k, ldw=k, ldy=ld, batch=parts, xb=kp, wb=kp, yb=rows * ld, y32=1)
    res = padded(r.standard_normal((rows, n)).astype(np.float32), ld)
    (bn, nw), (bb, nb), bres = g.w16(padded(r.standard_normal(n), ld)), g.w16(padded(r.standard_normal(n), ld)), g.raw(res)
    g.run("residual_norm", [bres, mix, bn, bb, h], rows=rows, width=n, ld=ld, eps=1e-3, has_mix=1, mix_parts=parts, has_h1=1, layer_norm=1)
    ref = res[:, :n] + x @ w.T
    assert np.abs(bres.to_numpy(np.float32, (rows, ld))[:, :n] - ref).max() <= 2e-6 * np.abs(ref).max()
    g.close(g.down(h, (rows, ld))[:, :n], plain.layer_norm(ref, nw[:n], nb[:n], 1e-3))


# ---- attention ----

def qk_case(g, r, rows, heads, kv, dim, dim_ld):
    k0, q0 = 0, kv * dim_ld
    ldu = q0 + heads * dim_ld + 64
    u = np.zeros((rows, ldu))
    u[:, k0:q0] = padded(r.standard_normal((rows, kv, dim)), dim_ld).reshape(rows, -1)
    u[:, q0:q0 + heads * dim_ld] = padded(r.standard_normal((rows, heads, dim)), dim_ld).reshape(rows, -1)
    return u, k0, q0, ldu


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("heads,kv,dim,rot_dims,scaled", [(4, 2, 24, 16, True), (3, 1, 64, 64, False), (8, 8, 100, 0, False), (2, 1, 130, 2, True)])
def test_queries_and_cache_rows(fk, act, heads, kv, dim, rot_dims, scaled):
    from fusekit_amd.layer_decoder import CausalAttention
    g, r = Rig(act), rng(dim)
    m = CausalAttention(heads=heads, kv_heads=kv, dim=dim, scale=1.0, rot_base=500.0, rot_dims=rot_dims, rot_scaling=stretch(original=64, fast=4.0, slow=0.5) if scaled else None)
    ld, T, cap, eps = m.dim_ld, 37, 50, 1e-3
    u, k0, q0, ldu = qk_case(g, r, T, heads, kv, dim, ld)
    (bwq, wq), (bwk, wk) = g.w16(padded(r.standard_normal((heads, dim)), ld)), g.w16(padded(r.standard_normal((kv, dim)), ld))
    K, V = g.zeros(kv * cap * ld), g.zeros(kv * cap * ld)
    freq, mag = m.rotation()
    fb = g.raw(freq if rot_dims else np.zeros(1))
    vu = (bf16_round(u) if act == 16 else u.astype(np.float32)).astype(np.float64)
    from fusekit_amd.checkpoint import layer_config_to_json
    from fumotar_helpers import model
    rot = layer_config_to_json(model([(m, None)]))["layers"][0]["mixer"]["rot"]
    kk, qq = vu[:, k0:q0].reshape(T, kv, ld)[..., :dim], vu[:, q0:q0 + heads * ld].reshape(T, heads, ld)[..., :dim]
    norm = lambda x, w: plain.rotate(plain.rms_norm(x.reshape(T, -1), w[:, :dim].reshape(-1), eps).reshape(x.shape), rot)
    refk, refq = norm(kk, wk), norm(qq, wq)
    at = 0
    for n in (1, 2, 33, 1):
        bu, _ = g.up(u[at:at + n])
        q = g.zeros(n * heads * ld)
        g.run("qk_store", [bu, bwq, bwk, fb, g.raw(np.array([at], np.uint32)), q, K, V], rows=n, heads=heads, kv_heads=kv, dim=dim, dim_ld=ld, rot_dims=rot_dims,
              ldu=ldu, k0=k0, q0=q0, capacity=cap, mag=mag, eps=eps)
        got = g.down(q, (n, heads, ld))
        g.close(got[..., :dim], refq[at:at + n])
        assert not got[..., dim:].any()
        at += n
    gk, gv = g.down(K, (kv, cap, ld)).transpose(1, 0, 2), g.down(V, (kv, cap, ld)).transpose(1, 0, 2)
    g.close(gk[:T, :, :dim], refk)
    assert np.array_equal(gv[:T, :, :dim], kk) and not gk[T:].any() and not gv[T:].any()   # values: the keys as projected


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("heads,kv,dim,ld", [(4, 2, 40, 64), (6, 1, 128, 128), (2, 2, 200, 256)])
def test_attention_rows_see_near_and_far_keys(fk, act, heads, kv, dim, ld):
    """Query i's score with one chosen key stands out, the chosen key being the first, the query's own, the one before it or
    one in the middle: a key that is missed or a future one that is seen changes the output altogether."""
    g, r = Rig(act), rng(dim)
    T, cap, scale = 150, 160, 1.0
    K = padded(r.standard_normal((kv, T, dim)) / np.sqrt(dim) * 1.0, ld)
    V = padded(r.standard_normal((kv, T, dim)), ld)
    q = np.zeros((T, heads, ld))
    target = np.zeros((T, heads), int)
    for i in range(T):
        for h in range(heads):
            target[i, h] = (0, i, max(i - 1, 0), i // 2, min(i, 63), min(i, 64))[(i + h) % 6]
            q[i, h] = 12.0 * K[h // (heads // kv), target[i, h]] / (K[h // (heads // kv), target[i, h]] ** 2).sum()
    q[np.arange(T) % 7 == 3] *= -1.0
    cap_pad = lambda a: np.concatenate([a, 30.0 + 0 * a[:, :cap - T]], 1)     # rows behind the sequence would dominate
    bk, vk = g.up(cap_pad(K))
    bv, vv = g.up(cap_pad(V))
    for at, n in ((0, 150), (0, 1), (149, 1), (63, 2), (40, 90), (128, 16)):
        bq, vq = g.up(q[at:at + n])
        ref = np.zeros((n, heads, ld))
        for h in range(heads):
            k, v = vk[h // (heads // kv)], vv[h // (heads // kv)]
            for i in range(n):
                s = k[:at + i + 1] @ vq[i, h] * scale
                e = np.exp(s - s.max())
                ref[i, h] = e / e.sum() @ v[:at + i + 1]
        off, kvl, ldo = g.raw(np.array([at], np.uint32)), g.raw(np.array([at + n], np.uint32)), heads * ld + 64
        out = g.zeros(n * ldo)
        g.run("gqa_rows", [bq, bk, bv, off, out], rows=n, heads=heads, kv_heads=kv, dim_ld=ld, capacity=cap, ldo=ldo, scale=scale)
        g.close(g.down(out, (n, ldo))[:, :heads * ld].reshape(n, heads, ld), ref)
        assert not g.down(out, (n, ldo))[:, heads * ld:].any()
        if act == 16 and ld <= 128:
            out = g.zeros(n * ldo)
            g.run("sdpa_prefill", [bq, bk, bv, kvl, out], rows=n, n_heads=heads, n_kv=kv, head_dim=ld, capacity=cap, scale=scale, ldo=ldo)
            g.close(g.down(out, (n, ldo))[:, :heads * ld].reshape(n, heads, ld), ref, 1e-2)
            assert not g.down(out, (n, ldo))[:, heads * ld:].any()


# ---- recurrences ----

@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("linear,bias,taps,channels", [(0, 0, 4, 96), (1, 1, 4, 64), (1, 1, 1, 40), (0, 0, 5, 130), (1, 0, 2, 68)])
def test_convolution_keeps_its_history(fk, act, linear, bias, taps, channels):
    g, r = Rig(act), rng(taps)
    T, ld = 80, pad(channels)
    u = r.standard_normal((T, ld))
    (bw, w), (bb, b) = g.w16(r.standard_normal((channels, taps))), g.w16(r.standard_normal(channels))
    hist = g.zeros(taps * ld)
    full = (bf16_round(u) if act == 16 else u.astype(np.float32)).astype(np.float64)
    ref = plain.causal_conv(full[:, :channels], w, b if bias else 0.0)
    ref = ref if linear else plain.silu(ref)
    at = 0
    for n in (1, 2, 1, 1, 3, 16, 2, 37, 1, 16):
        bu, _ = g.up(u[at:at + n])
        y = g.zeros(n * ld)
        g.run("ssm_conv", [bu, bw] + ([bb] if bias else []) + [hist, g.raw(np.array([at], np.uint32)), y], rows=n, channels=channels, taps=taps, ldu=ld, ldy=ld, ldh=ld,
              has_bias=bias, linear=linear, update=1)
        g.close(g.down(y, (n, ld))[:, :channels], ref[at:at + n])
        at += n
    assert at == T


def delta_case(r, T, heads, kv, dim, vdim):
    """Raw inputs of the recurrence; decays from none to everything within a token, keys that come back."""
    x = r.standard_normal((T, 2 * kv * dim + heads * vdim))
    x[T // 2:, kv * dim:2 * kv * dim] = x[:T - T // 2, kv * dim:2 * kv * dim]
    z = r.standard_normal((T, heads, dim)) * 2.0
    return x, z, np.linspace(-6, 3, heads), r.standard_normal((T, heads)) * 2.0


@pytest.mark.parametrize("act,form", [(32, "delta_scan"), (16, "delta_scan"), (16, "delta_chunk")])
@pytest.mark.parametrize("heads,kv,dim,vdim", [(2, 2, 32, 32), (4, 2, 20, 40), (6, 1, 64, 64), (2, 1, 128, 128), (3, 3, 96, 33), (1, 1, 200, 64), (2, 2, 256, 32), (2, 1, 150, 20)])
def test_delta_rule_in_portions(fk, act, form, heads, kv, dim, vdim):
    g, r = Rig(act), rng(heads * dim)
    dl, vl = pad(dim, 32), pad(vdim, 32)
    if form == "delta_chunk" and not g.native.delta_chunk_supported(dl, vl):
        pytest.skip("no chunked form of this shape")
    T, sl, nk, nd, nv = 260, pad(dim), kv * dl, heads * dl, heads * vl
    x, z, a_log, b = delta_case(r, T, heads, kv, dim, vdim)
    xs = np.concatenate([padded(x[:, i * kv * dim:(i + 1) * kv * dim].reshape(T, kv, dim), dl).reshape(T, nk) for i in (0, 1)]
                        + [padded(x[:, 2 * kv * dim:].reshape(T, heads, vdim), vl).reshape(T, nv)], 1)
    ldx, ldb = pad(xs.shape[1]), heads + 3
    xs = padded(xs, ldx)
    full = (bf16_round(xs) if act == 16 else xs.astype(np.float32)).astype(np.float64)
    (ba, va), (bd, vd) = g.w16(a_log), g.w16(padded(r.standard_normal((heads, dim)) - 2.0, dl))
    z32 = z.astype(np.float32)
    of = np.arange(heads) // (heads // kv)
    log_g = -np.exp(va)[:, None] * plain.softplus(z32.astype(np.float64) + vd[:, :dim])
    q = plain.unit(full[:, :nk].reshape(T, kv, dl)[..., :dim])[:, of] * dim ** -0.5
    k = plain.unit(full[:, nk:2 * nk].reshape(T, kv, dl)[..., :dim])[:, of]
    v = full[:, 2 * nk:2 * nk + nv].reshape(T, heads, vl)[..., :vdim]
    beta = plain.sigmoid(b.astype(np.float32).astype(np.float64))
    ref = plain.delta_recurrence(q, k, v, beta, log_g)
    state, at = g.zeros(nv * sl, 4), 0
    for m in (2, 70, 64, 1, 16, 107):
        bx, _ = g.up(xs[at:at + m])
        bz, bb = g.raw(padded(z32[at:at + m], dl)), g.raw(padded(b[at:at + m].astype(np.float32), ldb))
        qk, o = g.zeros(m * 2 * nk, 4), g.zeros(pad(m) * nv, 4)
        shape = dict(rows=m, heads=heads, kv_heads=kv, dim_ld=dl, ldx=ldx, ldb=ldb)
        g.run("delta_prep", [bx, bd, ba, bz, bb, qk], dim=dim, **shape)
        assert np.abs(bb.to_numpy(np.float32, (m, ldb))[:, :heads] - beta[at:at + m]).max() <= 1e-6
        lg = bz.to_numpy(np.float32, (m, heads, dl))[..., :dim] * np.log(2.0)
        assert (np.abs(lg - log_g[at:at + m]) <= 2e-6 * np.abs(log_g[at:at + m]) + 1e-7).all()
        bufs = [qk, bz, bb, (bx.ptr + 2 * nk * g.e, bx.nbytes - 2 * nk * g.e), state, o]
        if form == "delta_chunk":
            bufs.append(g.raw(np.full(g.native.delta_chunk_work_bytes(m, heads, dl, vl) // 4, 0x7fc07fc0, np.uint32)))   # NaNs: all that is read was written
        g.run(form, bufs, vdim_ld=vl, state_ld=sl, **shape)
        got = o.to_numpy(np.float32, (pad(m), heads, vl))[:m]
        assert np.abs(got[..., :vdim] - ref[at:at + m]).max() <= 2e-5 * np.abs(ref).max(), (m, np.abs(got[..., :vdim] - ref[at:at + m]).max() / np.abs(ref).max())
        assert not got[..., vdim:].any()
        at += m
    S = np.zeros((heads, dim, vdim))
    for t in range(T):
        S = np.exp(log_g[t])[..., None] * S
        S = S + k[t][..., None] * (beta[t][:, None] * (v[t] - np.einsum("hkv,hk->hv", S, k[t])))[:, None]
    got = state.to_numpy(np.float32, (heads, vl, sl)).transpose(0, 2, 1)
    assert np.abs(got[:, :dim, :vdim] - S).max() <= 2e-5 * np.abs(S).max() and not got[:, dim:].any() and not got[..., vdim:].any()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("blocks,block", [(1, 64), (3, 128), (5, 20)])
def test_linear_recurrence_in_portions(fk, act, blocks, block):
    g, r = Rig(act), rng(block)
    T, W = 270, blocks * block
    (brb, rb), (bib, ib), (bl, lam) = (g.w16(r.standard_normal(W)) for _ in range(3))
    lam[:4] = [-12.0, -8.0, 4.0, 9.0]                             # decays near one and near zero
    bl, lam = g.w16(lam)
    u, y, gates = r.standard_normal((T, W)), r.standard_normal((T, W)), (2.0 * r.standard_normal((T, blocks, 2, block))).astype(np.float32)
    full = (bf16_round(u) if act == 16 else u.astype(np.float32)).astype(np.float64)
    fy = (bf16_round(y) if act == 16 else y.astype(np.float32)).astype(np.float64)
    z = gates.astype(np.float64)
    S = plain.gated_recurrence(full, plain.sigmoid(z[:, :, 0].reshape(T, W) + rb), plain.sigmoid(z[:, :, 1].reshape(T, W) + ib), lam)
    state, at, ldy = g.zeros(W, 4), 0, W + 64
    for m in (1, 2, 31, 33, 64, 7, 132):
        bu, _ = g.up(u[at:at + m])
        by, _ = g.up(padded(y[at:at + m], ldy))
        g.run("lru_scan", [bu, g.raw(gates[at:at + m]), brb, bib, bl, state, by, g.zeros(-(-m // 32) * 2 * W, 4)], rows=m, width=W, block=block, ldx=W, ldy=ldy)
        g.close(g.down(by, (m, ldy))[:, :W], S[at:at + m] * fy[at:at + m], 4e-6 if act == 32 else None)
        at += m
        got = state.to_numpy(np.float32)
        assert np.abs(got - S[at - 1]).max() <= 4e-6 * np.abs(S).max()
    assert at == T


# ---- jobs of the fused launches ----

@pytest.mark.parametrize("width,n", [(72, 130), (1100, 70), (4500, 90)])
def test_joined_and_layer_normed_rows(fk, width, n):
    g, r = Rig(16), rng(n)
    ld = pad(width)
    x = padded((2.0 + r.standard_normal(width)).astype(np.float32), ld)
    (bw, w), (bo, ob) = g.w16(padded(r.standard_normal((n, width)), ld)), g.w16(r.standard_normal(n))
    (bn, nw), (bb, nb) = (g.w16(padded(r.standard_normal(width), ld)) for _ in range(2))
    y, tail = g.zeros(64), g.zeros(n - 64, 4)
    g.run("layer_jobs", [g.raw(x), bn, bb, bw, bo, y, tail], g0_mode=1, g0_n=n, g0_k=ld, g0_width=width, g0_eps=1e-4, g0_layer_norm=1, g0_n_act=64, g0_has_bias=1,
          g0_fn=1, g0_fn_begin=0, g0_fn_end=32, g0_fn2=2, g0_fn2_begin=48)
    h = bf16_round(plain.layer_norm(x[:width].astype(np.float64), nw[:width], nb[:width], 1e-4)).astype(np.float64)
    ref = w[:, :width] @ h + ob
    want = np.concatenate([plain.relu2(ref[:32]), ref[32:48], plain.gelu_tanh(ref[48:])])
    # a row element on the edge between two bf16 values may fall either way
    got = g.down(y, (64,))
    g.close(got[:32], want[:32], 1e-2)
    g.close(got[32:], want[32:64], 1e-2)
    assert np.abs(tail.to_numpy(np.float32) - want[64:]).max() <= 1e-2 * np.abs(want[64:]).max()
    (bj, wj), (b2, x2) = g.w16(np.concatenate([padded(r.standard_normal((n, width)), ld) for _ in range(2)], 1)), g.up(padded(r.standard_normal(width), ld))
    out = g.zeros(n, 4)
    g.run("layer_jobs", [g.raw(x), b2, bj, out], g0_mode=4, g0_n=n, g0_k=2 * ld, g0_width=width, g0_n_act=0)
    ref = wj @ np.concatenate([bf16_round(x).astype(np.float64), x2])
    assert np.abs(out.to_numpy(np.float32) - ref).max() <= 1e-5 * np.abs(ref).max()


@pytest.mark.parametrize("heads,kv,dim,vdim,rank,taps", [(2, 2, 32, 32, 8, 4), (4, 2, 20, 40, 70, 1), (2, 1, 128, 128, 128, 3), (3, 3, 200, 33, 24, 5)])
def test_delta_step_of_one_token(fk, heads, kv, dim, vdim, rank, taps):
    """The job of the fused launch against convolution, second decay projection and recurrence over a whole sequence."""
    g, r = Rig(16), rng(dim + rank)
    T, dl, vl, rl = 9, pad(dim, 32), pad(vdim, 32), pad(rank)
    sl, nk, nv = pad(dim), kv * dl, heads * vl
    ch = 2 * nk + nv
    heads_of = lambda a, n, d, ld: padded(a.reshape(a.shape[0], n, d), ld).reshape(a.shape[0], n * ld)
    raw = np.concatenate([heads_of(r.standard_normal((T, kv * dim)), kv, dim, dl), heads_of(r.standard_normal((T, kv * dim)), kv, dim, dl), heads_of(r.standard_normal((T, heads * vdim)), heads, vdim, vl)], 1)
    vraw = bf16_round(raw).astype(np.float64)
    bw, w = g.w16(r.standard_normal((ch, taps)))
    ba2, a2 = g.w16(padded(heads_of(r.standard_normal((rank, heads * dim)) * rank ** -0.5, heads, dim, dl).T, rl))
    (bd, vd), (bA, vA) = g.w16(heads_of(r.standard_normal((1, heads * dim)), heads, dim, dl)[0] - 1.0), g.w16(np.linspace(-3, 1, heads))
    va1 = bf16_round(padded(r.standard_normal((T, rank)), rl)).astype(np.float64)
    beta = r.standard_normal((T, heads)).astype(np.float32)
    y = bf16_round(plain.silu(plain.causal_conv(vraw, w, 0.0))).astype(np.float64)
    of = np.arange(heads) // (heads // kv)
    part = lambda a, n, ld, d: a.reshape(T, n, ld)[..., :d]
    q, k = plain.unit(part(y[:, :nk], kv, dl, dim))[:, of] * dim ** -0.5, plain.unit(part(y[:, nk:2 * nk], kv, dl, dim))[:, of]
    log_g = part(-np.repeat(np.exp(vA), dl) * plain.softplus(va1 @ a2.T + vd), heads, dl, dim)
    ref = plain.delta_recurrence(q, k, part(y[:, 2 * nk:], heads, vl, vdim), plain.sigmoid(beta.astype(np.float64)), log_g)
    state, hist, o = g.zeros(nv * sl, 4), g.zeros(taps * pad(ch)), g.zeros(nv, 4)
    for t in range(T):
        g.run("layer_jobs", [g.up(raw[t])[0], g.up(va1[t])[0], g.raw(beta[t]), bw, ba2, bd, bA, g.raw(np.array([t], np.uint32)), state, hist, o], delta_heads=heads, delta_kv_heads=kv,
              delta_dim=dim, delta_dim_ld=dl, delta_vdim_ld=vl, delta_state_ld=sl, delta_rank_ld=rl, delta_ldh=pad(ch), delta_taps=taps)
        got = o.to_numpy(np.float32, (heads, vl))
        # a convolution output on the edge between two bf16 values may fall either way
        assert np.abs(got[:, :vdim] - ref[t]).max() <= 5e-3 * np.abs(ref).max() and not got[:, vdim:].any()


@pytest.mark.parametrize("blocks,block,taps", [(1, 64, 4), (3, 128, 1), (2, 640, 5)])
def test_lru_step_of_one_token(fk, blocks, block, taps):
    g, r = Rig(16), rng(block)
    T, W = 8, blocks * block
    raw, y = r.standard_normal((T, W)), r.standard_normal((T, W))
    vraw, vy = bf16_round(raw).astype(np.float64), bf16_round(y).astype(np.float64)
    (bw, w), (bb, b), (bg, gates) = g.w16(r.standard_normal((W, taps))), g.w16(r.standard_normal(W)), g.w16(r.standard_normal((blocks, 2, block, block)) * block ** -0.5)
    (brb, rb), (bib, ib), (bl, lam) = (g.w16(r.standard_normal(W)) for _ in range(3))
    u = bf16_round(plain.causal_conv(vraw, w, b)).astype(np.float64)
    gate = [plain.sigmoid(plain.block_product(u, gates[:, i], bias.reshape(blocks, block))) for i, bias in ((0, rb), (1, ib))]
    S = plain.gated_recurrence(u, *gate, lam)
    state, hist = g.zeros(W, 4), g.zeros(taps * W)
    for t in range(T):
        by = g.up(y[t])[0]
        g.run("layer_jobs", [g.up(raw[t])[0], bw, bb, bg, brb, bib, bl, g.raw(np.array([t], np.uint32)), state, hist, by], lru_width=W, lru_block=block, lru_ldh=W, lru_taps=taps)
        assert np.abs(state.to_numpy(np.float32) - S[t]).max() <= 5e-3 * np.abs(S).max()
        g.close(g.down(by, (W,)), S[t] * vy[t], 1e-2)


def test_layer_out_normalises_heads(fk):
    g, r = Rig(16), rng(8)
    heads, dim, ld, ff, n = 3, 40, 64, 128, 77
    nv, ko = heads * ld, heads * ld + ff
    o = padded(r.standard_normal((heads, dim)).astype(np.float32), ld)
    (bz, z), (bh, hw) = g.up(r.standard_normal(nv)), g.w16(padded(r.standard_normal(dim), ld))
    (ba, row), (bw, w) = g.up(r.standard_normal(ko)), g.w16(r.standard_normal((n, ko)))
    x = r.standard_normal(n).astype(np.float32)
    bx = g.raw(x)
    g.run("layer_out", [bx, ba, bw, g.raw(o), bz, bh], n=n, ko=ko, norm_heads=heads, norm_dim=dim, norm_ld=ld, norm_eps=1e-4)
    first = np.zeros((heads, ld))
    first[:, :dim] = plain.rms_norm(o[:, :dim].astype(np.float64), hw[:dim], 1e-4) * plain.sigmoid(z.reshape(heads, ld)[:, :dim])
    ref = x + w @ np.concatenate([bf16_round(first.reshape(-1)).astype(np.float64), row[nv:]])
    assert np.abs(bx.to_numpy(np.float32) - ref).max() <= 4e-3 * np.abs(ref).max()


def test_bad_shapes_are_refused(fk):
    from fusekit_amd.native import FusekitError
    g = Rig(16)
    b, off = g.zeros(64 * 64), g.raw(np.zeros(1, np.uint32))
    cases = [("residual_norm", [b, b, b, b, b, b], dict(rows=1, width=40, ld=64, has_h1=1, has_h2=1, layer_norm=1)),
             ("residual_norm", [b, b], dict(rows=1, width=40, ld=64, ldcopy=32)),
             ("embed_rows", [off, b, b], dict(rows=1, width=40, vocab=4, ldw=40, ld=40)),
             ("embed_rows", [off, b, b, off, off, b], dict(rows=1, width=64, vocab=4, buckets=900)),          # table too small
             ("dense", [b, b, b], dict(rows=2, n=8, k=64, ldx=64, ldw=64, ldy=8, fn=3)),
             ("dense", [b, b, b], dict(rows=2, n=8, k=64, ldx=64, ldw=64, ldy=8, fn=1, fn_begin=2, fn_end=8)),
             ("qk_store", [b, b, b, b, off, b, b, b], dict(rows=1, heads=3, kv_heads=2, dim=8, dim_ld=8, ldu=64, q0=16, capacity=4)),
             ("qk_store", [b, b, b, b, off, b, b, b], dict(rows=1, heads=2, kv_heads=1, dim=8, dim_ld=8, rot_dims=9, ldu=64, q0=8, capacity=4)),
             ("gqa_rows", [b, b, b, off, b], dict(rows=1, heads=1, kv_heads=1, dim_ld=1024, capacity=2)),
             ("delta_scan", [b] * 6, dict(rows=1, heads=2, kv_heads=2, dim_ld=24, vdim_ld=32, state_ld=64, ldx=64)),
             ("delta_chunk", [b] * 7, dict(rows=64, heads=1, kv_heads=1, dim_ld=32, vdim_ld=32, state_ld=64, ldx=64)),   # workspace too small
             ("lru_scan", [b] * 8, dict(rows=1, width=64, block=48)),
             ("layer_jobs", [b, b, b, b, b, b, b, off, b, b, b], dict(lru_width=60, lru_block=20, lru_ldh=64, lru_taps=2))]
    for kernel, bufs, p in cases:
        with pytest.raises(FusekitError):
            g.run(kernel, bufs, **p)
