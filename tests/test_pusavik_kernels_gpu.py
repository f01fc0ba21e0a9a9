"""Every mechanism of the layer-list decoder alone, through its dispatch family, against the plain implementation."""
import numpy as np
import pytest

from oracle import pusavik as plain
from layer_rig import Rig, pad, padded
from pusavik_helpers import bf16_round, rng

pytestmark = pytest.mark.gpu


@pytest.mark.parametrize("act", [32, 16])
@pytest.mark.parametrize("rows,width,top", [(1, 40, 1), (5, 192, 3), (33, 300, 4)])
def test_residual_norm(fk, act, rows, width, top):
    g, r = Rig(act), rng(rows)
    ld, experts = pad(width), 3
    N = lambda *s: padded(r.standard_normal(s).astype(np.float32), ld)
    x, mix = N(rows, width), N(rows, width)
    eo, prev = N(rows * top, width), N(rows, width)
    step, w1, w2 = N(width), N(width), N(width)
    idx = r.integers(0, experts + 2, (rows, top)).astype(np.uint32)     # some identities
    wt = r.random((rows, top)).astype(np.float32)
    beo, veo = g.up(eo)
    bprev, vprev = g.up(prev)
    (bs, vs), (b1, v1), (b2, v2) = g.w16(step), g.w16(w1), g.w16(w2)
    bx, h1 = g.raw(x), g.zeros(rows * ld)
    g.run("residual_norm", [bx, g.raw(mix), beo, g.raw(wt), g.raw(idx), bprev, bs, b1, h1, b2, bprev], rows=rows, width=width, ld=ld, eps=1e-3,
          has_mix=1, top=top, experts=experts, has_step=1, has_h1=1, has_h2=1)
    y = x.astype(np.float64) + mix + vs
    veo = veo.reshape(rows, top, ld)
    for s in range(top):
        y += wt[:, s:s + 1] * np.where((idx[:, s] < experts)[:, None], veo[:, s], vprev)
    g2 = bx.to_numpy(np.float32, (rows, ld))
    assert np.abs(g2 - y).max() <= 1e-5 * np.abs(y).max()
    g.close(g.down(h1, (rows, ld))[:, :width], plain.rms_norm(y[:, :width], v1[:width], 1e-3))
    g.close(g.down(bprev, (rows, ld))[:, :width], plain.rms_norm(y[:, :width], v2[:width], 1e-3))   # h2 in the place of prev
    assert not g.down(h1, (rows, ld))[:, width:].any()


@pytest.mark.parametrize("act", [32, 16])
@pytest.mark.parametrize("rows,width,groups", [(1, 48, 1), (7, 120, 5), (40, 256, 8)])
def test_gated_group_norm(fk, act, rows, width, groups):
    g, r = Rig(act), rng(7)
    ld = pad(width)
    (by, y), (bz, z) = g.up(r.standard_normal((rows, ld))), g.up(r.standard_normal((rows, ld)))
    bw, w = g.w16(1 + 0.2 * r.standard_normal(width))
    out = g.zeros(rows * ld)
    g.run("group_norm", [by, bz, bw, out], rows=rows, width=width, groups=groups, ldx=ld, ldz=ld, ldy=ld, has_z=1, eps=1e-4)
    g.close(g.down(out, (rows, ld))[:, :width], plain.gated_group_norm(y[:, :width], z[:, :width], w, groups, 1e-4))


@pytest.mark.parametrize("act", [32, 16])
@pytest.mark.parametrize("rows", [1, 2, 8, 9, 31, 33, 64, 130])
@pytest.mark.parametrize("n,k,batch", [(1, 64, 1), (70, 64, 1), (129, 192, 1), (40, 128, 3), (3000, 64, 1)])
def test_dense(fk, act, rows, n, k, batch):
    g, r = Rig(act), rng(rows * n)
    ldx, ldy = batch * k, pad(batch * n, 4)
    bx, x = g.up(r.standard_normal((rows, ldx)))
    bw, w = g.w16(r.standard_normal((batch, n, k)) / np.sqrt(k))
    ref = np.concatenate([x[:, b * k:(b + 1) * k] @ w[b].T for b in range(batch)], 1)
    for y32 in (0, 1):
        y = g.zeros(rows * ldy, 4 if y32 else None)
        g.run("dense", [bx, bw, y], rows=rows, n=n, k=k, ldx=ldx, ldy=ldy, batch=batch, xb=k, wb=n * k, yb=n, y32=y32)
        got = y.to_numpy(np.float32, (rows, ldy)).astype(np.float64) if y32 else g.down(y, (rows, ldy))
        g.close(got[:, :batch * n], ref, 3e-6 if y32 else None)
        assert not got[:, batch * n:].any()


@pytest.mark.parametrize("rows,back,ring,offset", [(40, 9, 64, 100), (90, 30, 128, 7), (300, 255, 512, 1000), (64, 0, 64, 63)])
def test_dense_from_a_ring_transposed(fk, rows, back, ring, offset):
    g, r = Rig(16), rng(rows)
    n, k = 70, 64
    bx, x = g.up(r.standard_normal((ring, k)))
    bw, w = g.w16(r.standard_normal((n, k)) / 8)
    pos = offset - back + np.arange(rows)
    ref = x[pos % ring] @ w.T
    off = g.raw(np.array([offset], np.uint32))
    ldt = pad(rows)
    y, yt = g.zeros(rows * n), g.zeros(n * ldt)
    g.run("dense", [bx, bw, off, y], rows=rows, n=n, k=k, ldx=k, ldy=n, ring=ring, row_back=back)
    g.run("dense", [bx, bw, off, yt], rows=rows, n=n, k=k, ldx=k, ldy=ldt, ring=ring, row_back=back, transposed=1)
    live = pos >= 0
    g.close(g.down(y, (rows, n))[live], ref[live])
    g.close(g.down(yt, (n, ldt))[:, :rows].T[live], ref[live])


@pytest.mark.parametrize("outputs,top", [(2, 1), (5, 5), (15, 4), (64, 8), (65, 3), (200, 20), (700, 64)])
def test_router(fk, outputs, top):
    g, r = Rig(16), rng(outputs)
    rows, ld = 9, pad(outputs)
    z = padded(r.standard_normal((rows, outputs)).astype(np.float32) * 2, ld)
    bc, c = g.w16(r.standard_normal(outputs) * 0.05)          # large enough to change the choice
    idx, wt = g.zeros(rows * top, 4), g.zeros(rows * top, 4)
    g.run("route_rows", [g.raw(z), bc, idx, wt], rows=rows, outputs=outputs, top=top, ld=ld)
    gi, gw = idx.to_numpy(np.uint32, (rows, top)), wt.to_numpy(np.float32, (rows, top))
    changed = 0
    for t in range(rows):
        i, w = plain.route(z[t, :outputs].astype(np.float64), c, top)
        assert sorted(gi[t]) == sorted(i)
        assert np.allclose(gw[t][np.argsort(gi[t])], w[np.argsort(i)], rtol=2e-5)
        changed += set(i) != set(plain.route(z[t, :outputs].astype(np.float64), 0 * c, top)[0])
    assert changed or top == outputs or outputs < 14
    # the decode list's router job
    one_i, one_w = g.zeros(top, 4), g.zeros(top, 4)
    g.run("layer_jobs", [g.raw(z[3, :outputs]), bc, one_i, one_w], route_outputs=outputs, route_top=top)
    assert sorted(one_i.to_numpy(np.uint32)) == sorted(gi[3])
    assert np.allclose(np.sort(one_w.to_numpy(np.float32)), np.sort(gw[3]), rtol=2e-6)


def test_router_equal_scores_take_the_lower_index(fk):
    g = Rig(16)
    z, c = np.zeros((1, 192), np.float32), g.w16(np.zeros(130))[0]
    idx, wt = g.zeros(5, 4), g.zeros(5, 4)
    g.run("route_rows", [g.raw(z), c, idx, wt], rows=1, outputs=130, top=5, ld=192)
    assert list(idx.to_numpy(np.uint32)) == [0, 1, 2, 3, 4] and np.allclose(wt.to_numpy(np.float32), 0.2)
    g.run("layer_jobs", [g.raw(z[0]), c, idx, wt], route_outputs=130, route_top=5)
    assert list(idx.to_numpy(np.uint32)) == [0, 1, 2, 3, 4]


@pytest.mark.parametrize("act,grouped", [(32, 0), (16, 0), (16, 32), (16, 64), (16, 128)])
@pytest.mark.parametrize("rows,top,experts,n", [(3, 2, 4, 40), (50, 3, 5, 72), (160, 4, 3, 130)])
def test_experts(fk, act, grouped, rows, top, experts, n):
    g, r = Rig(act), rng(rows)
    k, routes = 128, rows * top
    bx, x = g.up(r.standard_normal((rows, k)))
    (bg, wg), (bu, wu) = g.w16(r.standard_normal((experts, n, k)) / 11), g.w16(r.standard_normal((experts, n, k)) / 11)
    idx = r.integers(0, experts + 1, (rows, top)).astype(np.uint32)     # the last is an identity: left alone
    idx[0] = 0                                                          # and an expert that is chosen twice by one token
    bi = g.raw(idx)
    groups = []
    if grouped:
        groups = [g.zeros(routes, 4), g.zeros((routes // grouped + experts) * 4, 4), g.zeros(1, 4)]
        g.run("route_group", [bi] + groups, routes=routes, experts=experts, tile_rows=grouped)
        assert sorted(groups[0].to_numpy(np.uint32)[:(idx < experts).sum()]) == sorted(np.flatnonzero(idx.ravel() < experts))
    ldy = pad(n)
    y, y1 = g.zeros(routes * ldy), g.zeros(routes * ldy)
    p = dict(routes=routes, experts=experts, n=n, k=k, ldx=k, ldw=k, ldy=ldy, x_div=top, grouped=int(grouped > 0), tile_rows=grouped or 64)
    g.run("experts", [bx, bg, bu, bi] + groups + [y], pair=1, **p)
    g.run("experts", [bx, bg, bi] + groups + [y1], **p)
    got, got1 = g.down(y, (routes, ldy)), g.down(y1, (routes, ldy))
    ref, ref1 = np.zeros((routes, n)), np.zeros((routes, n))
    for q, e in enumerate(idx.ravel()):
        if e < experts:
            a = x[q // top] @ wg[e].T
            ref[q], ref1[q] = plain.silu(a) * (x[q // top] @ wu[e].T), a
    g.close(got[:, :n], ref)
    g.close(got1[:, :n], ref1)


# ---- latent attention: every form, keys that stand out at chosen distances ----

class Attn:
    def __init__(self, act, heads, dim, rot, vdim, rank, window, rows, offset, seed=0):
        self.g, self.r = Rig(act), rng(seed)
        self.heads, self.dim, self.rot, self.vdim, self.rank, self.window, self.rows, self.offset = heads, dim, rot, vdim, rank, window, rows, offset
        self.dim_ld, self.rot_ld, self.vdim_ld, self.rank_ld = pad(dim, 32), pad(rot, 32), pad(vdim, 32), pad(rank)
        self.ldc, self.hs = self.rank_ld + self.rot_ld, self.dim_ld + self.rot_ld
        self.ring = 1 << (window + rows - 2).bit_length()
        T = offset + rows
        self.scale = (dim + rot) ** -0.5
        self.c, self.kr = self.r.standard_normal((T, rank)), self.r.standard_normal((T, rot))
        self.q = self.r.standard_normal((rows, heads, dim + rot))
        self.uk, self.uv = self.r.standard_normal((heads, dim, rank)) / np.sqrt(rank), self.r.standard_normal((heads, vdim, rank)) / np.sqrt(rank)
        self.sink = self.r.standard_normal(heads) + 1

    def stand_out(self, row, distance, head=0, strength=6.0):
        """Makes the rotated key part `distance` behind a row point along that row's query."""
        p = self.offset + row - distance
        v = self.q[row, head, self.dim:]
        self.kr[p] = v / np.linalg.norm(v) ** 2 * strength / self.scale

    def go(self):
        """Latent sums of each form against the plain softmax over W_uk c; returns {form: outputs [rows, heads, vdim]}, ref."""
        g = self.g
        H, R = self.heads, self.rows
        to = lambda a: bf16_round(a).astype(np.float64)
        A = (lambda a: to(a)) if g.act == 16 else (lambda a: np.asarray(a, np.float32).astype(np.float64))
        c, kr, q, uk, uv, sink = A(self.c), A(self.kr), A(self.q), to(self.uk), to(self.uv), to(self.sink)
        ref = np.zeros((R, H, self.vdim))
        for h in range(H):
            k, v = c @ uk[h].T, c @ uv[h].T
            for i in range(R):
                p = self.offset + i
                lo = max(0, p - self.window + 1)
                s = (k[lo:p + 1] @ q[i, h, :self.dim] + kr[lo:p + 1] @ q[i, h, self.dim:]) * self.scale
                ref[i, h] = plain.sink_softmax(s, sink[h]) @ v[lo:p + 1]
        cache = np.zeros((self.ring, self.ldc))
        for p in range(max(0, self.offset + R - self.ring), self.offset + R):
            cache[p % self.ring, :self.rank], cache[p % self.ring, self.rank_ld:self.rank_ld + self.rot] = c[p], kr[p]
        bc, _ = g.up(np.concatenate([cache.ravel(), np.zeros(128)]))
        ldq = pad(H * self.hs)
        qq = np.zeros((R, ldq))
        for h in range(H):
            qq[:, h * self.hs:h * self.hs + self.dim] = q[:, h, :self.dim]
            qq[:, h * self.hs + self.dim_ld:h * self.hs + self.dim_ld + self.rot] = q[:, h, self.dim:]
        bq, _ = g.up(np.concatenate([qq.ravel(), np.zeros(128)]))
        bs, off = g.w16(self.sink)[0], g.raw(np.array([self.offset], np.uint32))
        qa = np.zeros((R, H, self.rank_ld))
        qa[..., :self.rank] = np.einsum("rhd,hdk->rhk", q[..., :self.dim], uk)
        bqa, _ = g.up(qa)
        shape = dict(rows=R, heads=H, hs=self.hs, dim_ld=self.dim_ld, rot=self.rot, rank_ld=self.rank_ld, ldc=self.ldc, ldq=ldq, ring=self.ring,
                     window=self.window, scale=self.scale)
        out = {}

        def lift(b):
            return np.einsum("rhk,hvk->rhv", g.down(b, (R, H, self.rank_ld))[..., :self.rank], uv)

        o = g.zeros(R * H * self.rank_ld)
        g.run("latent_attn", [bqa, bq, bc, bs, off, o], rank=self.rank, **shape)
        out["rows"] = lift(o)
        if g.act == 16 and g.native.latent_split_supported(self.rank_ld, self.ldc):
            for span in {64, 64 * -(-self.window // 64)}:
                splits = -(-self.window // span)
                part, o = g.zeros(R * splits * H * (self.rank_ld + 2), 4), g.zeros(R * H * self.rank_ld)
                g.run("latent_split", [bqa, bq, bc, off, part, bs, o], splits=splits, span=span, combine=1, **shape)
                out[f"split {span}"] = lift(o)
        if g.act == 16 and g.native.latent_prefill_supported(self.dim_ld, self.rot_ld, self.vdim_ld):
            seen, ldk = self.window - 1 + R, H * self.dim_ld
            ldv = pad(seen + 64)
            wk, wv = np.zeros((H, self.dim_ld, self.rank_ld)), np.zeros((H, self.vdim_ld, self.rank_ld))
            wk[:, :self.dim, :self.rank], wv[:, :self.vdim, :self.rank] = uk, uv
            kx, vx = g.zeros(seen * ldk), g.zeros(H * self.vdim_ld * ldv)
            back = dict(ring=self.ring, row_back=self.window - 1, k=self.rank_ld, ldx=self.ldc)
            g.run("dense", [bc, g.w16(wk)[0], off, kx], rows=seen, n=ldk, ldy=ldk, **back)
            g.run("dense", [bc, g.w16(wv)[0], off, vx], rows=seen, n=H * self.vdim_ld, ldy=ldv, transposed=1, **back)
            ldo = pad(H * self.vdim_ld)
            o = g.zeros(R * ldo)
            g.run("latent_prefill", [bq, kx, vx, bc, bs, off, o], **{k: v for k, v in shape.items() if k not in ("hs", "rot")}, rot_ld=self.rot_ld,
                  vdim_ld=self.vdim_ld, ldk=ldk, ldv=ldv, ldo=ldo)
            out["prefill"] = g.down(o, (R, ldo))[:, :H * self.vdim_ld].reshape(R, H, self.vdim_ld)[..., :self.vdim]
        return out, ref


@pytest.mark.parametrize("act", [32, 16])
@pytest.mark.parametrize("shape", [dict(heads=3, dim=24, rot=12, vdim=20, rank=40), dict(heads=16, dim=48, rot=32, vdim=64, rank=100),
                                   dict(heads=20, dim=128, rot=64, vdim=128, rank=512), dict(heads=2, dim=96, rot=64, vdim=40, rank=200),
                                   dict(heads=1, dim=200, rot=32, vdim=250, rank=300)])
@pytest.mark.parametrize("window,rows,offset", [(1, 5, 0), (30, 70, 0), (64, 3, 200), (100, 33, 61), (130, 131, 500), (65, 1, 64)])
def test_latent_attention(fk, act, shape, window, rows, offset):
    a = Attn(act, window=window, rows=rows, offset=offset, **shape)
    out, ref = a.go()
    assert act == 32 or len(out) >= 2
    for form, got in out.items():
        err = np.abs(got - ref).max() / np.abs(ref).max()
        assert err <= (3e-6 if act == 32 else 2.5e-2), (form, err)


@pytest.mark.parametrize("act", [32, 16])
@pytest.mark.parametrize("window", [16, 63, 64, 65, 128, 129])
@pytest.mark.parametrize("rows,offset", [(1, 300), (70, 230), (7, 64)])
def test_latent_window_edge_and_far_key(fk, act, window, rows, offset):
    """One key stands out just inside, then just outside the window of the last row (and far inside that of others)."""
    seen = []
    for distance in (window - 1, window):
        if offset + rows - 1 - distance < 0:
            return
        a = Attn(act, heads=2, dim=32, rot=32, vdim=32, rank=64, window=window, rows=rows, offset=offset, seed=window)
        a.stand_out(rows - 1, distance)
        out, ref = a.go()
        for form, got in out.items():
            err = np.abs(got - ref).max() / np.abs(ref).max()
            assert err <= (3e-6 if act == 32 else 3e-2), (form, distance, err)
        seen.append(ref[rows - 1, 0])
    assert np.abs(seen[0] - seen[1]).max() > 0.2 * np.abs(seen[0]).max()    # the edge shows


def test_latent_first_tokens_and_sink(fk):
    for act in (32, 16):
        for rows, offset in ((4, 0), (2, 1), (80, 0)):
            a = Attn(act, heads=4, dim=32, rot=16, vdim=32, rank=64, window=48, rows=rows, offset=offset, seed=3)
            a.sink[:] = [-30.0, 0.0, 3.0, 30.0]        # absent, ordinary, strong, everything
            out, ref = a.go()
            assert np.abs(ref[:, 3]).max() < 1e-8
            for form, got in out.items():
                assert np.abs(got - ref).max() / np.abs(ref).max() <= (3e-6 if act == 32 else 2.5e-2), form
                assert np.abs(got[:, 3]).max() < 1e-6


@pytest.mark.parametrize("act", [32, 16])
@pytest.mark.parametrize("rows,offset", [(1, 0), (1, 5000), (6, 250)])
def test_latent_store(fk, act, rows, offset):
    g, r = Rig(act), rng(rows)
    rank, rot, rd, heads, dim, ring = 40, 20, 12, 3, 24, 256     # only the first 12 of the 20 are rotated
    rank_ld, ldc, hs, dim_ld = 64, 96, 64, 32
    ldkv, ldq = pad(rank + rot), pad(heads * hs)
    kv = r.standard_normal((rows, ldkv)).astype(np.float32)
    q = r.standard_normal((rows, ldq))
    bn, nw = g.w16(1 + 0.1 * r.standard_normal(rank))
    freq = 1000.0 ** (-2.0 * np.arange(rd // 2) / rd)
    bq, vq = g.up(q)
    cache, off = g.zeros(ring * ldc), g.raw(np.array([offset], np.uint32))
    g.run("latent_store", [g.raw(kv), bn, g.raw(freq), cache, bq, off], rows=rows, rank=rank, rank_ld=rank_ld, ldkv=ldkv, ldc=ldc, ring=ring,
          heads=heads, hs=hs, dim_ld=dim_ld, rot=rot, rot_dims=rd, ldq=ldq, eps=1e-5)
    pos = offset + np.arange(rows)
    got = g.down(cache, (ring, ldc))[pos % ring]
    k = kv.astype(np.float64)
    g.close(got[:, :rank], plain.rms_norm(k[:, :rank], nw, 1e-5))
    g.close(got[:, rank_ld:rank_ld + rot], plain.rotate_half(k[:, rank:rank + rot], pos, 1000.0, rd))
    gq = g.down(bq, (rows, ldq))
    for h in range(heads):
        s = vq[:, h * hs + dim_ld:h * hs + dim_ld + rot]
        g.close(gq[:, h * hs + dim_ld:h * hs + dim_ld + rot], plain.rotate_half(s, pos, 1000.0, rd))
        assert np.array_equal(gq[:, h * hs:h * hs + dim_ld], vq[:, h * hs:h * hs + dim_ld])


# ---- state-space mixer ----

@pytest.mark.parametrize("act", [32, 16])
@pytest.mark.parametrize("taps,channels", [(1, 20), (2, 36), (3, 10), (4, 260), (5, 24)])
def test_convolution_in_portions(fk, act, taps, channels):
    g, r = Rig(act), rng(taps)
    T, ld = 60, pad(channels)
    u = r.standard_normal((T, ld))
    (bw, w), (bb, b) = g.w16(r.standard_normal((channels, taps))), g.w16(r.standard_normal(channels))
    hist = g.zeros(taps * ld)
    ref, at = None, 0
    for n in (2, 1, 1, 20, 36):
        bu, vu = g.up(u[at:at + n])
        full = bf16_round(u) if act == 16 else u.astype(np.float32)
        ref = plain.silu(plain.causal_conv(full[:, :channels].astype(np.float64), w, b))
        y, off = g.zeros(n * ld), g.raw(np.array([at], np.uint32))
        g.run("ssm_conv", [bu, bw, bb, hist, off, y], rows=n, channels=channels, taps=taps, ldu=ld, ldy=ld, ldh=ld)
        g.close(g.down(y, (n, ld))[:, :channels], ref[at:at + n])
        # the history as the recurrence kernels leave it: position p in row p % taps
        h = g.down(hist, (taps, ld))
        for t in range(max(0, n - taps + 1), n):
            h[(at + t) % taps] = vu[t]
        hist = g.up(h)[0]
        at += n


@pytest.mark.parametrize("act,form", [(32, "ssm_scan"), (16, "ssm_scan"), (16, "ssm_chunk")])
@pytest.mark.parametrize("heads,groups,n,p", [(2, 1, 8, 4), (6, 3, 24, 12), (4, 2, 64, 32), (2, 2, 128, 64), (2, 1, 200, 100)])
def test_recurrence_in_portions(fk, act, form, heads, groups, n, p):
    g, r = Rig(act), rng(heads * n)
    if form == "ssm_chunk" and not g.native.ssm_chunk_supported(heads, p, n):
        pytest.skip("no chunked form of this shape")
    T, inner = 260, heads * p
    ch, sl = inner + 2 * groups * n, pad(n)
    ldx, ldt, ldy = pad(ch), pad(heads), pad(inner)
    xbc = padded(r.standard_normal((T, ch)).astype(np.float32), ldx)
    dt = padded((r.standard_normal((T, heads)) - 1).astype(np.float32), ldt)
    # decays from nearly none to nearly all within a few tokens
    (bdt, vdt), (ba, va), (bd, vd) = g.w16(r.standard_normal(heads) * 0.3), g.w16(np.linspace(-5, 2, heads)), g.w16(r.standard_normal(heads))
    full = (bf16_round(xbc) if act == 16 else xbc).astype(np.float64)
    gi = np.arange(heads) // (heads // groups)
    ref = plain.ssd_recurrence(full[:, :inner].reshape(T, heads, p), full[:, inner:inner + groups * n].reshape(T, groups, n)[:, gi],
                               full[:, inner + groups * n:ch].reshape(T, groups, n)[:, gi], plain.softplus(dt[:, :heads].astype(np.float64) + vdt), va, vd)
    state, hist = g.zeros(heads * p * sl, 4), g.zeros(3 * ldx)
    at = 0
    for m in (2, 70, 64, 1, 123):
        bx, _ = g.up(xbc[at:at + m])
        y, off = g.zeros(m * ldy), g.raw(np.array([at], np.uint32))
        bufs = [bx, g.raw(dt[at:at + m]), bdt, ba, bd, bx, off, state, hist, y]
        if form == "ssm_chunk":
            bufs += [g.zeros(-(-m // 64) * heads * p * sl, 4), g.zeros(-(-m // 64) * heads, 4)]
        g.run(form, bufs, rows=m, heads=heads, groups=groups, n=n, p=p, state_ld=sl, ldx=ldx, lddt=ldt, ldy=ldy, ldu=ldx, ldh=ldx, channels=ch, taps=3)
        g.close(g.down(y, (m, ldy))[:, :inner].reshape(m, heads, p), ref[at:at + m], 1e-5 if act == 32 else 6e-3)
        at += m
    # the state itself is fp32 in either form
    S = np.zeros((heads, n, p))
    dts = plain.softplus(dt[:, :heads].astype(np.float64) + vdt)
    for t in range(T):
        for h in range(heads):
            S[h] = np.exp(-np.exp(va[h]) * dts[t, h]) * S[h] + dts[t, h] * np.outer(full[t, inner + gi[h] * n:inner + (gi[h] + 1) * n], full[t, h * p:(h + 1) * p])
    got = state.to_numpy(np.float32, (heads, p, sl))
    assert np.abs(got[..., :n].transpose(0, 2, 1) - S).max() <= 2e-5 * np.abs(S).max()
    assert not got[..., n:].any()
    h = g.down(hist, (3, ldx))
    for t in (T - 2, T - 1):
        assert np.array_equal(h[t % 3, :ch], full[t, :ch])


def test_bad_shapes_are_refused(fk):
    from fusekit_amd.native import FusekitError
    g = Rig(16)
    b = g.zeros(64 * 64)
    off = g.raw(np.zeros(1, np.uint32))
    cases = [("dense", [b, b, b], dict(rows=2, n=4, k=40, ldx=64, ldw=64, ldy=4)),
             ("dense", [b, b, b], dict(rows=80, n=4, k=64, ldx=64, ldw=64, ldy=4)),                      # x too small
             ("dense", [b, b, off, b], dict(rows=2, n=4, k=64, ldx=64, ldw=64, ldy=4, ring=48)),         # no power of two
             ("residual_norm", [b], dict(rows=1, width=40, ld=40)),
             ("group_norm", [b, b, b], dict(rows=1, width=10, groups=3, ldx=64, ldy=64)),
             ("route_rows", [b, b, b, b], dict(rows=1, outputs=4, top=5)),
             ("latent_attn", [b, b, b, b, off, b], dict(rows=9, heads=1, hs=64, dim_ld=32, rot=16, rank=10, rank_ld=32, ldc=64, ldq=64, ring=16, window=9)),
             ("ssm_scan", [b] * 10, dict(rows=1, heads=3, groups=2, n=8, p=4, state_ld=64, ldx=64, lddt=64, ldy=64, ldu=64, ldh=64, channels=44, taps=2)),
             ("layer_jobs", [], {}),
             ("layer_out", [b], dict(n=0))]
    for kernel, bufs, p in cases:
        with pytest.raises(FusekitError):
            g.run(kernel, bufs, **p)
