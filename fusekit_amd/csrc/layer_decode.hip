// One decoded token of the layer-list decoder in few launches (bf16).
//
// Two kernels.  `layer_jobs_kernel` runs several independent jobs of a layer side by side, each on its own range of
// workgroups, so that what only depends on the previous launch shares one:
//   * matrix-vector products whose input row is formed while it is staged in LDS -- an RMS norm of the fp32 residual
//     row, a gated norm in groups, the combination of the attention's partial rows -- with the first weight rows
//     already requested;
//   * the gate / up pair of the chosen experts;
//   * the router's softmax and choice, the latent cache row;
//   * a step of a state-space mixer, a gated delta rule or a gated linear recurrence, with its convolution and gates.
// `layer_out_kernel` closes a layer: per element of the residual row the mixer's output projection, the weighted down
// projections of the chosen experts and the identities' share, added to the row in fp32.
//
// A latent-attention layer is six launches (norms + down projections + router | queries, cache row, choice | queries
// into the latent space, gate / up | attention | W_uv | output), a state-space layer four.  A joint layer is the norm with
// the joint input projection, the recurrence's step (or the cache rows and the attention), the joint output projection.
#include "column_device.hpp"
#include "layer_decode.hpp"
#include "lru_device.hpp"
#include "split_device.hpp"

namespace fk {

namespace {

typedef uint32_t ld_u32x4_t __attribute__((ext_vector_type(4)));

constexpr int kJobBlock = 256;
static_assert(kMaxSplits <= kMaxGateGroups, "both lists share the LDS behind the reduction words");
constexpr uint32_t kAhead = 4;   // pieces of two rows in flight per wave: a piece is 64 lanes x 16 bytes = 512 elements

__device__ __forceinline__ float dot8(ld_u32x4_t a, ld_u32x4_t b, float s) {
    s = dot2_bf16(a[0], b[0], s);
    s = dot2_bf16(a[1], b[1], s);
    s = dot2_bf16(a[2], b[2], s);
    return dot2_bf16(a[3], b[3], s);
}

// Two matrix rows per turn against the staged row, `turns` turns, as one stream of pieces: four pieces of both rows are
// in flight, a piece is multiplied and its register takes the piece four ahead.  `rows(turn, w0, w1)` gives a turn's
// rows, `emit(turn, s0, s1)` takes its sums.  start() issues the first requests and may be called before the row is
// staged.  Lanes past a row's end read its last 16 bytes and add nothing; the stream is padded to whole groups of four
// pieces with repeats of its last.
template <typename Rows>
struct PairStream {
    const Rows& rows;
    uint32_t pieces, per_row, total, lane;
    ld_u32x4_t v[kAhead][2];
    uint32_t ft = 0, fi = 0, fetched = 0;

    __device__ PairStream(const Rows& r, uint32_t k, uint32_t turns, uint32_t l)
        : rows(r), pieces(k / 8u), per_row((k + 511u) / 512u), total(turns * ((k + 511u) / 512u)), lane(l) {}
    __device__ __forceinline__ void fetch(uint32_t u) {
        const uint16_t *w0, *w1;
        rows(ft, w0, w1);
        const uint32_t c = fi * 64u + lane, at = (c < pieces ? c : pieces - 1u) * 8u;
        v[u][0] = *reinterpret_cast<const ld_u32x4_t*>(w0 + at);
        v[u][1] = *reinterpret_cast<const ld_u32x4_t*>(w1 + at);
        if (++fetched < total && ++fi == per_row) { fi = 0; ++ft; }
    }
    __device__ __forceinline__ void start() {
#pragma unroll
        for (uint32_t u = 0; u < kAhead; ++u) fetch(u);
    }
    template <typename Emit>
    __device__ __forceinline__ void run(const uint16_t* xs, const Emit& emit) {
        float s0 = 0.f, s1 = 0.f;
        uint32_t ut = 0, ui = 0, used = 0;
        auto use = [&](uint32_t u) __attribute__((always_inline)) {
            const uint32_t c = ui * 64u + lane;
            if (used < total && c < pieces) {
                const ld_u32x4_t x = *reinterpret_cast<const ld_u32x4_t*>(xs + c * 8u);
                s0 = dot8(v[u][0], x, s0);
                s1 = dot8(v[u][1], x, s1);
            }
        };
        auto step = [&]() __attribute__((always_inline)) {
            if (used < total && ++ui == per_row) {
                emit(ut, wave_sum(s0), wave_sum(s1));
                s0 = s1 = 0.f;
                ui = 0;
                ++ut;
            }
            ++used;
        };
        const uint32_t groups = (total + kAhead - 1u) / kAhead;
        for (uint32_t g = 0; g + 1u < groups; ++g) {
#pragma unroll
            for (uint32_t u = 0; u < kAhead; ++u) {
                use(u);
                fetch(u);
                step();
            }
        }
#pragma unroll
        for (uint32_t u = 0; u < kAhead; ++u) {
            use(u);
            step();
        }
    }
};

// The input row of a product, as bf16 in LDS.  k elements are written (zeros past the width).
__device__ void stage_row(const GemvJob& j, uint32_t head, uint32_t first_block, uint16_t* xs, float* red) {
    const uint32_t tid = threadIdx.x;
    if (j.mode == kRowPlain) {
        const uint16_t* x = reinterpret_cast<const uint16_t*>(j.x) + (size_t)head * j.x_head;
        for (uint32_t c = tid * 8u; c < j.k; c += kJobBlock * 8u) *reinterpret_cast<ld_u32x4_t*>(xs + c) = *reinterpret_cast<const ld_u32x4_t*>(x + c);
    } else if (j.mode == kRowNorm) {
        const float* x = reinterpret_cast<const float*>(j.x);
        const uint16_t* step = reinterpret_cast<const uint16_t*>(j.x2);
        float ss = 0.f;
        constexpr uint32_t kHold = 4;   // 4096 elements stay in registers between the two passes
        float4 held[kHold];
        auto load = [&](uint32_t c) __attribute__((always_inline)) {
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (c + 4u <= j.width && j.vec) v = *reinterpret_cast<const float4*>(x + c);
            else {
                v.x = c < j.width ? x[c] : 0.f; v.y = c + 1u < j.width ? x[c + 1u] : 0.f;
                v.z = c + 2u < j.width ? x[c + 2u] : 0.f; v.w = c + 3u < j.width ? x[c + 3u] : 0.f;
            }
            if (step) {
                const float4 s = act_load4(step + c);
                v.x += s.x; v.y += s.y; v.z += s.z; v.w += s.w;
            }
            return v;
        };
#pragma unroll
        for (uint32_t i = 0; i < kHold; ++i) {
            const uint32_t c = (tid + i * kJobBlock) * 4u;
            held[i] = c < j.k ? load(c) : make_float4(0.f, 0.f, 0.f, 0.f);
            ss = fmaf(held[i].x, held[i].x, ss); ss = fmaf(held[i].y, held[i].y, ss);
            ss = fmaf(held[i].z, held[i].z, ss); ss = fmaf(held[i].w, held[i].w, ss);
        }
        for (uint32_t c = (tid + kHold * kJobBlock) * 4u; c < j.k; c += kJobBlock * 4u) {
            const float4 v = load(c);
            ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
        }
        float mean = 0.f;
        if (j.nb) {   // layer norm: ss becomes the sum of the squared deviations
            float sum = 0.f;
#pragma unroll
            for (uint32_t i = 0; i < kHold; ++i) sum += (held[i].x + held[i].y) + (held[i].z + held[i].w);
            for (uint32_t c = (tid + kHold * kJobBlock) * 4u; c < j.k; c += kJobBlock * 4u) {
                const float4 v = load(c);
                sum += (v.x + v.y) + (v.z + v.w);
            }
            mean = block_sum<kJobBlock>(sum, red + 4) / (float)j.width;
            ss = 0.f;
            auto dev = [&](uint32_t c, float4 v) __attribute__((always_inline)) {
                const float d[4] = {v.x - mean, v.y - mean, v.z - mean, v.w - mean};
#pragma unroll
                for (uint32_t e = 0; e < 4; ++e) ss = c + e < j.width ? fmaf(d[e], d[e], ss) : ss;
            };
#pragma unroll
            for (uint32_t i = 0; i < kHold; ++i) dev((tid + i * kJobBlock) * 4u, held[i]);
            for (uint32_t c = (tid + kHold * kJobBlock) * 4u; c < j.k; c += kJobBlock * 4u) dev(c, load(c));
        }
        ss = block_sum<kJobBlock>(ss, red);
        const float r = 1.0f / sqrtf(ss / (float)j.width + j.eps);
        auto put = [&](uint32_t c, float4 v) __attribute__((always_inline)) {
            const float4 w = act_load4(j.nw + c), b = j.nb ? act_load4(j.nb + c) : make_float4(0.f, 0.f, 0.f, 0.f);
            v.x = (v.x - mean) * r; v.y = (v.y - mean) * r; v.z = (v.z - mean) * r; v.w = (v.w - mean) * r;
            const uint2 o = make_uint2(pack_bf16(fmaf(v.x, w.x, b.x), fmaf(v.y, w.y, b.y)), pack_bf16(fmaf(v.z, w.z, b.z), fmaf(v.w, w.w, b.w)));
            *reinterpret_cast<uint2*>(xs + c) = o;
            if (j.keep && first_block) *reinterpret_cast<uint2*>(j.keep + c) = o;
        };
#pragma unroll
        for (uint32_t i = 0; i < kHold; ++i) {
            const uint32_t c = (tid + i * kJobBlock) * 4u;
            if (c < j.k) put(c, held[i]);
        }
        for (uint32_t c = (tid + kHold * kJobBlock) * 4u; c < j.k; c += kJobBlock * 4u) put(c, load(c));
    } else if (j.mode == kRowGated) {
        const uint16_t *y = reinterpret_cast<const uint16_t*>(j.x), *z = reinterpret_cast<const uint16_t*>(j.x2);
        const uint32_t part = j.width / j.groups;
        float* sums = red + 8;          // one mean square per group (at most kMaxGateGroups)
        // a wave takes whole groups when there are several, else the block shares each
        if (j.groups >= 4u) {
            const uint32_t lane = tid & 63u, wave = tid >> 6;
            for (uint32_t g = wave; g < j.groups; g += 4u) {
                float ss = 0.f;
                for (uint32_t c = g * part + lane; c < (g + 1u) * part; c += 64u) {
                    const float v = act_load(y + c) * silu(act_load(z + c));
                    ss = fmaf(v, v, ss);
                }
                ss = wave_sum(ss);
                if (lane == 0) sums[g] = 1.0f / sqrtf(ss / (float)part + j.eps);
            }
        } else {
            for (uint32_t g = 0; g < j.groups; ++g) {
                float ss = 0.f;
                for (uint32_t c = g * part + tid; c < (g + 1u) * part; c += kJobBlock) {
                    const float v = act_load(y + c) * silu(act_load(z + c));
                    ss = fmaf(v, v, ss);
                }
                ss = block_sum<kJobBlock>(ss, red);
                __syncthreads();
                if (tid == 0) sums[g] = 1.0f / sqrtf(ss / (float)part + j.eps);
            }
        }
        __syncthreads();
        for (uint32_t c = tid; c < j.k; c += kJobBlock) {
            float v = 0.f;
            if (c < j.width) v = act_load(y + c) * silu(act_load(z + c)) * sums[c / part] * bf16_bits_to_f32(j.nw[c]);
            act_store(xs + c, v);
        }
    } else if (j.mode == kRowJoin) {
        const float* x = reinterpret_cast<const float*>(j.x);
        const uint16_t* second = reinterpret_cast<const uint16_t*>(j.x2);
        const uint32_t half = j.k / 2u;
        for (uint32_t c = tid * 4u; c < half; c += kJobBlock * 4u) {
            float v[4];
#pragma unroll
            for (uint32_t e = 0; e < 4; ++e) v[e] = c + e < j.width ? x[c + e] : 0.f;
            *reinterpret_cast<uint2*>(xs + c) = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]));
            *reinterpret_cast<uint2*>(xs + half + c) = *reinterpret_cast<const uint2*>(second + c);
        }
    } else {   // kRowCombine: the partial rows of one head, [splits][heads][pl] = latent sums | maximum | sum
        const float* p = reinterpret_cast<const float*>(j.x) + (size_t)head * j.pl;
        const size_t ss = (size_t)j.heads * j.pl;
        float* w = red + 8;
        split_weights(p + j.k, ss, j.splits, bf16_bits_to_f32(j.nw[head]), w);   // nw: the sinks
        __syncthreads();
        for (uint32_t c = tid * 2u; c < j.k; c += kJobBlock * 2u) {
            float v0 = 0.f, v1 = 0.f;
#pragma unroll 8
            for (uint32_t s = 0; s < j.splits; ++s) {
                const float2 q = *reinterpret_cast<const float2*>(p + s * ss + c);
                v0 = fmaf(w[s], q.x, v0);
                v1 = fmaf(w[s], q.y, v1);
            }
            *reinterpret_cast<uint32_t*>(xs + c) = pack_bf16(v0, v1);
        }
    }
}

// Softmax over `outputs` logits and the choice of `top`, by one wave.
template <int PER>
__device__ void route_wave(const RouteJob& a, uint32_t lane) {
    float s[PER], choice[PER], mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        const uint32_t e = lane + (uint32_t)i * 64u;
        s[i] = e < a.outputs ? a.logits[e] : -INFINITY;
        choice[i] = e < a.outputs ? bf16_bits_to_f32(a.correction[e]) : 0.f;
        mx = fmaxf(mx, s[i]);
    }
    mx = wave_max(mx);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        s[i] = expf(s[i] - mx);
        sum += s[i];
    }
    sum = wave_sum(sum);
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        s[i] /= sum;
        choice[i] = lane + (uint32_t)i * 64u < a.outputs ? choice[i] + s[i] : -INFINITY;
    }
    float mine = 0.f, total = 0.f;
    uint32_t mine_i = 0;
    for (uint32_t t = 0; t < a.top; ++t) {
        float best = choice[0], bs = s[0];
        uint32_t bi = lane;
#pragma unroll
        for (int i = 1; i < PER; ++i)
            if (choice[i] > best) { best = choice[i]; bs = s[i]; bi = lane + (uint32_t)i * 64u; }
        const float top = wave_max(best);
        uint64_t who = __builtin_amdgcn_ballot_w64(best == top);
        uint32_t win = 0;
        if (who) {
            uint32_t from = (uint32_t)__builtin_ctzll(who);
            win = (uint32_t)__builtin_amdgcn_readlane((int)bi, (int)from);
            for (who &= who - 1ull; who; who &= who - 1ull) {   // equal scores: the lower index
                const uint32_t l = (uint32_t)__builtin_ctzll(who), o = (uint32_t)__builtin_amdgcn_readlane((int)bi, (int)l);
                if (o < win) { win = o; from = l; }
            }
            const float w = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(bs), (int)from));
            if (lane == t) { mine = w; mine_i = win; }
            total += w;
            if (lane == from) {
#pragma unroll
                for (int i = 0; i < PER; ++i)
                    if (lane + (uint32_t)i * 64u == win) choice[i] = -INFINITY;
            }
        }
    }
    if (lane < a.top) {
        a.index[lane] = mine_i;
        a.weight[lane] = mine / (total + 1e-20f);
    }
}

// The cache row of one position: the normalised latent and the rotated key part.
__device__ void store_row(const StoreJob& a, float* red, float* cs) {
    const uint32_t tid = threadIdx.x, pos = *a.offset, half = a.rot_dims / 2u;
    uint16_t* row = a.cache + (size_t)(pos & (a.ring - 1u)) * a.ldc;
    for (uint32_t i = tid; i < half; i += kJobBlock) {
        position_cos_sin(pos, a.freq[i], cs[2 * i], cs[2 * i + 1]);
        a.tab[2 * i] = cs[2 * i];
        a.tab[2 * i + 1] = cs[2 * i + 1];
    }
    float ss = 0.f;
    for (uint32_t c = tid; c < a.rank; c += kJobBlock) ss = fmaf(a.kv[c], a.kv[c], ss);
    ss = block_sum<kJobBlock>(ss, red);
    const float r = 1.0f / sqrtf(ss / (float)a.rank + a.eps);
    for (uint32_t c = tid; c < a.rank; c += kJobBlock) act_store(row + c, a.kv[c] * r * bf16_bits_to_f32(a.norm[c]));
    const float* s = a.kv + a.rank;
    for (uint32_t i = tid; i < a.rot; i += kJobBlock) {
        float v = s[i];
        if (i < half) v = s[i] * cs[2 * i] - s[i + half] * cs[2 * i + 1];
        else if (i < a.rot_dims) v = s[i] * cs[2 * (i - half)] + s[i - half] * cs[2 * (i - half) + 1];
        act_store(row + a.rank_ld + i, v);
    }
}

// One token of one head and sixteen value columns: the convolution of the columns it needs, then the state.
// The history ring holds `taps` rows: this token's row takes the place of the one that has left the convolution, so the
// rows other workgroups still read are never the one written.
__device__ void scan_step(const ScanJob& a, uint32_t h, uint32_t pt, float* sm) {
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, pos = *a.offset;
    const uint32_t inner = a.heads * a.p, per = a.heads / a.groups, g = h / per, p0 = pt * 16u;
    const uint32_t slot = pos % a.taps;
    float *xs = sm, *B = sm + 16, *C = B + a.state_ld;   // 16 columns of x, then B and C padded to state_ld
    const uint32_t pl = p0 + wave * 4u + (lane >> 4), nl = (lane & 15u) * 4u;
    const bool live = pl < a.p;
    const uint32_t p = live ? pl : a.p - 1u, ni = a.state_ld / 64u;
    float* state = a.state + ((size_t)h * a.p + p) * a.state_ld + nl;
    float4 S[4];
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i)
        if (i < ni) S[i] = *reinterpret_cast<const float4*>(state + 64u * i);
    for (uint32_t i = tid; i < 16u + 2u * a.state_ld; i += kJobBlock) {
        uint32_t ch = 0xffffffffu;
        bool write = false;
        if (i < 16u) {
            if (p0 + i < a.p) { ch = h * a.p + p0 + i; write = true; }
        } else if (i < 16u + a.state_ld) {
            if (i - 16u < a.n) { ch = inner + g * a.n + i - 16u; write = h % per == 0u && pt == 0u; }
        } else if (i - 16u - a.state_ld < a.n) {
            ch = inner + (a.groups + g) * a.n + i - 16u - a.state_ld;
            write = h % per == 0u && pt == 0u;
        }
        float v = 0.f;
        if (ch != 0xffffffffu) {
            const uint16_t raw = a.u[ch];
            v = bf16_bits_to_f32(a.b[ch]);
            const uint16_t* w = a.w + (size_t)ch * a.taps;
            for (uint32_t k = 0; k + 1u < a.taps; ++k) {
                const uint32_t back = a.taps - 1u - k;
                if (back <= pos) v = fmaf(bf16_bits_to_f32(w[k]), bf16_bits_to_f32(a.hist[(size_t)((pos - back) % a.taps) * a.ldh + ch]), v);
            }
            v = round_bf16(silu(fmaf(bf16_bits_to_f32(w[a.taps - 1u]), bf16_bits_to_f32(raw), v)));
            if (write) a.hist[(size_t)slot * a.ldh + ch] = raw;
        }
        sm[i] = v;
    }
    const float dt = softplus(a.dt[h] + bf16_bits_to_f32(a.dt_bias[h])), decay = expf(-expf(bf16_bits_to_f32(a.a_log[h])) * dt);
    __syncthreads();
    const float x = xs[wave * 4u + (lane >> 4)], sx = dt * x;
    float out = 0.f;
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i) {
        if (i >= ni) break;
        const float4 b = *reinterpret_cast<const float4*>(B + nl + 64u * i), c = *reinterpret_cast<const float4*>(C + nl + 64u * i);
        S[i].x = fmaf(decay, S[i].x, sx * b.x); S[i].y = fmaf(decay, S[i].y, sx * b.y);
        S[i].z = fmaf(decay, S[i].z, sx * b.z); S[i].w = fmaf(decay, S[i].w, sx * b.w);
        out = fmaf(S[i].x, c.x, out); out = fmaf(S[i].y, c.y, out);
        out = fmaf(S[i].z, c.z, out); out = fmaf(S[i].w, c.w, out);
        if (live) *reinterpret_cast<float4*>(state + 64u * i) = S[i];
    }
    out = group_sum(out, 16);
    if (live && nl == 0) act_store(a.y + (size_t)h * a.p + p, fmaf(bf16_bits_to_f32(a.d[h]), x, out));
}

// The convolution of one channel for the token at `pos`; its raw input takes the ring row of the one that has left.
__device__ __forceinline__ float conv_token(const uint16_t* u, const uint16_t* w, const uint16_t* b, uint16_t* hist, uint32_t ch, uint32_t taps, uint32_t ldh,
                                            uint32_t pos, bool write) {
    const uint16_t raw = u[ch];
    const uint16_t* k = w + (size_t)ch * taps;
    float v = b ? bf16_bits_to_f32(b[ch]) : 0.f;
    const uint32_t slot = pos % taps;
    if (taps <= 4u) {   // every request ahead of the first use; rows before the start are multiplied away
        uint16_t past[3], w3[3];
#pragma unroll
        for (uint32_t i = 0; i < 3; ++i) {
            const uint32_t back = i + 1u, at = slot >= back ? slot - back : slot + taps - back;
            const bool in = back < taps;
            past[i] = hist[(size_t)(in ? at : 0u) * ldh + ch];
            w3[i] = k[in ? taps - 1u - back : 0u];
        }
#pragma unroll
        for (uint32_t i = 3; i-- > 0;)
            if (i + 1u < taps && i + 1u <= pos) v = fmaf(bf16_bits_to_f32(w3[i]), bf16_bits_to_f32(past[i]), v);
    } else {
        for (uint32_t i = 0; i + 1u < taps; ++i) {
            const uint32_t back = taps - 1u - i;
            if (back <= pos) v = fmaf(bf16_bits_to_f32(k[i]), bf16_bits_to_f32(hist[(size_t)((pos - back) % taps) * ldh + ch]), v);
        }
    }
    v = fmaf(bf16_bits_to_f32(k[taps - 1u]), bf16_bits_to_f32(raw), v);
    if (write) hist[(size_t)slot * ldh + ch] = raw;
    return v;
}

// One token of one head and sixteen value columns of a gated delta rule (the layout of delta.hip).  Every workgroup of a
// head forms its unit vectors and decays itself: the second decay projection is dim x rank, out of the L2 for all but one.
__device__ void delta_step(const DeltaJob& a, uint32_t h, uint32_t pt, float* sm) {
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, pos = *a.offset;
    const uint32_t per = a.heads / a.kv_heads, g = h / per, nk = a.kv_heads * a.dim_ld, p0 = pt * 16u;
    float *qs = sm, *ks = qs + a.state_ld, *gs = ks + a.state_ld, *vs = gs + a.state_ld;
    const uint32_t pl = wave * 4u + (lane >> 4), nl = (lane & 15u) * 4u, ni = a.state_ld / 64u;
    float* state = a.state + ((size_t)h * a.vdim_ld + p0 + pl) * a.state_ld + nl;
    float4 S[4];
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i)
        if (i < ni) S[i] = *reinterpret_cast<const float4*>(state + 64u * i);
    // decays: four lanes per row of the projection
    for (uint32_t d = tid >> 2; d < a.state_ld; d += kJobBlock / 4u) {
        float z = 0.f;
        if (d < a.dim_ld) {
            const uint16_t* row = a.a2 + ((size_t)h * a.dim_ld + d) * a.rank_ld;
#pragma unroll 4
            for (uint32_t c = (tid & 3u) * 8u; c < a.rank_ld; c += 32u)
                z = dot8(*reinterpret_cast<const ld_u32x4_t*>(row + c), *reinterpret_cast<const ld_u32x4_t*>(a.a1 + c), z);
        }
        z = group_sum(z, 4);
        if ((tid & 3u) == 0)
            gs[d] = d < a.dim_ld ? expf(-expf(bf16_bits_to_f32(a.a_log[h])) * softplus(z + bf16_bits_to_f32(a.dt_bias[(size_t)h * a.dim_ld + d]))) : 0.f;
    }
    for (uint32_t i = tid; i < 2u * a.state_ld + 16u; i += kJobBlock) {
        uint32_t ch = 0xffffffffu, at = i;
        bool write = h % per == 0u && pt == 0u;
        if (i < a.state_ld) {
            if (i < a.dim_ld) ch = g * a.dim_ld + i;
        } else if (i < 2u * a.state_ld) {
            if (i - a.state_ld < a.dim_ld) ch = nk + g * a.dim_ld + i - a.state_ld;
        } else {
            ch = 2u * nk + h * a.vdim_ld + p0 + i - 2u * a.state_ld;
            at = i + a.state_ld;   // behind the decays
            write = true;
        }
        sm[at] = ch != 0xffffffffu ? round_bf16(silu(conv_token(a.u, a.w, nullptr, a.hist, ch, a.taps, a.ldh, pos, write))) : 0.f;
    }
    const float beta = sigmoid(a.beta[h]);
    __syncthreads();
    float qq = 0.f, kk = 0.f;
    for (uint32_t c = lane; c < a.state_ld; c += 64u) {
        qq = fmaf(qs[c], qs[c], qq);
        kk = fmaf(ks[c], ks[c], kk);
    }
    const float fq = 1.0f / (sqrtf(wave_sum(qq) + 1e-6f) * sqrtf((float)a.dim)), fk = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
    float sk = 0.f, sq = 0.f, kq = 0.f;
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i) {
        if (i >= ni) break;
        const float4 k = *reinterpret_cast<const float4*>(ks + nl + 64u * i), q = *reinterpret_cast<const float4*>(qs + nl + 64u * i);
        const float4 d = *reinterpret_cast<const float4*>(gs + nl + 64u * i);
        S[i].x *= d.x; S[i].y *= d.y; S[i].z *= d.z; S[i].w *= d.w;
        sk = fmaf(S[i].x, k.x, sk); sk = fmaf(S[i].y, k.y, sk); sk = fmaf(S[i].z, k.z, sk); sk = fmaf(S[i].w, k.w, sk);
        sq = fmaf(S[i].x, q.x, sq); sq = fmaf(S[i].y, q.y, sq); sq = fmaf(S[i].z, q.z, sq); sq = fmaf(S[i].w, q.w, sq);
        kq = fmaf(k.x, q.x, kq); kq = fmaf(k.y, q.y, kq); kq = fmaf(k.z, q.z, kq); kq = fmaf(k.w, q.w, kq);
    }
    sk = group_sum(sk, 16) * fk;
    sq = group_sum(sq, 16) * fq;
    kq = group_sum(kq, 16) * fk * fq;
    const float u = beta * (vs[pl] - sk), uk = u * fk;
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i) {
        if (i >= ni) break;
        const float4 k = *reinterpret_cast<const float4*>(ks + nl + 64u * i);
        S[i].x = fmaf(k.x, uk, S[i].x); S[i].y = fmaf(k.y, uk, S[i].y); S[i].z = fmaf(k.z, uk, S[i].z); S[i].w = fmaf(k.w, uk, S[i].w);
        *reinterpret_cast<float4*>(state + 64u * i) = S[i];
    }
    if (nl == 0) a.o[(size_t)h * a.vdim_ld + p0 + pl] = fmaf(kq, u, sq);
}

// One token of some channels of one diagonal block: the convolution of the whole block, their gates, then a thread per
// channel, whose state and constants have been on their way since the start.
__device__ void lru_token(const LruJob& a, uint32_t part, uint32_t sub, uint16_t* xs, float* gates) {
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, pos = *a.offset;
    const uint32_t c0 = sub * kLruRows, count = a.block - c0 < kLruRows ? a.block - c0 : kLruRows;
    const uint32_t turns = wave < count ? (count - wave + 3u) / 4u : 0u, mine = part * a.block + c0 + (tid < count ? tid : 0u);
    const uint16_t *wr = a.gates + (size_t)part * 2u * a.block * a.block, *wi = wr + (size_t)a.block * a.block;
    auto rows = [&](uint32_t t, const uint16_t*& w0, const uint16_t*& w1) __attribute__((always_inline)) {
        const uint32_t r = wave + t * 4u, rr = c0 + (r < count ? r : count - 1u);
        w0 = wr + (size_t)rr * a.block;
        w1 = wi + (size_t)rr * a.block;
    };
    PairStream<decltype(rows)> st(rows, a.block, turns, lane);
    st.start();
    const float rb = bf16_bits_to_f32(a.rb[mine]), ib = bf16_bits_to_f32(a.ib[mine]), y = act_load(a.y + mine);
    const uint16_t lam = a.lam[mine];
    float S = a.state[mine];
    for (uint32_t i = tid; i < a.block; i += kJobBlock)
        act_store(xs + i, conv_token(a.u, a.w, a.b, a.hist, part * a.block + i, a.taps, a.ldh, pos, i - c0 < count));
    __syncthreads();
    if (turns)
        st.run(xs, [&](uint32_t t, float zr, float zi) __attribute__((always_inline)) {
            const uint32_t r = wave + t * 4u;
            if (lane == 0 && r < count) {
                gates[r] = zr;
                gates[kLruRows + r] = zi;
            }
        });
    __syncthreads();
    if (tid >= count) return;
    float decay, add;
    lru_step_fast(gates[tid] + rb, gates[kLruRows + tid] + ib, lru_rate(lam), act_load(xs + c0 + tid), decay, add);
    S = fmaf(decay, S, add);
    a.state[mine] = S;
    act_store(a.y + mine, S * y);
}

__global__ __launch_bounds__(kJobBlock) void layer_jobs_kernel(const LayerJobsArgs a) {
    extern __shared__ __align__(16) uint16_t lds[];
    __shared__ __align__(16) float red[8 + kMaxGateGroups];
    const uint32_t b = blockIdx.x, lane = threadIdx.x & 63u, wave = threadIdx.x >> 6;
    for (uint32_t i = 0; i < kMaxGemvJobs; ++i) {
        const GemvJob& j = a.gemv[i];
        if (b - j.first >= j.blocks) continue;
        const uint32_t local = b - j.first, head = j.rows_per_head ? local / j.blocks_per_head : 0u;
        uint32_t row0, count;
        if (j.rows_per_head) {
            const uint32_t part = local - head * j.blocks_per_head;
            row0 = part * j.rows_per_block;
            count = j.rows_per_head - row0 < j.rows_per_block ? j.rows_per_head - row0 : j.rows_per_block;
            row0 += head * j.rows_per_head;
        } else {
            row0 = local * j.rows_per_block;
            count = j.n - row0 < j.rows_per_block ? j.n - row0 : j.rows_per_block;
        }
        const uint32_t turns = wave * 2u < count ? (count - wave * 2u + 7u) / 8u : 0u;
        auto rows = [&](uint32_t t, const uint16_t*& w0, const uint16_t*& w1) __attribute__((always_inline)) {
            const uint32_t r = wave * 2u + t * 8u, ra = r < count ? r : count - 1u, rb = r + 1u < count ? r + 1u : count - 1u;
            w0 = j.w + (size_t)(row0 + ra) * j.ldw;
            w1 = j.w + (size_t)(row0 + rb) * j.ldw;
        };
        PairStream<decltype(rows)> st(rows, j.k, turns, lane);
        st.start();   // the first weight rows are on their way while the input row is formed
        stage_row(j, head, local == 0u, lds, red);
        __syncthreads();
        if (!turns) return;
        const uint32_t y0 = row0 + head * (j.y_head - j.rows_per_head);   // y_head equals rows_per_head without heads
        st.run(lds, [&](uint32_t t, float s0, float s1) __attribute__((always_inline)) {
            const uint32_t r = wave * 2u + t * 8u + lane;
            if (lane < 2u && r < count) {
                const float v = column_value(j.out, row0 + r, lane ? s1 : s0);
                if (row0 + r >= j.n_act) j.y32[y0 + r - j.n_act] = v;
                else reinterpret_cast<uint16_t*>(j.y)[y0 + r] = (uint16_t)f32_to_bf16_bits(v);
            }
        });
        return;
    }
    if (b - a.pair.first < a.pair.blocks) {
        const PairJob& j = a.pair;
        const uint32_t local = b - j.first, slot = local / j.blocks_per_slot, part = local - slot * j.blocks_per_slot;
        const uint32_t e = j.index[slot];
        if (e >= j.experts) return;   // an identity
        const uint32_t row0 = part * j.rows_per_block, end = row0 + j.rows_per_block < j.n ? row0 + j.rows_per_block : j.n;
        const uint16_t *wa = j.wa + (size_t)e * j.n * j.ldw, *wb = j.wb + (size_t)e * j.n * j.ldw;
        const uint32_t turns = row0 + wave < end ? (end - row0 - wave + 3u) / 4u : 0u;
        auto rows = [&](uint32_t t, const uint16_t*& w0, const uint16_t*& w1) __attribute__((always_inline)) {
            const uint32_t r = row0 + wave + t * 4u, rr = r < end ? r : end - 1u;
            w0 = wa + (size_t)rr * j.ldw;
            w1 = wb + (size_t)rr * j.ldw;
        };
        PairStream<decltype(rows)> st(rows, j.k, turns, lane);
        st.start();
        for (uint32_t c = threadIdx.x * 8u; c < j.k; c += kJobBlock * 8u) *reinterpret_cast<ld_u32x4_t*>(lds + c) = *reinterpret_cast<const ld_u32x4_t*>(j.x + c);
        __syncthreads();
        if (!turns) return;
        st.run(lds, [&](uint32_t t, float s0, float s1) __attribute__((always_inline)) {
            if (lane == 0) j.y[(size_t)slot * j.ldy + row0 + wave + t * 4u] = (uint16_t)f32_to_bf16_bits(silu(s0) * s1);
        });
        return;
    }
    if (b - a.route.first < a.route.blocks) {
        if (wave) return;
        if (a.route.outputs <= 64u) route_wave<1>(a.route, lane);
        else if (a.route.outputs <= 128u) route_wave<2>(a.route, lane);
        else if (a.route.outputs <= 256u) route_wave<4>(a.route, lane);
        else route_wave<16>(a.route, lane);
        return;
    }
    if (b - a.store.first < a.store.blocks) {
        store_row(a.store, red, reinterpret_cast<float*>(lds));
        return;
    }
    if (b - a.scan.first < a.scan.blocks) {
        const uint32_t local = b - a.scan.first, pts = (a.scan.p + 15u) / 16u;
        scan_step(a.scan, local / pts, local % pts, reinterpret_cast<float*>(lds));
        return;
    }
    if (b - a.delta.first < a.delta.blocks) {
        const uint32_t local = b - a.delta.first, pts = a.delta.vdim_ld / 16u;
        delta_step(a.delta, local / pts, local % pts, reinterpret_cast<float*>(lds));
        return;
    }
    if (b - a.lru.first < a.lru.blocks) {
        const uint32_t local = b - a.lru.first;
        lru_token(a.lru, local / a.lru.blocks_per_part, local % a.lru.blocks_per_part, lds, red);
    }
}

// One wave per residual element.  The products of a row -- the mixer's output projection and one down projection per
// chosen expert -- are a list of 64-lane pieces walked as one stream, eight requests ahead.
struct OutItem {
    const uint16_t* w;     // row 0 of the matrix, at the item's first element
    uint32_t ldw, x, pieces;   // x: element in the staged inputs; pieces: 16-byte pieces of the item (at most 64)
    float scale;
};
constexpr uint32_t kOutAhead = 8;

__global__ __launch_bounds__(kJobBlock) void layer_out_kernel(const LayerOutArgs a) {
    extern __shared__ __align__(16) uint16_t lds[];   // items, then the inputs: attention row | expert rows
    OutItem* items = reinterpret_cast<OutItem*>(lds);
    uint16_t* xs = lds + a.max_items * (sizeof(OutItem) / 2u);
    __shared__ uint32_t n_items;
    __shared__ float id_scale;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const uint32_t per_o = (a.ko + 511u) / 512u, per_e = (a.kf + 511u) / 512u;
    if (wave == 0) {
        uint32_t at = 0;
        if (a.wo) {
            for (uint32_t i = lane; i < per_o; i += 64u) {
                const uint32_t left = a.ko / 8u - i * 64u;
                items[i] = OutItem{a.wo + (size_t)i * 512u, a.ldo, i * 512u, left < 64u ? left : 64u, 1.0f};
            }
            at = per_o;
        }
        float idw = 0.f;
        const uint32_t my_e = lane < a.top ? a.index[lane] : 0u;
        const float my_w = lane < a.top ? a.weight[lane] : 0.f;
        for (uint32_t s = 0; s < a.top; ++s) {
            const uint32_t e = (uint32_t)__builtin_amdgcn_readlane((int)my_e, (int)s);
            const float w = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(my_w), (int)s));
            if (e >= a.experts) { idw += w; continue; }
            for (uint32_t i = lane; i < per_e; i += 64u) {
                const uint32_t left = a.kf / 8u - i * 64u;
                items[at + i] = OutItem{a.wd + (size_t)e * a.n * a.kf + (size_t)i * 512u, a.kf, (a.wo ? a.ko : 0u) + s * a.kf + i * 512u, left < 64u ? left : 64u, w};
            }
            at += per_e;
        }
        if (lane == 0) { n_items = at; id_scale = idw; }
    }
    const uint32_t base = a.wo ? a.ko : 0u;
    uint32_t formed = 0;
    if (a.ho) {
        formed = a.heads * a.hld;
        for (uint32_t h = wave; h < a.heads; h += 4u) {
            const float* o = a.ho + (size_t)h * a.hld;
            float ss = 0.f;
            for (uint32_t c = lane * 2u; c < a.hld; c += 128u) {
                const float2 v = *reinterpret_cast<const float2*>(o + c);
                ss = fmaf(v.x, v.x, ss);
                ss = fmaf(v.y, v.y, ss);
            }
            const float k = 1.0f / sqrtf(wave_sum(ss) / (float)a.hdim + a.heps);
            for (uint32_t c = lane * 2u; c < a.hld; c += 128u) {
                const float2 v = *reinterpret_cast<const float2*>(o + c);
                const uint32_t w = *reinterpret_cast<const uint32_t*>(a.hw + c), z = *reinterpret_cast<const uint32_t*>(a.hz + (size_t)h * a.hld + c);
                *reinterpret_cast<uint32_t*>(xs + (size_t)h * a.hld + c) = pack_bf16(v.x * k * bf16_lo(w) * sigmoid(bf16_lo(z)), v.y * k * bf16_hi(w) * sigmoid(bf16_hi(z)));
            }
        }
    }
    if (a.wo)
        for (uint32_t c = formed + tid * 8u; c < a.ko; c += kJobBlock * 8u) *reinterpret_cast<ld_u32x4_t*>(xs + c) = *reinterpret_cast<const ld_u32x4_t*>(a.att + c);
    for (uint32_t c = tid * 8u; c < a.top * a.kf; c += kJobBlock * 8u) *reinterpret_cast<ld_u32x4_t*>(xs + base + c) = *reinterpret_cast<const ld_u32x4_t*>(a.eh + c);
    __syncthreads();
    const uint32_t n = n_items;
    for (uint32_t row = blockIdx.x * 4u + wave; row < a.n; row += gridDim.x * 4u) {
        ld_u32x4_t p[kOutAhead];
        float s = 0.f;
        auto fetch = [&](uint32_t i) __attribute__((always_inline)) {
            const OutItem& it = items[i < n ? i : n - 1u];
            return *reinterpret_cast<const ld_u32x4_t*>(it.w + (size_t)row * it.ldw + (lane < it.pieces ? lane : it.pieces - 1u) * 8u);
        };
        if (n) {
#pragma unroll
            for (uint32_t u = 0; u < kOutAhead; ++u) p[u] = fetch(u);
            auto use = [&](uint32_t u, uint32_t i) __attribute__((always_inline)) {
                if (i < n) {
                    const OutItem& it = items[i];
                    if (lane < it.pieces) s = fmaf(it.scale, dot8(p[u], *reinterpret_cast<const ld_u32x4_t*>(xs + it.x + lane * 8u), 0.f), s);
                }
            };
            const uint32_t groups = (n + kOutAhead - 1u) / kOutAhead;
            for (uint32_t g = 0; g + 1u < groups; ++g) {
#pragma unroll
                for (uint32_t u = 0; u < kOutAhead; ++u) {
                    use(u, g * kOutAhead + u);
                    p[u] = fetch((g + 1u) * kOutAhead + u);
                }
            }
#pragma unroll
            for (uint32_t u = 0; u < kOutAhead; ++u) use(u, (groups - 1u) * kOutAhead + u);
        }
        s = wave_sum(s);
        if (lane == 0) {
            float add = s;
            if (a.mix) add += a.mix[row];
            if (id_scale != 0.f) add = fmaf(id_scale, bf16_bits_to_f32(a.h2[row]), add);
            float x = a.x[row];
            if (a.step) x += bf16_bits_to_f32(a.step[row]);
            a.x[row] = x + add;
        }
    }
}

}  // namespace

fk_status plan_layer_jobs(LayerJobsArgs& a, Launch* out) {
    uint32_t blocks = 0, lds = 64;
    // The serial jobs first: they are the longest chains.
    auto take = [&](uint32_t& first, uint32_t n) { first = blocks; blocks += n; };
    if (a.scan.u) {
        ScanJob& j = a.scan;
        if (!j.groups || j.heads % j.groups || j.state_ld % 64 || j.state_ld < j.n || j.state_ld > kMaxSsmState || !j.p || !j.taps) return set_error(FK_ERR_UNSUPPORTED, "layer jobs: state-space shape");
        j.blocks = j.heads * ((j.p + 15) / 16);
        take(j.first, j.blocks);
        lds = std::max(lds, (16u + 2u * j.state_ld) * 4u);
    }
    if (a.delta.u) {
        DeltaJob& j = a.delta;
        if (!j.kv_heads || j.heads % j.kv_heads || j.dim_ld % 32 || j.vdim_ld % 32 || j.state_ld % 64 || j.state_ld < j.dim_ld || j.state_ld > kMaxSsmState ||
            j.rank_ld % 8 || !j.taps)
            return set_error(FK_ERR_UNSUPPORTED, "layer jobs: delta rule shape");
        j.blocks = j.heads * (j.vdim_ld / 16);
        take(j.first, j.blocks);
        lds = std::max(lds, (3u * j.state_ld + 16u) * 4u);
    }
    if (a.lru.u) {
        LruJob& j = a.lru;
        if (!j.block || j.block % kRowPad || j.width % j.block || !j.taps) return set_error(FK_ERR_UNSUPPORTED, "layer jobs: linear recurrence shape");
        j.blocks_per_part = (j.block + kLruRows - 1) / kLruRows;
        j.blocks = j.width / j.block * j.blocks_per_part;
        take(j.first, j.blocks);
        lds = std::max(lds, j.block * 2u);
    }
    if (a.route.logits) {
        if (a.route.outputs > kMaxRouterOutputs || a.route.top > kMaxRouterTop || !a.route.top || a.route.top > a.route.outputs) return set_error(FK_ERR_UNSUPPORTED, "layer jobs: router shape");
        a.route.blocks = 1;
        take(a.route.first, 1);
    }
    if (a.store.kv) {
        const StoreJob& j = a.store;
        if (!j.ring || (j.ring & (j.ring - 1)) || j.rot_dims % 2 || j.rot_dims > j.rot || j.rank > j.rank_ld || j.rank_ld + j.rot > j.ldc) return set_error(FK_ERR_INVALID, "layer jobs: cache row shape");
        a.store.blocks = 1;
        take(a.store.first, 1);
        lds = std::max(lds, j.rot_dims * 4u + 16u);
    }
    for (uint32_t i = 0; i < kMaxGemvJobs; ++i) {
        GemvJob& j = a.gemv[i];
        j.blocks = 0;
        if (!j.w) continue;
        if (j.k % kRowPad || j.ldw < j.k || j.ldw % 8 || j.width > j.k || !j.n) return set_error(FK_ERR_INVALID, "layer jobs: product shape");
        if (j.mode == kRowGated && (!j.groups || j.groups > kMaxGateGroups || j.width % j.groups)) return set_error(FK_ERR_UNSUPPORTED, "layer jobs: at most 64 norm groups");
        if (j.mode == kRowCombine && (!j.rows_per_head || !j.splits || j.splits > kMaxSplits)) return set_error(FK_ERR_INVALID, "layer jobs: combination of what");
        if (j.mode == kRowJoin && (!j.x2 || j.k % (2 * kRowPad) || j.width > j.k / 2)) return set_error(FK_ERR_INVALID, "layer jobs: joined rows");
        if (j.out.fn > kFnMax || j.out.fn2 > kFnMax) return set_error(FK_ERR_INVALID, "layer jobs: column function");
        if (j.rows_per_head && j.n % j.rows_per_head) return set_error(FK_ERR_INVALID, "layer jobs: rows per head");
        if (!j.rows_per_head) j.y_head = 0;
        else if (j.y_head < j.rows_per_head) return set_error(FK_ERR_INVALID, "layer jobs: outputs per head");
        // rows per block: enough blocks to fill the device, few enough that forming the row does not dominate
        const uint32_t rows = j.rows_per_head ? j.rows_per_head : j.n, heads = j.rows_per_head ? j.n / j.rows_per_head : 1;
        uint32_t per = 8;
        while (per < 128 && (uint64_t)heads * ((rows + per - 1) / per) > 1024) per *= 2;
        if (j.mode == kRowCombine) per = std::max(per, 32u);
        j.rows_per_block = per;
        j.blocks_per_head = (rows + per - 1) / per;
        j.blocks = heads * j.blocks_per_head;
        take(j.first, j.blocks);
        lds = std::max(lds, j.k * 2u);
    }
    a.pair.blocks = 0;
    if (a.pair.wa) {
        PairJob& j = a.pair;
        if (j.k % kRowPad || j.ldw < j.k || j.ldw % 8 || !j.n || !j.top) return set_error(FK_ERR_INVALID, "layer jobs: expert shape");
        uint32_t per = 4;
        while (per < 64 && (uint64_t)j.top * ((j.n + per - 1) / per) > 2048) per *= 2;
        j.rows_per_block = per;
        j.blocks_per_slot = (j.n + per - 1) / per;
        j.blocks = j.top * j.blocks_per_slot;
        take(j.first, j.blocks);
        lds = std::max(lds, j.k * 2u);
    }
    if (!blocks) return set_error(FK_ERR_INVALID, "layer jobs: no job");
    if (lds > 60u * 1024u) return set_error(FK_ERR_UNSUPPORTED, "layer jobs: rows of at most 30720 elements");
    out->func = (const void*)&layer_jobs_kernel;
    out->grid = dim3(blocks, 1, 1);
    out->block = dim3(kJobBlock, 1, 1);
    out->shmem = lds;
    out->set_args(a);
    return FK_OK;
}

fk_status plan_layer_out(LayerOutArgs& a, Launch* out) {
    if (!a.x || !a.n || (a.wo && (!a.att || a.ko % kRowPad || a.ldo < a.ko)) || (a.top && (!a.eh || !a.wd || !a.index || !a.weight || !a.h2 || a.kf % kRowPad || !a.kf)))
        return set_error(FK_ERR_INVALID, "layer out: bad arguments");
    if (a.ho && (!a.hz || !a.hw || !a.wo || !a.hdim || a.hld % 8 || a.hld < a.hdim || (uint64_t)a.heads * a.hld > a.ko)) return set_error(FK_ERR_INVALID, "layer out: heads to normalise");
    if (!a.wo) a.ko = 0;
    if (!a.top) a.kf = 0;
    a.max_items = ((a.ko + 511) / 512 + a.top * ((a.kf + 511) / 512) + 2) / 2 * 2;   // even: the inputs behind stay 16-byte aligned
    const uint64_t lds = (uint64_t)a.max_items * sizeof(OutItem) + ((uint64_t)a.ko + (uint64_t)a.top * a.kf) * 2u + 16;
    if (lds > 60u * 1024u) return set_error(FK_ERR_UNSUPPORTED, "layer out: inputs of a row beyond 60 KB");
    out->func = (const void*)&layer_out_kernel;
    out->grid = dim3(std::min((a.n + 3u) / 4u, 1024u), 1, 1);
    out->block = dim3(kJobBlock, 1, 1);
    out->shmem = (uint32_t)lds;
    out->set_args(a);
    return FK_OK;
}

}  // namespace fk
