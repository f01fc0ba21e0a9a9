// The gated delta rule of a long portion, chunk by chunk on the matrix cores.
//
// With c_t the running sum of a chunk's log decays (per key channel), S the state the chunk starts from and
//     A[t, s] = sum_d k_t k_s exp(c_t - c_s)  (s < t),      B[t, s] = sum_d q_t k_s exp(c_t - c_s)  (s <= t),
// the recurrence over 64 tokens is
//     (I + beta A) U = beta (V - (k exp(c)) S)           the values each token writes
//     O = (q exp(c)) S + B U
//     S <- exp(c_last) S + sum_s k_s exp(c_last - c_s) u_s^T
// Two launches.  The first, side by side over chunks and heads, forms A and B, solves the triangular system for the two
// right-hand sides beta k exp(c) (giving W) and beta V (giving U0), so that U = U0 - W S.  The second walks the chunks of
// a head and a slice of its value columns in order: the state stays in accumulators, two products with it, two with U.
//
// No exponent is ever positive: inside a 16 x 16 diagonal block every pair of tokens has its own exponential; below the
// diagonal both factors are taken against the last token before the later block.
// The recurrence is kept in 32 bits: values enter a bf16 instruction as the sum of two bf16 halves (three products),
// accumulation, states and the triangular solution are fp32.
#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

namespace {

typedef __bf16 dc_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float dc_f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t dc_u32x4_t __attribute__((ext_vector_type(4)));

constexpr uint32_t kDc = kDeltaChunk, kDcStep = 32, kDcTs = kDc + 4, kDcUs = kDc + 8;

__device__ __forceinline__ dc_f32x4_t dc_mfma(dc_u32x4_t a, dc_u32x4_t b, dc_f32x4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(dc_bf16x8_t, a), __builtin_bit_cast(dc_bf16x8_t, b), c, 0, 0, 0);
}
// a . b with both operands as two halves; the product of the low halves is below fp32's own rounding.
__device__ __forceinline__ dc_f32x4_t dc_mfma3(dc_u32x4_t ah, dc_u32x4_t al, dc_u32x4_t bh, dc_u32x4_t bl, dc_f32x4_t c) {
    return dc_mfma(ah, bh, dc_mfma(ah, bl, dc_mfma(al, bh, c)));
}
__device__ __forceinline__ void dc_split2(float x, float y, uint32_t& hi, uint32_t& lo) {
    hi = pack_bf16(x, y);
    lo = pack_bf16(x - bf16_lo(hi), y - bf16_hi(hi));
}

// Where a (chunk, head) keeps what the first launch leaves to the second.
struct DcWork {
    uint16_t *w, *q, *k, *b;   // high halves; the low ones follow: [64][dim], [64][dim], [dim][64], [64][64]
    float *u0, *gamma;         // [64][vdim], [dim]
};
__host__ __device__ inline size_t dc_work_bytes(uint32_t dim, uint32_t vdim) { return (size_t)kDc * dim * 12 + kDc * kDc * 4 + (size_t)kDc * vdim * 4 + dim * 4; }
__device__ __forceinline__ DcWork dc_work(const DeltaChunkArgs& a, uint32_t chunk, uint32_t h) {
    unsigned char* p = reinterpret_cast<unsigned char*>(a.work) + ((size_t)chunk * a.heads + h) * dc_work_bytes(a.dim_ld, a.vdim_ld);
    DcWork w;
    const size_t n = (size_t)kDc * a.dim_ld;
    w.w = reinterpret_cast<uint16_t*>(p);
    w.q = w.w + 2 * n;
    w.k = w.q + 2 * n;
    w.b = w.k + 2 * n;
    w.u0 = reinterpret_cast<float*>(w.b + 2 * kDc * kDc);
    w.gamma = w.u0 + (size_t)kDc * a.vdim_ld;
    return w;
}

__global__ __launch_bounds__(256) void delta_intra_kernel(const DeltaChunkArgs a) {
    __shared__ __align__(16) float kt[kDcStep * kDcTs], qt[kDcStep * kDcTs], ct[kDcStep * kDcTs];   // [channel][token]
    __shared__ __align__(16) float A[kDc * kDcTs];
    __shared__ float beta[kDc];
    const uint32_t h = blockIdx.x, chunk = blockIdx.y, t0 = chunk * kDc, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const uint32_t l16 = lane & 15u, kq = lane >> 4, dim = a.dim_ld, vdim = a.vdim_ld, nk = a.kv_heads * dim;
    const uint32_t live = a.rows - t0 < kDc ? a.rows - t0 : kDc;
    const float* K = a.qk + (size_t)t0 * 2u * nk + nk + (size_t)(h / (a.heads / a.kv_heads)) * dim;
    const float* Q = K - nk;
    const float* G = a.decay + ((size_t)t0 * a.heads + h) * dim;
    const size_t ldk = 2u * (size_t)nk, ldg = (size_t)a.heads * dim;
    const DcWork w = dc_work(a, chunk, h);
    if (tid < kDc) beta[tid] = tid < live ? a.beta[(size_t)(t0 + tid) * a.ldb + h] : 0.f;   // tokens past the pass write nothing

    // ---- A and B: wave w owns the w-th diagonal block and up to two of the six blocks below the diagonal
    float da[4] = {0.f, 0.f, 0.f, 0.f}, db[4] = {0.f, 0.f, 0.f, 0.f};
    dc_f32x4_t oa[2], ob[2];
#pragma unroll
    for (int p = 0; p < 2; ++p) oa[p] = ob[p] = dc_f32x4_t{0.f, 0.f, 0.f, 0.f};
    const uint32_t dt = wave * 16u + (lane >> 2), ds = wave * 16u + (lane & 3u) * 4u;
    auto block_of = [](uint32_t p, uint32_t& i, uint32_t& j) __attribute__((always_inline)) {   // (1,0) (2,0) (2,1) (3,0) (3,1) (3,2)
        i = p == 0 ? 1u : p < 3 ? 2u : 3u;
        j = p == 0 ? 0u : p < 3 ? p - 1u : p - 3u;
    };
    for (uint32_t d0 = 0; d0 < dim; d0 += kDcStep) {
        __syncthreads();
#pragma unroll
        for (uint32_t i = 0; i < 2; ++i) {
            const uint32_t idx = tid + 256u * i, t = idx >> 3, d = (idx & 7u) * 4u;
            float4 kv = make_float4(0.f, 0.f, 0.f, 0.f), qv = kv, gv = kv;
            if (t < live) {
                kv = *reinterpret_cast<const float4*>(K + t * ldk + d0 + d);
                qv = *reinterpret_cast<const float4*>(Q + t * ldk + d0 + d);
                gv = *reinterpret_cast<const float4*>(G + t * ldg + d0 + d);
            }
            const uint32_t at = d * kDcTs + t;
            kt[at] = kv.x; kt[at + kDcTs] = kv.y; kt[at + 2 * kDcTs] = kv.z; kt[at + 3 * kDcTs] = kv.w;
            qt[at] = qv.x; qt[at + kDcTs] = qv.y; qt[at + 2 * kDcTs] = qv.z; qt[at + 3 * kDcTs] = qv.w;
            ct[at] = gv.x; ct[at + kDcTs] = gv.y; ct[at + 2 * kDcTs] = gv.z; ct[at + 3 * kDcTs] = gv.w;
        }
        __syncthreads();
#pragma unroll
        for (uint32_t i = 0; i < kDcStep / 4u; ++i) {   // running sums over the tokens, one per lane
            float* row = ct + (wave * (kDcStep / 4u) + i) * kDcTs;
            float v = row[lane];
#pragma unroll
            for (int o = 1; o < kWave; o <<= 1) {
                const float u = __shfl_up(v, o, kWave);
                if (lane >= (uint32_t)o) v += u;
            }
            row[lane] = v;
        }
        __syncthreads();
#pragma unroll 4
        for (uint32_t d = 0; d < kDcStep; ++d) {
            const float kv = kt[d * kDcTs + dt], qv = qt[d * kDcTs + dt], cv = ct[d * kDcTs + dt];
            const float4 ks = *reinterpret_cast<const float4*>(kt + d * kDcTs + ds), cs = *reinterpret_cast<const float4*>(ct + d * kDcTs + ds);
            const float ksv[4] = {ks.x, ks.y, ks.z, ks.w}, csv[4] = {cs.x, cs.y, cs.z, cs.w};
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float f = __builtin_amdgcn_exp2f(fminf(cv - csv[e], 0.f)) * ksv[e];   // later tokens are dropped below
                da[e] = fmaf(kv, f, da[e]);
                db[e] = fmaf(qv, f, db[e]);
            }
        }
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            if (wave + 4u * p >= 6u) break;
            uint32_t i, j;
            block_of(wave + 4u * p, i, j);
            dc_u32x4_t sh, sl, th, tl, qh, ql;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                float s[2], t[2], q[2];
#pragma unroll
                for (int x = 0; x < 2; ++x) {
                    const uint32_t d = (kq * 8u + (uint32_t)(2 * e + x)) * kDcTs;
                    const float ref = ct[d + 16u * i - 1u], f = __builtin_amdgcn_exp2f(ct[d + 16u * i + l16] - ref);
                    s[x] = kt[d + 16u * j + l16] * __builtin_amdgcn_exp2f(ref - ct[d + 16u * j + l16]);
                    t[x] = kt[d + 16u * i + l16] * f;
                    q[x] = qt[d + 16u * i + l16] * f;
                }
                uint32_t hi, lo;
                dc_split2(s[0], s[1], hi, lo); sh[e] = hi; sl[e] = lo;
                dc_split2(t[0], t[1], hi, lo); th[e] = hi; tl[e] = lo;
                dc_split2(q[0], q[1], hi, lo); qh[e] = hi; ql[e] = lo;
            }
            oa[p] = dc_mfma3(sh, sl, th, tl, oa[p]);   // rows s, columns t: a lane ends with four adjacent s of one t
            ob[p] = dc_mfma3(sh, sl, qh, ql, ob[p]);
        }
    }
    __syncthreads();
    auto put_b = [&](uint32_t t, uint32_t s, const float* v) __attribute__((always_inline)) {
        uint32_t h0, l0, h1, l1;
        dc_split2(v[0], v[1], h0, l0);
        dc_split2(v[2], v[3], h1, l1);
        *reinterpret_cast<uint2*>(w.b + t * kDc + s) = make_uint2(h0, h1);
        *reinterpret_cast<uint2*>(w.b + kDc * kDc + t * kDc + s) = make_uint2(l0, l1);
    };
    {
        float m[4], v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            m[e] = ds + (uint32_t)e < dt ? beta[dt] * da[e] : 0.f;
            v[e] = ds + (uint32_t)e <= dt ? db[e] : 0.f;
        }
        *reinterpret_cast<float4*>(A + dt * kDcTs + ds) = make_float4(m[0], m[1], m[2], m[3]);
        put_b(dt, ds, v);
    }
#pragma unroll
    for (int p = 0; p < 2; ++p) {
        if (wave + 4u * p >= 6u) break;
        uint32_t i, j;
        block_of(wave + 4u * p, i, j);
        const uint32_t t = 16u * i + l16, s = 16u * j + kq * 4u;
        const float f = beta[t], v[4] = {ob[p][0], ob[p][1], ob[p][2], ob[p][3]}, none[4] = {0.f, 0.f, 0.f, 0.f};
        *reinterpret_cast<float4*>(A + t * kDcTs + s) = make_float4(f * oa[p][0], f * oa[p][1], f * oa[p][2], f * oa[p][3]);
        put_b(t, s, v);
        put_b(16u * j + l16, 16u * i + kq * 4u, none);   // above the diagonal
    }
    __syncthreads();

    // ---- the triangular system, a thread per column of the right-hand sides
    for (uint32_t col = tid; col < dim + vdim; col += 256u) {
        float X[kDc];
        if (col < dim) {
            float c = 0.f;
#pragma unroll
            for (uint32_t t = 0; t < kDc; ++t) {
                const uint32_t r = t < live ? t : live - 1u;
                c += t < live ? G[r * ldg + col] : 0.f;
                const float e = __builtin_amdgcn_exp2f(c), q = Q[r * ldk + col] * e;
                X[t] = beta[t] * K[r * ldk + col] * e;
                const uint32_t hi = f32_to_bf16_bits(q);
                w.q[t * dim + col] = (uint16_t)hi;
                w.q[(kDc + t) * dim + col] = (uint16_t)f32_to_bf16_bits(q - bf16_bits_to_f32(hi));
            }
            const float last = c;
            w.gamma[col] = __builtin_amdgcn_exp2f(last);
            c = 0.f;
            uint16_t* kd = w.k + (size_t)col * kDc;
#pragma unroll
            for (uint32_t t = 0; t < kDc; t += 8u) {
                dc_u32x4_t hi, lo;
#pragma unroll
                for (uint32_t e = 0; e < 4; ++e) {
                    float v[2];
#pragma unroll
                    for (uint32_t x = 0; x < 2; ++x) {
                        const uint32_t s = t + 2u * e + x, r = s < live ? s : live - 1u;
                        c += s < live ? G[r * ldg + col] : 0.f;
                        v[x] = K[r * ldk + col] * __builtin_amdgcn_exp2f(fminf(last - c, 0.f));
                    }
                    uint32_t h2, l2;
                    dc_split2(v[0], v[1], h2, l2);
                    hi[e] = h2;
                    lo[e] = l2;
                }
                *reinterpret_cast<dc_u32x4_t*>(kd + t) = hi;
                *reinterpret_cast<dc_u32x4_t*>(kd + (size_t)dim * kDc + t) = lo;
            }
        } else {
            const uint16_t* v = a.v + (size_t)t0 * a.ldx + (size_t)h * vdim + col - dim;
#pragma unroll
            for (uint32_t t = 0; t < kDc; ++t) X[t] = beta[t] * act_load(v + (size_t)(t < live ? t : live - 1u) * a.ldx);
        }
#pragma unroll
        for (uint32_t t = 1; t < kDc; ++t) {
            float x0 = X[t], x1 = 0.f;
#pragma unroll
            for (uint32_t s = 0; s + 4u <= t; s += 4u) {
                const float4 m = *reinterpret_cast<const float4*>(A + t * kDcTs + s);
                x0 = fmaf(-m.x, X[s], x0); x1 = fmaf(-m.y, X[s + 1u], x1);
                x0 = fmaf(-m.z, X[s + 2u], x0); x1 = fmaf(-m.w, X[s + 3u], x1);
            }
#pragma unroll
            for (uint32_t s = t & ~3u; s < t; ++s) x0 = fmaf(-A[t * kDcTs + s], X[s], x0);
            X[t] = x0 + x1;
        }
        if (col < dim) {
#pragma unroll
            for (uint32_t t = 0; t < kDc; ++t) {
                const uint32_t hi = f32_to_bf16_bits(X[t]);
                w.w[t * dim + col] = (uint16_t)hi;
                w.w[(kDc + t) * dim + col] = (uint16_t)f32_to_bf16_bits(X[t] - bf16_bits_to_f32(hi));
            }
        } else {
#pragma unroll
            for (uint32_t t = 0; t < kDc; ++t) w.u0[t * vdim + col - dim] = X[t];
        }
    }
}

// KD: key channels / 32; VT: 16-wide tiles of value columns of the block.
template <int KD, int VT>
__global__ __launch_bounds__(256) void delta_inter_kernel(const DeltaChunkArgs a) {
    constexpr uint32_t DIM = KD * 32u, SS = DIM + 8u;
    constexpr int ND = (2 * KD + 3) / 4;   // 16-channel tiles of the state per wave
    __shared__ __align__(16) uint16_t sh[VT * 16 * SS], sl[VT * 16 * SS], uh[VT * 16 * kDcUs], ul[VT * 16 * kDcUs];
    const uint32_t h = blockIdx.x, v0 = blockIdx.y * (VT * 16u), tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, kq = lane >> 4;
    const uint32_t chunks = (a.rows + kDc - 1u) / kDc, nv = a.heads * a.vdim_ld;
    float* state = a.state + ((size_t)h * a.vdim_ld + v0 + l16) * a.state_ld + kq * 4u;

    dc_f32x4_t S[ND][VT];
#pragma unroll
    for (int i = 0; i < ND; ++i)
#pragma unroll
        for (int v = 0; v < VT; ++v)
            S[i][v] = wave + 4u * i < 2u * KD ? *reinterpret_cast<const dc_f32x4_t*>(state + (size_t)(v * 16) * a.state_ld + (wave + 4u * i) * 16u) : dc_f32x4_t{0.f, 0.f, 0.f, 0.f};
    dc_u32x4_t wo[KD][2], qo[KD][2], bo[2][2], ko[ND][2][2];
    dc_f32x4_t u0[VT], gm[ND];
    auto fetch_rows = [&](uint32_t chunk) __attribute__((always_inline)) {
        const DcWork w = dc_work(a, chunk, h);
        const uint32_t at = (wave * 16u + l16) * DIM + kq * 8u;
#pragma unroll
        for (int s = 0; s < KD; ++s)
#pragma unroll
            for (int x = 0; x < 2; ++x) {
                wo[s][x] = *reinterpret_cast<const dc_u32x4_t*>(w.w + x * kDc * DIM + at + s * 32);
                qo[s][x] = *reinterpret_cast<const dc_u32x4_t*>(w.q + x * kDc * DIM + at + s * 32);
            }
#pragma unroll
        for (int v = 0; v < VT; ++v)
#pragma unroll
            for (int r = 0; r < 4; ++r) u0[v][r] = w.u0[(wave * 16u + kq * 4u + r) * a.vdim_ld + v0 + v * 16 + l16];
    };
    auto fetch_columns = [&](uint32_t chunk) __attribute__((always_inline)) {
        const DcWork w = dc_work(a, chunk, h);
#pragma unroll
        for (int s = 0; s < 2; ++s)
#pragma unroll
            for (int x = 0; x < 2; ++x) {
                bo[s][x] = *reinterpret_cast<const dc_u32x4_t*>(w.b + x * kDc * kDc + (wave * 16u + l16) * kDc + s * 32 + kq * 8u);
#pragma unroll
                for (int i = 0; i < ND; ++i) {
                    const uint32_t d = wave + 4u * i < 2u * KD ? (wave + 4u * i) * 16u : 0u;
                    ko[i][s][x] = *reinterpret_cast<const dc_u32x4_t*>(w.k + (x * DIM + d + l16) * kDc + s * 32 + kq * 8u);
                }
            }
#pragma unroll
        for (int i = 0; i < ND; ++i) gm[i] = *reinterpret_cast<const dc_f32x4_t*>(w.gamma + (wave + 4u * i < 2u * KD ? (wave + 4u * i) * 16u : 0u) + kq * 4u);
    };
    fetch_rows(0);
    for (uint32_t chunk = 0; chunk < chunks; ++chunk) {
#pragma unroll
        for (int i = 0; i < ND; ++i)
            if (wave + 4u * i < 2u * KD) {
#pragma unroll
                for (int v = 0; v < VT; ++v) {
                    uint32_t h0, l0, h1, l1;
                    dc_split2(S[i][v][0], S[i][v][1], h0, l0);
                    dc_split2(S[i][v][2], S[i][v][3], h1, l1);
                    const uint32_t at = (v * 16u + l16) * SS + (wave + 4u * i) * 16u + kq * 4u;
                    *reinterpret_cast<uint2*>(sh + at) = make_uint2(h0, h1);
                    *reinterpret_cast<uint2*>(sl + at) = make_uint2(l0, l1);
                }
            }
        __syncthreads();
        fetch_columns(chunk);
        dc_f32x4_t pw[VT], pq[VT];
#pragma unroll
        for (int v = 0; v < VT; ++v) pw[v] = pq[v] = dc_f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KD; ++s)
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const uint32_t at = (v * 16u + l16) * SS + s * 32u + kq * 8u;
                const dc_u32x4_t bh = *reinterpret_cast<const dc_u32x4_t*>(sh + at), bl = *reinterpret_cast<const dc_u32x4_t*>(sl + at);
                pw[v] = dc_mfma3(wo[s][0], wo[s][1], bh, bl, pw[v]);
                pq[v] = dc_mfma3(qo[s][0], qo[s][1], bh, bl, pq[v]);
            }
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            uint32_t h0, l0, h1, l1;
            dc_split2(u0[v][0] - pw[v][0], u0[v][1] - pw[v][1], h0, l0);
            dc_split2(u0[v][2] - pw[v][2], u0[v][3] - pw[v][3], h1, l1);
            const uint32_t at = (v * 16u + l16) * kDcUs + wave * 16u + kq * 4u;
            *reinterpret_cast<uint2*>(uh + at) = make_uint2(h0, h1);
            *reinterpret_cast<uint2*>(ul + at) = make_uint2(l0, l1);
        }
        __syncthreads();
        if (chunk + 1u < chunks) fetch_rows(chunk + 1u);
#pragma unroll
        for (int i = 0; i < ND; ++i)
#pragma unroll
            for (int v = 0; v < VT; ++v)
#pragma unroll
                for (int r = 0; r < 4; ++r) S[i][v][r] *= gm[i][r];
#pragma unroll
        for (int s = 0; s < 2; ++s)
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const uint32_t at = (v * 16u + l16) * kDcUs + s * 32u + kq * 8u;
                const dc_u32x4_t bh = *reinterpret_cast<const dc_u32x4_t*>(uh + at), bl = *reinterpret_cast<const dc_u32x4_t*>(ul + at);
                pq[v] = dc_mfma3(bo[s][0], bo[s][1], bh, bl, pq[v]);
#pragma unroll
                for (int i = 0; i < ND; ++i) S[i][v] = dc_mfma3(ko[i][s][0], ko[i][s][1], bh, bl, S[i][v]);
            }
#pragma unroll
        for (int v = 0; v < VT; ++v)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const uint32_t t = chunk * kDc + wave * 16u + kq * 4u + r;
                if (t < a.rows) a.o[(size_t)t * nv + (size_t)h * a.vdim_ld + v0 + v * 16 + l16] = pq[v][r];
            }
    }
#pragma unroll
    for (int i = 0; i < ND; ++i)
#pragma unroll
        for (int v = 0; v < VT; ++v)
            if (wave + 4u * i < 2u * KD) *reinterpret_cast<dc_f32x4_t*>(state + (size_t)(v * 16) * a.state_ld + (wave + 4u * i) * 16u) = S[i][v];
}

template <int VT>
const void* inter_func(uint32_t kd) {
    switch (kd) {
        case 1: return (const void*)&delta_inter_kernel<1, VT>;
        case 2: return (const void*)&delta_inter_kernel<2, VT>;
        case 3: return (const void*)&delta_inter_kernel<3, VT>;
        case 4: return (const void*)&delta_inter_kernel<4, VT>;
        case 6: return (const void*)&delta_inter_kernel<6, VT>;
        case 8: return (const void*)&delta_inter_kernel<8, VT>;
        default: return nullptr;
    }
}

}  // namespace

uint64_t delta_chunk_work_bytes(uint32_t rows, uint32_t heads, uint32_t dim_ld, uint32_t vdim_ld) {
    return (uint64_t)((rows + kDc - 1) / kDc) * heads * dc_work_bytes(dim_ld, vdim_ld);
}

bool delta_chunk_supported(uint32_t dim_ld, uint32_t vdim_ld) { return dim_ld % 32 == 0 && vdim_ld % 32 == 0 && vdim_ld && inter_func<1>(dim_ld / 32); }

fk_status plan_delta_chunk(const DeltaChunkArgs& a, Launch* out) {
    if (!a.qk || !a.decay || !a.beta || !a.v || !a.state || !a.o || !a.work || !a.rows || !a.heads || !a.kv_heads) return set_error(FK_ERR_INVALID, "delta chunks: bad arguments");
    if (a.heads % a.kv_heads || a.ldb < a.heads || a.state_ld % 4 || a.state_ld < a.dim_ld) return set_error(FK_ERR_INVALID, "delta chunks: bad shape");
    if (!delta_chunk_supported(a.dim_ld, a.vdim_ld)) return set_error(FK_ERR_UNSUPPORTED, "delta chunks: key width 32, 64, 96, 128, 192 or 256, value width a multiple of 32");
    const uint32_t chunks = (a.rows + kDc - 1) / kDc;
    if (chunks > 65535) return set_error(FK_ERR_UNSUPPORTED, "delta chunks: too many rows");
    out->func = (const void*)&delta_intra_kernel;
    out->grid = dim3(a.heads, chunks, 1);
    out->block = dim3(256, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    Launch seq;
    const uint32_t vt = (uint64_t)a.heads * (a.vdim_ld / 32) >= 128 ? 2 : 1;   // narrower slices where that leaves compute units without a block
    seq.func = vt == 2 ? inter_func<2>(a.dim_ld / 32) : inter_func<1>(a.dim_ld / 32);
    seq.grid = dim3(a.heads, a.vdim_ld / (16 * vt), 1);
    seq.block = dim3(256, 1, 1);
    seq.set_args(a);
    out->then.push_back(seq);
    return FK_OK;
}

}  // namespace fk
