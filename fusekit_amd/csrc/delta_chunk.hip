// The gated delta rule of a long portion, chunk by chunk on the matrix cores.
//
// With c_t the running sum of a chunk's log decays (per key channel), S the state the chunk starts from and
//     A[t, s] = sum_d k_t k_s exp(c_t - c_s)  (s < t),      B[t, s] = sum_d q_t k_s exp(c_t - c_s)  (s <= t),
// the recurrence over 64 tokens is
//     (I + beta A) U = beta (V - (k exp(c)) S)           the values each token writes
//     O = (q exp(c)) S + B U
//     S <- exp(c_last) S + sum_s k_s exp(c_last - c_s) u_s^T
// Two launches.  The first, side by side over chunks and heads, forms A and B, inverts the triangular matrix (T, in fp32
// instructions: the diagonal blocks by substitution, the blocks below them by products) and multiplies W = T beta k exp(c)
// and U0 = T beta V, so that U = U0 - W S.  The second walks the chunks of a head and a slice of its value columns in
// order: the state stays in accumulators, two products with it, two with U, the operands of the next chunk on their way.
//
// A and B come in 16 x 16 blocks whose pairwise exponentials are split into two factors against the last token before the
// later block, so that no exponent below the diagonal is positive.  In a diagonal block the earlier token's factor grows;
// where some channel decays by more than 2^64 within the block, every pair gets an exponential of its own instead.
// The recurrence is kept in 32 bits: values enter a bf16 instruction as the sum of two bf16 halves (three products),
// accumulation, states and the triangular inverse are fp32.
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

// LDS traffic of one wave with itself: the hardware runs it in order, the fence keeps the compiler from reordering it.
__device__ __forceinline__ void dc_lds_order() {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// Where a (chunk, head) keeps what the first launch leaves to the second.  Matrices lie in the order in which a wave reads
// them as an operand: 16 rows x 32 columns after another, in each the 64 lanes' eight elements (dc_at).
struct DcWork {
    uint16_t *w, *q, *k, *b;   // high halves; the low ones follow: [64][dim], [64][dim], [dim][64], [64][64]
    float *u0, *gamma;         // [64][vdim] in tiles of 16 x 16, [dim]
};
__device__ __forceinline__ uint32_t dc_at(uint32_t row, uint32_t col, uint32_t width) {
    return ((row >> 4) * (width >> 5) + (col >> 5)) * 512u + ((((col >> 3) & 3u) << 4) + (row & 15u)) * 8u + (col & 7u);
}
// U0: a lane of the second launch holds four adjacent tokens of one value column.
__device__ __forceinline__ uint32_t dc_u0_at(uint32_t t, uint32_t v, uint32_t vdim) {
    return ((v >> 4) * 4u + (t >> 4)) * 256u + ((((t >> 2) & 3u) << 4) + (v & 15u)) * 4u + (t & 3u);
}
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

// A slice of 32 channels of the chunk: keys, queries and log decays, requested as they lie and staged as [channel][token].
struct DcSlice {
    float4 k[2], q[2], g[2];
};

__global__ __launch_bounds__(256, 2) void delta_intra_kernel(const DeltaChunkArgs a) {
    __shared__ __align__(16) float kt[kDcStep * kDcTs], qt[kDcStep * kDcTs], ct[kDcStep * kDcTs];   // [channel][token]
    __shared__ __align__(16) float A[kDc * kDcTs], T[kDc * kDcTs];
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

    auto fetch = [&](DcSlice& x, uint32_t d0) __attribute__((always_inline)) {
#pragma unroll
        for (uint32_t i = 0; i < 2; ++i) {
            const uint32_t idx = tid + 256u * i, t = idx >> 3, d = d0 + (idx & 7u) * 4u;
            x.k[i] = x.q[i] = x.g[i] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (t < live) {
                x.k[i] = *reinterpret_cast<const float4*>(K + t * ldk + d);
                x.q[i] = *reinterpret_cast<const float4*>(Q + t * ldk + d);
                x.g[i] = *reinterpret_cast<const float4*>(G + t * ldg + d);
            }
        }
    };
    // staged with the decays summed over the tokens (one token per lane); between two barriers of the caller
    auto stage = [&](const DcSlice& x) __attribute__((always_inline)) {
#pragma unroll
        for (uint32_t i = 0; i < 2; ++i) {
            const uint32_t idx = tid + 256u * i, at = (idx & 7u) * 4u * kDcTs + (idx >> 3);
            kt[at] = x.k[i].x; kt[at + kDcTs] = x.k[i].y; kt[at + 2 * kDcTs] = x.k[i].z; kt[at + 3 * kDcTs] = x.k[i].w;
            qt[at] = x.q[i].x; qt[at + kDcTs] = x.q[i].y; qt[at + 2 * kDcTs] = x.q[i].z; qt[at + 3 * kDcTs] = x.q[i].w;
            ct[at] = x.g[i].x; ct[at + kDcTs] = x.g[i].y; ct[at + 2 * kDcTs] = x.g[i].z; ct[at + 3 * kDcTs] = x.g[i].w;
        }
        __syncthreads();
        float v[kDcStep / 4u];
        float* row = ct + wave * (kDcStep / 4u) * kDcTs + lane;
#pragma unroll
        for (uint32_t i = 0; i < kDcStep / 4u; ++i) v[i] = row[i * kDcTs];
#pragma unroll
        for (int o = 1; o < kWave; o <<= 1)
#pragma unroll
            for (uint32_t i = 0; i < kDcStep / 4u; ++i) {
                const float u = __shfl_up(v[i], o, kWave);
                if (lane >= (uint32_t)o) v[i] += u;
            }
#pragma unroll
        for (uint32_t i = 0; i < kDcStep / 4u; ++i) row[i * kDcTs] = v[i];
    };

    // ---- A and B: wave w owns the w-th diagonal block and up to two of the six blocks below the diagonal
    dc_f32x4_t oa[3], ob[3];   // rows s, columns t: a lane holds four adjacent s of one t; [2]: the diagonal block
#pragma unroll
    for (int p = 0; p < 3; ++p) oa[p] = ob[p] = dc_f32x4_t{0.f, 0.f, 0.f, 0.f};
    auto block_of = [](uint32_t p, uint32_t& i, uint32_t& j) __attribute__((always_inline)) {   // (1,0) (2,0) (2,1) (3,0) (3,1) (3,2)
        i = p == 0 ? 1u : p < 3 ? 2u : 3u;
        j = p == 0 ? 0u : p < 3 ? p - 1u : p - 3u;
    };
    auto product = [&](uint32_t i, uint32_t j, dc_f32x4_t& pa, dc_f32x4_t& pb) __attribute__((always_inline)) {
        dc_u32x4_t sh, sl, th, tl, qh, ql;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            float sv[2], tv[2], qv[2];
#pragma unroll
            for (int y = 0; y < 2; ++y) {
                const uint32_t d = (kq * 8u + (uint32_t)(2 * e + y)) * kDcTs;
                const float ref = i ? ct[d + 16u * i - 1u] : 0.f, f = __builtin_amdgcn_exp2f(ct[d + 16u * i + l16] - ref);
                sv[y] = kt[d + 16u * j + l16] * __builtin_amdgcn_exp2f(ref - ct[d + 16u * j + l16]);
                tv[y] = kt[d + 16u * i + l16] * f;
                qv[y] = qt[d + 16u * i + l16] * f;
            }
            uint32_t hi, lo;
            dc_split2(sv[0], sv[1], hi, lo); sh[e] = hi; sl[e] = lo;
            dc_split2(tv[0], tv[1], hi, lo); th[e] = hi; tl[e] = lo;
            dc_split2(qv[0], qv[1], hi, lo); qh[e] = hi; ql[e] = lo;
        }
        pa = dc_mfma3(sh, sl, th, tl, pa);
        pb = dc_mfma3(sh, sl, qh, ql, pb);
    };
    const uint32_t dt = wave * 16u + l16, ds = wave * 16u + kq * 4u;
    DcSlice x;
    fetch(x, 0);
    for (uint32_t d0 = 0; d0 < dim; d0 += kDcStep) {
        __syncthreads();
        stage(x);
        __syncthreads();
        fetch(x, d0 + kDcStep < dim ? d0 + kDcStep : 0u);   // the second walk starts over
        const float* cr = ct + (lane & 31u) * kDcTs;
        const bool steep = (wave ? cr[16u * wave - 1u] : 0.f) - cr[16u * wave + 15u] > 64.f;
        if (__builtin_amdgcn_ballot_w64(steep) == 0) {
            product(wave, wave, oa[2], ob[2]);
        } else {
#pragma unroll 4
            for (uint32_t d = 0; d < kDcStep; ++d) {
                const float kv = kt[d * kDcTs + dt], qv = qt[d * kDcTs + dt], cv = ct[d * kDcTs + dt];
                const float4 ks = *reinterpret_cast<const float4*>(kt + d * kDcTs + ds), cs = *reinterpret_cast<const float4*>(ct + d * kDcTs + ds);
                const float ksv[4] = {ks.x, ks.y, ks.z, ks.w}, csv[4] = {cs.x, cs.y, cs.z, cs.w};
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float f = __builtin_amdgcn_exp2f(fminf(cv - csv[e], 0.f)) * ksv[e];   // later tokens are dropped below
                    oa[2][e] = fmaf(kv, f, oa[2][e]);
                    ob[2][e] = fmaf(qv, f, ob[2][e]);
                }
            }
        }
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            if (wave + 4u * p >= 6u) break;
            uint32_t i, j;
            block_of(wave + 4u * p, i, j);
            product(i, j, oa[p], ob[p]);
        }
    }
    auto put_b = [&](uint32_t t, uint32_t s, const float* v) __attribute__((always_inline)) {
        uint32_t h0, l0, h1, l1;
        dc_split2(v[0], v[1], h0, l0);
        dc_split2(v[2], v[3], h1, l1);
        const uint32_t at = dc_at(t, s, kDc);
        *reinterpret_cast<uint2*>(w.b + at) = make_uint2(h0, h1);
        *reinterpret_cast<uint2*>(w.b + kDc * kDc + at) = make_uint2(l0, l1);
    };
    const float4 zero4 = make_float4(0.f, 0.f, 0.f, 0.f);
    {
        float m[4], v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            m[e] = ds + (uint32_t)e < dt ? beta[dt] * oa[2][e] : 0.f;
            v[e] = ds + (uint32_t)e <= dt ? ob[2][e] : 0.f;
        }
        *reinterpret_cast<float4*>(A + dt * kDcTs + ds) = make_float4(m[0], m[1], m[2], m[3]);
        put_b(dt, ds, v);
    }
#pragma unroll
    for (int p = 0; p < 2; ++p) {
        if (wave + 4u * p >= 6u) break;
        uint32_t i, j;
        block_of(wave + 4u * p, i, j);
        const uint32_t t = 16u * i + l16, sx = 16u * j + kq * 4u;
        const float f = beta[t], v[4] = {ob[p][0], ob[p][1], ob[p][2], ob[p][3]}, none[4] = {0.f, 0.f, 0.f, 0.f};
        *reinterpret_cast<float4*>(A + t * kDcTs + sx) = make_float4(f * oa[p][0], f * oa[p][1], f * oa[p][2], f * oa[p][3]);
        put_b(t, sx, v);
        put_b(16u * j + l16, 16u * i + kq * 4u, none);   // above the diagonal
        *reinterpret_cast<float4*>(T + (16u * j + l16) * kDcTs + 16u * i + kq * 4u) = zero4;
    }
    __syncthreads();

    // ---- T = (I + A)^-1.  Wave w: column l16 of the w-th diagonal block by substitution ...
    {
        const float* M = A + wave * 16u * (kDcTs + 1u);
        float c[16];
#pragma unroll
        for (uint32_t t = 0; t < 16; ++t) {
            float v = t == l16 ? 1.f : 0.f;
#pragma unroll
            for (uint32_t s = 0; s < t; ++s) v = fmaf(-M[t * kDcTs + s], c[s], v);
            c[t] = v;
        }
        if (kq == 0) {
#pragma unroll
            for (uint32_t t = 0; t < 16; ++t) T[(wave * 16u + t) * kDcTs + wave * 16u + l16] = c[t];
        }
    }
    __syncthreads();
    // ... then the blocks below it: T_ij = -T_ii sum_k A_ik T_kj, j <= k < i
    for (uint32_t i = wave + 1u; i < 4u; ++i) {
        dc_f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
        for (uint32_t k = wave; k < i; ++k)
#pragma unroll
            for (uint32_t s = 0; s < 16; s += 4)
                acc = __builtin_amdgcn_mfma_f32_16x16x4f32(A[(16u * i + l16) * kDcTs + 16u * k + s + kq], T[(16u * k + s + kq) * kDcTs + 16u * wave + l16], acc, 0, 0, 0);
        float* out = T + (16u * i + kq * 4u) * kDcTs + 16u * wave + l16;
#pragma unroll
        for (int r = 0; r < 4; ++r) out[r * kDcTs] = -acc[r];
        dc_lds_order();
        acc = dc_f32x4_t{0.f, 0.f, 0.f, 0.f};
        float b[4];
#pragma unroll
        for (uint32_t s = 0; s < 4; ++s) b[s] = T[(16u * i + 4u * s + kq) * kDcTs + 16u * wave + l16];
#pragma unroll
        for (uint32_t s = 0; s < 4; ++s) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(T[(16u * i + l16) * kDcTs + 16u * i + 4u * s + kq], b[s], acc, 0, 0, 0);
        dc_lds_order();
#pragma unroll
        for (int r = 0; r < 4; ++r) out[r * kDcTs] = acc[r];
        dc_lds_order();
    }
    __syncthreads();
    // T beta as an operand: wave w takes the 16-wide column tile w % 2 of a slice, the token tiles w / 2 and w / 2 + 2
    const uint32_t n = wave & 1u, tw = wave >> 1;
    dc_u32x4_t th[2][2], tl[2][2];
#pragma unroll
    for (uint32_t p = 0; p < 2; ++p)
#pragma unroll
        for (uint32_t s = 0; s <= p; ++s) {   // T is lower triangular
            const float* row = T + ((tw + 2u * p) * 16u + l16) * kDcTs + s * 32u + kq * 8u;
            const float* be = beta + s * 32u + kq * 8u;
#pragma unroll
            for (uint32_t e = 0; e < 4; ++e) {
                uint32_t hi, lo;
                dc_split2(row[2 * e] * be[2 * e], row[2 * e + 1] * be[2 * e + 1], hi, lo);
                th[p][s][e] = hi;
                tl[p][s][e] = lo;
            }
        }
    // the first values, on their way while the slices are formed
    const uint16_t* V = a.v + (size_t)t0 * a.ldx + (size_t)h * vdim + (tid & 3u) * 8u;
    auto fetch_v = [&](uint32_t c0) __attribute__((always_inline)) {
        return (tid >> 2) < live ? *reinterpret_cast<const dc_u32x4_t*>(V + (size_t)(tid >> 2) * a.ldx + c0) : dc_u32x4_t{0u, 0u, 0u, 0u};
    };
    dc_u32x4_t vr = fetch_v(0);

    // ---- the operands of the second launch, a slice at a time
    for (uint32_t d0 = 0; d0 < dim; d0 += kDcStep) {
        __syncthreads();
        stage(x);
        __syncthreads();
        if (d0 + kDcStep < dim) fetch(x, d0 + kDcStep);
        // W[t][d]: rows d, columns t, so that a lane ends with four adjacent d of one t
        {
            dc_f32x4_t acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
            for (uint32_t s = 0; s < 2; ++s) {
                const uint32_t at = (n * 16u + l16) * kDcTs + s * 32u + kq * 8u;
                dc_u32x4_t hi, lo;
#pragma unroll
                for (uint32_t e = 0; e < 4; ++e) {
                    uint32_t h2, l2;
                    dc_split2(kt[at + 2 * e] * __builtin_amdgcn_exp2f(ct[at + 2 * e]), kt[at + 2 * e + 1] * __builtin_amdgcn_exp2f(ct[at + 2 * e + 1]), h2, l2);
                    hi[e] = h2;
                    lo[e] = l2;
                }
#pragma unroll
                for (uint32_t p = s; p < 2; ++p) acc[p] = dc_mfma3(hi, lo, th[p][s], tl[p][s], acc[p]);
            }
#pragma unroll
            for (uint32_t p = 0; p < 2; ++p) {
                uint32_t h0, l0, h1, l1;
                dc_split2(acc[p][0], acc[p][1], h0, l0);
                dc_split2(acc[p][2], acc[p][3], h1, l1);
                uint16_t* out = w.w + dc_at((tw + 2u * p) * 16u + l16, d0 + n * 16u + kq * 4u, dim);
                *reinterpret_cast<uint2*>(out) = make_uint2(h0, h1);
                *reinterpret_cast<uint2*>(out + kDc * dim) = make_uint2(l0, l1);
            }
        }
        {   // queries: eight channels of the token `lane`
            dc_u32x4_t hi, lo;
#pragma unroll
            for (uint32_t e = 0; e < 4; ++e) {
                const uint32_t at = (wave * 8u + 2u * e) * kDcTs + lane;
                uint32_t h2, l2;
                dc_split2(qt[at] * __builtin_amdgcn_exp2f(ct[at]), qt[at + kDcTs] * __builtin_amdgcn_exp2f(ct[at + kDcTs]), h2, l2);
                hi[e] = h2;
                lo[e] = l2;
            }
            uint16_t* out = w.q + dc_at(lane, d0 + wave * 8u, dim);
            *reinterpret_cast<dc_u32x4_t*>(out) = hi;
            *reinterpret_cast<dc_u32x4_t*>(out + kDc * dim) = lo;
        }
        {   // keys decayed to the end of the chunk: eight tokens of one channel
            const uint32_t d = (tid & 15u) + ((tid >> 7) << 4), sx = ((tid >> 4) & 7u) * 8u, at = d * kDcTs + sx;
            const float last = ct[d * kDcTs + kDc - 1u];
            dc_u32x4_t hi, lo;
#pragma unroll
            for (uint32_t e = 0; e < 4; ++e) {
                uint32_t h2, l2;
                dc_split2(kt[at + 2 * e] * __builtin_amdgcn_exp2f(fminf(last - ct[at + 2 * e], 0.f)),
                          kt[at + 2 * e + 1] * __builtin_amdgcn_exp2f(fminf(last - ct[at + 2 * e + 1], 0.f)), h2, l2);
                hi[e] = h2;
                lo[e] = l2;
            }
            uint16_t* out = w.k + dc_at(d0 + d, sx, kDc);
            *reinterpret_cast<dc_u32x4_t*>(out) = hi;
            *reinterpret_cast<dc_u32x4_t*>(out + (size_t)dim * kDc) = lo;
            if (sx == 0) w.gamma[d0 + d] = __builtin_amdgcn_exp2f(last);
        }
    }
    // U0[t][v], 32 value columns at a time: rows t, columns v
    uint16_t* vt = reinterpret_cast<uint16_t*>(kt);   // [value column][token]
    for (uint32_t c0 = 0; c0 < vdim; c0 += 32u) {
        __syncthreads();
#pragma unroll
        for (uint32_t e = 0; e < 4; ++e) {
            uint16_t* p = vt + ((tid & 3u) * 8u + 2u * e) * kDcUs + (tid >> 2);
            p[0] = (uint16_t)vr[e];
            p[kDcUs] = (uint16_t)(vr[e] >> 16);
        }
        __syncthreads();
        if (c0 + 32u < vdim) vr = fetch_v(c0 + 32u);
        dc_f32x4_t acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (uint32_t s = 0; s < 2; ++s) {
            const dc_u32x4_t v = *reinterpret_cast<const dc_u32x4_t*>(vt + (n * 16u + l16) * kDcUs + s * 32u + kq * 8u);
#pragma unroll
            for (uint32_t p = s; p < 2; ++p) acc[p] = dc_mfma(th[p][s], v, dc_mfma(tl[p][s], v, acc[p]));
        }
#pragma unroll
        for (uint32_t p = 0; p < 2; ++p)
            *reinterpret_cast<dc_f32x4_t*>(w.u0 + dc_u0_at((tw + 2u * p) * 16u + kq * 4u, c0 + n * 16u + l16, vdim)) = acc[p];
    }
}

// One wave's part of the second launch: WRITER waves form U (16 tokens each), the others the outputs; every wave holds its
// 16-channel tiles of the state (where there are more waves than tiles, two waves hold the same one).  Without branches,
// so that every wait counts exactly the requests it needs: those of the next chunk stay on their way across the barriers.
template <int KD, int VT, bool WRITER>
__device__ __forceinline__ void delta_walk(const DeltaChunkArgs& a, uint32_t wave, uint16_t* sh, uint16_t* sl, uint16_t* uh, uint16_t* ul) {
    constexpr uint32_t DIM = KD * 32u, SS = DIM + 8u;
    constexpr int ND = (2 * KD + 7) / 8;
    const uint32_t h = blockIdx.x, v0 = blockIdx.y * (VT * 16u), lane = threadIdx.x & 63u, l16 = lane & 15u, kq = lane >> 4;
    const uint32_t chunks = (a.rows + kDc - 1u) / kDc, nv = a.heads * a.vdim_ld, tt = (wave & 3u) * 16u;
    float* state = a.state + ((size_t)h * a.vdim_ld + v0 + l16) * a.state_ld + kq * 4u;
    uint32_t d0[ND];
#pragma unroll
    for (int i = 0; i < ND; ++i) d0[i] = (wave + 8u * i) % (2u * KD) * 16u;

    dc_f32x4_t S[ND][VT];
#pragma unroll
    for (int i = 0; i < ND; ++i)
#pragma unroll
        for (int v = 0; v < VT; ++v) S[i][v] = *reinterpret_cast<const dc_f32x4_t*>(state + (size_t)(v * 16) * a.state_ld + d0[i]);
    // arrived before anything else is requested: a wait for them at the head of the loop would also wait for what is on its way
#pragma unroll
    for (int i = 0; i < ND; ++i)
#pragma unroll
        for (int v = 0; v < VT; ++v) asm volatile("" : "+v"(S[i][v]));
    struct Operands {
        dc_u32x4_t r[KD][2], b[2][2], k[ND][2][2];
        dc_f32x4_t u0[VT], g[ND];
    };
    auto fetch = [&](Operands& o, uint32_t chunk) __attribute__((always_inline)) {
        const DcWork w = dc_work(a, chunk < chunks ? chunk : chunks - 1u, h);
        const uint16_t* r = (WRITER ? w.w : w.q) + (tt >> 4) * (KD * 512u) + lane * 8u;
#pragma unroll
        for (int s = 0; s < KD; ++s)
#pragma unroll
            for (int x = 0; x < 2; ++x) o.r[s][x] = *reinterpret_cast<const dc_u32x4_t*>(r + x * kDc * DIM + s * 512);
        if (WRITER) {
#pragma unroll
            for (int v = 0; v < VT; ++v) o.u0[v] = *reinterpret_cast<const dc_f32x4_t*>(w.u0 + (((v0 >> 4) + v) * 4u + (tt >> 4)) * 256u + lane * 4u);
        }
#pragma unroll
        for (int i = 0; i < ND; ++i) o.g[i] = *reinterpret_cast<const dc_f32x4_t*>(w.gamma + d0[i] + kq * 4u);
#pragma unroll
        for (int s = 0; s < 2; ++s)
#pragma unroll
            for (int x = 0; x < 2; ++x) {
                if (!WRITER) o.b[s][x] = *reinterpret_cast<const dc_u32x4_t*>(w.b + x * kDc * kDc + ((tt >> 4) * 2u + s) * 512u + lane * 8u);
#pragma unroll
                for (int i = 0; i < ND; ++i) o.k[i][s][x] = *reinterpret_cast<const dc_u32x4_t*>(w.k + x * DIM * kDc + ((d0[i] >> 4) * 2u + s) * 512u + lane * 8u);
            }
    };
    auto step = [&](const Operands& o, Operands& next, uint32_t chunk) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < ND; ++i)
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                uint32_t h0, l0, h1, l1;
                dc_split2(S[i][v][0], S[i][v][1], h0, l0);
                dc_split2(S[i][v][2], S[i][v][3], h1, l1);
                const uint32_t at = (v * 16u + l16) * SS + d0[i] + kq * 4u;
                *reinterpret_cast<uint2*>(sh + at) = make_uint2(h0, h1);
                *reinterpret_cast<uint2*>(sl + at) = make_uint2(l0, l1);
            }
        fetch(next, chunk + 1u);
        __syncthreads();
        dc_f32x4_t p[VT];
#pragma unroll
        for (int v = 0; v < VT; ++v) p[v] = dc_f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KD; ++s)
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const uint32_t at = (v * 16u + l16) * SS + s * 32u + kq * 8u;
                p[v] = dc_mfma3(o.r[s][0], o.r[s][1], *reinterpret_cast<const dc_u32x4_t*>(sh + at), *reinterpret_cast<const dc_u32x4_t*>(sl + at), p[v]);
            }
        if (WRITER) {
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                uint32_t h0, l0, h1, l1;
                dc_split2(o.u0[v][0] - p[v][0], o.u0[v][1] - p[v][1], h0, l0);
                dc_split2(o.u0[v][2] - p[v][2], o.u0[v][3] - p[v][3], h1, l1);
                const uint32_t at = (v * 16u + l16) * kDcUs + tt + kq * 4u;
                *reinterpret_cast<uint2*>(uh + at) = make_uint2(h0, h1);
                *reinterpret_cast<uint2*>(ul + at) = make_uint2(l0, l1);
            }
        }
#pragma unroll
        for (int i = 0; i < ND; ++i)
#pragma unroll
            for (int v = 0; v < VT; ++v)
#pragma unroll
                for (int e = 0; e < 4; ++e) S[i][v][e] *= o.g[i][e];
        __syncthreads();
#pragma unroll
        for (int s = 0; s < 2; ++s)
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const uint32_t at = (v * 16u + l16) * kDcUs + s * 32u + kq * 8u;
                const dc_u32x4_t bh = *reinterpret_cast<const dc_u32x4_t*>(uh + at), bl = *reinterpret_cast<const dc_u32x4_t*>(ul + at);
#pragma unroll
                for (int i = 0; i < ND; ++i) S[i][v] = dc_mfma3(o.k[i][s][0], o.k[i][s][1], bh, bl, S[i][v]);
                if (!WRITER) p[v] = dc_mfma3(o.b[s][0], o.b[s][1], bh, bl, p[v]);
            }
        if (!WRITER) {   // whole chunks: the rows past the pass are written too
#pragma unroll
            for (int v = 0; v < VT; ++v)
#pragma unroll
                for (int e = 0; e < 4; ++e) a.o[(size_t)(chunk * kDc + tt + kq * 4u + e) * nv + (size_t)h * a.vdim_ld + v0 + v * 16 + l16] = p[v][e];
        }
    };
    Operands even, odd;
    fetch(even, 0);
    uint32_t chunk = 0;
    for (; chunk + 1u < chunks; chunk += 2u) {
        step(even, odd, chunk);
        step(odd, even, chunk + 1u);
    }
    if (chunk < chunks) step(even, odd, chunk);
#pragma unroll
    for (int i = 0; i < ND; ++i)
#pragma unroll
        for (int v = 0; v < VT; ++v) *reinterpret_cast<dc_f32x4_t*>(state + (size_t)(v * 16) * a.state_ld + d0[i]) = S[i][v];
}

// KD: key channels / 32; VT: 16-wide tiles of value columns of the block.
template <int KD, int VT>
__global__ __launch_bounds__(512) void delta_inter_kernel(const DeltaChunkArgs a) {
    __shared__ __align__(16) uint16_t sh[VT * 16 * (KD * 32 + 8)], sl[VT * 16 * (KD * 32 + 8)], uh[VT * 16 * kDcUs], ul[VT * 16 * kDcUs];
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
    if (wave < 4u) delta_walk<KD, VT, true>(a, wave, sh, sl, uh, ul);   // both halves pass the same barriers
    else delta_walk<KD, VT, false>(a, wave, sh, sl, uh, ul);
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
    if (a.heads % a.kv_heads || a.ldb < a.heads || a.state_ld % 4 || a.state_ld < a.dim_ld || a.ldx % 8 || ((uintptr_t)a.v & 15u)) return set_error(FK_ERR_INVALID, "delta chunks: bad shape");
    if (!delta_chunk_supported(a.dim_ld, a.vdim_ld)) return set_error(FK_ERR_UNSUPPORTED, "delta chunks: key width 32, 64, 96, 128, 192 or 256, value width a multiple of 32");
    const uint32_t chunks = (a.rows + kDc - 1) / kDc;
    if (chunks > 65535) return set_error(FK_ERR_UNSUPPORTED, "delta chunks: too many rows");
    out->func = (const void*)&delta_intra_kernel;
    out->grid = dim3(a.heads, chunks, 1);
    out->block = dim3(256, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    Launch seq;
    const uint32_t vt = (uint64_t)a.heads * (a.vdim_ld / 32) >= 64 ? 2 : 1;   // a wider slice reads the operands less often
    seq.func = vt == 2 ? inter_func<2>(a.dim_ld / 32) : inter_func<1>(a.dim_ld / 32);
    seq.grid = dim3(a.heads, a.vdim_ld / (16 * vt), 1);
    seq.block = dim3(512, 1, 1);
    seq.set_args(a);
    out->then.push_back(seq);
    return FK_OK;
}

}  // namespace fk
