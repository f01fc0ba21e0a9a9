// Gated delta rule with one decay per head and key channel:
//     S <- g S,  u = beta (v - S^T k),  S <- S + k u^T,  o = S^T q
// per token and head, g along the key channels, S [key, value] in fp32.  With A = g S the two read-outs need one pass over
// the state: o = A^T q + (k . q) u.
//
// The state of a head is stored as [vdim_ld][state_ld], like the state-space mixer's: sixteen lanes share one value column
// and hold four adjacent key channels each (per 64), so both sums of a step stay inside a row of sixteen lanes.
#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

namespace {

constexpr int kDeltaBlock = 256;
constexpr float kUnitEps = 1e-6f;

// Unit vectors, log2 decays and step sizes of one row.
template <typename T>
__global__ __launch_bounds__(kDeltaBlock) void delta_prep_kernel(const DeltaPrepArgs a) {
    const uint32_t r = blockIdx.x, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const T* x = reinterpret_cast<const T*>(a.xc) + (size_t)r * a.ldx;
    const uint32_t nk = a.kv_heads * a.dim_ld;
    float* qk = a.qk + (size_t)r * 2u * nk;
    const float q_scale = 1.0f / sqrtf((float)a.dim);
    for (uint32_t i = wave; i < 2u * a.kv_heads; i += kDeltaBlock / kWave) {   // the query heads, then the key heads
        const T* s = x + (size_t)i * a.dim_ld;
        float ss = 0.f;
        for (uint32_t d = lane * 4u; d < a.dim_ld; d += kWave * 4u) {
            const float4 v = act_load4(s + d);
            ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
        }
        float f = 1.0f / sqrtf(wave_sum(ss) + kUnitEps);
        if (i < a.kv_heads) f *= q_scale;
        for (uint32_t d = lane * 4u; d < a.dim_ld; d += kWave * 4u) {
            const float4 v = act_load4(s + d);
            *reinterpret_cast<float4*>(qk + (size_t)i * a.dim_ld + d) = make_float4(v.x * f, v.y * f, v.z * f, v.w * f);
        }
    }
    const uint32_t n = a.heads * a.dim_ld;
    float* g = a.decay + (size_t)r * n;
    for (uint32_t c = tid * 4u; c < n; c += kDeltaBlock * 4u) {
        const float rate = -1.4426950408889634f * expf(bf16_bits_to_f32(a.a_log[c / a.dim_ld]));
        const float4 z = *reinterpret_cast<const float4*>(g + c), b = act_load4(a.dt_bias + c);
        *reinterpret_cast<float4*>(g + c) = make_float4(rate * softplus(z.x + b.x), rate * softplus(z.y + b.y), rate * softplus(z.z + b.z), rate * softplus(z.w + b.w));
    }
    for (uint32_t h = tid; h < a.heads; h += kDeltaBlock) {
        float* b = a.beta + (size_t)r * a.ldb + h;
        *b = sigmoid(*b);
    }
}

template <typename T, int NI>
__global__ __launch_bounds__(kDeltaBlock) void delta_scan_kernel(const DeltaScanArgs a) {
    const uint32_t h = blockIdx.x, lane = threadIdx.x & 63u, wave = threadIdx.x >> 6;
    const uint32_t p = blockIdx.y * 16u + wave * 4u + (lane >> 4), nl = (lane & 15u) * 4u;   // vdim_ld is a multiple of 32
    const uint32_t nk = a.kv_heads * a.dim_ld, g = h / (a.heads / a.kv_heads), nd = a.heads * a.dim_ld;
    float* state = a.state + ((size_t)h * a.vdim_ld + p) * a.state_ld + nl;
    const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
    float4 S[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) S[i] = *reinterpret_cast<const float4*>(state + 64 * i);
    struct Row {
        float4 q[NI], k[NI], g[NI];
        float v, beta;
    };
    auto fetch = [&](uint32_t r, Row& w) __attribute__((always_inline)) {
        const float *qk = a.qk + (size_t)r * 2u * nk + (size_t)g * a.dim_ld, *d = a.decay + (size_t)r * nd + (size_t)h * a.dim_ld;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const uint32_t c = nl + 64u * i;
            const bool in = c < a.dim_ld;
            w.q[i] = in ? *reinterpret_cast<const float4*>(qk + c) : zero;
            w.k[i] = in ? *reinterpret_cast<const float4*>(qk + nk + c) : zero;
            w.g[i] = in ? *reinterpret_cast<const float4*>(d + c) : zero;
        }
        w.v = act_load(reinterpret_cast<const T*>(a.v) + (size_t)r * a.ldx + (size_t)h * a.vdim_ld + p);
        w.beta = a.beta[(size_t)r * a.ldb + h];
    };
    constexpr uint32_t kDeep = NI <= 2 ? 4 : 2;   // rows on their way
    Row in[kDeep];
#pragma unroll
    for (uint32_t e = 0; e < kDeep; ++e) fetch(e < a.rows ? e : a.rows - 1u, in[e]);
    float* o = a.o + (size_t)h * a.vdim_ld + p;
    const size_t ldo = (size_t)a.heads * a.vdim_ld;
    auto step = [&](uint32_t r, const Row& w) __attribute__((always_inline)) {
        float sk = 0.f, sq = 0.f, kq = 0.f;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            S[i].x *= exp2f(w.g[i].x); S[i].y *= exp2f(w.g[i].y); S[i].z *= exp2f(w.g[i].z); S[i].w *= exp2f(w.g[i].w);
            sk = fmaf(S[i].x, w.k[i].x, sk); sk = fmaf(S[i].y, w.k[i].y, sk); sk = fmaf(S[i].z, w.k[i].z, sk); sk = fmaf(S[i].w, w.k[i].w, sk);
            sq = fmaf(S[i].x, w.q[i].x, sq); sq = fmaf(S[i].y, w.q[i].y, sq); sq = fmaf(S[i].z, w.q[i].z, sq); sq = fmaf(S[i].w, w.q[i].w, sq);
            kq = fmaf(w.k[i].x, w.q[i].x, kq); kq = fmaf(w.k[i].y, w.q[i].y, kq); kq = fmaf(w.k[i].z, w.q[i].z, kq); kq = fmaf(w.k[i].w, w.q[i].w, kq);
        }
        sk = group_sum(sk, 16);
        sq = group_sum(sq, 16);
        kq = group_sum(kq, 16);
        const float u = w.beta * (w.v - sk);
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            S[i].x = fmaf(w.k[i].x, u, S[i].x); S[i].y = fmaf(w.k[i].y, u, S[i].y);
            S[i].z = fmaf(w.k[i].z, u, S[i].z); S[i].w = fmaf(w.k[i].w, u, S[i].w);
        }
        if (nl == 0) o[(size_t)r * ldo] = fmaf(kq, u, sq);
    };
    for (uint32_t r0 = 0; r0 < a.rows; r0 += kDeep) {
#pragma unroll
        for (uint32_t e = 0; e < kDeep; ++e) {
            if (r0 + e < a.rows) step(r0 + e, in[e]);
            fetch(r0 + e + kDeep < a.rows ? r0 + e + kDeep : a.rows - 1u, in[e]);
        }
    }
#pragma unroll
    for (int i = 0; i < NI; ++i) *reinterpret_cast<float4*>(state + 64 * i) = S[i];
}

template <typename T>
const void* scan_func(uint32_t ni) {
    switch (ni) {
        case 1: return (const void*)&delta_scan_kernel<T, 1>;
        case 2: return (const void*)&delta_scan_kernel<T, 2>;
        case 3: return (const void*)&delta_scan_kernel<T, 3>;
        default: return (const void*)&delta_scan_kernel<T, 4>;
    }
}

}  // namespace

fk_status plan_delta_prep(const DeltaPrepArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "delta prep: act must be 16 or 32");
    if (!a.xc || !a.dt_bias || !a.a_log || !a.decay || !a.beta || !a.qk || !a.rows || !a.heads || !a.kv_heads || !a.dim) return set_error(FK_ERR_INVALID, "delta prep: bad arguments");
    if (a.heads % a.kv_heads || a.dim_ld % 32 || a.dim_ld < a.dim || a.ldx % 4 || a.ldb < a.heads) return set_error(FK_ERR_INVALID, "delta prep: bad shape");
    out->func = act == 16 ? (const void*)&delta_prep_kernel<uint16_t> : (const void*)&delta_prep_kernel<float>;
    out->grid = dim3(a.rows, 1, 1);
    out->block = dim3(kDeltaBlock, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    return FK_OK;
}

fk_status plan_delta_scan(const DeltaScanArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "delta scan: act must be 16 or 32");
    if (!a.qk || !a.decay || !a.beta || !a.v || !a.state || !a.o || !a.rows || !a.heads || !a.kv_heads) return set_error(FK_ERR_INVALID, "delta scan: bad arguments");
    if (a.heads % a.kv_heads || a.dim_ld % 32 || a.vdim_ld % 32 || !a.vdim_ld || a.ldb < a.heads || a.state_ld % 64 || a.state_ld < a.dim_ld)
        return set_error(FK_ERR_INVALID, "delta scan: bad shape");
    if (a.state_ld > kMaxSsmState || a.vdim_ld / 16u > 65535) return set_error(FK_ERR_UNSUPPORTED, "delta scan: key width at most 256");
    const uint32_t ni = a.state_ld / 64u;
    out->func = act == 16 ? scan_func<uint16_t>(ni) : scan_func<float>(ni);
    out->grid = dim3(a.heads, a.vdim_ld / 16u, 1);
    out->block = dim3(kDeltaBlock, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    return FK_OK;
}

}  // namespace fk
