// Grouped-query attention of the layer-list decoder around the shared attention kernels: the launch that turns a joint
// projection into rotated queries and cache rows, and a row-by-row attention for every head width and for fp32.
//
// bf16 attention itself is sdpa_decode (one row) and sdpa_prefill (portions); heads are padded with zeros to the widths
// they take, which changes no score and no output.
#include <algorithm>

#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

namespace {

constexpr int kGqaBlock = 256;
constexpr uint32_t kGqaWaves = kGqaBlock / kWave, kGqaTile = 64, kMaxRotPairs = 512;

// A block forms the two mean squares of its row, then its waves take heads in turn; a row's heads are dealt to gridDim.y
// blocks (one for a portion, one wave per head for a single row).
template <typename T>
__global__ __launch_bounds__(kGqaBlock) void qk_store_kernel(const QkStoreArgs a) {
    __shared__ float red[kGqaWaves + 1], red2[kGqaWaves + 1];
    __shared__ float cs[2 * kMaxRotPairs];
    const uint32_t r = blockIdx.x, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, pos = *a.offset + r, half = a.rot_dims / 2u;
    if (pos >= a.capacity) return;
    const T* row = reinterpret_cast<const T*>(a.u) + (size_t)r * a.ldu;
    const uint32_t nq = a.heads * a.dim_ld, nk = a.kv_heads * a.dim_ld;
    for (uint32_t i = tid; i < half; i += kGqaBlock) {
        float c, s;
        position_cos_sin(pos, a.freq[i], c, s);
        cs[2 * i] = c * a.mag;
        cs[2 * i + 1] = s * a.mag;
    }
    float sq = 0.f, sk = 0.f;
    for (uint32_t c = tid * 4u; c < nq; c += kGqaBlock * 4u) {
        const float4 v = act_load4(row + a.q0 + c);
        sq = fmaf(v.x, v.x, sq); sq = fmaf(v.y, v.y, sq); sq = fmaf(v.z, v.z, sq); sq = fmaf(v.w, v.w, sq);
    }
    for (uint32_t c = tid * 4u; c < nk; c += kGqaBlock * 4u) {
        const float4 v = act_load4(row + a.k0 + c);
        sk = fmaf(v.x, v.x, sk); sk = fmaf(v.y, v.y, sk); sk = fmaf(v.z, v.z, sk); sk = fmaf(v.w, v.w, sk);
    }
    const float rq = 1.0f / sqrtf(block_sum<kGqaBlock>(sq, red) / (float)(a.heads * a.dim) + a.eps);
    const float rk = 1.0f / sqrtf(block_sum<kGqaBlock>(sk, red2) / (float)(a.kv_heads * a.dim) + a.eps);
    for (uint32_t h = blockIdx.y * kGqaWaves + wave; h < a.heads + a.kv_heads; h += kGqaWaves * gridDim.y) {
        const bool key = h >= a.heads;
        const uint32_t n = key ? h - a.heads : h;
        const T* src = row + (key ? a.k0 : a.q0) + (size_t)n * a.dim_ld;
        const uint16_t* w = (key ? a.wk : a.wq) + (size_t)n * a.dim_ld;
        const float f = key ? rk : rq;
        const size_t at = ((size_t)n * a.capacity + pos) * a.dim_ld;
        T* dst = key ? reinterpret_cast<T*>(a.cache_k) + at : reinterpret_cast<T*>(a.q) + (size_t)r * nq + (size_t)n * a.dim_ld;
        T* val = reinterpret_cast<T*>(a.cache_v) + at;
        for (uint32_t d = lane; d < a.dim_ld; d += kWave) {
            const T raw = src[d];
            const float v = act_load(&raw) * f * bf16_bits_to_f32(w[d]);
            float o = v;
            if (d < a.rot_dims) {
                const bool low = d < half;
                const uint32_t i = low ? d : d - half, p = low ? d + half : d - half;
                const float other = act_load(src + p) * f * bf16_bits_to_f32(w[p]);
                o = low ? v * cs[2 * i] - other * cs[2 * i + 1] : v * cs[2 * i] + other * cs[2 * i + 1];
            }
            act_store(dst + d, o);
            if (key) val[d] = raw;
        }
    }
}

// Keys 64 at a time: sixteen lanes per key form the scores, every wave reduces the 64 of them, then wave w adds values
// w, w + 4, .. of the tile; the waves' sums meet at the end.
template <typename T>
__global__ __launch_bounds__(kGqaBlock) void gqa_rows_kernel(const GqaRowsArgs a) {
    __shared__ __align__(16) float q[kMaxGqaDim], acc_s[kGqaWaves][kMaxGqaDim];
    __shared__ float s[kGqaTile], p[kGqaTile];
    const uint32_t h = blockIdx.x, r = blockIdx.y, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const uint32_t pos = *a.offset + r, seen = pos + 1u < a.capacity ? pos + 1u : a.capacity;
    const size_t base = (size_t)(h / (a.heads / a.kv_heads)) * a.capacity * a.dim_ld;
    const T *K = reinterpret_cast<const T*>(a.cache_k) + base, *V = reinterpret_cast<const T*>(a.cache_v) + base;
    const T* qr = reinterpret_cast<const T*>(a.q) + ((size_t)r * a.heads + h) * a.dim_ld;
    for (uint32_t d = tid; d < a.dim_ld; d += kGqaBlock) q[d] = act_load(qr + d);
    constexpr uint32_t kPer = kMaxGqaDim / kWave;
    float acc[kPer];
#pragma unroll
    for (uint32_t i = 0; i < kPer; ++i) acc[i] = 0.f;
    float m = -INFINITY, l = 0.f;
    __syncthreads();
    for (uint32_t j0 = 0; j0 < seen; j0 += kGqaTile) {
        for (uint32_t t = tid >> 4; t < kGqaTile; t += kGqaBlock / 16u) {
            const uint32_t j = j0 + t < seen ? j0 + t : seen - 1u;
            float v = 0.f;
            for (uint32_t d = (lane & 15u) * 4u; d < a.dim_ld; d += 64u) {
                const float4 k = act_load4(K + (size_t)j * a.dim_ld + d), x = *reinterpret_cast<const float4*>(q + d);
                v = fmaf(k.x, x.x, v); v = fmaf(k.y, x.y, v); v = fmaf(k.z, x.z, v); v = fmaf(k.w, x.w, v);
            }
            v = group_sum(v, 16);
            if ((lane & 15u) == 0) s[t] = j0 + t < seen ? v * a.scale : -INFINITY;
        }
        __syncthreads();
        const float mine = s[lane], top = fmaxf(m, wave_max(mine)), alpha = expf(m - top), e = expf(mine - top);
        l = l * alpha + wave_sum(e);
        m = top;
        if (wave == 0) p[lane] = e;
#pragma unroll
        for (uint32_t i = 0; i < kPer; ++i) acc[i] *= alpha;
        __syncthreads();
        const uint32_t live = seen - j0 < kGqaTile ? seen - j0 : kGqaTile;
        for (uint32_t t = wave; t < live; t += kGqaWaves) {
            const float w = p[t];
            const T* v = V + (size_t)(j0 + t) * a.dim_ld;
#pragma unroll
            for (uint32_t i = 0; i < kPer; ++i)
                if (lane + i * 64u < a.dim_ld) acc[i] = fmaf(w, act_load(v + lane + i * 64u), acc[i]);
        }
        // the next tile's scores go to `s`, which nobody reads any more; `p` is rewritten behind the next barrier
    }
#pragma unroll
    for (uint32_t i = 0; i < kPer; ++i)
        if (lane + i * 64u < a.dim_ld) acc_s[wave][lane + i * 64u] = acc[i];
    __syncthreads();
    T* out = reinterpret_cast<T*>(a.out) + (size_t)r * a.ldo + (size_t)h * a.dim_ld;
    for (uint32_t d = tid; d < a.dim_ld; d += kGqaBlock)
        act_store(out + d, ((acc_s[0][d] + acc_s[1][d]) + (acc_s[2][d] + acc_s[3][d])) / l);
}

}  // namespace

fk_status plan_qk_store(const QkStoreArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "qk store: act must be 16 or 32");
    if (!a.u || !a.wq || !a.wk || !a.freq || !a.q || !a.cache_k || !a.cache_v || !a.offset || !a.rows || !a.heads || !a.kv_heads || !a.capacity)
        return set_error(FK_ERR_INVALID, "qk store: bad arguments");
    if (a.heads % a.kv_heads || a.dim_ld < a.dim || a.dim_ld % 4 || a.rot_dims % 2 || a.rot_dims > a.dim || a.ldu % 4 || a.k0 % 4 || a.q0 % 4 ||
        a.q0 + a.heads * a.dim_ld > a.ldu || a.k0 + a.kv_heads * a.dim_ld > a.ldu)
        return set_error(FK_ERR_INVALID, "qk store: bad shape");
    if (a.rot_dims > 2 * kMaxRotPairs) return set_error(FK_ERR_UNSUPPORTED, "qk store: at most 1024 rotated dimensions");
    out->func = act == 16 ? (const void*)&qk_store_kernel<uint16_t> : (const void*)&qk_store_kernel<float>;
    out->grid = dim3(a.rows, std::min((a.heads + a.kv_heads + kGqaWaves - 1) / kGqaWaves, std::max(1u, 2048u / a.rows)), 1);   // enough blocks to fill the device
    out->block = dim3(kGqaBlock, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    return FK_OK;
}

fk_status plan_gqa_rows(const GqaRowsArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "gqa rows: act must be 16 or 32");
    if (!a.q || !a.cache_k || !a.cache_v || !a.offset || !a.out || !a.rows || !a.heads || !a.kv_heads || !a.capacity)
        return set_error(FK_ERR_INVALID, "gqa rows: bad arguments");
    if (a.heads % a.kv_heads || a.dim_ld % 4 || !a.dim_ld || a.ldo < a.heads * a.dim_ld) return set_error(FK_ERR_INVALID, "gqa rows: bad shape");
    if (a.dim_ld > kMaxGqaDim || a.rows > 65535) return set_error(FK_ERR_UNSUPPORTED, "gqa rows: heads of at most 512, at most 65535 rows");
    out->func = act == 16 ? (const void*)&gqa_rows_kernel<uint16_t> : (const void*)&gqa_rows_kernel<float>;
    out->grid = dim3(a.heads, a.rows, 1);
    out->block = dim3(kGqaBlock, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    return FK_OK;
}

}  // namespace fk
