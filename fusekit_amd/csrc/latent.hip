// Latent attention: the cache of a layer holds one normalised latent and one rotated key part per position, shared by
// all heads.  A query can meet it in two ways, which differ by rounding only:
//   * in the latent space -- q is carried through W_uk once per head, so scores are dot products with the cached
//     latents and the weighted sum of latents is left to W_uv (decoding and short portions: nothing is formed per key);
//   * with keys and values formed from the latents for the positions a pass can see (long portions: the pass shares
//     them, latent_prefill.hip).
// `window` counts the positions a query can attend to, its own among them.  The softmax has a sink, a per-head score
// that enters the denominator only.
#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

namespace {

constexpr int kLatBlock = 256;

// One block per row: normalises the latent into the cache row, rotates the key part into it and the queries in place.
template <typename T>
__global__ __launch_bounds__(kLatBlock) void latent_store_kernel(const LatentStoreArgs a) {
    extern __shared__ float cs_sn[];   // rot_dims floats: cos, sin per pair
    __shared__ float red[kLatBlock / kWave + 1];
    const uint32_t r = blockIdx.x, pos = *a.offset + r, half = a.rot_dims / 2u;
    const float* kv = a.kv + (size_t)r * a.ldkv;
    T* row = reinterpret_cast<T*>(a.cache) + (size_t)(pos & (a.ring - 1u)) * a.ldc;
    for (uint32_t i = threadIdx.x; i < half; i += kLatBlock) position_cos_sin(pos, a.freq[i], cs_sn[2 * i], cs_sn[2 * i + 1]);
    float ss = 0.f;
    for (uint32_t c = threadIdx.x; c < a.rank; c += kLatBlock) ss = fmaf(kv[c], kv[c], ss);
    ss = block_sum<kLatBlock>(ss, red);   // its barrier also publishes the table
    const float k = 1.0f / sqrtf(ss / (float)a.rank + a.eps);
    for (uint32_t c = threadIdx.x; c < a.rank; c += kLatBlock) act_store(row + c, kv[c] * k * bf16_bits_to_f32(a.norm[c]));
    for (uint32_t i = threadIdx.x; i < a.rot; i += kLatBlock) {
        const float* s = kv + a.rank;
        float v = s[i];
        if (i < half) v = s[i] * cs_sn[2 * i] - s[i + half] * cs_sn[2 * i + 1];
        else if (i < a.rot_dims) v = s[i] * cs_sn[2 * (i - half)] + s[i - half] * cs_sn[2 * (i - half) + 1];
        act_store(row + a.rank_ld + i, v);
    }
    T* q = reinterpret_cast<T*>(a.q) + (size_t)r * a.ldq;
    for (uint32_t t = threadIdx.x; t < a.heads * half; t += kLatBlock) {
        const uint32_t h = t / half, i = t - h * half;
        T* s = q + (size_t)h * a.hs + a.dim_ld;
        const float u = act_load(s + i), v = act_load(s + i + half), cs = cs_sn[2 * i], sn = cs_sn[2 * i + 1];
        act_store(s + i, u * cs - v * sn);
        act_store(s + i + half, v * cs + u * sn);
    }
}

// One block per (head, row), any width: 256 positions at a time, a wave per position for the scores, a thread per
// latent element for the sum.
constexpr uint32_t kLatTile = 256, kLatMaxPer = 8;   // latent widths up to 2048
template <typename T, typename Q>
__global__ __launch_bounds__(kLatBlock) void latent_attn_kernel(const LatentAttnArgs a) {
    extern __shared__ __align__(16) float sm[];   // qa [rank_ld] | q rotated [ldc - rank_ld] | scores [kLatTile]
    __shared__ float red[kLatBlock / kWave + 1];
    const uint32_t h = blockIdx.x, r = blockIdx.y, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const uint32_t pos = *a.offset + r, lo = pos + 1u > a.window ? pos + 1u - a.window : 0u, rot_ld = a.ldc - a.rank_ld;
    float *qa = sm, *qr = sm + a.rank_ld, *sc = qr + rot_ld;
    const Q* gqa = reinterpret_cast<const Q*>(a.qa) + ((size_t)r * a.heads + h) * a.rank_ld;
    const T* gq = reinterpret_cast<const T*>(a.q) + (size_t)r * a.ldq + (size_t)h * a.hs + a.dim_ld;
    for (uint32_t c = tid; c < a.rank_ld; c += kLatBlock) qa[c] = act_load(gqa + c);
    for (uint32_t c = tid; c < rot_ld; c += kLatBlock) qr[c] = c < a.rot ? act_load(gq + c) : 0.f;
    __syncthreads();
    const T* cache = reinterpret_cast<const T*>(a.cache);
    float acc[kLatMaxPer] = {};
    float m = -INFINITY, l = 0.f;
    for (uint32_t j0 = lo; j0 <= pos; j0 += kLatTile) {
        const uint32_t cnt = pos + 1u - j0 < kLatTile ? pos + 1u - j0 : kLatTile;
        for (uint32_t j = wave; j < cnt; j += kLatBlock / kWave) {
            const T* row = cache + (size_t)((j0 + j) & (a.ring - 1u)) * a.ldc;
            float s = 0.f;
            for (uint32_t c = lane * 4u; c < a.ldc; c += kWave * 4u) {   // qa and qr lie one behind the other, as the row does
                const float4 k = act_load4(row + c), q = *reinterpret_cast<const float4*>(sm + c);
                s = fmaf(k.x, q.x, s); s = fmaf(k.y, q.y, s); s = fmaf(k.z, q.z, s); s = fmaf(k.w, q.w, s);
            }
            s = wave_sum(s);
            if (lane == 0) sc[j] = s * a.scale;
        }
        __syncthreads();
        const float mine = tid < cnt ? sc[tid] : -INFINITY;
        const float mt = block_max<kLatBlock>(mine, red);
        const float m_new = fmaxf(m, mt), alpha = expf(m - m_new);
        const float p = tid < cnt ? expf(mine - m_new) : 0.f;
        sc[tid] = p;
        l = l * alpha + block_sum<kLatBlock>(p, red);
#pragma unroll
        for (uint32_t i = 0; i < kLatMaxPer; ++i) acc[i] *= alpha;
        m = m_new;
        for (uint32_t j = 0; j < cnt; ++j) {
            const T* row = cache + (size_t)((j0 + j) & (a.ring - 1u)) * a.ldc;
            const float pj = sc[j];
#pragma unroll
            for (uint32_t i = 0; i < kLatMaxPer; ++i) {
                const uint32_t c = tid + i * kLatBlock;
                if (c < a.rank) acc[i] = fmaf(pj, act_load(row + c), acc[i]);
            }
        }
        __syncthreads();
    }
    const float sink = bf16_bits_to_f32(a.sink[h]), top = fmaxf(m, sink);
    const float f = expf(m - top) / (l * expf(m - top) + expf(sink - top));
    T* out = reinterpret_cast<T*>(a.out) + ((size_t)r * a.heads + h) * a.rank_ld;
#pragma unroll
    for (uint32_t i = 0; i < kLatMaxPer; ++i) {
        const uint32_t c = tid + i * kLatBlock;
        if (c < a.rank) act_store(out + c, acc[i] * f);
    }
}

}  // namespace

fk_status plan_latent_store(const LatentStoreArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "latent store: act must be 16 or 32");
    if (!a.kv || !a.norm || !a.freq || !a.cache || !a.q || !a.offset || !a.rows || !a.rank || !a.heads)
        return set_error(FK_ERR_INVALID, "latent store: bad arguments");
    if (a.rot_dims % 2 || a.rot_dims > a.rot || a.rank > a.rank_ld || a.rank_ld + a.rot > a.ldc)
        return set_error(FK_ERR_INVALID, "latent store: the rotated dimensions must be even and the parts within the cache row");
    if (!a.ring || (a.ring & (a.ring - 1)) || a.rows > a.ring) return set_error(FK_ERR_INVALID, "latent store: the ring must be a power of two of at least `rows`");
    if (a.rot_dims > 8192) return set_error(FK_ERR_UNSUPPORTED, "latent store: at most 8192 rotated dimensions");
    out->func = act == 16 ? (const void*)&latent_store_kernel<uint16_t> : (const void*)&latent_store_kernel<float>;
    out->grid = dim3(a.rows);
    out->block = dim3(kLatBlock, 1, 1);
    out->shmem = a.rot_dims * 4u + 16u;
    out->set_args(a);
    return FK_OK;
}

fk_status plan_latent_attn(const LatentAttnArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "latent attention: act must be 16 or 32");
    if (!a.qa || !a.q || !a.cache || !a.sink || !a.out || !a.offset || !a.rows || !a.heads || !a.window)
        return set_error(FK_ERR_INVALID, "latent attention: bad arguments");
    if (!a.ring || (a.ring & (a.ring - 1)) || (uint64_t)a.window + a.rows - 1u > a.ring)
        return set_error(FK_ERR_INVALID, "latent attention: the ring must be a power of two of at least window + rows - 1");
    if (a.rank_ld % 4 || a.ldc % 4 || a.rank > a.rank_ld || a.rank_ld + a.rot > a.ldc) return set_error(FK_ERR_INVALID, "latent attention: bad row layout");
    if (a.rank > kLatMaxPer * kLatBlock || a.rows > 65535) return set_error(FK_ERR_UNSUPPORTED, "latent attention: latent width at most 2048, rows at most 65535");
    const uint32_t lds = (a.ldc + kLatTile) * 4u;
    if (lds > 60u * 1024u) return set_error(FK_ERR_UNSUPPORTED, "latent attention: cache row too wide");
    out->func = act == 16 ? (const void*)&latent_attn_kernel<uint16_t, uint16_t> : (const void*)&latent_attn_kernel<float, float>;
    out->grid = dim3(a.heads, a.rows);
    out->block = dim3(kLatBlock, 1, 1);
    out->shmem = lds;
    out->set_args(a);
    return FK_OK;
}

}  // namespace fk
