// Latent attention of a few query rows on the matrix cores: the window is split over workgroups, the partial rows are
// combined afterwards (by the product with W_uv that consumes them, or by latent_combine_kernel).
//
// All heads share the cached latents, so a workgroup takes 16 heads of one query row and walks its positions 64 at a
// time.  A wave loads the rows of 16 positions once, straight into the operand layout of
//     S^T[position, head] = K . Q^T        (16 x 16 x 32, K: [latent | rotated key part])
// and writes the latents, transposed, to LDS for
//     O^T[latent, head] += C^T[latent, position] . P^T[position, head]
// two neighbouring positions exchanging halves so that whole 32-bit words are written; latents beyond 256 go in a second
// turn through the same LDS.  A lane owns one head in both products, so the running maximum and the rescale stay in it.
#include "act_device.hpp"
#include "layered.hpp"
#include "split_device.hpp"

namespace fk {

namespace {

typedef __bf16 ls_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float ls_f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t ls_u32x4_t __attribute__((ext_vector_type(4)));

constexpr uint32_t kLsTile = 64, kLsCs = kLsTile + 8, kLsHalf = 256;

__device__ __forceinline__ ls_f32x4_t ls_mfma(ls_u32x4_t a, ls_u32x4_t b, ls_f32x4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(ls_bf16x8_t, a), __builtin_bit_cast(ls_bf16x8_t, b), c, 0, 0, 0);
}

// S: steps of 32 over the cache row; HALVES: turns of 256 latents.
template <int S, int HALVES>
__global__ __launch_bounds__(256) void latent_split_kernel(const LatentSplitArgs a) {
    constexpr uint32_t QS = S * 32u + 8u;
    __shared__ __align__(16) uint16_t qs[16 * QS];
    __shared__ __align__(16) uint16_t ct[kLsHalf * kLsCs];
    __shared__ __align__(16) uint16_t ps[16 * kLsCs];
    __shared__ float wmax[4][16], wsum[4][16];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, kq = lane >> 4;
    const uint32_t split = blockIdx.x, h0 = blockIdx.y * 16u, r = blockIdx.z;
    const uint32_t pos = *a.offset + r, lo = pos + 1u > a.window ? pos + 1u - a.window : 0u;
    const uint32_t j0 = lo + split * a.span, j1 = j0 + a.span < pos + 1u ? j0 + a.span : pos + 1u;
    const uint32_t pl = a.rank_ld + 2u;
    float* part = a.part + ((size_t)r * a.splits + split) * a.heads * pl;
    if (j0 > pos) {   // nothing of the window here
        const uint32_t hs = a.heads - h0 < 16u ? a.heads - h0 : 16u;
        for (uint32_t i = tid; i < hs * pl; i += 256u) part[(size_t)h0 * pl + i] = i % pl == a.rank_ld ? -INFINITY : 0.f;
        return;
    }
    auto load_k = [&](uint32_t j, ls_u32x4_t* k) __attribute__((always_inline)) {
        uint32_t p = j + wave * 16u + l16;
        p = p < j1 ? p : j1 - 1u;
        const uint16_t* row = a.cache + (size_t)(p & (a.ring - 1u)) * a.ldc + kq * 8u;
#pragma unroll
        for (int s = 0; s < S; ++s) k[s] = (uint32_t)s * 32u < a.ldc ? *reinterpret_cast<const ls_u32x4_t*>(row + s * 32) : ls_u32x4_t{0u, 0u, 0u, 0u};
    };
    ls_u32x4_t k[S];
    load_k(j0, k);
    for (uint32_t i = tid; i < 16u * (S * 4u); i += 256u) {   // [carried query | rotated part | zeros], 16 bytes at a time
        const uint32_t h = i / (S * 4u), c = (i % (S * 4u)) * 8u;
        ls_u32x4_t v = {0u, 0u, 0u, 0u};
        if (h0 + h < a.heads && c < a.ldc)
            v = c < a.rank_ld ? *reinterpret_cast<const ls_u32x4_t*>(a.qa + ((size_t)r * a.heads + h0 + h) * a.rank_ld + c)
                              : *reinterpret_cast<const ls_u32x4_t*>(a.q + (size_t)r * a.ldq + (size_t)(h0 + h) * a.hs + a.dim_ld + c - a.rank_ld);
        *reinterpret_cast<ls_u32x4_t*>(qs + h * QS + c) = v;
    }
    __syncthreads();
    if (a.tab) {   // the queries arrive unrotated
        const uint32_t half = a.rot_dims / 2u;
        for (uint32_t i = tid; i < 16u * half; i += 256u) {
            const uint32_t h = i / half, d = i - h * half;
            uint16_t* q = qs + h * QS + a.rank_ld + d;
            const float u = act_load(q), v = act_load(q + half), cs = a.tab[2 * d], sn = a.tab[2 * d + 1];
            act_store(q, u * cs - v * sn);
            act_store(q + half, v * cs + u * sn);
        }
        __syncthreads();
    }

    const float scale2 = a.scale * 1.4426950408889634f;
    float m_run = -INFINITY, l_run = 0.f;
    ls_f32x4_t o[HALVES][4];
#pragma unroll
    for (int f = 0; f < HALVES; ++f)
#pragma unroll
        for (int t = 0; t < 4; ++t) o[f][t] = ls_f32x4_t{0.f, 0.f, 0.f, 0.f};

    for (uint32_t j = j0; j < j1; j += kLsTile) {
        ls_f32x4_t s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < S; ++i) s = ls_mfma(k[i], *reinterpret_cast<const ls_u32x4_t*>(qs + l16 * QS + i * 32 + kq * 8u), s);
        float sv[4], mt = -INFINITY;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            sv[e] = j + wave * 16u + kq * 4u + (uint32_t)e < j1 ? s[e] * scale2 : -INFINITY;
            mt = fmaxf(mt, sv[e]);
        }
        mt = fmaxf(mt, __shfl_xor(mt, 16, kWave));
        mt = fmaxf(mt, __shfl_xor(mt, 32, kWave));
        if (kq == 0) wmax[wave][l16] = mt;
        // the latents of this wave's positions, transposed: the even lane of a pair writes dimensions 0..3, the odd 4..7
        auto transpose = [&](int f) __attribute__((always_inline)) {
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                if (f * 8 + i >= S) break;
                const ls_u32x4_t v = k[f * 8 + i < S ? f * 8 + i : 0];
                ls_u32x4_t w;
#pragma unroll
                for (int e = 0; e < 4; ++e) w[e] = (uint32_t)__builtin_amdgcn_update_dpp(0, (int)v[e], 0xB1, 0xF, 0xF, true);   // lane ^ 1
                const bool odd = l16 & 1u;
                const uint32_t a0 = odd ? w[2] : v[0], a1 = odd ? w[3] : v[1], b0 = odd ? v[2] : w[0], b1 = odd ? v[3] : w[1];
                uint16_t* q = ct + (i * 32u + kq * 8u + (odd ? 4u : 0u)) * kLsCs + wave * 16u + (l16 & ~1u);
                *reinterpret_cast<uint32_t*>(q) = (a0 & 0xffffu) | (b0 << 16);
                *reinterpret_cast<uint32_t*>(q + kLsCs) = (a0 >> 16) | (b0 & 0xffff0000u);
                *reinterpret_cast<uint32_t*>(q + 2 * kLsCs) = (a1 & 0xffffu) | (b1 << 16);
                *reinterpret_cast<uint32_t*>(q + 3 * kLsCs) = (a1 >> 16) | (b1 & 0xffff0000u);
            }
        };
        transpose(0);
        __syncthreads();
        const float m_tile = fmaxf(fmaxf(wmax[0][l16], wmax[1][l16]), fmaxf(wmax[2][l16], wmax[3][l16]));
        const float m_new = fmaxf(m_run, m_tile), alpha = __builtin_amdgcn_exp2f(m_run - m_new);   // a tile holds a visible position
        float p[4], sum = 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            p[e] = __builtin_amdgcn_exp2f(sv[e] - m_new);
            sum += p[e];
        }
        *reinterpret_cast<uint2*>(ps + l16 * kLsCs + wave * 16u + kq * 4u) = make_uint2(pack_bf16(p[0], p[1]), pack_bf16(p[2], p[3]));
        sum += __shfl_xor(sum, 16, kWave);
        sum += __shfl_xor(sum, 32, kWave);
        if (kq == 0) wsum[wave][l16] = sum;
        m_run = m_new;
#pragma unroll
        for (int f = 0; f < HALVES; ++f)
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int e = 0; e < 4; ++e) o[f][t][e] *= alpha;
        __syncthreads();
        l_run = l_run * alpha + ((wsum[0][l16] + wsum[1][l16]) + (wsum[2][l16] + wsum[3][l16]));
        ls_u32x4_t pf[2];
#pragma unroll
        for (int u = 0; u < 2; ++u) pf[u] = *reinterpret_cast<const ls_u32x4_t*>(ps + l16 * kLsCs + u * 32 + kq * 8u);
#pragma unroll
        for (int f = 0; f < HALVES; ++f) {
            if (f > 0) {
                __syncthreads();
                transpose(f);
                __syncthreads();
            }
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const uint32_t c = (wave * 4u + t) * 16u;
                if (f * kLsHalf + c >= a.rank_ld) break;
#pragma unroll
                for (int u = 0; u < 2; ++u)
                    o[f][t] = ls_mfma(*reinterpret_cast<const ls_u32x4_t*>(ct + (c + l16) * kLsCs + u * 32 + kq * 8u), pf[u], o[f][t]);
            }
        }
        if (j + kLsTile < j1) {
            load_k(j + kLsTile, k);
            __syncthreads();
        }
    }
    if (h0 + l16 >= a.heads) return;
    float* out = part + (size_t)(h0 + l16) * pl;
#pragma unroll
    for (int f = 0; f < HALVES; ++f)
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            const uint32_t c = f * kLsHalf + (wave * 4u + t) * 16u + kq * 4u;
            if (c < a.rank_ld) {   // rows of rank_ld + 2 floats: 8-byte aligned
                *reinterpret_cast<float2*>(out + c) = make_float2(o[f][t][0], o[f][t][1]);
                *reinterpret_cast<float2*>(out + c + 2) = make_float2(o[f][t][2], o[f][t][3]);
            }
        }
    if (wave == 0 && kq == 0) {
        out[a.rank_ld] = m_run * 0.6931471805599453f;
        out[a.rank_ld + 1u] = l_run;
    }
}

// Partial rows -> the latent sum of one (head, row), with the sink in the denominator.
__global__ __launch_bounds__(256) void latent_combine_kernel(const LatentSplitArgs a) {
    __shared__ float w[kMaxSplits];
    const uint32_t h = blockIdx.x, r = blockIdx.y, pl = a.rank_ld + 2u;
    const float* p = a.part + ((size_t)r * a.splits * a.heads + h) * pl;
    const size_t ss = (size_t)a.heads * pl;
    split_weights(p + a.rank_ld, ss, a.splits, bf16_bits_to_f32(a.sink[h]), w);
    __syncthreads();
    for (uint32_t c = threadIdx.x * 2u; c < a.rank_ld; c += 512u) {
        float v0 = 0.f, v1 = 0.f;
#pragma unroll 8
        for (uint32_t s = 0; s < a.splits; ++s) {
            const float2 q = *reinterpret_cast<const float2*>(p + s * ss + c);
            v0 = fmaf(w[s], q.x, v0);
            v1 = fmaf(w[s], q.y, v1);
        }
        *reinterpret_cast<uint32_t*>(a.out + ((size_t)r * a.heads + h) * a.rank_ld + c) = pack_bf16(v0, v1);
    }
}

struct LsForm {
    uint32_t ldc, rank;
    const void* f;
};
const LsForm kLsForms[] = {{4 * 32, 256, (const void*)&latent_split_kernel<4, 1>}, {10 * 32, 256, (const void*)&latent_split_kernel<10, 1>},
                           {18 * 32, 512, (const void*)&latent_split_kernel<18, 2>}};

}  // namespace

bool latent_split_supported(uint32_t rank_ld, uint32_t ldc) {
    if (rank_ld % 32 || ldc % 32) return false;
    for (const LsForm& f : kLsForms)
        if (ldc <= f.ldc && rank_ld <= f.rank) return true;
    return false;
}

fk_status plan_latent_split(LatentSplitArgs& a, bool combine, Launch* out) {
    if (!a.qa || !a.q || !a.cache || !a.part || !a.offset || !a.rows || !a.heads || !a.window || (combine && (!a.out || !a.sink)))
        return set_error(FK_ERR_INVALID, "latent split: bad arguments");
    if (!a.ring || (a.ring & (a.ring - 1)) || (uint64_t)a.window + a.rows - 1u > a.ring) return set_error(FK_ERR_INVALID, "latent split: ring too small");
    if (!a.splits || !a.span || a.span % kLsTile || (uint64_t)a.splits * a.span < a.window) return set_error(FK_ERR_INVALID, "latent split: the splits must cover the window in whole tiles");
    if (a.rot_dims % 2 || a.rot_dims > a.rot || a.rank_ld + a.rot > a.ldc) return set_error(FK_ERR_INVALID, "latent split: bad row layout");
    if (!latent_split_supported(a.rank_ld, a.ldc)) return set_error(FK_ERR_UNSUPPORTED, "latent split: cache rows of at most 512 + 64 elements");
    if (a.rows > 65535 || a.splits > kMaxSplits) return set_error(FK_ERR_UNSUPPORTED, "latent split: too many rows or splits");
    for (const LsForm& f : kLsForms)
        if (a.ldc <= f.ldc && a.rank_ld <= f.rank) {
            out->func = f.f;
            break;
        }
    out->grid = dim3(a.splits, (a.heads + 15) / 16, a.rows);
    out->block = dim3(256, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    if (combine) {
        Launch c;
        c.func = (const void*)&latent_combine_kernel;
        c.grid = dim3(a.heads, a.rows, 1);
        c.block = dim3(256, 1, 1);
        c.set_args(a);
        out->then.push_back(c);
    }
    return FK_OK;
}

}  // namespace fk
