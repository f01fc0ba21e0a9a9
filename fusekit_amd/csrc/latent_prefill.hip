// Sliding-window attention of a portion of a prompt, with keys and values formed from the cached latents once per pass
// (they are shared by the rows of the pass), on the matrix cores.
//
// One block = one head x 64 or 128 query rows, a 16- or 32-row tile per wave; the four waves walk the same 64-position
// steps, whose key rows [unrotated part | rotated part shared by the heads] and transposed value rows are staged in
// LDS, the next step being on its way in registers.  Per step a wave computes
//     S^T[kv, q] = K[kv, :] . Q[q, :]        then        O^T[d, q] += V^T[d, kv] . P^T[kv, q]
// with 16 x 16 x 32 instructions: a lane owns one query (column) in both, and the score registers are the second
// product's right operand as they lie, because the order of kv inside an instruction is free as long as both operands
// agree (lane group g holds kv 4 g .. 4 g + 3 of two neighbouring 16-position tiles).
// Positions are counted from the first one the pass can see: t = position - *offset + window - 1; row r of the pass sees
// t in [r, r + window - 1], from the start of the sequence.  The sink joins the denominator at the end.
#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

namespace {

typedef __bf16 lp_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float lp_f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t lp_u32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t lp_u32x2_t __attribute__((ext_vector_type(2)));

constexpr uint32_t kLpStep = 64, kLpVs = kLpStep + 8;

// KD: steps of 32 over the query / key width; VD: 16-wide tiles of the value width; QT: query tiles per wave.
template <int KD, int VD, int QT>
__global__ __launch_bounds__(256) void latent_prefill_kernel(const LatentPrefillArgs a) {
    constexpr uint32_t KS = KD * 32u + 8u;                     // staged key row, padded
    constexpr int KP = KD * 4, NK = (64 * KP + 255) / 256;     // 16-byte pieces per key row, per thread
    constexpr int NV = (VD * 16 * 8 + 255) / 256;
    __shared__ __align__(16) uint16_t kt[kLpStep * KS];
    __shared__ __align__(16) uint16_t vt[VD * 16 * kLpVs];

    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, kq = lane >> 4;
    const uint32_t h = blockIdx.x % a.heads, tiles = (a.rows + 64u * QT - 1u) / (64u * QT);
    const uint32_t tile = tiles - 1u - blockIdx.x / a.heads, r0 = tile * 64u * QT;
    const uint32_t r_end = r0 + 64u * QT < a.rows ? r0 + 64u * QT : a.rows;   // one past the block's last row
    const uint32_t pos0 = *a.offset, W1 = a.window - 1u;
    const uint32_t t_min = pos0 < W1 ? W1 - pos0 : 0u;                       // the sequence starts here
    const uint32_t t_lo = (r0 > t_min ? r0 : t_min) & ~7u, t_end = r_end + W1;

    // queries: lane (q = l16, kq) holds 8 elements at 32 s + 8 kq
    const uint32_t rq0 = r0 + wave * 16u * QT;
    lp_u32x4_t qf[QT][KD];
    uint32_t row[QT];
#pragma unroll
    for (int q = 0; q < QT; ++q) {
        row[q] = rq0 + (uint32_t)q * 16u + l16;
        const uint32_t rr = row[q] < a.rows ? row[q] : a.rows - 1u;   // rows past the pass repeat its last one; never stored
        const uint16_t* p = a.q + (size_t)rr * a.ldq + (size_t)h * (a.dim_ld + a.rot_ld) + kq * 8u;
#pragma unroll
        for (int s = 0; s < KD; ++s)
            qf[q][s] = (uint32_t)s * 32u < a.dim_ld + a.rot_ld ? *reinterpret_cast<const lp_u32x4_t*>(p + s * 32) : lp_u32x4_t{0u, 0u, 0u, 0u};
    }

    lp_u32x4_t kr[NK], vr[NV];
    const uint32_t kp_dim = a.dim_ld / 8u, kp_all = (a.dim_ld + a.rot_ld) / 8u;
    auto fetch = [&](uint32_t t0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < NK; ++i) {
            const uint32_t idx = tid + 256u * i, j = idx / KP, pc = idx % KP;
            uint32_t t = t0 + j;
            t = t < t_end ? t : t_end - 1u;
            lp_u32x4_t v = {0u, 0u, 0u, 0u};
            if (idx < 64u * KP) {
                if (pc < kp_dim) v = *reinterpret_cast<const lp_u32x4_t*>(a.k + (size_t)t * a.ldk + (size_t)h * a.dim_ld + pc * 8u);
                else if (pc < kp_all)
                    v = *reinterpret_cast<const lp_u32x4_t*>(a.cache + (size_t)((pos0 + t - W1) & (a.ring - 1u)) * a.ldc + a.rank_ld + (pc - kp_dim) * 8u);
            }
            kr[i] = v;
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const uint32_t idx = tid + 256u * i, d = idx >> 3, pc = idx & 7u;
            lp_u32x4_t v = {0u, 0u, 0u, 0u};
            if (d < a.vdim_ld && d < VD * 16u) v = *reinterpret_cast<const lp_u32x4_t*>(a.vt + ((size_t)h * a.vdim_ld + d) * a.ldv + t0 + pc * 8u);
            vr[i] = v;
        }
    };
    auto stage = [&]() __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < NK; ++i) {
            const uint32_t idx = tid + 256u * i;
            if (idx < 64u * KP) *reinterpret_cast<lp_u32x4_t*>(kt + (idx / KP) * KS + (idx % KP) * 8u) = kr[i];
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const uint32_t idx = tid + 256u * i;
            if ((idx >> 3) < VD * 16u) *reinterpret_cast<lp_u32x4_t*>(vt + (idx >> 3) * kLpVs + (idx & 7u) * 8u) = vr[i];
        }
    };

    const float scale2 = a.scale * 1.4426950408889634f;
    float m_run[QT], l_run[QT];
    lp_f32x4_t o[QT][VD];
#pragma unroll
    for (int q = 0; q < QT; ++q) {
        m_run[q] = -INFINITY;
        l_run[q] = 0.f;
#pragma unroll
        for (int d = 0; d < VD; ++d) o[q][d] = lp_f32x4_t{0.f, 0.f, 0.f, 0.f};
    }

    fetch(t_lo);
    for (uint32_t t0 = t_lo; t0 < t_end; t0 += kLpStep) {
        __syncthreads();
        stage();
        __syncthreads();
        if (t0 + kLpStep < t_end) fetch(t0 + kLpStep);

        lp_f32x4_t s[QT][4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
#pragma unroll
            for (int q = 0; q < QT; ++q) s[q][j] = lp_f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int d = 0; d < KD; ++d) {
                const lp_u32x4_t kf = *reinterpret_cast<const lp_u32x4_t*>(kt + (j * 16u + l16) * KS + d * 32u + kq * 8u);
#pragma unroll
                for (int q = 0; q < QT; ++q)
                    s[q][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(lp_bf16x8_t, kf), __builtin_bit_cast(lp_bf16x8_t, qf[q][d]), s[q][j], 0, 0, 0);
            }
        }
        uint32_t pk[QT][8];   // 16 probabilities per lane and query tile, in register order
#pragma unroll
        for (int q = 0; q < QT; ++q) {
            const uint32_t first = rq0 + (uint32_t)q * 16u;   // the tile's rows: first .. first + 15
            const bool whole = t0 >= first + 15u && t0 >= t_min && t0 + kLpStep - 1u <= first + W1;
            const uint32_t lo = row[q] > t_min ? row[q] : t_min, hi = row[q] + W1;
            float sv[16], mt = -INFINITY;
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    float v = s[q][j][r] * scale2;
                    if (!whole) {
                        const uint32_t t = t0 + (uint32_t)(j * 16 + r) + kq * 4u;
                        if (t < lo || t > hi) v = -INFINITY;
                    }
                    sv[j * 4 + r] = v;
                    mt = fmaxf(mt, v);
                }
            mt = fmaxf(mt, __shfl_xor(mt, 16, kWave));
            mt = fmaxf(mt, __shfl_xor(mt, 32, kWave));
            // the reference moves only when a step's maximum has outgrown it by 2^8: accumulators are rescaled rarely
            const bool grow = mt > m_run[q] + 8.0f;
            const float m_new = grow ? mt : m_run[q], m_ref = m_new == -INFINITY ? 0.f : m_new;
            const float alpha = grow ? __builtin_amdgcn_exp2f(m_run[q] - m_ref) : 1.0f;
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const float p0 = __builtin_amdgcn_exp2f(sv[2 * i] - m_ref), p1 = __builtin_amdgcn_exp2f(sv[2 * i + 1] - m_ref);
                sum += p0 + p1;
                pk[q][i] = pack_bf16(p0, p1);
            }
            l_run[q] = l_run[q] * alpha + sum;
            m_run[q] = m_new;
            if (__builtin_amdgcn_ballot_w64(alpha != 1.0f) != 0) {
#pragma unroll
                for (int d = 0; d < VD; ++d)
#pragma unroll
                    for (int r = 0; r < 4; ++r) o[q][d][r] *= alpha;
            }
        }
#pragma unroll
        for (int c = 0; c < 2; ++c)
#pragma unroll
            for (int d = 0; d < VD; ++d) {
                const uint16_t* p = vt + (d * 16u + l16) * kLpVs + c * 32u + kq * 4u;
                const lp_u32x2_t v0 = *reinterpret_cast<const lp_u32x2_t*>(p), v1 = *reinterpret_cast<const lp_u32x2_t*>(p + 16);
                const lp_u32x4_t vf = {v0[0], v0[1], v1[0], v1[1]};
#pragma unroll
                for (int q = 0; q < QT; ++q) {
                    const lp_u32x4_t pf = {pk[q][c * 4], pk[q][c * 4 + 1], pk[q][c * 4 + 2], pk[q][c * 4 + 3]};
                    o[q][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(lp_bf16x8_t, vf), __builtin_bit_cast(lp_bf16x8_t, pf), o[q][d], 0, 0, 0);
                }
            }
    }

    const float sink = bf16_bits_to_f32(a.sink[h]) * 1.4426950408889634f;
#pragma unroll
    for (int q = 0; q < QT; ++q) {
        float l = l_run[q];
        l += __shfl_xor(l, 16, kWave);
        l += __shfl_xor(l, 32, kWave);
        const float top = fmaxf(m_run[q], sink), e = __builtin_amdgcn_exp2f(m_run[q] - top);
        const float f = e / (l * e + __builtin_amdgcn_exp2f(sink - top));
        if (row[q] >= a.rows) continue;
        uint16_t* out = a.out + (size_t)row[q] * a.ldo + (size_t)h * a.vdim_ld + kq * 4u;
#pragma unroll
        for (int d = 0; d < VD; ++d)
            if (d * 16u < a.vdim_ld)
                *reinterpret_cast<uint2*>(out + d * 16) = make_uint2(pack_bf16(o[q][d][0] * f, o[q][d][1] * f), pack_bf16(o[q][d][2] * f, o[q][d][3] * f));
    }
}

struct LpForm {
    uint32_t kd, vd;
    const void *one, *two;
};
#define FK_LP_FORM(KD, VD) {KD, VD, (const void*)&latent_prefill_kernel<KD, VD, 1>, (const void*)&latent_prefill_kernel<KD, VD, 2>}
const LpForm kLpForms[] = {FK_LP_FORM(2, 4), FK_LP_FORM(4, 4), FK_LP_FORM(4, 8), FK_LP_FORM(6, 8), FK_LP_FORM(8, 8),
                           {8, 16, (const void*)&latent_prefill_kernel<8, 16, 1>, nullptr}};   // two tiles would not fit the registers

const LpForm* lp_form(uint32_t dim_ld, uint32_t rot_ld, uint32_t vdim_ld) {
    for (const LpForm& f : kLpForms)
        if (dim_ld + rot_ld <= f.kd * 32u && vdim_ld <= f.vd * 16u) return &f;
    return nullptr;
}

}  // namespace

bool latent_prefill_supported(uint32_t dim_ld, uint32_t rot_ld, uint32_t vdim_ld) { return lp_form(dim_ld, rot_ld, vdim_ld) != nullptr; }

fk_status plan_latent_prefill(const LatentPrefillArgs& a, Launch* out) {
    if (!a.q || !a.k || !a.vt || !a.cache || !a.sink || !a.out || !a.offset || !a.rows || !a.heads || !a.window)
        return set_error(FK_ERR_INVALID, "latent prefill: bad arguments");
    if (a.dim_ld % 32 || a.rot_ld % 32 || a.vdim_ld % 32 || a.ldq % 8 || a.ldk % 8 || a.ldv % 8 || a.ldc % 8 || a.rank_ld % 8 || a.ldo % 4)
        return set_error(FK_ERR_INVALID, "latent prefill: head parts must be padded to 32, rows to 8 elements");
    if (!a.ring || (a.ring & (a.ring - 1)) || (uint64_t)a.window + a.rows - 1u > a.ring) return set_error(FK_ERR_INVALID, "latent prefill: ring too small");
    if ((uint64_t)a.window - 1 + a.rows + kLpStep > a.ldv) return set_error(FK_ERR_INVALID, "latent prefill: ldv must cover a step past the last position");
    const LpForm* f = lp_form(a.dim_ld, a.rot_ld, a.vdim_ld);
    if (!f) return set_error(FK_ERR_UNSUPPORTED, "latent prefill: head widths beyond 256");
    // two tiles per wave share every staged key; one where that leaves compute units without a block
    const bool two = f->two && (uint64_t)((a.rows + 127) / 128) * a.heads >= 512;
    const uint64_t g = (uint64_t)((a.rows + (two ? 127 : 63)) / (two ? 128 : 64)) * a.heads;
    if (g > 0x7fffffffull) return set_error(FK_ERR_UNSUPPORTED, "latent prefill: too many blocks");
    out->func = two ? f->two : f->one;
    out->grid = dim3((uint32_t)g, 1, 1);
    out->block = dim3(256, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    return FK_OK;
}

}  // namespace fk
