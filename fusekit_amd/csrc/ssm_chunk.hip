// The state-space recurrence of a long portion, chunk by chunk on the matrix cores.
//
// With da_t = -exp(a_log) dt_t and c_t its running sum inside a chunk of 64 tokens,
//     y_t   = sum_(s <= t) exp(c_t - c_s) dt_s (C_t . B_s) x_s  +  exp(c_t) S_in^T C_t  +  D x_t
//     S_out = exp(c_last) S_in + sum_t exp(c_last - c_t) dt_t B_t x_t^T
// three launches: every chunk's own contribution to the state; a pass over the chunks that turns contributions into
// the states the chunks start from (and leaves the final state); every chunk's outputs.
//
// The recurrence is kept in fp32: decays, step sizes and states are fp32, and where such a value is an operand of a
// bf16 matrix instruction it enters as the sum of two bf16 halves (16 bits of mantissa), with fp32 accumulation.  x, B
// and C are bf16 as the convolution left them.
#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

namespace {

typedef __bf16 sc_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float sc_f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t sc_u32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t sc_u32x2_t __attribute__((ext_vector_type(2)));

constexpr uint32_t kL = 64, kTs = kL + 8;   // tokens per chunk, stride of a transposed row

__device__ __forceinline__ sc_f32x4_t mfma(sc_u32x4_t a, sc_u32x4_t b, sc_f32x4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(sc_bf16x8_t, a), __builtin_bit_cast(sc_bf16x8_t, b), c, 0, 0, 0);
}

// dt and the running log decay of the chunk's tokens (one per lane of a wave); tokens past the pass neither decay nor add.
__device__ __forceinline__ void chunk_steps(const SsmChunkArgs& a, uint32_t h, uint32_t t0, uint32_t lane, float& dt, float& cum) {
    const uint32_t t = t0 + lane;
    dt = t < a.rows ? softplus(a.dt[(size_t)t * a.lddt + h] + bf16_bits_to_f32(a.dt_bias[h])) : 0.f;
    cum = -expf(bf16_bits_to_f32(a.a_log[h])) * dt;
#pragma unroll
    for (int o = 1; o < kWave; o <<= 1) {
        const float u = __shfl_up(cum, o, kWave);
        if (lane >= (uint32_t)o) cum += u;
    }
}

__device__ __forceinline__ void split_bf16(float v, uint32_t& hi, uint32_t& lo) {
    hi = f32_to_bf16_bits(v);
    lo = f32_to_bf16_bits(v - bf16_bits_to_f32(hi));
}

// Contribution of one chunk to one head's state: [p][n] = sum_t (w_t x_t[p]) B_t[n].  NS: 16-wide tiles of n per wave.
template <int PT, int NT>
__global__ __launch_bounds__(256) void ssm_chunk_state_kernel(const SsmChunkArgs a) {
    __shared__ __align__(16) uint16_t xh[PT * 16 * kTs], xl[PT * 16 * kTs], bt[NT * 16 * kTs];
    __shared__ float w[kL];
    const uint32_t h = blockIdx.x, chunk = blockIdx.y, t0 = chunk * kL, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const uint32_t l16 = lane & 15u, kq = lane >> 4, inner = a.heads * a.p, g = h / (a.heads / a.groups);
    if (wave == 0) {
        float dt, cum;
        chunk_steps(a, h, t0, lane, dt, cum);
        const float last = __shfl(cum, kWave - 1, kWave);
        w[lane] = expf(last - cum) * dt;
        if (lane == 0) a.decay[(size_t)chunk * a.heads + h] = expf(last);
    }
    __syncthreads();
    const uint32_t live = a.rows - t0 < kL ? a.rows - t0 : kL;
    // four adjacent columns of one token per thread and turn, written transposed
    constexpr uint32_t PC = PT * 4, NC = NT * 4;
    for (uint32_t i = tid; i < kL * PC; i += 256u) {
        const uint32_t t = i / PC, p = (i % PC) * 4u;
        float v[4] = {0.f, 0.f, 0.f, 0.f};
        if (t < live && p < a.p) {
            const float4 x = act_load4(a.xbc + (size_t)(t0 + t) * a.ldx + (size_t)h * a.p + p);
            v[0] = x.x * w[t]; v[1] = x.y * w[t]; v[2] = x.z * w[t]; v[3] = x.w * w[t];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            uint32_t hi, lo;
            split_bf16(v[e], hi, lo);
            xh[(p + e) * kTs + t] = (uint16_t)hi;
            xl[(p + e) * kTs + t] = (uint16_t)lo;
        }
    }
    for (uint32_t i = tid; i < kL * NC; i += 256u) {
        const uint32_t t = i / NC, n = (i % NC) * 4u;
        uint2 v = make_uint2(0u, 0u);
        if (t < live && n < a.n) v = *reinterpret_cast<const uint2*>(a.xbc + (size_t)(t0 + t) * a.ldx + inner + (size_t)g * a.n + n);
        bt[n * kTs + t] = (uint16_t)v.x;
        bt[(n + 1u) * kTs + t] = (uint16_t)(v.x >> 16);
        bt[(n + 2u) * kTs + t] = (uint16_t)v.y;
        bt[(n + 3u) * kTs + t] = (uint16_t)(v.y >> 16);
    }
    __syncthreads();
    // rows n first: a lane ends with four adjacent n of one p
    float* out = a.chunks + (((size_t)chunk * a.heads + h) * a.p) * a.state_ld;
    for (uint32_t nt = wave; nt < NT; nt += 4u) {
        if (nt * 16u >= a.state_ld) break;
        sc_f32x4_t acc[PT];
#pragma unroll
        for (int i = 0; i < PT; ++i) acc[i] = sc_f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (uint32_t k = 0; k < 2; ++k) {
            const sc_u32x4_t b = *reinterpret_cast<const sc_u32x4_t*>(bt + (nt * 16u + l16) * kTs + k * 32u + kq * 8u);
#pragma unroll
            for (int i = 0; i < PT; ++i) {
                acc[i] = mfma(b, *reinterpret_cast<const sc_u32x4_t*>(xh + (i * 16u + l16) * kTs + k * 32u + kq * 8u), acc[i]);
                acc[i] = mfma(b, *reinterpret_cast<const sc_u32x4_t*>(xl + (i * 16u + l16) * kTs + k * 32u + kq * 8u), acc[i]);
            }
        }
#pragma unroll
        for (int i = 0; i < PT; ++i) {
            const uint32_t p = i * 16u + l16;
            if (p < a.p) *reinterpret_cast<float4*>(out + (size_t)p * a.state_ld + nt * 16u + kq * 4u) = make_float4(acc[i][0], acc[i][1], acc[i][2], acc[i][3]);
        }
    }
}

// One thread per four adjacent state elements: walks the chunks, leaves in each chunk's place the state it starts from.
__global__ __launch_bounds__(256) void ssm_chunk_pass_kernel(const SsmChunkArgs a) {
    const uint32_t per_head = a.p * a.state_ld / 4u, i = blockIdx.x * 256u + threadIdx.x, total = a.heads * per_head;
    if (i < total) {
        const uint32_t h = i / per_head, chunks = (a.rows + kL - 1u) / kL;
        float4* st = reinterpret_cast<float4*>(a.state) + i;
        float4 S = *st;
        float4* c = reinterpret_cast<float4*>(a.chunks) + i;
        constexpr uint32_t kAhead = 4;
        for (uint32_t k0 = 0; k0 < chunks; k0 += kAhead) {
            float4 d[kAhead];
            float e[kAhead];
#pragma unroll
            for (uint32_t u = 0; u < kAhead; ++u) {
                const uint32_t k = k0 + u < chunks ? k0 + u : chunks - 1u;
                d[u] = c[(size_t)k * total];
                e[u] = a.decay[(size_t)k * a.heads + h];
            }
#pragma unroll
            for (uint32_t u = 0; u < kAhead; ++u) {
                if (k0 + u >= chunks) break;
                c[(size_t)(k0 + u) * total] = S;
                S.x = fmaf(e[u], S.x, d[u].x); S.y = fmaf(e[u], S.y, d[u].y);
                S.z = fmaf(e[u], S.z, d[u].z); S.w = fmaf(e[u], S.w, d[u].w);
            }
        }
        *st = S;
    }
    // the convolution's history: the last taps - 1 rows of the pass
    const uint32_t keep = a.rows < a.taps - 1u ? a.rows : a.taps - 1u, pos = *a.offset;
    for (uint32_t t = a.rows - keep; t < a.rows; ++t)
        for (uint32_t ch = i; ch < a.channels; ch += gridDim.x * 256u)
            a.hist[(size_t)((pos + t) % a.taps) * a.ldh + ch] = a.u[(size_t)t * a.ldu + ch];
}

// Outputs of one chunk of one head; wave w owns tokens 16 w .. 16 w + 15 (the columns of every product).
template <int PT, int NS>
__global__ __launch_bounds__(256) void ssm_chunk_out_kernel(const SsmChunkArgs a) {
    __shared__ __align__(16) uint16_t xt[PT * 16 * kTs];
    __shared__ float cum_s[kL], dt_s[kL];
    const uint32_t h = blockIdx.x, chunk = blockIdx.y, t0 = chunk * kL, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const uint32_t l16 = lane & 15u, kq = lane >> 4, inner = a.heads * a.p, g = h / (a.heads / a.groups);
    const uint32_t live = a.rows - t0 < kL ? a.rows - t0 : kL;
    if (wave == 0) {
        float dt, cum;
        chunk_steps(a, h, t0, lane, dt, cum);
        cum_s[lane] = cum;
        dt_s[lane] = dt;
    }
    constexpr uint32_t PC = PT * 4;
    for (uint32_t i = tid; i < kL * PC; i += 256u) {
        const uint32_t t = i / PC, p = (i % PC) * 4u;
        uint2 v = make_uint2(0u, 0u);
        if (t < live && p < a.p) v = *reinterpret_cast<const uint2*>(a.xbc + (size_t)(t0 + t) * a.ldx + (size_t)h * a.p + p);
        xt[p * kTs + t] = (uint16_t)v.x;
        xt[(p + 1u) * kTs + t] = (uint16_t)(v.x >> 16);
        xt[(p + 2u) * kTs + t] = (uint16_t)v.y;
        xt[(p + 3u) * kTs + t] = (uint16_t)(v.y >> 16);
    }
    const uint16_t* Brow = a.xbc + inner + (size_t)g * a.n + kq * 8u;
    const uint16_t* Crow = Brow + (size_t)a.groups * a.n;
    const sc_u32x4_t zero = {0u, 0u, 0u, 0u};
    const uint32_t tc = wave * 16u + l16, t_my = t0 + (tc < live ? tc : live - 1u);   // tokens past the pass repeat the last; never stored
    sc_u32x4_t cf[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s)
        cf[s] = (uint32_t)s * 32u + kq * 8u < a.n ? *reinterpret_cast<const sc_u32x4_t*>(Crow + (size_t)t_my * a.ldx + s * 32) : zero;
    // the state the chunk starts from
    sc_f32x4_t y[PT];
    const float* S = a.chunks + (((size_t)chunk * a.heads + h) * a.p) * a.state_ld + kq * 8u;
#pragma unroll
    for (int i = 0; i < PT; ++i) {
        y[i] = sc_f32x4_t{0.f, 0.f, 0.f, 0.f};
        const uint32_t p = i * 16u + l16, pc = p < a.p ? p : a.p - 1u;
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            if ((uint32_t)s * 32u >= a.state_ld) break;
            const float4 v0 = *reinterpret_cast<const float4*>(S + (size_t)pc * a.state_ld + s * 32), v1 = *reinterpret_cast<const float4*>(S + (size_t)pc * a.state_ld + s * 32 + 4);
            const float v[8] = {v0.x, v0.y, v0.z, v0.w, v1.x, v1.y, v1.z, v1.w};
            sc_u32x4_t hi, lo;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                hi[e] = pack_bf16(v[2 * e], v[2 * e + 1]);
                lo[e] = pack_bf16(v[2 * e] - bf16_lo(hi[e]), v[2 * e + 1] - bf16_hi(hi[e]));
            }
            y[i] = mfma(hi, cf[s], y[i]);
            y[i] = mfma(lo, cf[s], y[i]);
        }
    }
    __syncthreads();
    const float ct = cum_s[tc], et = expf(ct);
#pragma unroll
    for (int i = 0; i < PT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) y[i][r] *= et;
    // tokens of the chunk up to this wave's, 32 at a time
    for (uint32_t s0 = 0; s0 <= wave * 16u; s0 += 32u) {
        sc_u32x4_t mh, ml;
#pragma unroll
        for (int b = 0; b < 2; ++b) {
            const uint32_t sr = s0 + b * 16u + l16, s_my = t0 + (sr < live ? sr : live - 1u);
            sc_f32x4_t gt = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < NS; ++s) {
                const sc_u32x4_t bf = (uint32_t)s * 32u + kq * 8u < a.n ? *reinterpret_cast<const sc_u32x4_t*>(Brow + (size_t)s_my * a.ldx + s * 32) : zero;
                gt = mfma(bf, cf[s], gt);
            }
            float m[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const uint32_t s = s0 + b * 16u + kq * 4u + (uint32_t)r;
                m[r] = s <= tc ? gt[r] * expf(ct - cum_s[s]) * dt_s[s] : 0.f;   // dt is 0 past the pass
            }
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const uint32_t hi = pack_bf16(m[2 * e], m[2 * e + 1]);
                mh[b * 2 + e] = hi;
                ml[b * 2 + e] = pack_bf16(m[2 * e] - bf16_lo(hi), m[2 * e + 1] - bf16_hi(hi));
            }
        }
#pragma unroll
        for (int i = 0; i < PT; ++i) {
            const uint16_t* p = xt + (i * 16u + l16) * kTs + s0 + kq * 4u;
            const sc_u32x2_t x0 = *reinterpret_cast<const sc_u32x2_t*>(p), x1 = *reinterpret_cast<const sc_u32x2_t*>(p + 16);
            const sc_u32x4_t xf = {x0[0], x0[1], x1[0], x1[1]};
            y[i] = mfma(xf, mh, y[i]);
            y[i] = mfma(xf, ml, y[i]);
        }
    }
    if (tc >= live) return;
    const float D = bf16_bits_to_f32(a.d[h]);
    uint16_t* out = a.y + (size_t)(t0 + tc) * a.ldy + (size_t)h * a.p + kq * 4u;
#pragma unroll
    for (int i = 0; i < PT; ++i) {
        const uint32_t p = i * 16u + kq * 4u;
        if (p >= a.p) continue;
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = fmaf(D, bf16_bits_to_f32(xt[(p + r) * kTs + tc]), y[i][r]);
        *reinterpret_cast<uint2*>(out + i * 16) = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]));
    }
}

// Smallest compiled widths that hold p values and n state rows.
struct ChunkForm {
    uint32_t p, n;
    const void *state, *out;
};
#define FK_CHUNK_FORM(PT, NS) {PT * 16, NS * 32, (const void*)&ssm_chunk_state_kernel<PT, NS * 2>, (const void*)&ssm_chunk_out_kernel<PT, NS>}
const ChunkForm kChunkForms[] = {FK_CHUNK_FORM(2, 2), FK_CHUNK_FORM(2, 4), FK_CHUNK_FORM(4, 2), FK_CHUNK_FORM(4, 4), FK_CHUNK_FORM(8, 4), FK_CHUNK_FORM(4, 8), FK_CHUNK_FORM(8, 8)};

const ChunkForm* chunk_form(uint32_t p, uint32_t n) {
    for (const ChunkForm& f : kChunkForms)
        if (p <= f.p && n <= f.n) return &f;
    return nullptr;
}

}  // namespace

bool ssm_chunk_supported(uint32_t heads, uint32_t p, uint32_t n) { return p % 4 == 0 && n % 8 == 0 && (heads * p) % 8 == 0 && chunk_form(p, n); }

fk_status plan_ssm_chunk(const SsmChunkArgs& a, Launch* out) {
    if (!a.xbc || !a.dt || !a.dt_bias || !a.a_log || !a.d || !a.state || !a.y || !a.u || !a.hist || !a.offset || !a.chunks || !a.decay || !a.rows || !a.taps)
        return set_error(FK_ERR_INVALID, "ssm chunks: bad arguments");
    if (!a.groups || a.heads % a.groups || a.state_ld % 64 || a.state_ld < a.n) return set_error(FK_ERR_INVALID, "ssm chunks: bad shape");
    if (!ssm_chunk_supported(a.heads, a.p, a.n) || a.ldx % 8 || a.ldy % 4)
        return set_error(FK_ERR_UNSUPPORTED, "ssm chunks: vdim a multiple of 4 up to 128, state of 8 up to 256, heads * vdim of 8");
    const ChunkForm* f = chunk_form(a.p, a.n);
    const uint32_t chunks = (a.rows + kL - 1) / kL;
    if (chunks > 65535) return set_error(FK_ERR_UNSUPPORTED, "ssm chunks: too many rows");
    out->func = f->state;
    out->grid = dim3(a.heads, chunks, 1);
    out->block = dim3(256, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    Launch pass;
    pass.func = (const void*)&ssm_chunk_pass_kernel;
    pass.grid = dim3((a.heads * a.p * (a.state_ld / 4) + 255) / 256, 1, 1);
    pass.block = dim3(256, 1, 1);
    pass.set_args(a);
    Launch fin;
    fin.func = f->out;
    fin.grid = dim3(a.heads, chunks, 1);
    fin.block = dim3(256, 1, 1);
    fin.set_args(a);
    out->then.push_back(pass);
    out->then.push_back(fin);
    return FK_OK;
}

}  // namespace fk
