// State-space mixer with one scalar decay per head (Mamba-2): the short causal convolution and the recurrence
//     S <- a S + d (B (x) x),   y = C . S + D x,   d = softplus(dt + bias), a = exp(-d exp(a_log))
// per token, with S in fp32.  The state of a head is stored as [vdim][state, padded]: sixteen lanes share one value column and
// hold four adjacent state rows each, so a step's reduction stays inside a row of sixteen lanes and the state of a
// column moves as whole 16-byte words.
#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

namespace {

// A thread owns one column and walks kConvRows rows, its window of inputs and its weights in registers (up to kConvTaps).
constexpr uint32_t kConvRows = 16, kConvTaps = 4;
template <typename T>
__global__ __launch_bounds__(256) void ssm_conv_rows_kernel(const SsmConvArgs a) {
    const uint32_t c = (blockIdx.x * 256u + threadIdx.x) * 4u, r0 = blockIdx.y * kConvRows;
    if (c >= a.channels) return;
    const uint32_t pos0 = *a.offset;
    const T* u = reinterpret_cast<const T*>(a.u) + c;
    const T* hist = reinterpret_cast<const T*>(a.hist) + c;
    float w[kConvTaps][4], x[kConvTaps][4], b[4];
#pragma unroll
    for (uint32_t k = 0; k < kConvTaps; ++k)   // right-aligned: the last entry meets the current row
#pragma unroll
        for (uint32_t e = 0; e < 4; ++e) w[k][e] = k + a.taps >= kConvTaps ? bf16_bits_to_f32(a.w[(size_t)(c + e) * a.taps + k + a.taps - kConvTaps]) : 0.f;
#pragma unroll
    for (uint32_t e = 0; e < 4; ++e) b[e] = a.b ? bf16_bits_to_f32(a.b[c + e]) : 0.f;
    auto input = [&](int32_t r) __attribute__((always_inline)) {   // row r of the pass; before it: the history, zeros before the start
        if (r >= 0) return act_load4(u + (size_t)r * a.ldu);
        const int32_t p = (int32_t)pos0 + r;
        if (p < 0 || -r >= (int32_t)a.taps) return make_float4(0.f, 0.f, 0.f, 0.f);
        return act_load4(hist + (size_t)((uint32_t)p % a.taps) * a.ldh);
    };
    auto put = [&](float (&d)[4], float4 v) __attribute__((always_inline)) { d[0] = v.x; d[1] = v.y; d[2] = v.z; d[3] = v.w; };
#pragma unroll
    for (uint32_t k = 0; k + 1u < kConvTaps; ++k) put(x[k + 1], input((int32_t)(r0 + k) - (int32_t)(kConvTaps - 1u)));
    if (a.update && r0 == 0u) {   // these threads alone read the history of their columns, and have done so
        for (uint32_t t = a.rows - (a.taps - 1u); t < a.rows; ++t)
            act_store4(reinterpret_cast<T*>(a.hist) + (size_t)((pos0 + t) % a.taps) * a.ldh + c, act_load4(u + (size_t)t * a.ldu));
    }
    T* y = reinterpret_cast<T*>(a.y) + c;
#pragma unroll
    for (uint32_t i = 0; i < kConvRows; ++i) {
        const uint32_t r = r0 + i;
        if (r >= a.rows) break;
#pragma unroll
        for (uint32_t k = 0; k + 1u < kConvTaps; ++k)
#pragma unroll
            for (uint32_t e = 0; e < 4; ++e) x[k][e] = x[k + 1][e];
        put(x[kConvTaps - 1], act_load4(u + (size_t)r * a.ldu));
        float s[4];
#pragma unroll
        for (uint32_t e = 0; e < 4; ++e) {
            s[e] = b[e];
#pragma unroll
            for (uint32_t k = 0; k < kConvTaps; ++k) s[e] = fmaf(w[k][e], x[k][e], s[e]);
            if (!a.linear) s[e] = silu(s[e]);
        }
        act_store4(y + (size_t)r * a.ldy, make_float4(s[0], s[1], s[2], s[3]));
    }
}

template <typename T>
__global__ __launch_bounds__(256) void ssm_conv_kernel(const SsmConvArgs a) {
    const uint32_t c = blockIdx.x * 256u + threadIdx.x, r = blockIdx.y;
    if (c >= a.channels) return;
    const uint32_t pos = *a.offset + r;
    const T* u = reinterpret_cast<const T*>(a.u);
    const T* hist = reinterpret_cast<const T*>(a.hist);
    float s = a.b ? bf16_bits_to_f32(a.b[c]) : 0.f;
    for (uint32_t k = 0; k < a.taps; ++k) {
        const uint32_t back = a.taps - 1u - k;
        if (back > pos) continue;   // before the first token: zero
        const float v = back <= r ? act_load(u + (size_t)(r - back) * a.ldu + c) : act_load(hist + (size_t)((pos - back) % a.taps) * a.ldh + c);
        s = fmaf(bf16_bits_to_f32(a.w[(size_t)c * a.taps + k]), v, s);
    }
    act_store(reinterpret_cast<T*>(a.y) + (size_t)r * a.ldy + c, a.linear ? s : silu(s));
    // a single row takes the place of the one that has left the convolution, which nobody reads
    if (a.update && a.rows == 1u) reinterpret_cast<T*>(a.hist)[(size_t)(pos % a.taps) * a.ldh + c] = u[c];
}

// The history after a pass of several rows: its last taps - 1 rows.
template <typename T>
__global__ __launch_bounds__(256) void ssm_conv_history_kernel(const SsmConvArgs a) {
    const uint32_t c = blockIdx.x * 256u + threadIdx.x, pos = *a.offset;
    if (c >= a.channels) return;
    const uint32_t keep = a.rows < a.taps - 1u ? a.rows : a.taps - 1u;
    for (uint32_t t = a.rows - keep; t < a.rows; ++t)
        reinterpret_cast<T*>(a.hist)[(size_t)((pos + t) % a.taps) * a.ldh + c] = reinterpret_cast<const T*>(a.u)[(size_t)t * a.ldu + c];
}

// Four adjacent values of a row of `n`, zeros past its end.
template <typename T>
__device__ __forceinline__ float4 load4_upto(const T* p, uint32_t i, uint32_t n, bool whole) {
    if (i >= n) return make_float4(0.f, 0.f, 0.f, 0.f);
    if (whole) return act_load4(p + i);
    float4 v = make_float4(act_load(p + i), 0.f, 0.f, 0.f);
    if (i + 1u < n) v.y = act_load(p + i + 1u);
    if (i + 2u < n) v.z = act_load(p + i + 2u);
    if (i + 3u < n) v.w = act_load(p + i + 3u);
    return v;
}

template <typename T, int NI>
__global__ __launch_bounds__(256) void ssm_scan_kernel(const SsmScanArgs a) {
    const uint32_t h = blockIdx.x, lane = threadIdx.x & 63u, wave = threadIdx.x >> 6;
    const uint32_t p_raw = blockIdx.y * 16u + wave * 4u + (lane >> 4), nl = (lane & 15u) * 4u;
    const bool live = p_raw < a.p;
    const uint32_t p = live ? p_raw : a.p - 1u;
    const uint32_t inner = a.heads * a.p, g = h / (a.heads / a.groups);
    const bool whole = ((a.n | inner) & 3u) == 0;
    const T* x0 = reinterpret_cast<const T*>(a.xbc);
    const float bias = bf16_bits_to_f32(a.dt_bias[h]), rate = expf(bf16_bits_to_f32(a.a_log[h])), D = bf16_bits_to_f32(a.d[h]);
    float* state = a.state + ((size_t)h * a.p + p) * a.state_ld + nl;
    float4 S[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) S[i] = *reinterpret_cast<const float4*>(state + 64 * i);
    auto fetch = [&](uint32_t r, float4* B, float4* C, float& x, float& dt) __attribute__((always_inline)) {
        const T* row = x0 + (size_t)r * a.ldx;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            B[i] = load4_upto(row + inner + g * a.n, nl + 64u * i, a.n, whole);
            C[i] = load4_upto(row + inner + (a.groups + g) * a.n, nl + 64u * i, a.n, whole);
        }
        x = act_load(row + (size_t)h * a.p + p);
        dt = a.dt[(size_t)r * a.lddt + h];
    };
    float4 B[NI], C[NI], Bn[NI], Cn[NI];
    float x, dt, xn = 0.f, dtn = 0.f;
    fetch(0, B, C, x, dt);
    T* y = reinterpret_cast<T*>(a.y) + (size_t)h * a.p + p;
    for (uint32_t r = 0; r < a.rows; ++r) {
        fetch(r + 1u < a.rows ? r + 1u : r, Bn, Cn, xn, dtn);
        const float step = softplus(dt + bias), decay = expf(-rate * step), sx = step * x;
        float out = 0.f;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            S[i].x = fmaf(decay, S[i].x, sx * B[i].x); S[i].y = fmaf(decay, S[i].y, sx * B[i].y);
            S[i].z = fmaf(decay, S[i].z, sx * B[i].z); S[i].w = fmaf(decay, S[i].w, sx * B[i].w);
            out = fmaf(S[i].x, C[i].x, out); out = fmaf(S[i].y, C[i].y, out);
            out = fmaf(S[i].z, C[i].z, out); out = fmaf(S[i].w, C[i].w, out);
        }
        out = group_sum(out, 16);
        if (live && nl == 0) act_store(y + (size_t)r * a.ldy, fmaf(D, x, out));
#pragma unroll
        for (int i = 0; i < NI; ++i) { B[i] = Bn[i]; C[i] = Cn[i]; }
        x = xn;
        dt = dtn;
    }
    if (live) {
#pragma unroll
        for (int i = 0; i < NI; ++i) *reinterpret_cast<float4*>(state + 64 * i) = S[i];
    }
    // the convolution's history: the last taps - 1 rows of the pass
    const uint32_t keep = a.rows < a.taps - 1u ? a.rows : a.taps - 1u, pos = *a.offset;
    const uint32_t t0 = (blockIdx.y * gridDim.x + blockIdx.x) * 256u + threadIdx.x, nt = gridDim.x * gridDim.y * 256u;
    for (uint32_t t = a.rows - keep; t < a.rows; ++t)
        for (uint32_t c = t0; c < a.channels; c += nt)
            reinterpret_cast<T*>(a.hist)[(size_t)((pos + t) % a.taps) * a.ldh + c] = reinterpret_cast<const T*>(a.u)[(size_t)t * a.ldu + c];
}

template <typename T>
const void* scan_func(uint32_t ni) {
    switch (ni) {
        case 1: return (const void*)&ssm_scan_kernel<T, 1>;
        case 2: return (const void*)&ssm_scan_kernel<T, 2>;
        case 3: return (const void*)&ssm_scan_kernel<T, 3>;
        default: return (const void*)&ssm_scan_kernel<T, 4>;
    }
}

}  // namespace

fk_status plan_ssm_conv(const SsmConvArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "ssm conv: act must be 16 or 32");
    if (!a.u || !a.w || !a.hist || !a.y || !a.offset || !a.rows || !a.channels || !a.taps) return set_error(FK_ERR_INVALID, "ssm conv: bad arguments");
    if (a.rows > 65535) return set_error(FK_ERR_UNSUPPORTED, "ssm conv: at most 65535 rows");
    const uintptr_t align = act == 16 ? 7 : 15;   // four elements per access
    if (a.rows >= kConvRows && a.taps <= kConvTaps && a.channels % 4 == 0 && a.ldu % 4 == 0 && a.ldy % 4 == 0 && a.ldh % 4 == 0 &&
        (((uintptr_t)a.u | (uintptr_t)a.hist | (uintptr_t)a.y) & align) == 0) {
        out->func = act == 16 ? (const void*)&ssm_conv_rows_kernel<uint16_t> : (const void*)&ssm_conv_rows_kernel<float>;
        out->grid = dim3((a.channels / 4u + 255u) / 256u, (a.rows + kConvRows - 1u) / kConvRows);
    } else {
        out->func = act == 16 ? (const void*)&ssm_conv_kernel<uint16_t> : (const void*)&ssm_conv_kernel<float>;
        out->grid = dim3((a.channels + 255u) / 256u, a.rows);
        if (a.update && a.rows > 1u && a.taps > 1u) {
            Launch h;
            h.func = act == 16 ? (const void*)&ssm_conv_history_kernel<uint16_t> : (const void*)&ssm_conv_history_kernel<float>;
            h.grid = dim3((a.channels + 255u) / 256u, 1, 1);
            h.block = dim3(256, 1, 1);
            h.set_args(a);
            out->then.push_back(h);
        }
    }
    out->block = dim3(256, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    return FK_OK;
}

fk_status plan_ssm_scan(const SsmScanArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "ssm scan: act must be 16 or 32");
    if (!a.xbc || !a.dt || !a.dt_bias || !a.a_log || !a.d || !a.state || !a.y || !a.u || !a.hist || !a.offset || !a.rows || !a.p || !a.n || !a.taps)
        return set_error(FK_ERR_INVALID, "ssm scan: bad arguments");
    if (!a.groups || a.heads % a.groups) return set_error(FK_ERR_INVALID, "ssm scan: heads must be a multiple of groups");
    if (a.n > kMaxSsmState || a.state_ld % 64 || a.state_ld < a.n || a.state_ld > kMaxSsmState) return set_error(FK_ERR_UNSUPPORTED, "ssm scan: state width at most 256");
    if ((a.p + 15u) / 16u > 65535) return set_error(FK_ERR_UNSUPPORTED, "ssm scan: head too wide");
    const uint32_t ni = a.state_ld / 64u;
    out->func = act == 16 ? scan_func<uint16_t>(ni) : scan_func<float>(ni);
    out->grid = dim3(a.heads, (a.p + 15u) / 16u);
    out->block = dim3(256, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    return FK_OK;
}

}  // namespace fk
