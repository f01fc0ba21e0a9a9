// One step of the real-gated linear recurrent unit, shared by the kernels that run it over a pass and for one token.
#pragma once
#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

// log a per unit of r
__device__ __forceinline__ float lru_rate(uint16_t lam) { return -8.0f * softplus(bf16_bits_to_f32(lam)); }

// zr, zi: the gates before their sigmoids.  1 - a^2 is formed without cancellation.
__device__ __forceinline__ void lru_step(float zr, float zi, float rate, float u, float& decay, float& add) {
    const float log_a = rate * sigmoid(zr);
    decay = expf(log_a);
    add = sqrtf(-expm1f(2.0f * log_a)) * sigmoid(zi) * u;
}

// The same with the hardware's exponential, reciprocal and root (within a few units of the last place) and, near
// a = 1, the series of 1 - exp(x) = -x (1 + x/2 (1 + x/3 (1 + x/4 ..))): nine terms for |x| < 1/2.
__device__ __forceinline__ void lru_step_fast(float zr, float zi, float rate, float u, float& decay, float& add) {
    constexpr float kLog2e = 1.4426950408889634f;
    const float r = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-kLog2e * zr)), i = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-kLog2e * zi));
    const float log_a = rate * r, x = 2.0f * log_a;
    decay = __builtin_amdgcn_exp2f(kLog2e * log_a);
    float s = 1.0f;
    s = fmaf(x * (1.0f / 9.0f), s, 1.0f); s = fmaf(x * 0.125f, s, 1.0f); s = fmaf(x * (1.0f / 7.0f), s, 1.0f); s = fmaf(x * (1.0f / 6.0f), s, 1.0f);
    s = fmaf(x * 0.2f, s, 1.0f); s = fmaf(x * 0.25f, s, 1.0f); s = fmaf(x * (1.0f / 3.0f), s, 1.0f); s = fmaf(x * 0.5f, s, 1.0f);
    const float rest = x > -0.5f ? -x * s : fmaf(-decay, decay, 1.0f);
    add = __builtin_amdgcn_sqrtf(rest) * i * u;
}

}  // namespace fk
