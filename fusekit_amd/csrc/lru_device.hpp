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

}  // namespace fk
