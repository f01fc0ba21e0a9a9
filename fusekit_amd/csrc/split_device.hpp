// Weights of the partial rows of a split attention, shared by the kernels that combine them.
#pragma once
#include "fk_device.hpp"

namespace fk {

// ml[s * stride] and ml[s * stride + 1] are the maximum and the sum of split s; w[s] becomes exp(maximum) over the whole
// denominator, in which the sink counts once.  Wave 0 does the work; the caller's barrier publishes w.
__device__ __forceinline__ void split_weights(const float* ml, size_t stride, uint32_t splits, float sink, float* w) {
    if (threadIdx.x >= (uint32_t)kWave) return;
    const uint32_t s = threadIdx.x;
    const float m = s < splits ? ml[s * stride] : -INFINITY, l = s < splits ? ml[s * stride + 1] : 0.f;
    const float top = fmaxf(wave_max(m), sink), e = expf(m - top);
    const float total = wave_sum(e * l) + expf(sink - top);
    if (s < splits) w[s] = e / total;
}

}  // namespace fk
