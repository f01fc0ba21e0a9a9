// Activation element access for kernels that serve bf16 and fp32 activations with one body.
#pragma once
#include "fk_device.hpp"

namespace fk {

__device__ __forceinline__ float act_load(const uint16_t* p) { return bf16_bits_to_f32(*p); }
__device__ __forceinline__ float act_load(const float* p) { return *p; }
__device__ __forceinline__ void act_store(uint16_t* p, float v) { *p = (uint16_t)f32_to_bf16_bits(v); }
__device__ __forceinline__ void act_store(float* p, float v) { *p = v; }

// Four adjacent elements, aligned to their own size.
__device__ __forceinline__ float4 act_load4(const uint16_t* p) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    return make_float4(bf16_lo(v.x), bf16_hi(v.x), bf16_lo(v.y), bf16_hi(v.y));
}
__device__ __forceinline__ float4 act_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ void act_store4(uint16_t* p, float4 v) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16(v.x, v.y), pack_bf16(v.z, v.w));
}
__device__ __forceinline__ void act_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }

__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu(float z) { return z / (1.0f + expf(-z)); }
// log(1 + exp(z)) without overflow and without losing small results.
__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

// 0.5 z (1 + tanh(t)) = z sigmoid(2 t), t = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_tanh(float z) {
    const float t = 0.7978845608028654f * fmaf(0.044715f * z * z, z, z);
    return z * sigmoid(2.0f * t);
}

// cos / sin of position * freq.  The angle is formed and reduced in double, so its error does not grow with the
// position; the evaluation is fp32.
__device__ __forceinline__ void position_cos_sin(uint32_t pos, double freq, float& cs, float& sn) {
    const double a = (double)pos * freq;
    const double turns = rint(a * 0.15915494309189535);
    sincosf((float)(a - turns * 6.283185307179586), &sn, &cs);
}

}  // namespace fk
