// Column functions of the layer-list decoder's products.
#pragma once
#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

__device__ __forceinline__ uint32_t column_fn(const ColumnOut& o, uint32_t n) { return n >= o.begin && n < o.end ? o.fn : n >= o.begin2 ? o.fn2 : (uint32_t)kFnNone; }

__device__ __forceinline__ float apply_fn(uint32_t fn, float v) {
    if (fn == kFnRelu2) {
        v = fmaxf(v, 0.f);
        return v * v;
    }
    return fn == kFnGelu ? gelu_tanh(v) : v;
}

// What becomes of one column's sum before it is stored.
__device__ __forceinline__ float column_value(const ColumnOut& o, uint32_t n, float v) {
    if (o.bias) v += bf16_bits_to_f32(o.bias[n]);
    return apply_fn(column_fn(o, n), v);
}

}  // namespace fk
