// Device helpers of the kernels for unquantized models: bf16 rounding, accurate activations, and the store that ends a
// group product.
#pragma once
#include "it_device.h"
#include "kernels_float.h"

namespace itk {

IT_DEV uint16_t to_bf16(float f) { return __builtin_bit_cast(uint16_t, (__bf16)f); }
// the library's exponential (about 1 ulp over the whole range): what 32-bit mode and everything inside a recurrence use
IT_DEV float silu_exact(float z) { return z / (1.0f + expf(-z)); }
IT_DEV float softplus_exact(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

IT_DEV float sigmoid_exact(float z) { return 1.0f / (1.0f + expf(-z)); }
IT_DEV float act_of(int act, float z) { return act == ACT_RELU ? fmaxf(z, 0.0f) : silu_exact(z); }

IT_DEV void group_store(const GroupMat& m, int t, int j, float v) {
    v *= m.scale;
    const GroupOut& o = m.o;
    if (o.f32) o.f32[(int64_t)t * m.n_out + j] = v;
    if (o.half) o.half[(int64_t)t * pad8(m.n_out) + j] = to_bf16(v);
    if (o.slab) {
        const int64_t row = (o.row_dyn ? *o.row_dyn : o.row) + t;
        const int64_t at = row * o.row_stride + (j / o.head_dim) * o.head_stride + j % o.head_dim;
        if (o.slab_f32) ((float*)o.slab)[at] = v;
        else ((uint16_t*)o.slab)[at] = it_f32_to_f16(v);
    }
}

}  // namespace itk
