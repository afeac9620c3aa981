// fp32 matrix-core products of 16 x 16 tiles, for recurrences whose operands stay 32-bit.
#pragma once
#include "it_device.h"

namespace itk {

typedef float v4f __attribute__((ext_vector_type(4)));
// D = A(16 x 4) B(4 x 16) + C: lane l gives A[l % 16][l / 16] and B[l / 16][l % 16], and holds D[4 * (l / 16) + i][l % 16].
// The order of k is free as long as both operands agree: four products in turn take k = 4 (l / 16) + 0 .. 3 of a stretch of
// 16, so that a lane's operands are 16 bytes in a row.
IT_DEV v4f mfma4(float a, float b, v4f c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
IT_DEV v4f mfma16(const float4& a, const float4& b, v4f c) {
    c = mfma4(a.x, b.x, c);
    c = mfma4(a.y, b.y, c);
    c = mfma4(a.z, b.z, c);
    return mfma4(a.w, b.w, c);
}
// four elements of a row of n from k on, zeros past its end
IT_DEV float4 row4(const float* q, int k, int n, bool vec) {
    if (vec) return k < n ? *(const float4*)(q + k) : make_float4(0.f, 0.f, 0.f, 0.f);
    return make_float4(k < n ? q[k] : 0.0f, k + 1 < n ? q[k + 1] : 0.0f, k + 2 < n ? q[k + 2] : 0.0f, k + 3 < n ? q[k + 3] : 0.0f);
}

}  // namespace itk
