// Rows of unquantized matrices read eight elements at a time, whatever their type and alignment, and the launch switch over both.
#pragma once
#include "it_device.h"
#include "it_reduce.h"
#include "kernels_float.h"

namespace itk {

template <int FMT> struct Raw8 { uint4 a; };
template <> struct Raw8<W_F32> { uint4 a, b; };

template <int FMT> IT_DEV const uint8_t* row_at(const uint8_t* w, int64_t row, int n_in) {
    return w + row * n_in * (FMT == W_F32 ? 4 : 2);
}
// a weight is read once a token: it need not stay in the caches
typedef uint32_t u4 __attribute__((ext_vector_type(4)));
IT_DEV uint4 stream16(const void* p) {
    const u4 v = __builtin_nontemporal_load((const u4*)p);
    return make_uint4(v.x, v.y, v.z, v.w);
}
// eight elements of a row from k on; AL: the row length is a multiple of 8 and the rows are 16-byte aligned
template <int FMT, bool AL> IT_DEV Raw8<FMT> load8(const uint8_t* row, int k, int n_in) {
    Raw8<FMT> r{};
    if (AL) {
        if (k < n_in) {
            if constexpr (FMT == W_F32) {
                r.a = stream16((const float*)row + k);
                r.b = stream16((const float*)row + k + 4);
            } else {
                r.a = stream16((const uint16_t*)row + k);
            }
        }
    } else {
        uint32_t v[8];
#pragma unroll
        for (int e = 0; e < 8; e++) {
            if (FMT == W_F32) v[e] = k + e < n_in ? ((const uint32_t*)row)[k + e] : 0u;
            else v[e] = k + e < n_in ? ((const uint16_t*)row)[k + e] : 0u;
        }
        if constexpr (FMT == W_F32) {
            r.a = make_uint4(v[0], v[1], v[2], v[3]);
            r.b = make_uint4(v[4], v[5], v[6], v[7]);
        } else {
            r.a = make_uint4(v[0] | (v[1] << 16), v[2] | (v[3] << 16), v[4] | (v[5] << 16), v[6] | (v[7] << 16));
        }
    }
    return r;
}
template <int FMT> IT_DEV void widen8(const Raw8<FMT>& r, float* f) {
    if constexpr (FMT == W_F32) {
        const uint32_t v[8] = {r.a.x, r.a.y, r.a.z, r.a.w, r.b.x, r.b.y, r.b.z, r.b.w};
#pragma unroll
        for (int e = 0; e < 8; e++) f[e] = __uint_as_float(v[e]);
    } else {
        const uint32_t v[4] = {r.a.x, r.a.y, r.a.z, r.a.w};
#pragma unroll
        for (int e = 0; e < 4; e++) {
            if (FMT == W_BF16) {
                f[2 * e] = __uint_as_float(v[e] << 16);
                f[2 * e + 1] = __uint_as_float(v[e] & 0xffff0000u);
            } else {
                f[2 * e] = it_f16_to_f32((uint16_t)(v[e] & 0xffffu));
                f[2 * e + 1] = it_f16_to_f32((uint16_t)(v[e] >> 16));
            }
        }
    }
}

IT_DEV float block_sum(float v, float* red) {   // 256 threads
    v = group_sum<64>(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

inline bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

// one call per (format, alignment)
#define IT_BY_FORMAT(fmt, al, CALL)                                                    \
    do {                                                                               \
        if ((fmt) == W_BF16) { if (al) { CALL(W_BF16, true); } else { CALL(W_BF16, false); } } \
        else if ((fmt) == W_F16) { if (al) { CALL(W_F16, true); } else { CALL(W_F16, false); } } \
        else { if (al) { CALL(W_F32, true); } else { CALL(W_F32, false); } }           \
    } while (0)

}  // namespace itk
