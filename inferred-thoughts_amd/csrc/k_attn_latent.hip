// Latent attention: a token's cache row is [latent c | rotated key part k_r], one row for all heads.  A head's key is
// [uk_h c | k_r], its value uv_h c.  Two forms, the same sums in another order:
//
//   few queries:  (q_n . uk_h c) = (uk_h^T q_n) . c, so the queries are taken to the latent's space (latent_prep_k), attend to
//       the rows as they are cached, the row's first `rank` elements being the values (attend_shared_split_k, or
//       attend_bias_plain_k), and uv_h is applied to the sum (latent_value_k).  A row is read once for all heads.
//   many queries: the visible rows become keys and values of every head (latent_keys_k and two matrix products), which
//       attend_bias_batch_k takes.
//
// The rotation turns neighbouring dimensions (2i, 2i + 1) by the angle table's row of the position.
#include <algorithm>

#include "it_device.h"
#include "it_float.h"
#include "it_reduce.h"
#include "it_rows8.h"
#include "kernels_float.h"

namespace itk {
namespace {

typedef _Float16 h8 __attribute__((ext_vector_type(8)));
typedef float v16f __attribute__((ext_vector_type(16)));
constexpr float LOG2E = 1.4426950408889634f;

IT_DEV void slab_store(const LatentP& p, int64_t at, float v) {
    if (p.slab_f32) ((float*)p.slab)[at] = v;
    else ((uint16_t*)p.slab)[at] = it_f32_to_f16(v);
}
// element i of a rotated part x at position pos
IT_DEV float rotated(const LatentP& p, const float* x, int i, int64_t pos) {
    if (i >= p.n_rot) return x[i];
    const float2 cs = p.table[pos * (p.n_rot >> 1) + (i >> 1)];
    const float u = x[i & ~1], v = x[i | 1];
    return i & 1 ? fmaf(v, cs.x, u * cs.y) : fmaf(u, cs.x, -(v * cs.y));
}
// the cache row of token t, by the whole block
IT_DEV void cache_row(const LatentP& p, int t, int64_t pos, float* red) {
    const int tid = threadIdx.x;
    const float* x = p.kv + (int64_t)t * p.k_dim();
    const int64_t at = pos * p.row_stride;
    float ss = 0.0f;
    for (int i = tid; i < p.rank; i += 256) ss = fmaf(x[i], x[i], ss);
    const float rinv = 1.0f / sqrtf(block_sum(ss, red) / (float)p.rank + p.eps);
    for (int i = tid; i < p.rank; i += 256) slab_store(p, at + i, x[i] * rinv * p.kv_norm[i]);
    for (int i = tid; i < p.rot; i += 256) slab_store(p, at + p.rank + i, rotated(p, x + p.rank, i, pos));
}

// ---------------------------------------------------------------- few queries: into the latent's space
// a block: 128 latent elements of one head, 16 lanes of eight; the head's rows of uk dealt to 16 groups
constexpr int RB = 128;
template <int FMT, bool AL>
__global__ __launch_bounds__(256) void latent_prep_k(LatentP p, int slices, float* __restrict__ qa) {
    __shared__ float part[16][RB + 1], red[4];
    const int tid = threadIdx.x, t = blockIdx.y;
    const int64_t pos = (p.n_pos_dyn ? *p.n_pos_dyn - p.n_tok : p.pos) + t;
    if ((int)blockIdx.x == p.heads * slices) {
        cache_row(p, t, pos, red);
        return;
    }
    const int h = blockIdx.x / slices, r0 = (blockIdx.x % slices) * RB, dg = tid >> 4, c = r0 + (tid & 15) * 8;
    const float* q = p.q + ((int64_t)t * p.heads + h) * (p.dim + p.rot);
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; e++) acc[e] = 0.0f;
#pragma unroll 4
    for (int d = dg; d < p.dim; d += 16) {
        float f[8];
        widen8<FMT>(load8<FMT, AL>(row_at<FMT>(p.uk, h * p.dim + d, p.rank), c, p.rank), f);
        const float x = q[d];
#pragma unroll
        for (int e = 0; e < 8; e++) acc[e] = fmaf(f[e], x, acc[e]);
    }
#pragma unroll
    for (int e = 0; e < 8; e++) part[dg][(tid & 15) * 8 + e] = acc[e];
    __syncthreads();
    float* o = qa + ((int64_t)t * p.heads + h) * p.k_dim();
    if (tid < RB && r0 + tid < p.rank) {
        float v = 0.0f;
#pragma unroll
        for (int i = 0; i < 16; i++) v += part[i][tid];
        o[r0 + tid] = v;
    }
    if (r0 == 0)
        for (int i = tid; i < p.rot; i += 256) o[p.rank + i] = rotated(p, q + p.dim, i, pos);
}

// ---------------------------------------------------------------- many queries
__global__ __launch_bounds__(256) void latent_rows_k(LatentP p, float* __restrict__ q) {
    __shared__ float red[4];
    const int tid = threadIdx.x, t = blockIdx.x, half = p.n_rot >> 1;
    const int64_t pos = (int64_t)p.pos + t;
    if (p.kv) cache_row(p, t, pos, red);
    float* row = q + (int64_t)t * p.heads * (p.dim + p.rot) + p.dim;
    for (int i = tid; i < p.heads * half; i += 256) {
        float* x = row + (i / half) * (p.dim + p.rot) + 2 * (i % half);
        const float2 cs = p.table[pos * half + i % half];
        const float u = x[0], v = x[1];
        x[0] = fmaf(u, cs.x, -(v * cs.y));
        x[1] = fmaf(v, cs.x, u * cs.y);
    }
}

__global__ __launch_bounds__(256) void latent_keys_k(LatentP p, int first, uint16_t* __restrict__ c16, uint16_t* __restrict__ k, int ks) {
    const int tid = threadIdx.x, rp = pad8(p.rank), tail = ks - p.dim;
    const int64_t key = blockIdx.x;
    const uint16_t* row = (const uint16_t*)p.slab + (first + key) * p.row_stride;
    for (int i = tid; i < rp; i += 256) c16[key * rp + i] = i < p.rank ? to_bf16(it_f16_to_f32(row[i])) : 0;
    for (int i = tid; i < p.heads * tail; i += 256) {
        const int h = i / tail, j = i % tail;
        k[(key * p.heads + h) * ks + p.dim + j] = j < p.rot ? row[p.rank + j] : 0;
    }
}

// ---------------------------------------------------------------- few queries, split over rows that all heads share
// partial of (query, head, split): [v_dim padded to 32 sums][maximum in the log2 domain][sum]
// A block: one query's chunk of up to 32 heads (the columns of every product), one range of keys, 32 of them at a time.  The
// waves share the scores' sum over the elements of a row (each takes every fourth 16 of them); then each holds all scores and
// owns the output dims 32 w .. (+ 128).  Keys, values and the scaled query are f16, a probability enters the second product
// as an f16 pair, and the operands' layouts are those of attend_bias_split_k.
constexpr int KT = 32;
constexpr int SPLIT_MAX = 256;
template <int NDW>
__global__ __launch_bounds__(256) void attend_shared_split_k(BiasAttnP a, int n_split, int chunks, int kp, float* __restrict__ part) {
    extern __shared__ __align__(16) uint16_t lds[];
    const int RS = kp + 8, NS = kp / 16, rp = (a.v_dim + 31) & ~31, ND = rp / 32;
    uint16_t *Ks = lds, *Qs = lds + KT * RS;            // [32][RS] each
    float* red = (float*)(lds + 2 * KT * RS);           // [wave][16][64]
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), c = lane & 31, g = lane >> 5;
    const int cw = (a.n_head + chunks - 1) / chunks, h0 = (blockIdx.x % chunks) * cw, t = blockIdx.x / chunks, nh = min(cw, a.n_head - h0);
    const int split = blockIdx.y;
    const int pos = (a.n_pos_dyn ? *a.n_pos_dyn : a.n_pos) - a.n_q + t, n_pos = pos + 1;
    const int seen = a.window ? max(0, n_pos - a.window) : 0, kpb = max(KT, ((n_pos - seen + n_split - 1) / n_split + 15) & ~15);
    const int k0 = seen + split * kpb, k1 = min(n_pos, k0 + kpb);
    const int64_t head_stride = (int64_t)n_split * (rp + 2);
    float* my = part + (((int64_t)t * a.n_head + h0) * n_split + split) * (rp + 2);
    if (k0 >= k1) {
        if (tid < nh) {
            my[tid * head_stride + rp] = -INFINITY;
            my[tid * head_stride + rp + 1] = 0.0f;
        }
        return;
    }
    const float qsc = a.scale * LOG2E;
    for (int row = tid >> 6; row < 32; row += 4)
        for (int d = lane; d < kp; d += 64) {
            const float v = row < nh && d < a.k_dim ? a.q[((int64_t)t * a.n_head + h0 + row) * a.k_dim + d] * qsc : 0.0f;
            Qs[row * RS + d] = __builtin_bit_cast(uint16_t, (_Float16)v);
        }
    v16f o[NDW];
#pragma unroll
    for (int dw = 0; dw < NDW; dw++)
#pragma unroll
        for (int i = 0; i < 16; i++) o[dw][i] = 0.0f;
    float m = -INFINITY, l = 0.0f;
    const int nseg = kp / 8;
    for (int key0 = k0; key0 < k1; key0 += KT) {
        __syncthreads();   // the rows before are read
        for (int row = tid >> 6; row < KT; row += 4) {
            const uint16_t* src = (const uint16_t*)a.k + (int64_t)(key0 + row) * a.k_stride;
            for (int seg = lane; seg < nseg; seg += 64)
                *(uint4*)(Ks + row * RS + seg * 8) = key0 + row < k1 && seg * 8 < a.k_stride ? *(const uint4*)(src + seg * 8) : make_uint4(0, 0, 0, 0);
        }
        __syncthreads();
        v16f sc;
#pragma unroll
        for (int i = 0; i < 16; i++) sc[i] = 0.0f;
        for (int s = w; s < NS; s += 4)
            sc = __builtin_amdgcn_mfma_f32_32x32x16_f16(*(const h8*)(Ks + c * RS + 16 * s + 8 * g), *(const h8*)(Qs + c * RS + 16 * s + 8 * g), sc, 0, 0, 0);
#pragma unroll
        for (int i = 0; i < 16; i++) red[(w * 16 + i) * 64 + lane] = sc[i];
        __syncthreads();
        float mt = -INFINITY;
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const float v = (red[i * 64 + lane] + red[(16 + i) * 64 + lane]) + (red[(32 + i) * 64 + lane] + red[(48 + i) * 64 + lane]);
            sc[i] = key0 + 8 * (i >> 2) + 4 * g + (i & 3) < k1 ? v : -INFINITY;
            mt = fmaxf(mt, sc[i]);
        }
        mt = fmaxf(mt, __shfl_xor(mt, 32, 64));   // (the tile's first key is always seen)
        const float m_new = fmaxf(m, mt), alpha = __builtin_amdgcn_exp2f(m - m_new);
        h8 ph[2], pl[2];
        float psum = 0.0f;
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const float p = __builtin_amdgcn_exp2f(sc[i] - m_new);
            psum += p;
            const _Float16 hi = (_Float16)p;
            ph[i >> 3][i & 7] = hi;
            pl[i >> 3][i & 7] = (_Float16)(p - (float)hi);
        }
        l = l * alpha + psum;
        m = m_new;
#pragma unroll
        for (int dw = 0; dw < NDW; dw++) {
            const int dt = w + 4 * dw;
            if (dt < ND) {
                const int d = min(32 * dt + c, kp - 1);   // (a dim past the row's end is not stored)
#pragma unroll
                for (int i = 0; i < 16; i++) o[dw][i] *= alpha;
#pragma unroll
                for (int j = 0; j < 2; j++) {
                    const uint16_t* vp = Ks + (16 * j + 4 * g) * RS + d;
                    h8 vf;
#pragma unroll
                    for (int e = 0; e < 8; e++) vf[e] = __builtin_bit_cast(_Float16, vp[(8 * (e >> 2) + (e & 3)) * RS]);
                    o[dw] = __builtin_amdgcn_mfma_f32_32x32x16_f16(vf, ph[j], o[dw], 0, 0, 0);
                    o[dw] = __builtin_amdgcn_mfma_f32_32x32x16_f16(vf, pl[j], o[dw], 0, 0, 0);
                }
            }
        }
    }
    l += __shfl_xor(l, 32, 64);
    if (c >= nh) return;
    float* p = my + c * head_stride;
#pragma unroll
    for (int dw = 0; dw < NDW; dw++) {
        const int dt = w + 4 * dw;
        if (dt < ND) {
#pragma unroll
            for (int i4 = 0; i4 < 4; i4++) {
                float* q = p + 32 * dt + 8 * i4 + 4 * g;   // 8-byte aligned: the partial's size is even
                *(float2*)q = make_float2(o[dw][4 * i4], o[dw][4 * i4 + 1]);
                *(float2*)(q + 2) = make_float2(o[dw][4 * i4 + 2], o[dw][4 * i4 + 3]);
            }
        }
    }
    if (w == 0 && g == 0) {
        p[rp] = m;
        p[rp + 1] = l;
    }
}

// ---------------------------------------------------------------- the values' matrix, behind the merge
// a block: 32 output dims of one (query, head), a wave eight of them, four at a time
template <int FMT, bool AL>
__global__ __launch_bounds__(256) void latent_value_k(LatentP p, BiasAttnP a, const float* __restrict__ part, int n_split, float* __restrict__ out) {
    extern __shared__ __align__(16) float ol[];   // [rank padded to 8]
    __shared__ float wsplit[SPLIT_MAX], red[8];
    __shared__ int seen;
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int h = blockIdx.x % p.heads;
    if (n_split) {
        const int rp = (p.rank + 31) & ~31, st = rp + 2;
        const float* q = part + (int64_t)blockIdx.x * n_split * st;
        const float ms = tid < n_split ? q[(int64_t)tid * st + rp] : -INFINITY, ls = tid < n_split ? q[(int64_t)tid * st + rp + 1] : 0.0f;
        float m = group_max<64>(ms);
        if (tid == 0) seen = 0;
        if (lane == 0) red[4 + w] = m;
        __syncthreads();
        m = fmaxf(fmaxf(red[4], red[5]), fmaxf(red[6], red[7]));
        const float wgt = ms != -INFINITY ? __builtin_amdgcn_exp2f(ms - m) : 0.0f;
        if (ms != -INFINITY) atomicMax(&seen, tid + 1);   // the splits with keys come first
        wsplit[tid] = wgt;
        float l = block_sum(ls * wgt, red);
        if (a.sink) l += __builtin_amdgcn_exp2f((a.sinks ? a.sinks[h] * LOG2E : 0.0f) - m);
        const int n = seen;
        for (int r = tid; r < pad8(p.rank); r += 256) {
            float acc = 0.0f;
            if (r < p.rank) {
#pragma unroll 8
                for (int s = 0; s < n; s++) acc = fmaf(q[(int64_t)s * st + r], wsplit[s], acc);
            }
            ol[r] = acc / l;
        }
    } else {
        for (int r = tid; r < pad8(p.rank); r += 256) ol[r] = r < p.rank ? part[(int64_t)blockIdx.x * p.rank + r] : 0.0f;
    }
    __syncthreads();
    const float gate = p.gate ? sigmoid_exact(p.gate[blockIdx.x]) : 1.0f;
#pragma unroll
    for (int half = 0; half < 2; half++) {
        const int j0 = blockIdx.y * 32 + w * 8 + half * 4;
        float acc[4] = {0.f, 0.f, 0.f, 0.f};
        for (int k = lane * 8; k < p.rank; k += 512) {
            const float4 x0 = *(const float4*)(ol + k), x1 = *(const float4*)(ol + k + 4);
            const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
            for (int i = 0; i < 4; i++) {
                float f[8];
                widen8<FMT>(load8<FMT, AL>(row_at<FMT>(p.uv, (int64_t)h * p.vdim + min(j0 + i, p.vdim - 1), p.rank), k, p.rank), f);
#pragma unroll
                for (int e = 0; e < 8; e++) acc[i] = fmaf(f[e], x[e], acc[i]);
            }
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            acc[i] = group_sum<64>(acc[i]);
            if (lane == i && j0 + i < p.vdim) out[(int64_t)blockIdx.x * p.vdim + j0 + i] = acc[i] * gate;
        }
    }
}

int padded_row(const BiasAttnP& a) { return (a.k_dim + 15) & ~15; }
size_t shared_lds(const BiasAttnP& a) { return (size_t)2 * KT * (padded_row(a) + 8) * sizeof(uint16_t) + 4 * 16 * 64 * sizeof(float); }
template <class F> bool allow_lds(F* fn, size_t lds) {
    if (lds <= 64 * 1024) return true;
    if (hipFuncSetAttribute((const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess) return true;
    (void)hipGetLastError();
    return false;
}

}  // namespace

void latent_prep(const LatentP& p, float* qa, hipStream_t s) {
    const bool al = p.rank % 8 == 0 && aligned16(p.uk);
    const int slices = (p.rank + RB - 1) / RB;
    const dim3 grid(p.heads * slices + (p.kv ? 1 : 0), p.n_tok);
#define IT_CALL(F, A) hipLaunchKernelGGL((latent_prep_k<F, A>), grid, dim3(256), 0, s, p, slices, qa)
    IT_BY_FORMAT(p.uk_fmt, al, IT_CALL);
#undef IT_CALL
}
void latent_rows(const LatentP& p, float* q, hipStream_t s) { hipLaunchKernelGGL(latent_rows_k, dim3(p.n_tok), dim3(256), 0, s, p, q); }
void latent_keys(const LatentP& p, int first, int n_keys, uint16_t* c16, uint16_t* k, int ks, hipStream_t s) {
    hipLaunchKernelGGL(latent_keys_k, dim3(n_keys), dim3(256), 0, s, p, first, c16, k, ks);
}
void latent_value(const LatentP& p, const BiasAttnP& a, const float* part, int n_split, float* out, hipStream_t s) {
    const bool al = p.rank % 8 == 0 && aligned16(p.uv);
    const dim3 grid(p.n_tok * p.heads, (p.vdim + 31) / 32);
    const size_t lds = pad8(p.rank) * sizeof(float);
#define IT_CALL(F, A) hipLaunchKernelGGL((latent_value_k<F, A>), grid, dim3(256), lds, s, p, a, part, n_split, out)
    IT_BY_FORMAT(p.uv_fmt, al, IT_CALL);
#undef IT_CALL
}

// one row for all heads, the values its first elements; rows of whole 16-byte pieces; no bias, no temperature
bool attend_shared_takes(const BiasAttnP& a) {
    return !a.kv_f32 && a.k == a.v && a.n_head_kv == 1 && a.v_dim <= a.k_dim && a.k_stride % 8 == 0 && a.k_dim <= a.k_stride && !a.slopes &&
           a.temp_coef == 0.0f && aligned16(a.k) && a.v_dim <= 1024 && shared_lds(a) <= 156 * 1024;
}
int attend_shared_splits(const BiasAttnP& a, int n_pos_max) {
    const int most = a.window ? std::min(a.window, n_pos_max) : n_pos_max;
    return std::max(1, std::min(SPLIT_MAX, (most + 63) / 64));
}
size_t attend_shared_scratch_floats(const BiasAttnP& a, int n_split) {
    return (size_t)a.n_q * a.n_head * n_split * (((a.v_dim + 31) & ~31) + 2);
}
bool attend_shared_split(const BiasAttnP& a, int n_split, float* scratch, hipStream_t s) {
    if (!attend_shared_takes(a) || n_split < 1 || n_split > SPLIT_MAX || !a.q || !a.k) return false;
    const int chunks = (a.n_head + 31) / 32, ndw = (((a.v_dim + 31) / 32) + 3) / 4, kp = padded_row(a);
    const size_t lds = shared_lds(a);
    const dim3 grid((unsigned)(a.n_q * chunks), n_split);
#define IT_CALL(N)                                                                                                        \
    do {                                                                                                                  \
        if (!allow_lds(attend_shared_split_k<N>, lds)) return false;                                                       \
        hipLaunchKernelGGL(attend_shared_split_k<N>, grid, dim3(256), lds, s, a, n_split, chunks, kp, scratch);            \
    } while (0)
    if (ndw <= 1) IT_CALL(1);
    else if (ndw <= 2) IT_CALL(2);
    else if (ndw <= 4) IT_CALL(4);
    else IT_CALL(8);
#undef IT_CALL
    return true;
}

}  // namespace itk
