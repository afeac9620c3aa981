// Latent attention: a token's cache row is [latent c | rotated key part k_r], one row for all heads.  A head's key is
// [uk_h c | k_r], its value uv_h c.  Two forms, the same sums in another order:
//
//   few queries:  (q_n . uk_h c) = (uk_h^T q_n) . c, so the queries are taken to the latent's space (latent_prep_k), attend to
//       the rows as they are cached, the row's first `rank` elements being the values (attend_shared_split_k, or
//       attend_bias_plain_k), and uv_h is applied to the outcome (latent_value_k).  A row is read once for all heads.
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
constexpr int RANK_MAX = 4096;

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
__global__ __launch_bounds__(256) void latent_prep_k(LatentP p, int slices, float* __restrict__ qa, uint16_t* __restrict__ q16, int kp, float qsc) {
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
    const int64_t th = (int64_t)t * p.heads + h;
    auto store = [&](int i, float v) {
        if (q16) q16[th * kp + i] = it_f32_to_f16(v * qsc);
        else qa[th * p.k_dim() + i] = v;
    };
    if (tid < RB && r0 + tid < p.rank) {
        float v = 0.0f;
#pragma unroll
        for (int i = 0; i < 16; i++) v += part[i][tid];
        store(r0 + tid, v);
    }
    if (r0 == 0) {
        for (int i = tid; i < p.rot; i += 256) store(p.rank + i, rotated(p, q + p.dim, i, pos));
        if (q16 && tid < kp - p.k_dim()) q16[th * kp + p.k_dim() + tid] = 0;
    }
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
// The partials of a call: sums [query][head][split][v_dim padded to 32], behind them [query][head][split][maximum in the log2
// domain, sum].
struct Partials {
    float *sums, *ml;
    int rp, n_split;
    IT_DEV const float* sums_of(int64_t qh) const { return sums + qh * n_split * rp; }
    IT_DEV float* at(int64_t qh, int split) const { return sums + (qh * n_split + split) * rp; }
    IT_DEV float* ml_at(int64_t qh, int split) const { return ml + (qh * n_split + split) * 2; }
};
// A block: one query's chunk of up to 32 heads (the columns of every product), one range of keys, 32 of them at a time.  The
// waves share the scores' sum over the elements of a row (each takes every fourth 16 of them); then each holds all scores and
// owns the output dims 32 w .. (+ 128).  Keys, values and the scaled query (q16, rows of kp) are f16, a probability enters the
// second product as an f16 pair, and the operands' layouts are those of attend_bias_split_k.
// NDW: output tiles a wave; KR: 16-byte pieces a thread moves for 32 rows.
constexpr int KT = 32;
constexpr int SPLIT_MAX = 256;
template <int KR> struct RowPieces {
    uint4 r[KR];
    int nseg, dq, dr, row0, seg0;
    IT_DEV RowPieces(int n) : nseg(n), dq(256 / n), dr(256 % n), row0(threadIdx.x / n), seg0(threadIdx.x % n) {}
    // f(i, row, seg) of this thread's pieces
    template <class F> IT_DEV void each(F f) {
        int row = row0, seg = seg0;
#pragma unroll
        for (int i = 0; i < KR; i++) {
            f(i, row, seg);
            row += dq;
            seg += dr;
            if (seg >= nseg) seg -= nseg, row++;
        }
    }
    // `rows` rows from src on, `stride` elements apart and as long at most; zeros for the rest of 32
    IT_DEV void fetch(const uint16_t* src, int64_t stride, int rows) {
        each([&](int i, int row, int seg) __attribute__((always_inline)) {
            r[i] = row < rows && seg * 8 < stride ? *(const uint4*)(src + row * stride + seg * 8) : make_uint4(0, 0, 0, 0);
        });
    }
    IT_DEV void stash(uint16_t* to, int rs) {
        each([&](int i, int row, int seg) __attribute__((always_inline)) {
            if (row < KT) *(uint4*)(to + row * rs + seg * 8) = r[i];
        });
    }
};
template <int NDW, int KR>
__global__ __launch_bounds__(256) void attend_shared_split_k(BiasAttnP a, const uint16_t* __restrict__ q16, int chunks, int kp, Partials part) {
    extern __shared__ __align__(16) uint16_t lds[];
    const int RS = kp + 8, NS = kp / 16, ND = part.rp / 32;
    uint16_t *Ks = lds, *Qs = lds + KT * RS;            // [32][RS] each
    float* red = (float*)(lds + 2 * KT * RS);           // [wave][16][64]
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), c = lane & 31, g = lane >> 5;
    const int cw = (a.n_head + chunks - 1) / chunks, h0 = (blockIdx.x % chunks) * cw, t = blockIdx.x / chunks, nh = min(cw, a.n_head - h0);
    const int split = blockIdx.y, n_split = part.n_split;
    const int pos = (a.n_pos_dyn ? *a.n_pos_dyn : a.n_pos) - a.n_q + t, n_pos = pos + 1;
    const int seen = a.window ? max(0, n_pos - a.window) : 0, kpb = max(KT, ((n_pos - seen + n_split - 1) / n_split + 15) & ~15);
    const int k0 = seen + split * kpb, k1 = min(n_pos, k0 + kpb);
    const int64_t qh = (int64_t)t * a.n_head + h0;
    if (k0 >= k1) {
        if (tid < nh) {
            float* ml = part.ml_at(qh + tid, split);
            ml[0] = -INFINITY;
            ml[1] = 0.0f;
        }
        return;
    }
    RowPieces<KR> kr(kp / 8);
    {
        RowPieces<KR> qr(kp / 8);
        qr.fetch(q16 + qh * kp, kp, nh);
        kr.fetch((const uint16_t*)a.k + (int64_t)k0 * a.k_stride, a.k_stride, k1 - k0);
        qr.stash(Qs, RS);
    }
    v16f o[NDW];
#pragma unroll
    for (int dw = 0; dw < NDW; dw++)
#pragma unroll
        for (int i = 0; i < 16; i++) o[dw][i] = 0.0f;
    float m = -INFINITY, l = 0.0f;
    for (int key0 = k0; key0 < k1; key0 += KT) {
        kr.stash(Ks, RS);
        __syncthreads();
        if (key0 + KT < k1) kr.fetch((const uint16_t*)a.k + (int64_t)(key0 + KT) * a.k_stride, a.k_stride, k1 - key0 - KT);
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
        __syncthreads();   // the rows are read: the next ones may land
    }
    l += __shfl_xor(l, 32, 64);
    if (c >= nh) return;
    float* p = part.at(qh + c, split);
#pragma unroll
    for (int dw = 0; dw < NDW; dw++) {
        const int dt = w + 4 * dw;
        if (dt < ND) {
#pragma unroll
            for (int i4 = 0; i4 < 4; i4++)
                *(float4*)(p + 32 * dt + 8 * i4 + 4 * g) = make_float4(o[dw][4 * i4], o[dw][4 * i4 + 1], o[dw][4 * i4 + 2], o[dw][4 * i4 + 3]);
        }
    }
    if (w == 0 && g == 0) {
        float* ml = part.ml_at(qh + c, split);
        ml[0] = m;
        ml[1] = l;
    }
}

// One block per (query, head, 64 elements): 16 groups of threads over the splits, every one's first pieces in flight before it is
// known which splits hold anything
constexpr int EARLY = 8;
__global__ __launch_bounds__(256) void attend_shared_merge_k(BiasAttnP a, Partials part, float* __restrict__ out) {
    __shared__ float wsplit[SPLIT_MAX], red[8], sums[16][64];
    __shared__ int seen[4];
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, grp = tid >> 4, r = blockIdx.y * 64 + (tid & 15) * 4;
    const float* q = part.sums_of(blockIdx.x) + min(r, part.rp - 4);
    float4 v[EARLY];
#pragma unroll
    for (int i = 0; i < EARLY; i++) v[i] = grp + 16 * i < part.n_split ? *(const float4*)(q + (int64_t)(grp + 16 * i) * part.rp) : make_float4(0.f, 0.f, 0.f, 0.f);
    const bool has = tid < part.n_split;
    const float* ml = part.ml_at(blockIdx.x, has ? tid : 0);
    const float ms = has ? ml[0] : -INFINITY, ls = has ? ml[1] : 0.0f;
    float m = group_max<64>(ms);
    const int live = __popcll(__ballot(ms != -INFINITY));   // the splits with keys come first
    if (lane == 0) red[4 + w] = m, seen[w] = live;
    __syncthreads();
    m = fmaxf(fmaxf(red[4], red[5]), fmaxf(red[6], red[7]));
    const int n = (seen[0] + seen[1]) + (seen[2] + seen[3]), h = blockIdx.x % a.n_head;
    const float wgt = ms != -INFINITY ? __builtin_amdgcn_exp2f(ms - m) : 0.0f;
    wsplit[tid] = wgt;
    float l = block_sum(ls * wgt, red);
    if (a.sink) l += __builtin_amdgcn_exp2f((a.sinks ? a.sinks[h] * LOG2E : 0.0f) - m);
    float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
    auto add = [&](const float4& v, float x) { acc = make_float4(fmaf(v.x, x, acc.x), fmaf(v.y, x, acc.y), fmaf(v.z, x, acc.z), fmaf(v.w, x, acc.w)); };
#pragma unroll
    for (int i = 0; i < EARLY; i++)
        if (grp + 16 * i < n) add(v[i], wsplit[grp + 16 * i]);
#pragma unroll 8
    for (int s = grp + 16 * EARLY; s < n; s += 16) add(*(const float4*)(q + (int64_t)s * part.rp), wsplit[s]);
    *(float4*)(&sums[grp][(tid & 15) * 4]) = acc;
    __syncthreads();
    if (tid < 64 && (int)blockIdx.y * 64 + tid < a.v_dim) {
        float t = 0.0f;
#pragma unroll
        for (int i = 0; i < 16; i++) t += sums[i][tid];
        out[(int64_t)blockIdx.x * a.v_dim + blockIdx.y * 64 + tid] = t / l;
    }
}

// ---------------------------------------------------------------- the values' matrix
// A block: 32 output dims of one (query, head), a wave eight of them
template <int FMT, bool AL>
__global__ __launch_bounds__(256) void latent_value_k(LatentP p, const float* __restrict__ ol, float* __restrict__ out) {
    __shared__ __align__(16) float xs[RANK_MAX];
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int h = blockIdx.x % p.heads, j0 = blockIdx.y * 32 + w * 8;
    const uint8_t* row[8];
    Raw8<FMT> first[8];
#pragma unroll
    for (int i = 0; i < 8; i++) {
        row[i] = row_at<FMT>(p.uv, (int64_t)h * p.vdim + min(j0 + i, p.vdim - 1), p.rank);
        first[i] = load8<FMT, AL>(row[i], lane * 8, p.rank);
    }
    const float gate = p.gate ? sigmoid_exact(p.gate[blockIdx.x]) : 1.0f;
    for (int r = tid; r < pad8(p.rank); r += 256) xs[r] = r < p.rank ? ol[(int64_t)blockIdx.x * p.rank + r] : 0.0f;
    __syncthreads();
    float acc[8];
#pragma unroll
    for (int i = 0; i < 8; i++) acc[i] = 0.0f;
    for (int k = lane * 8; k < p.rank; k += 512) {
        const float4 x0 = *(const float4*)(xs + k), x1 = *(const float4*)(xs + k + 4);
        const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
        for (int i = 0; i < 8; i++) {
            float f[8];
            widen8<FMT>(k < 512 ? first[i] : load8<FMT, AL>(row[i], k, p.rank), f);
#pragma unroll
            for (int e = 0; e < 8; e++) acc[i] = fmaf(f[e], x[e], acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < 8; i++) {
        acc[i] = group_sum<64>(acc[i]);
        if (lane == i && j0 + i < p.vdim) out[(int64_t)blockIdx.x * p.vdim + j0 + i] = acc[i] * gate;
    }
}

int padded_row(const BiasAttnP& a) { return (a.k_dim + 15) & ~15; }
Partials partials_of(const BiasAttnP& a, float* scratch, int n_split) {
    Partials p{scratch, nullptr, (a.v_dim + 31) & ~31, n_split};
    p.ml = scratch + (size_t)a.n_q * a.n_head * n_split * p.rp;
    return p;
}
size_t shared_lds(const BiasAttnP& a) { return (size_t)2 * KT * (padded_row(a) + 8) * sizeof(uint16_t) + 4 * 16 * 64 * sizeof(float); }
template <class F> bool allow_lds(F* fn, size_t lds) {
    if (lds <= 64 * 1024) return true;
    if (hipFuncSetAttribute((const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess) return true;
    (void)hipGetLastError();
    return false;
}

}  // namespace

void latent_prep(const LatentP& p, float* qa, uint16_t* q16, int kp, float scale, hipStream_t s) {
    const bool al = p.rank % 8 == 0 && aligned16(p.uk);
    const int slices = (p.rank + RB - 1) / RB;
    const dim3 grid(p.heads * slices + (p.kv ? 1 : 0), p.n_tok);
#define IT_CALL(F, A) hipLaunchKernelGGL((latent_prep_k<F, A>), grid, dim3(256), 0, s, p, slices, qa, q16, kp, scale * LOG2E)
    IT_BY_FORMAT(p.uk_fmt, al, IT_CALL);
#undef IT_CALL
}
void latent_rows(const LatentP& p, float* q, hipStream_t s) { hipLaunchKernelGGL(latent_rows_k, dim3(p.n_tok), dim3(256), 0, s, p, q); }
void latent_keys(const LatentP& p, int first, int n_keys, uint16_t* c16, uint16_t* k, int ks, hipStream_t s) {
    hipLaunchKernelGGL(latent_keys_k, dim3(n_keys), dim3(256), 0, s, p, first, c16, k, ks);
}
void latent_value(const LatentP& p, const float* ol, float* out, hipStream_t s) {
    const bool al = p.rank % 8 == 0 && aligned16(p.uv);
    const dim3 grid(p.n_tok * p.heads, (p.vdim + 31) / 32);
#define IT_CALL(F, A) hipLaunchKernelGGL((latent_value_k<F, A>), grid, dim3(256), 0, s, p, ol, out)
    IT_BY_FORMAT(p.uv_fmt, al, IT_CALL);
#undef IT_CALL
}

// one row for all heads, the values its first elements; rows of whole 16-byte pieces; no bias, no temperature
bool attend_shared_takes(const BiasAttnP& a) {
    return !a.kv_f32 && a.k == a.v && a.n_head_kv == 1 && a.v_dim <= a.k_dim && a.k_stride % 8 == 0 && a.k_dim <= a.k_stride && !a.slopes &&
           a.temp_coef == 0.0f && aligned16(a.k) && a.v_dim <= 1024 && a.k_dim <= 1088 && shared_lds(a) <= 156 * 1024;
}
int attend_shared_splits(const BiasAttnP& a, int n_pos_max) {
    const int most = a.window ? std::min(a.window, n_pos_max) : n_pos_max;
    return std::max(1, std::min(most <= 8192 ? 128 : SPLIT_MAX, (most + KT - 1) / KT));
}
int attend_shared_q_row(const BiasAttnP& a) { return padded_row(a); }
size_t attend_shared_scratch_floats(const BiasAttnP& a, int n_split) {
    return (size_t)a.n_q * a.n_head * n_split * (((a.v_dim + 31) & ~31) + 2);
}
bool attend_shared_split(const BiasAttnP& a, const uint16_t* q16, int n_split, float* scratch, float* out, hipStream_t s) {
    if (!attend_shared_takes(a) || n_split < 1 || n_split > SPLIT_MAX || !q16 || !a.k || !scratch) return false;
    const int chunks = (a.n_head + 31) / 32, ndw = (((a.v_dim + 31) / 32) + 3) / 4, kp = padded_row(a), kr = (KT * (kp / 8) + 255) / 256;
    const size_t lds = shared_lds(a);
    const dim3 grid((unsigned)(a.n_q * chunks), n_split);
    const Partials pt = partials_of(a, scratch, n_split);
#define IT_CALL(N, R)                                                                                                     \
    do {                                                                                                                  \
        if (!allow_lds(attend_shared_split_k<N, R>, lds)) return false;                                                    \
        hipLaunchKernelGGL((attend_shared_split_k<N, R>), grid, dim3(256), lds, s, a, q16, chunks, kp, pt);                \
        hipLaunchKernelGGL(attend_shared_merge_k, dim3((unsigned)(a.n_q * a.n_head), (pt.rp + 63) / 64), dim3(256), 0, s, a, pt, out); \
        return true;                                                                                                      \
    } while (0)
    if (ndw <= 1 && kr <= 3) IT_CALL(1, 3);
    if (ndw <= 2 && kr <= 5) IT_CALL(2, 5);
    if (ndw <= 4 && kr <= 9) IT_CALL(4, 9);
    IT_CALL(8, 17);   // (1088 elements: what the LDS holds)
#undef IT_CALL
}

}  // namespace itk
