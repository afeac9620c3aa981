// Attention with what the kernels of k_attn.hip and k_attn_prefill.hip do not have: a distance bias per head
// (score -= slope * (i - j)), a sink in the softmax's denominator (e^sink_h + sum exp(score)), a query temperature that grows
// with the position, a sliding window, and keys and values of different, arbitrary sizes.
//
//     score_ij = (temp(i) q_i . k_j) * scale - slope * (i - j),  i - window < j <= i
//     out_i = sum_j exp(score_ij) v_j / (e^sink_h + sum_j exp(score_ij))
//
// The heads of a cache row are k_stride (v_stride) elements apart, a multiple of eight with zeros behind the head's own
// elements, so that every 16-byte piece of a row is aligned whatever the head size.
//
// attend_bias_plain_k: one block per (query, head), 32-bit arithmetic, f16 or f32 slabs, any shape.
// attend_bias_split_k: up to 16 queries, split over the keys, f16 matrix cores; the partials are merged, and the sink
//     added, by attend_bias_merge_k.
// attend_bias_batch_k: many queries, one pass over the keys.
// The matrix-core kernels form S^T = K Q^T and O^T = V^T P^T as the kernels beside them do (32x32x16: lane l supplies
// eight k values of row l % 32, k group l / 32, for A and for B, and receives column l % 32 and rows
// 8 * (i / 4) + 4 * (l / 32) + i % 4), so the softmax of a query stays in a lane pair.  Keys, values and the scaled
// query are f16; scores, biases, maxima and sums are f32; a probability enters the second product as an f16 pair (high
// half and the remainder), so it keeps 22 bits.  The softmax runs on the visible keys alone and the sink joins at the
// end, where 2^-m is formed in f32: scores far below the sink's 0 keep their precision.
#include <algorithm>

#include "it_device.h"
#include "it_float.h"
#include "it_reduce.h"
#include "kernels_float.h"

namespace itk {
namespace {

typedef _Float16 h8 __attribute__((ext_vector_type(8)));
typedef float v16f __attribute__((ext_vector_type(16)));
constexpr float LOG2E = 1.4426950408889634f;
constexpr int KT = 64;       // keys per tile
constexpr int VS = KT + 4;   // row stride of V^T in LDS, in f16

IT_DEV float temperature(const BiasAttnP& a, int pos) {
    if (a.temp_coef == 0.0f) return 1.0f;
    return 1.0f + a.temp_coef * logf((float)((pos + 1) / a.temp_every + 1));
}

IT_DEV int first_seen(const BiasAttnP& a, int pos) { return a.window ? max(0, pos - a.window + 1) : 0; }
// the sink in the log2 domain, ahead of a maximum
IT_DEV float sink_share(const BiasAttnP& a, int head, float m) {
    return a.sink ? __builtin_amdgcn_exp2f((a.sinks ? a.sinks[head] * LOG2E : 0.0f) - m) : 0.0f;
}

// ---------------------------------------------------------------- 32-bit, any shape
IT_DEV float block_max(float v, float* red) {
    v = group_max<64>(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
}
IT_DEV float block_total(float v, float* red) {
    v = group_sum<64>(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

template <bool F32>
__global__ __launch_bounds__(256) void attend_bias_plain_k(BiasAttnP a, float* __restrict__ out) {
    extern __shared__ __align__(16) float lds[];
    float* qs = lds;                       // [k_dim]
    float* ps = lds + ((a.k_dim + 3) & ~3);   // [256]
    float* os = ps + 256;                  // [v_dim]
    __shared__ float red[4];
    const int tid = threadIdx.x, t = blockIdx.x / a.n_head, h = blockIdx.x % a.n_head;
    const int kvh = h / (a.n_head / a.n_head_kv);
    const int n_pos = a.n_pos_dyn ? *a.n_pos_dyn : a.n_pos, pos = n_pos - a.n_q + t;
    const int64_t krow = (int64_t)a.n_head_kv * a.k_stride, vrow = (int64_t)a.n_head_kv * a.v_stride;
    const float slope = a.slopes ? a.slopes[h] : 0.0f, temp = temperature(a, pos);
    for (int i = tid; i < a.k_dim; i += 256) qs[i] = a.q[((int64_t)t * a.n_head + h) * a.k_dim + i] * temp;
    for (int i = tid; i < a.v_dim; i += 256) os[i] = 0.0f;
    __syncthreads();
    float m = -INFINITY, l = 0.0f;
    for (int s0 = first_seen(a, pos); s0 <= pos; s0 += 256) {
        const int s = s0 + tid, live = min(256, pos + 1 - s0);
        float sc = -INFINITY;
        if (s <= pos) {
            const int64_t at = s * krow + (int64_t)kvh * a.k_stride;
            float dot = 0.0f;
            for (int i = 0; i < a.k_dim; i++)
                dot = fmaf(qs[i], F32 ? ((const float*)a.k)[at + i] : it_f16_to_f32(((const uint16_t*)a.k)[at + i]), dot);
            sc = dot * a.scale - slope * (float)(pos - s);
        }
        const float m_new = fmaxf(m, block_max(sc, red));
        const float p = s <= pos ? expf(sc - m_new) : 0.0f, alpha = expf(m - m_new);
        ps[tid] = p;
        l = l * alpha + block_total(p, red);   // (its barriers also publish ps)
        m = m_new;
        for (int i = tid; i < a.v_dim; i += 256) {
            float acc = os[i] * alpha;
            const int64_t at = (int64_t)s0 * vrow + (int64_t)kvh * a.v_stride + i;
            for (int c = 0; c < live; c++)
                acc = fmaf(ps[c], F32 ? ((const float*)a.v)[at + c * vrow] : it_f16_to_f32(((const uint16_t*)a.v)[at + c * vrow]), acc);
            os[i] = acc;
        }
        __syncthreads();
    }
    const float den = l + (a.sink ? expf((a.sinks ? a.sinks[h] : 0.0f) - m) : 0.0f);
    for (int i = tid; i < a.v_dim; i += 256) out[((int64_t)t * a.n_head + h) * a.v_dim + i] = os[i] / den;
}

// ---------------------------------------------------------------- tiles of K and V
// HD, HV: the key and value sizes rounded up to whole operands.  K rows go to LDS as stored, V transposed ([dim][key]); pieces
// past a head's stride are zeros.
template <int HD, int HV = HD> struct KvTile {
    static constexpr int KS = HD + 8;
    static constexpr int KSEG = KT * HD / 8 / 256;
    static constexpr int UNITS = (KT / 4) * (HV / 8);
    static constexpr int VU = (UNITS + 255) / 256;
    uint4 rk[KSEG], rv[VU][4];
    const uint16_t *kb, *vb;
    int64_t krow, vrow;
    int ks, vs, tid;
    IT_DEV KvTile(const BiasAttnP& a, int kvh)
        : kb((const uint16_t*)a.k + kvh * a.k_stride), vb((const uint16_t*)a.v + kvh * a.v_stride),
          krow((int64_t)a.n_head_kv * a.k_stride), vrow((int64_t)a.n_head_kv * a.v_stride), ks(a.k_stride), vs(a.v_stride),
          tid(threadIdx.x) {}
    // keys key0 .. key0 + 63, those from `end` on as zeros
    IT_DEV void fetch_k(int key0, int end) {
#pragma unroll
        for (int p = 0; p < KSEG; p++) {
            const int idx = tid + p * 256, key = key0 + idx / (HD / 8), seg = idx % (HD / 8);
            rk[p] = key < end && seg * 8 < ks ? *(const uint4*)(kb + key * krow + seg * 8) : make_uint4(0, 0, 0, 0);
        }
    }
    IT_DEV void fetch_v(int key0, int end) {
#pragma unroll
        for (int u = 0; u < VU; u++) {
            const int unit = tid + u * 256, ka = unit % (KT / 4), b = unit / (KT / 4);
#pragma unroll
            for (int c = 0; c < 4; c++) {
                const int key = key0 + 4 * ka + c;
                rv[u][c] = unit < UNITS && key < end && b * 8 < vs ? *(const uint4*)(vb + key * vrow + 8 * b) : make_uint4(0, 0, 0, 0);
            }
        }
    }
    IT_DEV void stash_k(uint16_t* Ks) {
#pragma unroll
        for (int p = 0; p < KSEG; p++) {
            const int idx = tid + p * 256, key = idx / (HD / 8), seg = idx % (HD / 8);
            *(uint4*)(Ks + key * KS + seg * 8) = rk[p];
        }
    }
    IT_DEV void stash_v(uint16_t* Vt) {
#pragma unroll
        for (int u = 0; u < VU; u++) {
            const int unit = tid + u * 256, ka = unit % (KT / 4), b = unit / (KT / 4);   // a wave's transposed writes: 16 key groups side by side
            if (unit >= UNITS) continue;
            const uint32_t x[4][4] = {{rv[u][0].x, rv[u][0].y, rv[u][0].z, rv[u][0].w},
                                      {rv[u][1].x, rv[u][1].y, rv[u][1].z, rv[u][1].w},
                                      {rv[u][2].x, rv[u][2].y, rv[u][2].z, rv[u][2].w},
                                      {rv[u][3].x, rv[u][3].y, rv[u][3].z, rv[u][3].w}};
#pragma unroll
            for (int p = 0; p < 4; p++) {   // dims 8b + 2p (low halves) and 8b + 2p + 1 (high halves) of the four keys
                const uint32_t lo0 = __builtin_amdgcn_perm(x[1][p], x[0][p], 0x05040100u), lo1 = __builtin_amdgcn_perm(x[3][p], x[2][p], 0x05040100u);
                const uint32_t hi0 = __builtin_amdgcn_perm(x[1][p], x[0][p], 0x07060302u), hi1 = __builtin_amdgcn_perm(x[3][p], x[2][p], 0x07060302u);
                *(uint2*)(Vt + (8 * b + 2 * p) * VS + 4 * ka) = make_uint2(lo0, lo1);
                *(uint2*)(Vt + (8 * b + 2 * p + 1) * VS + 4 * ka) = make_uint2(hi0, hi1);
            }
        }
    }
};

// scores of 64 keys against this lane's query column, biased and masked, and what the softmax makes of them
struct Softmax {
    float m = -INFINITY, l = 0.0f;
    // sc: raw products (already times scale * log2 e); key of (kk, i) = key0 + 32 kk + 8 (i / 4) + 4 g + i % 4; keys past
    // `last` or ahead of `first` are not seen; returns the factor of what was accumulated so far
    // MASKED: some key of the tile lies past `last` or ahead of `first`
    template <bool MASKED>
    IT_DEV float step(v16f (&sc)[2], int key0, int g, int first, int last, float pos, float slope2, h8 (&ph)[4], h8 (&pl)[4]) {
        const float at = -slope2 * (pos - (float)(key0 + 4 * g));   // the bias of the lane's first key; the others are whole steps on
        float mt = -INFINITY;
#pragma unroll
        for (int kk = 0; kk < 2; kk++)
#pragma unroll
            for (int i = 0; i < 16; i++) {
                const int off = 32 * kk + 8 * (i >> 2) + (i & 3);
                float v = sc[kk][i] + fmaf(slope2, (float)off, at);
                if (MASKED) v = key0 + 4 * g + off <= last && key0 + 4 * g + off >= first ? v : -INFINITY;
                sc[kk][i] = v;
                mt = fmaxf(mt, v);
            }
        mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
        const float m_new = fmaxf(m, mt);
        const float base = m_new == -INFINITY ? 0.0f : m_new;   // a tile of which this query sees nothing yet
        const float alpha = __builtin_amdgcn_exp2f(m - base);
        float psum = 0.0f;
#pragma unroll
        for (int kk = 0; kk < 2; kk++)
#pragma unroll
            for (int i = 0; i < 16; i++) {
                const float p = __builtin_amdgcn_exp2f(sc[kk][i] - base);
                psum += p;
                const _Float16 hi = (_Float16)p;
                ph[2 * kk + (i >> 3)][i & 7] = hi;
                pl[2 * kk + (i >> 3)][i & 7] = (_Float16)(p - (float)hi);
            }
        l = l * alpha + psum;
        m = m_new;
        return alpha;
    }
};

// ---------------------------------------------------------------- few queries, split over the keys
// partial of (query, head, split): [HD sums][maximum in the log2 domain][sum]
// A block: one query, one KV head's chunk of up to 32 query heads (its columns), one range of keys.  All four waves form the same
// scores; wave w owns output dims 32 w .. (+ 128).
template <int HD>
__global__ __launch_bounds__(256) void attend_bias_split_k(BiasAttnP a, int n_split, int chunks, float* __restrict__ part) {
    typedef KvTile<HD> Tile;
    constexpr int KS = Tile::KS, NS = HD / 16, ND = HD / 32, NDW = (ND + 3) / 4;
    extern __shared__ __align__(16) uint16_t dlds[];
    uint16_t* Ks = dlds;                 // [64][KS]
    uint16_t* Vt = dlds + KT * KS;       // [HD][VS]
    uint16_t* Qs = Vt + HD * VS;         // [32][KS]
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = lane & 31, g = lane >> 5;
    const int G = a.n_head / a.n_head_kv, cw = (G + chunks - 1) / chunks;
    int b = blockIdx.x;
    const int chunk = b % chunks;
    b /= chunks;
    const int kvh = b % a.n_head_kv, t = b / a.n_head_kv;
    const int first = chunk * cw, nh = min(cw, G - first);   // query heads of this block
    const int h0 = kvh * G + first, split = blockIdx.y;
    const int n_pos_last = a.n_pos_dyn ? *a.n_pos_dyn : a.n_pos;
    const int pos = n_pos_last - a.n_q + t, n_pos = pos + 1;
    const int seen = first_seen(a, pos), kpb = max(16, ((n_pos - seen + n_split - 1) / n_split + 15) & ~15);
    const int k0 = seen + split * kpb, k1 = min(n_pos, k0 + kpb);
    const int64_t head_stride = (int64_t)n_split * (HD + 2);
    float* my = part + (((int64_t)t * a.n_head + h0) * n_split + split) * (HD + 2);
    if (k0 >= k1) {
        if (tid < nh) {
            my[tid * head_stride + HD] = -INFINITY;
            my[tid * head_stride + HD + 1] = 0.0f;
        }
        return;
    }
    Tile tile(a, kvh);
    tile.fetch_k(k0, k1);
    tile.fetch_v(k0, k1);
    const float qsc = temperature(a, pos) * (a.scale * LOG2E);
    for (int i = tid; i < 32 * HD; i += 256) {
        const int row = i / HD, d = i % HD;
        const float v = row < nh && d < a.k_dim ? a.q[((int64_t)t * a.n_head + h0 + row) * a.k_dim + d] * qsc : 0.0f;
        Qs[row * KS + d] = __builtin_bit_cast(uint16_t, (_Float16)v);
    }
    const float slope2 = a.slopes && c < nh ? a.slopes[h0 + c] * LOG2E : 0.0f;
    v16f o[NDW];
#pragma unroll
    for (int dw = 0; dw < NDW; dw++)
#pragma unroll
        for (int i = 0; i < 16; i++) o[dw][i] = 0.0f;
    Softmax sm;
    const int n_kt = (k1 - k0 + KT - 1) / KT;
    for (int kt = 0; kt < n_kt; kt++) {
        const int key0 = k0 + kt * KT;
        tile.stash_k(Ks);
        tile.stash_v(Vt);
        __syncthreads();
        if (kt + 1 < n_kt) {
            tile.fetch_k(key0 + KT, k1);
            tile.fetch_v(key0 + KT, k1);
        }
        v16f sc[2];
#pragma unroll
        for (int kk = 0; kk < 2; kk++)
#pragma unroll
            for (int i = 0; i < 16; i++) sc[kk][i] = 0.0f;
#pragma unroll
        for (int s = 0; s < NS; s++) {
            const h8 qf = *(const h8*)(Qs + c * KS + 16 * s + 8 * g);
#pragma unroll
            for (int kk = 0; kk < 2; kk++)
                sc[kk] = __builtin_amdgcn_mfma_f32_32x32x16_f16(*(const h8*)(Ks + (32 * kk + c) * KS + 16 * s + 8 * g), qf, sc[kk], 0, 0, 0);
        }
        h8 ph[4], pl[4];
        const float alpha = key0 + KT <= k1 ? sm.step<false>(sc, key0, g, k0, k1 - 1, (float)pos, slope2, ph, pl)
                                            : sm.step<true>(sc, key0, g, k0, k1 - 1, (float)pos, slope2, ph, pl);
        if (kt > 0) {
#pragma unroll
            for (int dw = 0; dw < NDW; dw++)
#pragma unroll
                for (int i = 0; i < 16; i++) o[dw][i] *= alpha;
        }
#pragma unroll
        for (int dw = 0; dw < NDW; dw++) {
            const int dt = w + 4 * dw;
            if (dt < ND) {
#pragma unroll
                for (int j = 0; j < 4; j++) {
                    const uint16_t* vp = Vt + (32 * dt + c) * VS + 16 * j + 4 * g;
                    const uint2 v0 = *(const uint2*)vp, v1 = *(const uint2*)(vp + 8);
                    const h8 vf = __builtin_bit_cast(h8, make_uint4(v0.x, v0.y, v1.x, v1.y));
                    o[dw] = __builtin_amdgcn_mfma_f32_32x32x16_f16(vf, ph[j], o[dw], 0, 0, 0);
                    o[dw] = __builtin_amdgcn_mfma_f32_32x32x16_f16(vf, pl[j], o[dw], 0, 0, 0);
                }
            }
        }
        __syncthreads();   // the tiles are read: the next ones may land
    }
    const float l = sm.l + __shfl_xor(sm.l, 32, 64);
    if (c < nh) {
        float* p = my + c * head_stride;
#pragma unroll
        for (int dw = 0; dw < NDW; dw++) {
            const int dt = w + 4 * dw;
            if (dt < ND) {
#pragma unroll
                for (int i4 = 0; i4 < 4; i4++) {
                    float* q = p + 32 * dt + 8 * i4 + 4 * g;   // 8-byte aligned: the partial stride is even
                    *(float2*)q = make_float2(o[dw][4 * i4], o[dw][4 * i4 + 1]);
                    *(float2*)(q + 2) = make_float2(o[dw][4 * i4 + 2], o[dw][4 * i4 + 3]);
                }
            }
        }
        if (w == 0 && g == 0) {
            p[HD] = sm.m;
            p[HD + 1] = l;
        }
    }
}

// one block per (query, head, 32 output dims): the weights of up to 256 splits in LDS, eight groups of 32 threads over them
constexpr int SPLIT_MAX = 256;
__global__ __launch_bounds__(256) void attend_bias_merge_k(BiasAttnP a, const float* __restrict__ part, int n_split, int hd, float* __restrict__ out) {
    __shared__ float wsplit[SPLIT_MAX], red[4], accs[8][32];
    const int tid = threadIdx.x, sg = tid >> 5, i = tid & 31, d = blockIdx.y * 32 + i;
    const float* p = part + (int64_t)blockIdx.x * n_split * (hd + 2);
    const bool has = tid < n_split;
    const float ms = has ? p[(int64_t)tid * (hd + 2) + hd] : -INFINITY;
    const float ls = has ? p[(int64_t)tid * (hd + 2) + hd + 1] : 0.0f;
    float o[SPLIT_MAX / 8];   // every load in flight before the first wait
#pragma unroll
    for (int j = 0; j < SPLIT_MAX / 8; j++) {
        const int sp = sg + 8 * j;
        o[j] = sp < n_split ? p[(int64_t)sp * (hd + 2) + d] : 0.0f;
    }
    const float m = block_max(ms, red);
    const float wgt = ms != -INFINITY ? __builtin_amdgcn_exp2f(ms - m) : 0.0f;
    wsplit[tid] = wgt;
    const float l = block_total(ls * wgt, red) + sink_share(a, blockIdx.x % a.n_head, m);
    float acc = 0.0f;
#pragma unroll
    for (int j = 0; j < SPLIT_MAX / 8; j++) {
        const float ww = wsplit[sg + 8 * j];
        acc += ww != 0.0f ? o[j] * ww : 0.0f;   // a split without keys wrote no sums
    }
    accs[sg][i] = acc;
    __syncthreads();
    if (tid < 32 && d < a.v_dim) {
        const float r = ((accs[0][i] + accs[1][i]) + (accs[2][i] + accs[3][i])) + ((accs[4][i] + accs[5][i]) + (accs[6][i] + accs[7][i]));
        out[(int64_t)blockIdx.x * a.v_dim + d] = r / l;
    }
}

// ---------------------------------------------------------------- many queries
constexpr __host__ __device__ bool q_in_registers(int hd) { return hd <= 192; }
// A block: 128 (token, head) rows of one chunk of a KV head's query heads; a wave: 32 of them, their operands in registers (in
// LDS where heads are so large that the accumulators need them).
template <int HD, int HV>
__global__ __launch_bounds__(256) void attend_bias_batch_k(BiasAttnP a, int chunks, float* __restrict__ out32, uint16_t* __restrict__ out16) {
    typedef KvTile<HD, HV> Tile;
    constexpr int KS = Tile::KS, NS = HD / 16, ND = HV / 32;
    extern __shared__ __align__(16) uint16_t blds[];
    uint16_t* Ks = blds;                 // [64][KS]
    uint16_t* Vt = blds + KT * KS;       // [HV][VS]
    constexpr bool QREG = q_in_registers(HD);
    uint16_t* Qs = Vt + HV * VS;         // [128][KS], or nothing
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r = lane & 31, g = lane >> 5;
    const int G = a.n_head / a.n_head_kv, cw = (G + chunks - 1) / chunks, QT = 128 / cw;
    const int kvh = blockIdx.y / chunks, first = (blockIdx.y % chunks) * cw, nh = min(cw, G - first);
    const int n_qt = (a.n_q + QT - 1) / QT, qt = n_qt - 1 - (int)blockIdx.x;   // the longest rows first
    const int base_pos = a.n_pos - a.n_q;
    const int row = 32 * w + r, rt = row / cw, rh = row % cw;
    const int token = qt * QT + rt;
    const bool valid = rt < QT && token < a.n_q && rh < nh;
    const int head = kvh * G + first + (rh < nh ? rh : 0);
    const int pos = valid ? base_pos + token : base_pos;   // (a row without a query is not stored; it sees a key at least)
    const float slope2 = a.slopes ? a.slopes[head] * LOG2E : 0.0f;
    // this lane's query row, scaled: eight elements of every 16
    h8 qf[QREG ? NS : 1];
    {
        const float sq = valid ? temperature(a, pos) * (a.scale * LOG2E) : 0.0f;
        const float* q = a.q + ((int64_t)(valid ? token : 0) * a.n_head + head) * a.k_dim;
        const bool vec = a.k_dim % 4 == 0 && (reinterpret_cast<uintptr_t>(a.q) & 15) == 0;
#pragma unroll
        for (int s = 0; s < NS; s++) {
            const int d = 16 * s + 8 * g;
            float v[8];
            if (vec) {
                const float4 x0 = d < a.k_dim ? *(const float4*)(q + d) : make_float4(0.f, 0.f, 0.f, 0.f);
                const float4 x1 = d + 4 < a.k_dim ? *(const float4*)(q + d + 4) : make_float4(0.f, 0.f, 0.f, 0.f);
                v[0] = x0.x; v[1] = x0.y; v[2] = x0.z; v[3] = x0.w; v[4] = x1.x; v[5] = x1.y; v[6] = x1.z; v[7] = x1.w;
            } else {
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] = d + e < a.k_dim ? q[d + e] : 0.0f;
            }
            h8 x;
#pragma unroll
            for (int e = 0; e < 8; e++) x[e] = (_Float16)(v[e] * sq);
            if constexpr (QREG) qf[s] = x;
            else *(h8*)(Qs + row * KS + d) = x;   // (read by this wave alone)
        }
    }
    const int first_pos = base_pos + qt * QT, last_pos = base_pos + min(a.n_q, (qt + 1) * QT) - 1;
    const int n_kt = last_pos / KT + 1, kt0 = first_seen(a, first_pos) / KT, seen_by_all = first_seen(a, last_pos);
    const int seen = first_seen(a, pos);
    Tile tile(a, kvh);
    v16f o[ND];
#pragma unroll
    for (int dt = 0; dt < ND; dt++)
#pragma unroll
        for (int i = 0; i < 16; i++) o[dt][i] = 0.0f;
    Softmax sm;
    tile.fetch_k(kt0 * KT, a.n_pos);
    tile.fetch_v(kt0 * KT, a.n_pos);
    for (int kt = kt0; kt < n_kt; kt++) {
        tile.stash_k(Ks);
        tile.stash_v(Vt);
        __syncthreads();
        if (kt + 1 < n_kt) {
            tile.fetch_k((kt + 1) * KT, a.n_pos);
            tile.fetch_v((kt + 1) * KT, a.n_pos);
        }
        v16f sc[2];
#pragma unroll
        for (int kk = 0; kk < 2; kk++)
#pragma unroll
            for (int i = 0; i < 16; i++) sc[kk][i] = 0.0f;
#pragma unroll
        for (int s = 0; s < NS; s++) {
            h8 q;
            if constexpr (QREG) q = qf[s];
            else q = *(const h8*)(Qs + row * KS + 16 * s + 8 * g);
#pragma unroll
            for (int kk = 0; kk < 2; kk++)
                sc[kk] = __builtin_amdgcn_mfma_f32_32x32x16_f16(*(const h8*)(Ks + (32 * kk + r) * KS + 16 * s + 8 * g), q, sc[kk], 0, 0, 0);
            if ((s & 3) == 3) __builtin_amdgcn_sched_barrier(0);   // a few fragments in flight: registers are short
        }
        h8 ph[4], pl[4];
        const float alpha = kt * KT + KT - 1 <= first_pos && kt * KT >= seen_by_all
                                ? sm.step<false>(sc, kt * KT, g, seen, pos, (float)pos, slope2, ph, pl)
                                : sm.step<true>(sc, kt * KT, g, seen, pos, (float)pos, slope2, ph, pl);
        if (__any(alpha != 1.0f)) {
#pragma unroll
            for (int dt = 0; dt < ND; dt++)
#pragma unroll
                for (int i = 0; i < 16; i++) o[dt][i] *= alpha;
        }
#pragma unroll
        for (int dt = 0; dt < ND; dt++) {
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const uint16_t* vp = Vt + (32 * dt + r) * VS + 16 * j + 4 * g;
                const uint2 v0 = *(const uint2*)vp, v1 = *(const uint2*)(vp + 8);
                const h8 vf = __builtin_bit_cast(h8, make_uint4(v0.x, v0.y, v1.x, v1.y));
                o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_f16(vf, ph[j], o[dt], 0, 0, 0);
                o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_f16(vf, pl[j], o[dt], 0, 0, 0);
            }
            __builtin_amdgcn_sched_barrier(0);
        }
        __syncthreads();
    }
    const float l = sm.l + __shfl_xor(sm.l, 32, 64) + sink_share(a, head, sm.m);
    if (!valid) return;
    const float inv = (a.gate ? sigmoid_exact(a.gate[(int64_t)token * a.n_head + head]) : 1.0f) / l;
    const int width = a.n_head * a.v_dim;
#pragma unroll
    for (int dt = 0; dt < ND; dt++)
#pragma unroll
        for (int i4 = 0; i4 < 4; i4++) {
            const int d = 32 * dt + 8 * i4 + 4 * g;
            const float v[4] = {o[dt][4 * i4] * inv, o[dt][4 * i4 + 1] * inv, o[dt][4 * i4 + 2] * inv, o[dt][4 * i4 + 3] * inv};
            const int64_t at32 = (int64_t)token * width + head * a.v_dim + d, at16 = (int64_t)token * pad8(width) + head * a.v_dim + d;
            if (out16 && a.v_dim % 4 == 0) {
                if (d < a.v_dim)
                    *(uint2*)(out16 + at16) = make_uint2(to_bf16(v[0]) | ((uint32_t)to_bf16(v[1]) << 16), to_bf16(v[2]) | ((uint32_t)to_bf16(v[3]) << 16));
            } else if (out16) {
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (d + e < a.v_dim) out16[at16 + e] = to_bf16(v[e]);
            }
            if (out32) {
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (d + e < a.v_dim) out32[at32 + e] = v[e];
            }
        }
}

int padded_head(const BiasAttnP& a) {   // 0: larger than the matrix-core kernels take
    const int d = std::max(a.k_dim, a.v_dim);
    for (int hd : {32, 64, 96, 128, 192, 256})
        if (d <= hd) return hd;
    return 0;
}
size_t split_lds(int hd) { return ((size_t)(KT + 32) * (hd + 8) + (size_t)hd * VS) * sizeof(uint16_t); }
size_t batch_lds(int hd, int hv) { return ((size_t)(KT + (q_in_registers(hd) ? 0 : 128)) * (hd + 8) + (size_t)hv * VS) * sizeof(uint16_t); }
template <class F> bool allow_lds(F* fn, size_t lds) {
    if (lds <= 64 * 1024) return true;
    if (hipFuncSetAttribute((const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess) return true;
    (void)hipGetLastError();
    return false;
}

}  // namespace

void attend_bias_plain(const BiasAttnP& a, float* out, hipStream_t s) {
    const size_t lds = ((size_t)((a.k_dim + 3) & ~3) + 256 + a.v_dim) * sizeof(float);
    const dim3 grid((unsigned)(a.n_q * a.n_head));
    if (a.kv_f32) hipLaunchKernelGGL(attend_bias_plain_k<true>, grid, dim3(256), lds, s, a, out);
    else hipLaunchKernelGGL(attend_bias_plain_k<false>, grid, dim3(256), lds, s, a, out);
}

bool attend_bias_mfma_takes(const BiasAttnP& a) {
    auto al = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
    return !a.kv_f32 && padded_head(a) && a.k_stride % 8 == 0 && a.v_stride % 8 == 0 && al(a.k) && al(a.v);
}
int attend_bias_splits(int n_pos_max, int n_q) {
    (void)n_q;
    return std::max(1, std::min(SPLIT_MAX, (n_pos_max + KT - 1) / KT));
}
size_t attend_bias_scratch_floats(const BiasAttnP& a, int n_split) {
    return (size_t)a.n_q * a.n_head * n_split * (padded_head(a) + 2);
}

#define IT_HEAD(hd, CALL)                    \
    switch (hd) {                            \
        case 32: CALL(32); break;            \
        case 64: CALL(64); break;            \
        case 96: CALL(96); break;            \
        case 128: CALL(128); break;          \
        case 192: CALL(192); break;          \
        case 256: CALL(256); break;          \
        default: return false;               \
    }

bool attend_bias_split(const BiasAttnP& a, int n_split, float* scratch, float* out, hipStream_t s) {
    if (!attend_bias_mfma_takes(a) || n_split > SPLIT_MAX || !a.q || !a.k || !a.v) return false;
    const int hd = padded_head(a), G = a.n_head / a.n_head_kv, chunks = (G + 31) / 32;
    const dim3 grid((unsigned)(a.n_q * a.n_head_kv * chunks), n_split);
#define IT_CALL(HD)                                                                                                  \
    if (!allow_lds(attend_bias_split_k<HD>, split_lds(HD))) return false;                                             \
    hipLaunchKernelGGL(attend_bias_split_k<HD>, grid, dim3(256), split_lds(HD), s, a, n_split, chunks, scratch)
    IT_HEAD(hd, IT_CALL)
#undef IT_CALL
    hipLaunchKernelGGL(attend_bias_merge_k, dim3((unsigned)(a.n_q * a.n_head), (a.v_dim + 31) / 32), dim3(256), 0, s, a, scratch, n_split, hd, out);
    return true;
}

bool attend_bias_batch(const BiasAttnP& a, float* out32, uint16_t* out16, hipStream_t s) {
    if (!attend_bias_mfma_takes(a) || a.n_pos_dyn || !a.q || !a.k || !a.v) return false;
    const int hd = padded_head(a), G = a.n_head / a.n_head_kv, chunks = (G + 31) / 32, cw = (G + chunks - 1) / chunks, QT = 128 / cw;
    const dim3 grid((unsigned)((a.n_q + QT - 1) / QT), (unsigned)(a.n_head_kv * chunks));
#define IT_CALL2(HD, HV)                                                                                             \
    do {                                                                                                             \
        if (!allow_lds(attend_bias_batch_k<HD, HV>, batch_lds(HD, HV))) return false;                                 \
        hipLaunchKernelGGL((attend_bias_batch_k<HD, HV>), grid, dim3(256), batch_lds(HD, HV), s, a, chunks, out32, out16); \
        return true;                                                                                                 \
    } while (0)
    // (values shorter than keys: the pairs that latent attention makes of 64 + 32 and 128 + 64)
    if (hd == 96 && a.v_dim <= 64) IT_CALL2(96, 64);
    if (hd == 192 && a.v_dim <= 128) IT_CALL2(192, 128);
#define IT_CALL(HD) IT_CALL2(HD, HD)
    IT_HEAD(hd, IT_CALL)
#undef IT_CALL
#undef IT_CALL2
    return true;
}
#undef IT_HEAD

}  // namespace itk
