// Products of several unquantized matrices with the same activations (a norm's output feeding the query, key, value,
// gate and up projections of a parallel layer), and sums of products added to the residual stream.
//
// One token (decode): a launch per group.  Every block forms the normed input in LDS while its first weight rows are
// in flight; a wave then takes groups of R rows, 16 bytes of each row a lane, and finishes them where they belong:
// f32 rows, cache slabs, or act(gate) * up.  What an earlier sublayer left to be normed and added to the residual is added
// on the way in: every block forms the sum, the first one stores it, in another buffer than the one all of them read.  Activations stay f32 throughout, so the arithmetic is the same in
// 32-bit mode.  A few tokens: one weight row a wave, eight tokens a pass.  Many tokens take k_gemm_bf16.hip.
#include "it_device.h"
#include "it_float.h"
#include "it_reduce.h"
#include "it_rows8.h"
#include "kernels_float.h"

namespace itk {
namespace {

constexpr int CH = 512;   // elements of a row a wave takes at a time, eight a lane

// which matrix a group of rows belongs to
struct Groups {
    int first[GROUP_MAX + 1];
    int n;
};

constexpr int U = 4;   // row pieces of a wave in flight

template <int FMT, bool AL, int R>
__global__ __launch_bounds__(256) void group_gemv_k(GroupP p, Groups gs) {
    extern __shared__ __align__(16) float xs[];   // the input, zero past its end to a whole number of pieces
    __shared__ float red[4];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int n_ch = (p.n_in + CH - 1) / CH;
    const uint8_t* rp[R];
    Raw8<FMT> w[R][U];
    int mi = 0, j0 = 0;
    auto open = [&](int g) __attribute__((always_inline)) {
        mi = 0;
        while (mi + 1 < p.n_mats && g >= gs.first[mi + 1]) mi++;
        const GroupMat& m = p.m[mi];
        const int at = g - gs.first[mi];
        if (m.up) {
            j0 = at * (R / 2);
#pragma unroll
            for (int r = 0; r < R; r++) rp[r] = row_at<FMT>(r < R / 2 ? m.w : m.up, min(j0 + r % (R / 2), m.n_out - 1), p.n_in);
        } else {
            j0 = at * R;
#pragma unroll
            for (int r = 0; r < R; r++) rp[r] = row_at<FMT>(m.w, min(j0 + r, m.n_out - 1), p.n_in);
        }
    };
    auto load = [&](int c0) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int r = 0; r < R; r++) w[r][u] = load8<FMT, AL>(rp[r], (c0 + u) * CH + lane * 8, p.n_in);
    };
    int g = blockIdx.x * 4 + wave;
    if (g < gs.n) {
        open(g);
        load(0);
    }
    // the input while the first rows are on their way
    {
        float ss = 0.0f;
        if (p.add.y) {
            float *x0 = xs + n_ch * CH, sy = 0.0f;   // the residual behind the input
            if (p.n_in % 4 == 0) {
                for (int i = tid * 4; i < p.n_in; i += 1024) {
                    const float4 v = *(const float4*)(p.add.y + i);
                    *(float4*)(x0 + i) = *(const float4*)(p.x + i);
                    sy = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, sy))));
                    *(float4*)(xs + i) = v;
                }
                for (int i = p.n_in + tid * 4; i < n_ch * CH; i += 1024) *(float4*)(xs + i) = make_float4(0.f, 0.f, 0.f, 0.f);
            } else {
                for (int i = tid; i < n_ch * CH; i += 256) {
                    const float v = i < p.n_in ? p.add.y[i] : 0.0f;
                    if (i < p.n_in) x0[i] = p.x[i];
                    sy = fmaf(v, v, sy);
                    xs[i] = v;
                }
            }
            sy = block_sum(sy, red);   // (its barriers also publish xs and x0)
            const float r = p.add.mult / sqrtf(sy / (float)p.n_in + p.add.eps);
            for (int i = tid; i < p.n_in; i += 256) {
                const float v = fmaf(xs[i] * p.add.w[i], r, x0[i]);
                ss = fmaf(v, v, ss);
                xs[i] = v;
                if (blockIdx.x == 0) p.add.x_new[i] = v;
            }
        } else if (p.n_in % 4 == 0) {   // (device buffers are 16-byte aligned)
            for (int i = tid * 4; i < n_ch * CH; i += 1024) {
                const float4 v = i < p.n_in ? *(const float4*)(p.x + i) : make_float4(0.f, 0.f, 0.f, 0.f);
                ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
                *(float4*)(xs + i) = v;
            }
        } else {
            for (int i = tid; i < n_ch * CH; i += 256) {
                const float v = i < p.n_in ? p.x[i] : 0.0f;
                ss = fmaf(v, v, ss);
                xs[i] = v;
            }
        }
        if (p.norm_w) {
            ss = block_sum(ss, red);   // (its barriers also publish xs)
            const float rinv = 1.0f / sqrtf(ss / (float)p.n_in + p.eps);
            for (int i = tid; i < p.n_in; i += 256) xs[i] = xs[i] * rinv * p.norm_w[i];
        }
        __syncthreads();
    }
    for (bool first = true; g < gs.n; g += gridDim.x * 4, first = false) {
        if (!first) open(g);
        float acc[R];
#pragma unroll
        for (int r = 0; r < R; r++) acc[r] = 0.0f;
        for (int c0 = 0; c0 < n_ch; c0 += U) {
            if (!first || c0 > 0) load(c0);
#pragma unroll
            for (int u = 0; u < U; u++) {
                if (c0 + u < n_ch) {
                    const float4 x0 = *(const float4*)(xs + (c0 + u) * CH + lane * 8), x1 = *(const float4*)(xs + (c0 + u) * CH + lane * 8 + 4);
                    const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
                    for (int r = 0; r < R; r++) {
                        float f[8];
                        widen8<FMT>(w[r][u], f);
#pragma unroll
                        for (int e = 0; e < 8; e++) acc[r] = fmaf(f[e], x[e], acc[r]);
                    }
                }
            }
        }
#pragma unroll
        for (int r = 0; r < R; r++) acc[r] = group_sum<64>(acc[r]);
        const GroupMat& m = p.m[mi];
        // lane r finishes row r
        if (m.up) {
#pragma unroll
            for (int r = 0; r < R / 2; r++)
                if (lane == r && j0 + r < m.n_out) group_store(m, 0, j0 + r, act_of(m.act, acc[r]) * acc[R / 2 + r]);
        } else {
#pragma unroll
            for (int r = 0; r < R; r++)
                if (lane == r && j0 + r < m.n_out) group_store(m, 0, j0 + r, acc[r]);
        }
    }
}

// ---------------------------------------------------------------- one token: sum of products into the residual
// Eight waves a block, S of them on a group of R rows: the pieces of the terms' rows, one term behind the other, are dealt to
// them in turn, and so sit in LDS: piece q of the inputs at q * CH.
template <int FMT, bool AL, int R, int S>
__global__ __launch_bounds__(512) void res_gemv_k(ResP p) {
    constexpr int W = 8, UR = 8 / R;
    extern __shared__ __align__(16) float xs[];
    __shared__ float red[W], part_sum[W][R][RES_MAX];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int j0 = (blockIdx.x * (W / S) + wave / S) * R, s = wave % S;
    const int n0 = (p.t[0].n_in + CH - 1) / CH, n1 = p.n_terms > 1 ? (p.t[1].n_in + CH - 1) / CH : 0, nq = n0 + n1;
    const uint8_t* rp[RES_MAX][R];
#pragma unroll
    for (int r = 0; r < R; r++) {
        const int j = min(j0 + r, p.n_out - 1);
        rp[0][r] = row_at<FMT>(p.t[0].w, j, p.t[0].n_in);
        rp[1][r] = n1 ? row_at<FMT>(p.t[1].w, j, p.t[1].n_in) : rp[0][r];
    }
    Raw8<FMT> w[R][UR];
    auto load = [&](int q0) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < UR; u++) {
            const int q = q0 + s + S * u;
#pragma unroll
            for (int r = 0; r < R; r++) {
                if (q < n0) w[r][u] = load8<FMT, AL>(rp[0][r], q * CH + lane * 8, p.t[0].n_in);
                else if (q < nq) w[r][u] = load8<FMT, AL>(rp[1][r], (q - n0) * CH + lane * 8, p.t[1].n_in);
            }
        }
    };
    load(0);
    float* at = xs;
    for (int k = 0; k < p.n_terms; k++) {
        const int n = p.t[k].n_in, len = (n + CH - 1) / CH * CH;
        const float* in = p.t[k].in;
        if (n % 4 == 0) {   // (device buffers are 16-byte aligned)
            for (int i = tid * 4; i < len; i += 2048) *(float4*)(at + i) = i < n ? *(const float4*)(in + i) : make_float4(0.f, 0.f, 0.f, 0.f);
        } else {
            for (int i = tid; i < len; i += 512) at[i] = i < n ? in[i] : 0.0f;
        }
        at += len;
    }
    at = xs;
    for (int k = 0; k < p.n_terms; k++) {
        const ResTerm& t = p.t[k];
        if (t.norm_w) {   // a part of the row to one, two, four or all eight waves
            const int part = t.n_in / t.norm_groups, wpg = t.norm_groups > 4 ? 1 : t.norm_groups > 2 ? 2 : t.norm_groups > 1 ? 4 : 8;
            __syncthreads();
            for (int g0 = 0; g0 < t.norm_groups; g0 += W / wpg) {
                const int gi = g0 + wave / wpg, sub = wave % wpg;
                float* a = at + gi * part;
                float ss = 0.0f;
                if (gi < t.norm_groups)
                    for (int i = sub * 64 + lane; i < part; i += 64 * wpg) ss = fmaf(a[i], a[i], ss);
                ss = group_sum<64>(ss);
                if (wpg > 1) {
                    if (lane == 0) red[wave] = ss;
                    __syncthreads();
                    ss = 0.0f;
                    for (int i = 0; i < wpg; i++) ss += red[wave - sub + i];
                }
                const float rinv = 1.0f / sqrtf(ss / (float)part + t.eps);
                if (gi < t.norm_groups)
                    for (int i = sub * 64 + lane; i < part; i += 64 * wpg) {
                        const float v = a[i] * rinv * t.norm_w[t.norm_period == part ? i : gi * part + i];
                        a[i] = t.gate ? v * silu_exact(t.gate[gi * part + i]) : v;
                    }
            }
        }
        at += (t.n_in + CH - 1) / CH * CH;
    }
    __syncthreads();
    float acc[RES_MAX][R];
#pragma unroll
    for (int k = 0; k < RES_MAX; k++)
#pragma unroll
        for (int r = 0; r < R; r++) acc[k][r] = 0.0f;
    for (int q0 = 0; q0 < nq; q0 += S * UR) {
        if (q0) load(q0);
#pragma unroll
        for (int u = 0; u < UR; u++) {
            const int q = q0 + s + S * u;
            if (q >= nq) continue;
            const float4 x0 = *(const float4*)(xs + q * CH + lane * 8), x1 = *(const float4*)(xs + q * CH + lane * 8 + 4);
            const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
            for (int r = 0; r < R; r++) {
                float f[8], v = q < n0 ? acc[0][r] : acc[1][r];
                widen8<FMT>(w[r][u], f);
#pragma unroll
                for (int e = 0; e < 8; e++) v = fmaf(f[e], x[e], v);
                if (q < n0) acc[0][r] = v;
                else acc[1][r] = v;
            }
        }
    }
#pragma unroll
    for (int k = 0; k < RES_MAX; k++)
#pragma unroll
        for (int r = 0; r < R; r++) {
            acc[k][r] = group_sum<64>(acc[k][r]);
            if (S > 1 && lane == 0) part_sum[wave][r][k] = acc[k][r];
        }
    if (S > 1) __syncthreads();
    if (s) return;
#pragma unroll
    for (int r = 0; r < R; r++) {
        if (lane != r || j0 + r >= p.n_out) continue;
        float total = 0.0f;
        for (int k = 0; k < p.n_terms; k++) {
            float v = k ? acc[1][r] : acc[0][r];
            if (S > 1) {
                v = 0.0f;
                for (int i = 0; i < S; i++) v += part_sum[wave + i][r][k];
            }
            total += p.t[k].scale ? v * p.t[k].scale[j0 + r] : v;
        }
        p.x[j0 + r] = p.set ? total : p.x[j0 + r] + total;
    }
}

// ---------------------------------------------------------------- a few tokens
constexpr int NT = 8;

template <int FMT, bool AL>
IT_DEV void dot_rows(const uint8_t* row, const float* x, int n_in, int n_tok, int t0, int lane, float* acc) {
#pragma unroll
    for (int t = 0; t < NT; t++) acc[t] = 0.0f;
    for (int k = lane * 8; k < n_in; k += CH) {
        float f[8];
        widen8<FMT>(load8<FMT, AL>(row, k, n_in), f);
#pragma unroll
        for (int t = 0; t < NT; t++) {
            if (t0 + t < n_tok) {
                const float* xt = x + (int64_t)(t0 + t) * n_in + k;
#pragma unroll
                for (int e = 0; e < 8; e++)
                    if (AL || k + e < n_in) acc[t] = fmaf(f[e], xt[e], acc[t]);
            }
        }
    }
#pragma unroll
    for (int t = 0; t < NT; t++) acc[t] = group_sum<64>(acc[t]);
}

template <int FMT, bool AL>
__global__ __launch_bounds__(256) void group_rows_k(GroupP p, Groups gs) {   // a group is one row (one gate / up pair)
    const int lane = threadIdx.x & 63, g = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    if (g >= gs.n) return;
    int mi = 0;
    while (mi + 1 < p.n_mats && g >= gs.first[mi + 1]) mi++;
    const GroupMat& m = p.m[mi];
    const int j = g - gs.first[mi], t0 = blockIdx.y * NT;
    float a[NT], b[NT];
    dot_rows<FMT, AL>(row_at<FMT>(m.w, j, p.n_in), p.x, p.n_in, p.n_tok, t0, lane, a);
    if (m.up) dot_rows<FMT, AL>(row_at<FMT>(m.up, j, p.n_in), p.x, p.n_in, p.n_tok, t0, lane, b);
#pragma unroll
    for (int t = 0; t < NT; t++)
        if (lane == t && t0 + t < p.n_tok) group_store(m, t0 + t, j, m.up ? act_of(m.act, a[t]) * b[t] : a[t]);
}

template <int FMT, bool AL>
__global__ __launch_bounds__(256) void res_rows_k(ResP p) {
    const int lane = threadIdx.x & 63, j = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    if (j >= p.n_out) return;
    const int t0 = blockIdx.y * NT;
    float total[NT], a[NT];
#pragma unroll
    for (int t = 0; t < NT; t++) total[t] = 0.0f;
    for (int k = 0; k < p.n_terms; k++) {
        const ResTerm& q = p.t[k];
        dot_rows<FMT, AL>(row_at<FMT>(q.w, j, q.n_in), q.in, q.n_in, p.n_tok, t0, lane, a);
        const float sc = q.scale ? q.scale[j] : 1.0f;
#pragma unroll
        for (int t = 0; t < NT; t++) total[t] += a[t] * sc;
    }
#pragma unroll
    for (int t = 0; t < NT; t++)
        if (lane == t && t0 + t < p.n_tok) {
            float* x = p.x + (int64_t)(t0 + t) * p.n_out + j;
            *x = p.set ? total[t] : *x + total[t];
        }
}

// ---------------------------------------------------------------- norms, conversions, sums
__global__ __launch_bounds__(256) void norm_rows_k(const float* __restrict__ x, const float* __restrict__ w, int groups, float eps,
                                                   int nd, float* __restrict__ out32, uint16_t* __restrict__ out16) {
    __shared__ float red[4];
    const int part = nd / groups, g = blockIdx.y, tid = threadIdx.x;
    const int64_t row = blockIdx.x;
    const float* xr = x + row * nd + g * part;
    float rinv = 1.0f;
    if (w) {
        float ss = 0.0f;
        for (int i = tid; i < part; i += 256) ss = fmaf(xr[i], xr[i], ss);
        ss = block_sum(ss, red);
        rinv = 1.0f / sqrtf(ss / (float)part + eps);
    }
    for (int i = tid; i < part; i += 256) {
        const float v = w ? xr[i] * rinv * w[g * part + i] : xr[i];
        if (out32) out32[row * nd + g * part + i] = v;
        if (out16) out16[row * pad8(nd) + g * part + i] = to_bf16(v);
    }
    if (out16 && g == groups - 1 && tid < pad8(nd) - nd) out16[row * pad8(nd) + nd + tid] = 0;
}

// parts of whole float4s, rows of whole 16-byte bf16 pieces: a thread keeps its pieces between the two passes (up to 8,192
// elements a part)
template <int V>
__global__ __launch_bounds__(256) void norm_rows4_k(const float* __restrict__ x, const float* __restrict__ w, float eps, int part,
                                                    float* __restrict__ out32, uint16_t* __restrict__ out16) {
    __shared__ float red[4];
    const int tid = threadIdx.x, n4 = part >> 2;
    const int64_t at0 = ((int64_t)blockIdx.x * gridDim.y + blockIdx.y) * part;   // rows are `gridDim.y` parts
    const float4* xr = (const float4*)(x + at0);
    w += blockIdx.y * part;
    float4 v[V];
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < V; i++) {
        const int at = tid + i * 256;
        v[i] = at < n4 ? xr[at] : make_float4(0.f, 0.f, 0.f, 0.f);
        ss = fmaf(v[i].x, v[i].x, fmaf(v[i].y, v[i].y, fmaf(v[i].z, v[i].z, fmaf(v[i].w, v[i].w, ss))));
    }
    ss = block_sum(ss, red);
    const float rinv = 1.0f / sqrtf(ss / (float)part + eps);
#pragma unroll
    for (int i = 0; i < V; i++) {
        const int at = tid + i * 256;
        if (at >= n4) continue;
        const float4 ww = ((const float4*)w)[at];
        const float4 r = make_float4(v[i].x * rinv * ww.x, v[i].y * rinv * ww.y, v[i].z * rinv * ww.z, v[i].w * rinv * ww.w);
        if (out32) ((float4*)(out32 + at0))[at] = r;
        if (out16)
            ((uint2*)(out16 + at0))[at] = make_uint2(to_bf16(r.x) | ((uint32_t)to_bf16(r.y) << 16), to_bf16(r.z) | ((uint32_t)to_bf16(r.w) << 16));
    }
}

// a wave a part (a head's output, as a rule)
__global__ __launch_bounds__(256) void norm_gate_rows_k(const float* __restrict__ x, const float* __restrict__ w, int period, const float* __restrict__ gate,
                                                        int groups, float eps, int64_t n_parts, int nd, float* __restrict__ out32, uint16_t* __restrict__ out16) {
    const int part = nd / groups, lane = threadIdx.x & 63;
    const int64_t at = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (at >= n_parts) return;
    const int64_t row = at / groups;
    const int j0 = (int)(at % groups) * part;
    const float* xr = x + row * nd + j0;
    float ss = 0.0f;
    for (int i = lane; i < part; i += 64) ss = fmaf(xr[i], xr[i], ss);
    const float rinv = 1.0f / sqrtf(group_sum<64>(ss) / (float)part + eps);
    for (int i = lane; i < part; i += 64) {
        float v = xr[i] * rinv * w[period == part ? i : j0 + i];
        if (gate) v *= silu_exact(gate[row * nd + j0 + i]);
        if (out32) out32[row * nd + j0 + i] = v;
        if (out16) out16[row * pad8(nd) + j0 + i] = to_bf16(v);
    }
    if (out16 && j0 + part == nd && lane < pad8(nd) - nd) out16[row * pad8(nd) + nd + lane] = 0;
}

// the same for parts of whole float4s, rows of whole 16-byte bf16 pieces: a lane keeps its V pieces
template <int V>
__global__ __launch_bounds__(256) void norm_gate_rows4_k(const float* __restrict__ x, const float* __restrict__ w, int period, const float* __restrict__ gate,
                                                         int groups, float eps, int64_t n_parts, int nd, float* __restrict__ out32, uint16_t* __restrict__ out16) {
    const int part = nd / groups, n4 = part >> 2, lane = threadIdx.x & 63;
    const int64_t at = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (at >= n_parts) return;
    const int64_t at0 = at * part;   // (rows are `groups` parts)
    if (period != part) w += at % groups * part;
    float4 v[V], z[V];
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < V; i++) {
        const int k = lane + i * 64;
        v[i] = k < n4 ? ((const float4*)(x + at0))[k] : make_float4(0.f, 0.f, 0.f, 0.f);
        if (gate) z[i] = k < n4 ? ((const float4*)(gate + at0))[k] : make_float4(0.f, 0.f, 0.f, 0.f);
        ss = fmaf(v[i].x, v[i].x, fmaf(v[i].y, v[i].y, fmaf(v[i].z, v[i].z, fmaf(v[i].w, v[i].w, ss))));
    }
    const float rinv = 1.0f / sqrtf(group_sum<64>(ss) / (float)part + eps);
#pragma unroll
    for (int i = 0; i < V; i++) {
        const int k = lane + i * 64;
        if (k >= n4) continue;
        const float4 ww = ((const float4*)w)[k];
        float4 r = make_float4(v[i].x * rinv * ww.x, v[i].y * rinv * ww.y, v[i].z * rinv * ww.z, v[i].w * rinv * ww.w);
        if (gate) r = make_float4(r.x * silu_exact(z[i].x), r.y * silu_exact(z[i].y), r.z * silu_exact(z[i].z), r.w * silu_exact(z[i].w));
        if (out32) ((float4*)(out32 + at0))[k] = r;
        if (out16)
            ((uint2*)(out16 + at0))[k] = make_uint2(to_bf16(r.x) | ((uint32_t)to_bf16(r.y) << 16), to_bf16(r.z) | ((uint32_t)to_bf16(r.w) << 16));
    }
}

// V > 0: rows of whole float4s, a thread keeps its V pieces; V = 0: any row, through x_new
template <int V>
__global__ __launch_bounds__(256) void add_norm_rows_k(const float* __restrict__ x, AddNormed a, const float* __restrict__ w, float eps, int nd,
                                                       float* __restrict__ out32, uint16_t* __restrict__ out16) {
    __shared__ float red[4];
    const int tid = threadIdx.x;
    const int64_t row = blockIdx.x;
    const float *xr = x + row * nd, *yr = a.y + row * nd;
    float *xn = a.x_new + row * nd, sy = 0.0f, ss = 0.0f;
    if constexpr (V > 0) {
        const int n4 = nd >> 2;
        float4 xv[V], yv[V];
#pragma unroll
        for (int i = 0; i < V; i++) {
            const int at = tid + i * 256;
            xv[i] = at < n4 ? ((const float4*)xr)[at] : make_float4(0.f, 0.f, 0.f, 0.f);
            yv[i] = at < n4 ? ((const float4*)yr)[at] : make_float4(0.f, 0.f, 0.f, 0.f);
            sy = fmaf(yv[i].x, yv[i].x, fmaf(yv[i].y, yv[i].y, fmaf(yv[i].z, yv[i].z, fmaf(yv[i].w, yv[i].w, sy))));
        }
        const float r = a.mult / sqrtf(block_sum(sy, red) / (float)nd + a.eps);
#pragma unroll
        for (int i = 0; i < V; i++) {
            const int at = tid + i * 256;
            if (at >= n4) continue;
            const float4 ww = ((const float4*)a.w)[at];
            float4& v = xv[i];
            v = make_float4(fmaf(yv[i].x * ww.x, r, v.x), fmaf(yv[i].y * ww.y, r, v.y), fmaf(yv[i].z * ww.z, r, v.z), fmaf(yv[i].w * ww.w, r, v.w));
            ((float4*)xn)[at] = v;
            ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
        }
        if (!w) return;
        const float rinv = 1.0f / sqrtf(block_sum(ss, red) / (float)nd + eps);
#pragma unroll
        for (int i = 0; i < V; i++) {
            const int at = tid + i * 256;
            if (at >= n4) continue;
            const float4 ww = ((const float4*)w)[at], v = xv[i];
            const float4 h = make_float4(v.x * rinv * ww.x, v.y * rinv * ww.y, v.z * rinv * ww.z, v.w * rinv * ww.w);
            if (out32) ((float4*)(out32 + row * nd))[at] = h;
            if (out16)
                ((uint2*)(out16 + row * nd))[at] = make_uint2(to_bf16(h.x) | ((uint32_t)to_bf16(h.y) << 16), to_bf16(h.z) | ((uint32_t)to_bf16(h.w) << 16));
        }
    } else {
        for (int i = tid; i < nd; i += 256) sy = fmaf(yr[i], yr[i], sy);
        const float r = a.mult / sqrtf(block_sum(sy, red) / (float)nd + a.eps);
        for (int i = tid; i < nd; i += 256) {
            const float v = fmaf(yr[i] * a.w[i], r, xr[i]);
            xn[i] = v;
            ss = fmaf(v, v, ss);
        }
        if (!w) return;
        const float rinv = 1.0f / sqrtf(block_sum(ss, red) / (float)nd + eps);
        for (int i = tid; i < nd; i += 256) {   // (a thread's own elements)
            const float h = xn[i] * rinv * w[i];
            if (out32) out32[row * nd + i] = h;
            if (out16) out16[row * pad8(nd) + i] = to_bf16(h);
        }
        if (out16 && tid < pad8(nd) - nd) out16[row * pad8(nd) + nd + tid] = 0;
    }
}

__global__ void act_mul_k(float* __restrict__ a, const float* __restrict__ b, int64_t n, int act) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i < n) a[i] = act_of(act, a[i]) * b[i];
}

__global__ void widen_rows_k(const uint16_t* __restrict__ in, int nd, float* __restrict__ out, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i < n) out[i] = it_bf16_to_f32(in[i / nd * pad8(nd) + i % nd]);
}

__global__ void group_scatter_k(GroupMat m, const float* __restrict__ rows, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    group_store(m, (int)(i / m.n_out), (int)(i % m.n_out), rows[i]);
}

__global__ void scaled_residual_k(float* __restrict__ x, const float* __restrict__ a, const float* __restrict__ sa,
                                  const float* __restrict__ b, const float* __restrict__ sb, int set, int nd, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const int j = (int)(i % nd);
    float v = sa ? a[i] * sa[j] : a[i];
    if (b) v += sb ? b[i] * sb[j] : b[i];
    x[i] = set ? v : x[i] + v;
}

__global__ void add_rows_k(float* __restrict__ x, const float* __restrict__ rows, const float* __restrict__ vec, int nd, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    float v = x[i];
    if (rows) v += rows[i];
    if (vec) v += vec[i % nd];
    x[i] = v;
}

__global__ void gather_rows_k(const float* __restrict__ src, const int32_t* __restrict__ idx, int nd, float* __restrict__ out, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    out[i] = src[(int64_t)idx[i / nd] * nd + i % nd];
}

Groups groups_of(const GroupP& p, int rows_per_group) {
    Groups g{};
    for (int i = 0; i < p.n_mats; i++) {
        const int per = p.m[i].up ? (rows_per_group > 1 ? rows_per_group / 2 : 1) : rows_per_group;
        g.first[i + 1] = g.first[i] + (p.m[i].n_out + per - 1) / per;
    }
    g.n = g.first[p.n_mats];
    return g;
}
bool group_aligned(const GroupP& p) {
    bool al = p.n_in % 8 == 0;
    for (int i = 0; i < p.n_mats; i++) al = al && aligned16(p.m[i].w) && aligned16(p.m[i].up);
    return al;
}
bool res_aligned(const ResP& p) {
    bool al = true;
    for (int i = 0; i < p.n_terms; i++) al = al && p.t[i].n_in % 8 == 0 && aligned16(p.t[i].w);
    return al;
}
size_t padded(int n) { return (size_t)((n + CH - 1) / CH * CH); }
size_t group_lds(const GroupP& p) { return padded(p.n_in) * (p.add.y ? 2 : 1) * sizeof(float); }
constexpr size_t LDS_MAX = 144 * 1024;

template <class F> bool allow_lds(F* fn, size_t lds) {
    if (lds <= 64 * 1024) return true;
    if (hipFuncSetAttribute((const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)LDS_MAX) == hipSuccess) return true;
    (void)hipGetLastError();
    return false;
}

template <int FMT, bool AL> bool launch_group(const GroupP& p, hipStream_t s) {
    const size_t lds = group_lds(p);
    Groups g4 = groups_of(p, 4);
    if (g4.n >= 2048) {   // enough groups of four rows to keep every wave of the chip at work
        if (!allow_lds(group_gemv_k<FMT, AL, 4>, lds)) return false;
        hipLaunchKernelGGL((group_gemv_k<FMT, AL, 4>), dim3(min((g4.n + 3) / 4, 1024)), dim3(256), lds, s, p, g4);
    } else {
        Groups g2 = groups_of(p, 2);
        if (!allow_lds(group_gemv_k<FMT, AL, 2>, lds)) return false;
        hipLaunchKernelGGL((group_gemv_k<FMT, AL, 2>), dim3(min((g2.n + 3) / 4, 1024)), dim3(256), lds, s, p, g2);
    }
    return true;
}
// about one block a CU and eight rows in the making in it: rows shared by several waves where there are few, several rows a
// wave where there are many
template <int FMT, bool AL> bool launch_res(const ResP& p, hipStream_t s) {
    size_t lds = 0;
    for (int i = 0; i < p.n_terms; i++) lds += padded(p.t[i].n_in) * sizeof(float);
#define IT_RES(R, S)                                                                                        \
    do {                                                                                                    \
        if (!allow_lds(res_gemv_k<FMT, AL, R, S>, lds)) return false;                                       \
        const int per = 8 / S * R;                                                                          \
        hipLaunchKernelGGL((res_gemv_k<FMT, AL, R, S>), dim3((p.n_out + per - 1) / per), dim3(512), lds, s, p); \
        return true;                                                                                        \
    } while (0)
    if (p.n_out <= 512) IT_RES(1, 4);
    if (p.n_out <= 1024) IT_RES(1, 2);
    if (p.n_out <= 2048) IT_RES(1, 1);
    IT_RES(2, 1);
#undef IT_RES
}

}  // namespace

bool group_gemv_takes(const GroupP& p) { return p.n_tok == 1 && group_lds(p) <= LDS_MAX; }
bool group_gemv(const GroupP& p, hipStream_t s) {
    if (!group_gemv_takes(p)) return false;
    const bool al = group_aligned(p);
    bool ok = false;
#define IT_CALL(F, A) ok = launch_group<F, A>(p, s)
    IT_BY_FORMAT(p.fmt, al, IT_CALL);
#undef IT_CALL
    return ok;
}

bool res_gemv_takes(const ResP& p) {
    size_t lds = 0;
    for (int i = 0; i < p.n_terms; i++) lds += padded(p.t[i].n_in) * sizeof(float);
    return p.n_tok == 1 && lds <= LDS_MAX;
}
bool res_gemv(const ResP& p, hipStream_t s) {
    if (!res_gemv_takes(p)) return false;
    const bool al = res_aligned(p);
    bool ok = false;
#define IT_CALL(F, A) ok = launch_res<F, A>(p, s)
    IT_BY_FORMAT(p.fmt, al, IT_CALL);
#undef IT_CALL
    return ok;
}

void group_rows(const GroupP& p, hipStream_t s) {
    const Groups g = groups_of(p, 1);
    const bool al = group_aligned(p);
    const dim3 grid((g.n + 3) / 4, (p.n_tok + NT - 1) / NT);
#define IT_CALL(F, A) hipLaunchKernelGGL((group_rows_k<F, A>), grid, dim3(256), 0, s, p, g)
    IT_BY_FORMAT(p.fmt, al, IT_CALL);
#undef IT_CALL
}
void res_rows(const ResP& p, hipStream_t s) {
    const bool al = res_aligned(p);
    const dim3 grid((p.n_out + 3) / 4, (p.n_tok + NT - 1) / NT);
#define IT_CALL(F, A) hipLaunchKernelGGL((res_rows_k<F, A>), grid, dim3(256), 0, s, p)
    IT_BY_FORMAT(p.fmt, al, IT_CALL);
#undef IT_CALL
}

void norm_rows(const float* x, const float* w, int groups, float eps, int64_t n_rows, int nd, float* out32, uint16_t* out16, hipStream_t s) {
    if (n_rows <= 0) return;
    const int part = nd / groups;
    if (w && nd % 8 == 0 && part % 4 == 0 && part <= 8192 && aligned16(x) && aligned16(w) && aligned16(out32) && aligned16(out16)) {
        const dim3 grid((unsigned)n_rows, groups);
        if (part <= 1024) hipLaunchKernelGGL(norm_rows4_k<1>, grid, dim3(256), 0, s, x, w, eps, part, out32, out16);
        else if (part <= 2048) hipLaunchKernelGGL(norm_rows4_k<2>, grid, dim3(256), 0, s, x, w, eps, part, out32, out16);
        else if (part <= 4096) hipLaunchKernelGGL(norm_rows4_k<4>, grid, dim3(256), 0, s, x, w, eps, part, out32, out16);
        else hipLaunchKernelGGL(norm_rows4_k<8>, grid, dim3(256), 0, s, x, w, eps, part, out32, out16);
        return;
    }
    hipLaunchKernelGGL(norm_rows_k, dim3((unsigned)n_rows, groups), dim3(256), 0, s, x, w, groups, eps, nd, out32, out16);
}

void norm_gate_rows(const float* x, const float* w, int period, const float* gate, int groups, float eps, int64_t n_rows, int nd,
                    float* out32, uint16_t* out16, hipStream_t s) {
    if (n_rows <= 0) return;
    const int64_t parts = n_rows * groups;
    const int part = nd / groups;
    if (nd % 8 == 0 && part % 4 == 0 && part <= 1024 && aligned16(x) && aligned16(w) && aligned16(gate) && aligned16(out32) && aligned16(out16)) {
        const dim3 grid((unsigned)((parts + 3) / 4));
        if (part <= 256) hipLaunchKernelGGL(norm_gate_rows4_k<1>, grid, dim3(256), 0, s, x, w, period, gate, groups, eps, parts, nd, out32, out16);
        else hipLaunchKernelGGL(norm_gate_rows4_k<4>, grid, dim3(256), 0, s, x, w, period, gate, groups, eps, parts, nd, out32, out16);
        return;
    }
    hipLaunchKernelGGL(norm_gate_rows_k, dim3((unsigned)((parts + 3) / 4)), dim3(256), 0, s, x, w, period, gate, groups, eps, parts, nd, out32, out16);
}

void add_norm_rows(const float* x, const AddNormed& add, const float* norm_w, float eps, int64_t n_rows, int nd, float* out32,
                   uint16_t* out16, hipStream_t s) {
    if (n_rows <= 0) return;
    const dim3 grid((unsigned)n_rows), block(256);
    const bool al = nd % 8 == 0 && aligned16(x) && aligned16(add.y) && aligned16(add.x_new) && aligned16(add.w) && aligned16(norm_w) &&
                    aligned16(out32) && aligned16(out16);
#define IT_CALL(V) hipLaunchKernelGGL(add_norm_rows_k<V>, grid, block, 0, s, x, add, norm_w, eps, nd, out32, out16)
    if (!al || nd > 8192) IT_CALL(0);
    else if (nd <= 1024) IT_CALL(1);
    else if (nd <= 2048) IT_CALL(2);
    else if (nd <= 4096) IT_CALL(4);
    else IT_CALL(8);
#undef IT_CALL
}

static dim3 per_element(int64_t n) { return dim3((unsigned)((n + 255) / 256)); }
void widen_rows(const uint16_t* in, int64_t n_rows, int nd, float* out, hipStream_t s) {
    const int64_t n = n_rows * nd;
    hipLaunchKernelGGL(widen_rows_k, per_element(n), dim3(256), 0, s, in, nd, out, n);
}
void group_scatter(const GroupMat& m, const float* rows, int n_tok, hipStream_t s) {
    const int64_t n = (int64_t)n_tok * m.n_out;
    hipLaunchKernelGGL(group_scatter_k, per_element(n), dim3(256), 0, s, m, rows, n);
}
void scaled_residual(float* x, const float* a, const float* sa, const float* b, const float* sb, int set, int64_t n_rows, int nd, hipStream_t s) {
    const int64_t n = n_rows * nd;
    hipLaunchKernelGGL(scaled_residual_k, per_element(n), dim3(256), 0, s, x, a, sa, b, sb, set, nd, n);
}
void act_mul(float* a, const float* b, int64_t n, int act, hipStream_t s) {
    hipLaunchKernelGGL(act_mul_k, per_element(n), dim3(256), 0, s, a, b, n, act);
}
void add_rows(float* x, const float* rows, const float* vec, int64_t n_rows, int nd, hipStream_t s) {
    const int64_t n = n_rows * nd;
    hipLaunchKernelGGL(add_rows_k, per_element(n), dim3(256), 0, s, x, rows, vec, nd, n);
}
void gather_rows(const float* src, const int32_t* idx, int n_rows, int nd, float* out, hipStream_t s) {
    const int64_t n = (int64_t)n_rows * nd;
    hipLaunchKernelGGL(gather_rows_k, per_element(n), dim3(256), 0, s, src, idx, nd, out, n);
}

}  // namespace itk
