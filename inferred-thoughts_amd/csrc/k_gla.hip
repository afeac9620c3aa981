// Gated linear attention between its projections: a matrix state per head whose rows decay by a factor of their own,
//     alpha_t = sigmoid(a2 low_t + b)^(1 / tau),   S_t = diag(alpha_t) S_{t-1} + k_t v_t^T,   o_t = S_t^T q_t
// State [head][value dim][key dim], f32, as in k_ssd.hip: a value row's sum over the keys stays in 16 lanes.
//
// gla_step_k: one token, one launch; a block owns 16 value rows of a head and forms the head's decays by itself.
// gla_decay_k, gla_scan_k: several tokens, the recurrence one token after the other with the state in registers.
// gla_m_k, gla_chunk_state_k, gla_chunk_pass_k, gla_chunk_out_k: many tokens in chunks of 64 on the fp32 matrix cores.  With
// c_t = sum_{s<=t} ln alpha_s inside a chunk that starts from S0:
//     O = M V + (Q e^{c}) S0,   M_ts = sum_d q_t[d] k_s[d] e^{c_t[d] - c_s[d]} for s <= t
//     S = e^{c_L} S0 + sum_s (k_s e^{c_L - c_s}) v_s^T
// As in k_ssd.hip only S0 depends on the chunk before.  The exponents c_t - c_s depend on the channel and cannot be taken out of
// the sum over d, and e^{-c_s} alone can leave f32's range.  So a chunk is four stretches of 16 tokens: between two of them,
// M's operands are scaled by the decay up to and from the edge ahead of the later one, both at most 1; inside one, every
// exponent is formed on its own.  c is summed per stretch, and differences of nearby positions keep their precision.
#include <algorithm>

#include "it_device.h"
#include "it_float.h"
#include "it_mfma32.h"
#include "it_reduce.h"
#include "it_rows8.h"
#include "kernels_float.h"

namespace itk {
namespace {

constexpr int PR = 16;     // value rows per block
constexpr int D_MAX = 512;
constexpr int RANK_MAX = 1024;
constexpr int ST = 16;     // tokens of a stretch

IT_DEV float log_decay(float z, float inv_tau) { return -softplus_exact(-z) * inv_tau; }

// The key channels a lane of 16 holds: four in a row where rows are whole float4s
template <int NR, bool VEC> IT_DEV int channel(int l16, int i) { return VEC ? 4 * l16 + 64 * (i >> 2) + (i & 3) : l16 + 16 * i; }
template <int NR, bool VEC> IT_DEV void load_row(const float* p, int l16, int n, float (&x)[NR]) {
    if constexpr (VEC) {
#pragma unroll
        for (int i = 0; i < NR; i += 4) {
            const int c = channel<NR, true>(l16, i);
            const float4 v = c < n ? *(const float4*)(p + c) : make_float4(0.f, 0.f, 0.f, 0.f);
            x[i] = v.x; x[i + 1] = v.y; x[i + 2] = v.z; x[i + 3] = v.w;
        }
    } else {
#pragma unroll
        for (int i = 0; i < NR; i++) x[i] = l16 + 16 * i < n ? p[l16 + 16 * i] : 0.0f;
    }
}
template <int NR, bool VEC> IT_DEV void store_row(float* p, int l16, int n, const float (&x)[NR]) {
    if constexpr (VEC) {
#pragma unroll
        for (int i = 0; i < NR; i += 4) {
            const int c = channel<NR, true>(l16, i);
            if (c < n) *(float4*)(p + c) = make_float4(x[i], x[i + 1], x[i + 2], x[i + 3]);
        }
    } else {
#pragma unroll
        for (int i = 0; i < NR; i++)
            if (l16 + 16 * i < n) p[l16 + 16 * i] = x[i];
    }
}

// ---------------------------------------------------------------- one token
template <int FMT, bool AL, int NR, bool VEC>
__global__ __launch_bounds__(256) void gla_step_k(GlaP p) {
    __shared__ __align__(16) float al[D_MAX], qs[D_MAX], ks[D_MAX];
    const int tid = threadIdx.x, l16 = tid & 15, row = tid >> 4;
    const int slices = (p.vdim + PR - 1) / PR, h = blockIdx.x / slices, r = (blockIdx.x % slices) * PR + row;
    float* S = p.state + ((int64_t)h * p.vdim + min(r, p.vdim - 1)) * p.dim;
    float st[NR];
    load_row<NR, VEC>(S, l16, p.dim, st);
    const float v = p.v[h * p.vdim + min(r, p.vdim - 1)];
    for (int c = tid; c < p.dim; c += 256) {
        const int ch = h * p.dim + c;
        const uint8_t* w = row_at<FMT>(p.a2, ch, p.rank);
        float z = 0.0f;
        for (int k = 0; k < p.rank; k += 8) {
            float f[8];
            widen8<FMT>(load8<FMT, AL>(w, k, p.rank), f);
#pragma unroll
            for (int e = 0; e < 8; e++)
                if (AL || k + e < p.rank) z = fmaf(f[e], p.low[k + e], z);
        }
        al[c] = expf(log_decay(z + p.a2_b[ch], p.inv_tau));
        qs[c] = p.q[ch];
        ks[c] = p.k[ch];
    }
    __syncthreads();
    if (r >= p.vdim) return;   // (whole groups of 16 lanes)
    float y = 0.0f;
#pragma unroll
    for (int i = 0; i < NR; i++) {
        const int c = channel<NR, VEC>(l16, i);
        if (c < p.dim) {
            st[i] = fmaf(ks[c], v, al[c] * st[i]);
            y = fmaf(st[i], qs[c], y);
        }
    }
    store_row<NR, VEC>(S, l16, p.dim, st);
    y = group_sum<16>(y);
    if (l16 == 0) p.out[h * p.vdim + r] = y;
}

// ---------------------------------------------------------------- several tokens: decays
// a thread: one channel of 16 tokens
template <int FMT, bool AL>
__global__ __launch_bounds__(256) void gla_decay_k(GlaP p, int logs) {
    extern __shared__ __align__(16) float lows[];   // [16][rank padded to 8]
    const int tid = threadIdx.x, ch = blockIdx.x * 256 + tid, t0 = blockIdx.y * ST, nk = p.keys(), rp = (p.rank + 7) & ~7;
    for (int i = tid; i < ST * rp; i += 256) {
        const int t = i / rp, k = i % rp;
        lows[i] = t0 + t < p.n_tok && k < p.rank ? p.low[(int64_t)(t0 + t) * p.rank + k] : 0.0f;
    }
    __syncthreads();
    if (ch >= nk) return;
    float z[ST];
    const float b = p.a2_b[ch];
#pragma unroll
    for (int t = 0; t < ST; t++) z[t] = 0.0f;
    const uint8_t* w = row_at<FMT>(p.a2, ch, p.rank);
    for (int k = 0; k < p.rank; k += 8) {
        float f[8];
        widen8<FMT>(load8<FMT, AL>(w, k, p.rank), f);
#pragma unroll
        for (int t = 0; t < ST; t++) {
            const float4 a = *(const float4*)(lows + t * rp + k), c = *(const float4*)(lows + t * rp + k + 4);
            const float x[8] = {a.x, a.y, a.z, a.w, c.x, c.y, c.z, c.w};
#pragma unroll
            for (int e = 0; e < 8; e++) z[t] = fmaf(f[e], x[e], z[t]);
        }
    }
    float sum = 0.0f;
#pragma unroll
    for (int t = 0; t < ST; t++) {
        const float l = log_decay(z[t] + b, p.inv_tau);
        sum += l;
        if (t0 + t < p.n_tok) p.decay[(int64_t)(t0 + t) * nk + ch] = logs ? sum : expf(l);
    }
}

// ---------------------------------------------------------------- several tokens: one after the other
template <int NR, bool VEC>
__global__ __launch_bounds__(256) void gla_scan_k(GlaP p) {
    const int tid = threadIdx.x, l16 = tid & 15, row = tid >> 4;
    const int slices = (p.vdim + PR - 1) / PR, h = blockIdx.x / slices, r = (blockIdx.x % slices) * PR + row;
    if (r >= p.vdim) return;   // (whole groups of 16 lanes)
    const int nk = p.keys(), nv = p.values();
    float* S = p.state + ((int64_t)h * p.vdim + r) * p.dim;
    float st[NR], q[NR], k[NR], a[NR], v = 0.0f;
    load_row<NR, VEC>(S, l16, p.dim, st);
    auto fetch = [&](int t) __attribute__((always_inline)) {
        const int64_t at = (int64_t)t * nk + h * p.dim;
        load_row<NR, VEC>(p.q + at, l16, p.dim, q);
        load_row<NR, VEC>(p.k + at, l16, p.dim, k);
        load_row<NR, VEC>(p.decay + at, l16, p.dim, a);
        v = p.v[(int64_t)t * nv + h * p.vdim + r];
    };
    fetch(0);
    for (int t = 0; t < p.n_tok; t++) {
        float y = 0.0f;
#pragma unroll
        for (int i = 0; i < NR; i++) {
            st[i] = fmaf(k[i], v, a[i] * st[i]);
            y = fmaf(st[i], q[i], y);
        }
        if (t + 1 < p.n_tok) fetch(t + 1);
        y = group_sum<16>(y);
        if (l16 == 0) p.out[(int64_t)t * nv + h * p.vdim + r] = y;
    }
    store_row<NR, VEC>(S, l16, p.dim, st);
}

// ---------------------------------------------------------------- chunks of 64
constexpr int L = 64;
constexpr int PW = 64;      // value rows of a head per block
constexpr int XS = PW + 4;  // LDS row stride of the values
// a call's chunks are taken some at a time (ck0 ..): per turn
struct GlaWork {
    float* m;       // [chunk][head][t][s], tiles on or below the diagonal
    float* sums;    // [chunk][head][value row][dim]: a chunk's own sum, then its starting state
    float* last;    // [chunk][head][dim]: e^{c_L}
    int ck0, n_ck;
};
IT_DEV bool keys_vec(const GlaP& p) { return p.dim % 4 == 0; }
IT_DEV float4 exp4(const float4& a) { return make_float4(expf(a.x), expf(a.y), expf(a.z), expf(a.w)); }
IT_DEV float4 add4(const float4& a, const float4& b) { return make_float4(a.x + b.x, a.y + b.y, a.z + b.z, a.w + b.w); }
IT_DEV float4 sub4(const float4& a, const float4& b) { return make_float4(a.x - b.x, a.y - b.y, a.z - b.z, a.w - b.w); }
IT_DEV float4 mul4(const float4& a, const float4& b) { return make_float4(a.x * b.x, a.y * b.y, a.z * b.z, a.w * b.w); }

// M of one (chunk, head): a wave per 16 x 16 tile
__global__ __launch_bounds__(64) void gla_m_k(GlaP p, GlaWork wk) {
    const int lane = threadIdx.x, m = lane & 15, g = lane >> 4;
    const int rt = blockIdx.z < 1 ? 0 : blockIdx.z < 3 ? 1 : blockIdx.z < 6 ? 2 : 3, ct = blockIdx.z - rt * (rt + 1) / 2;
    const int ck = blockIdx.x, h = blockIdx.y, t0 = (wk.ck0 + ck) * L, nk = p.keys(), end = p.n_tok - 1;
    const bool vec = keys_vec(p);
    auto at = [&](const float* x, int t) { return x + (int64_t)min(t0 + t, end) * nk + h * p.dim; };
    float* out = wk.m + ((int64_t)ck * p.heads + h) * L * L;
    if (t0 + ST * rt > end) return;   // no token reads these rows
    if (rt != ct) {
        const float *q = at(p.q, ST * rt + m), *cq = at(p.decay, ST * rt + m), *k = at(p.k, ST * ct + m), *ck_ = at(p.decay, ST * ct + m);
        v4f acc = {0.f, 0.f, 0.f, 0.f};
        for (int d = 4 * g; d < p.dim + 4 * g; d += 16) {
            float4 e = sub4(row4(at(p.decay, ST * ct + ST - 1), d, p.dim, vec), row4(ck_, d, p.dim, vec));   // from the key to its stretch's end
            for (int j = ct + 1; j < rt; j++) e = add4(e, row4(at(p.decay, ST * j + ST - 1), d, p.dim, vec));
            acc = mfma16(mul4(row4(q, d, p.dim, vec), exp4(row4(cq, d, p.dim, vec))), mul4(row4(k, d, p.dim, vec), exp4(e)), acc);
        }
#pragma unroll
        for (int i = 0; i < 4; i++) out[(ST * rt + 4 * g + i) * L + ST * ct + m] = acc[i];
        return;
    }
    // row m, columns 4 g ..
    const float *q = at(p.q, ST * rt + m), *cq = at(p.decay, ST * rt + m);
    const float *k[4], *c[4];
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; i++) k[i] = at(p.k, ST * rt + 4 * g + i), c[i] = at(p.decay, ST * rt + 4 * g + i);
    for (int d = 0; d < p.dim; d += 4) {
        const float4 qv = row4(q, d, p.dim, vec), cv = row4(cq, d, p.dim, vec);
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float4 kv = row4(k[i], d, p.dim, vec), e = sub4(cv, row4(c[i], d, p.dim, vec));
            acc[i] = fmaf(qv.x * kv.x, fx_expf(fminf(e.x, 0.0f)), acc[i]);
            acc[i] = fmaf(qv.y * kv.y, fx_expf(fminf(e.y, 0.0f)), acc[i]);
            acc[i] = fmaf(qv.z * kv.z, fx_expf(fminf(e.z, 0.0f)), acc[i]);
            acc[i] = fmaf(qv.w * kv.w, fx_expf(fminf(e.w, 0.0f)), acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < 4; i++) out[(ST * rt + m) * L + ST * rt + 4 * g + i] = 4 * g + i <= m ? acc[i] : 0.0f;
}

// the log decay over stretch j of the chunk at t0 (0 past the call's end), all channels of a head, to LDS [4][np]
IT_DEV void stretches_of(const GlaP& p, int t0, int h, int np, float* tot) {
    for (int i = threadIdx.x; i < 4 * np; i += 256) {
        const int j = i / np, d = i % np;
        tot[i] = d < p.dim && t0 + ST * j < p.n_tok ? p.decay[(int64_t)min(t0 + ST * j + ST - 1, p.n_tok - 1) * p.keys() + h * p.dim + d] : 0.0f;
    }
}
// the chunk's values of this block's rows to LDS [token][XS]
IT_DEV void values_of(const GlaP& p, int t0, int h, int r0, float* xs) {
    const int nv = p.values();
    const bool vec = p.vdim % 4 == 0;
    for (int i = threadIdx.x; i < L * PW / 4; i += 256) {
        const int t = i / (PW / 4), r = i % (PW / 4) * 4;
        *(float4*)(xs + t * XS + r) = t0 + t < p.n_tok ? row4(p.v + (int64_t)(t0 + t) * nv + h * p.vdim, r0 + r, p.vdim, vec) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
}

// a chunk's own sum: wave w takes value rows 16 w ..
__global__ __launch_bounds__(256) void gla_chunk_state_k(GlaP p, GlaWork wk) {
    extern __shared__ __align__(16) float lds[];
    const int np = (p.dim + 15) & ~15, LS = np + 4;
    float *Ks = lds, *Xs = lds + L * LS, *tot = Xs + L * XS;
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), m = lane & 15, g = lane >> 4;
    const int slices = (p.vdim + PW - 1) / PW, h = blockIdx.y / slices, r0 = (blockIdx.y % slices) * PW;
    const int ck = blockIdx.x, t0 = (wk.ck0 + ck) * L, nk = p.keys();
    const bool vec = keys_vec(p);
    stretches_of(p, t0, h, np, tot);
    values_of(p, t0, h, r0, Xs);
    __syncthreads();
    for (int i = tid; i < L * (np / 4); i += 256) {
        const int t = i / (np / 4), k = i % (np / 4) * 4;
        float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
        if (t0 + t < p.n_tok) {
            const int64_t at = (int64_t)(t0 + t) * nk + h * p.dim;
            float4 e = sub4(*(const float4*)(tot + (t / ST) * np + k), row4(p.decay + at, k, p.dim, vec));   // from the token to the chunk's end
            for (int j = t / ST + 1; j < 4; j++) e = add4(e, *(const float4*)(tot + j * np + k));
            x = mul4(row4(p.k + at, k, p.dim, vec), exp4(e));
        }
        *(float4*)(Ks + t * LS + k) = x;
    }
    if (r0 == 0)
        for (int d = tid; d < p.dim; d += 256)
            wk.last[((int64_t)ck * p.heads + h) * p.dim + d] = expf((tot[d] + tot[np + d]) + (tot[2 * np + d] + tot[3 * np + d]));
    __syncthreads();
    if (r0 + 16 * w >= p.vdim) return;
    float a[L / 4];
#pragma unroll
    for (int s = 0; s < L / 4; s++) a[s] = Xs[(4 * s + g) * XS + 16 * w + m];
    float* out = wk.sums + (((int64_t)ck * p.heads + h) * p.vdim + r0 + 16 * w) * p.dim;
    for (int c = 0; c < np / 16; c++) {
        v4f acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < L / 4; s++) acc = mfma4(a[s], Ks[(4 * s + g) * LS + 16 * c + m], acc);
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (r0 + 16 * w + 4 * g + i < p.vdim && 16 * c + m < p.dim) out[(int64_t)(4 * g + i) * p.dim + 16 * c + m] = acc[i];
    }
}

// sums -> starting states, and the state after the last of them
template <int V>   // elements a thread carries (of one value row)
__global__ __launch_bounds__(256) void gla_chunk_pass_k(GlaP p, GlaWork wk) {
    constexpr int AHEAD = 8;
    typedef float fv __attribute__((ext_vector_type(V)));
    const int64_t per_head = (int64_t)p.vdim * p.dim, all = per_head * p.heads, e = ((int64_t)blockIdx.x * 256 + threadIdx.x) * V;
    if (e >= all) return;
    const float* last = wk.last + e / per_head * p.dim + e % p.dim;
    fv run = *(const fv*)(p.state + e);
    float* q = wk.sums + e;
    for (int c0 = 0; c0 < wk.n_ck; c0 += AHEAD) {
        fv v[AHEAD], gl[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; i++)
            if (c0 + i < wk.n_ck) {
                v[i] = *(const fv*)(q + (c0 + i) * all);
                gl[i] = *(const fv*)(last + (int64_t)(c0 + i) * p.keys());
            }
#pragma unroll
        for (int i = 0; i < AHEAD; i++)
            if (c0 + i < wk.n_ck) {
                *(fv*)(q + (c0 + i) * all) = run;
                run = run * gl[i] + v[i];
            }
    }
    *(fv*)(p.state + e) = run;
}

// the read-out: wave w takes stretch w of the chunk
__global__ __launch_bounds__(256) void gla_chunk_out_k(GlaP p, GlaWork wk) {
    extern __shared__ __align__(16) float lds[];
    const int np = (p.dim + 15) & ~15, LS = np + 4;
    float *Ss = lds, *Xs = lds + PW * LS, *tot = Xs + L * XS;   // [value row][LS], [token][XS], [4][np]
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), m = lane & 15, g = lane >> 4;
    const int slices = (p.vdim + PW - 1) / PW, h = blockIdx.y / slices, r0 = (blockIdx.y % slices) * PW;
    const int ck = blockIdx.x, t0 = (wk.ck0 + ck) * L, nk = p.keys(), nv = p.values();
    const bool vec = keys_vec(p);
    const int n_tile = (min(PW, p.vdim - r0) + 15) / 16;
    stretches_of(p, t0, h, np, tot);
    values_of(p, t0, h, r0, Xs);
    const float* s0 = wk.sums + (((int64_t)ck * p.heads + h) * p.vdim + r0) * p.dim;
    for (int i = tid; i < PW * (np / 4); i += 256) {
        const int r = i / (np / 4), k = i % (np / 4) * 4;
        *(float4*)(Ss + r * LS + k) = r0 + r < p.vdim ? row4(s0 + (int64_t)r * p.dim, k, p.dim, vec) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    const int tr = ST * w + m;
    const int64_t at = (int64_t)min(t0 + tr, p.n_tok - 1) * nk + h * p.dim;
    const float *qrow = p.q + at, *crow = p.decay + at;
    const float* mrow = wk.m + (((int64_t)ck * p.heads + h) * L + tr) * L;
    float4 mv[4];
#pragma unroll
    for (int j = 0; j < 4; j++) mv[j] = j <= w && t0 + ST * w < p.n_tok ? *(const float4*)(mrow + ST * j + 4 * g) : make_float4(0.f, 0.f, 0.f, 0.f);
    __syncthreads();
    v4f y[PW / 16];
#pragma unroll
    for (int x = 0; x < PW / 16; x++) y[x] = v4f{0.f, 0.f, 0.f, 0.f};
    for (int k = 4 * g; k < np; k += 16) {
        float4 e = row4(crow, k, p.dim, vec);
        for (int j = 0; j < w; j++) e = add4(e, *(const float4*)(tot + j * np + k));
        const float4 a = mul4(row4(qrow, k, p.dim, vec), exp4(e));
#pragma unroll
        for (int x = 0; x < PW / 16; x++)
            if (x < n_tile) y[x] = mfma16(a, *(const float4*)(Ss + (16 * x + m) * LS + k), y[x]);
    }
#pragma unroll
    for (int j = 0; j < 4; j++) {
        if (j > w) continue;
        const float* xk = Xs + (ST * j + 4 * g) * XS + m;
#pragma unroll
        for (int x = 0; x < PW / 16; x++)
            if (x < n_tile) y[x] = mfma16(mv[j], make_float4(xk[16 * x], xk[XS + 16 * x], xk[2 * XS + 16 * x], xk[3 * XS + 16 * x]), y[x]);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int t = t0 + ST * w + 4 * g + i;
        if (t >= p.n_tok) continue;
#pragma unroll
        for (int x = 0; x < PW / 16; x++) {
            const int r = r0 + 16 * x + m;
            if (x < n_tile && r < p.vdim) p.out[(int64_t)t * nv + h * p.vdim + r] = y[x][i];
        }
    }
}

size_t chunk_lds(int d) {
    const size_t np = (d + 15) & ~15;
    return (L * (np + 4) + L * XS + 4 * np) * sizeof(float);
}
// chunks a turn: their states are about what the last cache level holds
int at_a_time(const GlaP& p) {
    const int64_t one = (int64_t)p.heads * p.vdim * p.dim * sizeof(float);
    return (int)std::min<int64_t>((p.n_tok + L - 1) / L, std::max<int64_t>(8, (128 << 20) / one));
}
template <class F> bool allow_lds(F* fn, size_t lds) {
    if (lds <= 64 * 1024) return true;
    if (hipFuncSetAttribute((const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess) return true;
    (void)hipGetLastError();
    return false;
}
unsigned blocks(const GlaP& p) { return (unsigned)(p.heads * ((p.vdim + PR - 1) / PR)); }
bool a2_aligned(const GlaP& p) { return p.rank % 8 == 0 && aligned16(p.a2); }

// channels a lane of 16 holds
#define IT_BY_DIM(d, CALL)                                            \
    do {                                                              \
        if ((d) % 4) {                                                \
            if ((d) <= 32) { CALL(2, false); }                        \
            else if ((d) <= 128) { CALL(8, false); }                  \
            else { CALL(32, false); }                                 \
        } else if ((d) <= 64) { CALL(4, true); }                      \
        else if ((d) <= 128) { CALL(8, true); }                       \
        else if ((d) <= 256) { CALL(16, true); }                      \
        else { CALL(32, true); }                                      \
    } while (0)

}  // namespace

bool gla_takes(const GlaP& p) { return p.dim >= 1 && p.dim <= D_MAX && p.vdim >= 1 && p.rank >= 1 && p.rank <= RANK_MAX; }

void gla_step(const GlaP& p, hipStream_t s) {
    const bool al = a2_aligned(p);
#define IT_STEP(NR, VEC) hipLaunchKernelGGL((gla_step_k<FM, ALI, NR, VEC>), dim3(blocks(p)), dim3(256), 0, s, p)
#define IT_CALL(F, A)                        \
    do {                                     \
        constexpr int FM = F;                \
        constexpr bool ALI = A;              \
        IT_BY_DIM(p.dim, IT_STEP);           \
    } while (0)
    IT_BY_FORMAT(p.a2_fmt, al, IT_CALL);
#undef IT_CALL
#undef IT_STEP
}
void gla_decay(const GlaP& p, int logs, hipStream_t s) {
    const bool al = a2_aligned(p);
    const size_t lds = (size_t)ST * ((p.rank + 7) & ~7) * sizeof(float);   // 64 KB at most
    const dim3 grid((p.keys() + 255) / 256, (p.n_tok + ST - 1) / ST);
#define IT_CALL(F, A) hipLaunchKernelGGL((gla_decay_k<F, A>), grid, dim3(256), lds, s, p, logs)
    IT_BY_FORMAT(p.a2_fmt, al, IT_CALL);
#undef IT_CALL
}
void gla_scan(const GlaP& p, hipStream_t s) {
#define IT_CALL(NR, VEC) hipLaunchKernelGGL((gla_scan_k<NR, VEC>), dim3(blocks(p)), dim3(256), 0, s, p)
    IT_BY_DIM(p.dim, IT_CALL);
#undef IT_CALL
}

// (the LDS of a CU bounds the key size of the chunked form)
bool gla_chunk_takes(const GlaP& p) { return p.n_tok >= L && chunk_lds(p.dim) <= 156 * 1024; }
size_t gla_chunk_work_floats(const GlaP& p) { return (size_t)at_a_time(p) * p.heads * ((size_t)L * L + (size_t)p.vdim * p.dim + p.dim); }
bool gla_chunk(const GlaP& p, float* work, hipStream_t s) {
    const size_t lds = chunk_lds(p.dim);
    if (!allow_lds(gla_chunk_state_k, lds) || !allow_lds(gla_chunk_out_k, lds)) return false;
    const int all = (p.n_tok + L - 1) / L, turn = at_a_time(p);
    const int64_t elems = (int64_t)p.heads * p.vdim * p.dim;
    GlaWork wk{};
    wk.m = work;   // (whole 16-byte pieces; the sums and decays are where their rows are)
    wk.sums = work + (size_t)turn * p.heads * L * L;
    wk.last = wk.sums + (size_t)turn * elems;
    for (wk.ck0 = 0; wk.ck0 < all; wk.ck0 += turn) {
        wk.n_ck = std::min(turn, all - wk.ck0);
        const dim3 grid(wk.n_ck, p.heads * ((p.vdim + PW - 1) / PW)), block(256);
        hipLaunchKernelGGL(gla_m_k, dim3(wk.n_ck, p.heads, 10), dim3(64), 0, s, p, wk);
        hipLaunchKernelGGL(gla_chunk_state_k, grid, block, lds, s, p, wk);
        if (p.dim % 4 == 0) hipLaunchKernelGGL(gla_chunk_pass_k<4>, dim3((unsigned)((elems / 4 + 255) / 256)), block, 0, s, p, wk);
        else hipLaunchKernelGGL(gla_chunk_pass_k<1>, dim3((unsigned)((elems + 255) / 256)), block, 0, s, p, wk);
        hipLaunchKernelGGL(gla_chunk_out_k, grid, block, lds, s, p, wk);
    }
    return true;
}

}  // namespace itk
