// The Mamba-2 mixer between its projections (state-space duality):
//     [z | x | B | C | dt] = u;  x, B, C = silu(causal conv + bias);  dt = softplus(dt + bias)
//     S_t = e^{a_t} S_{t-1} + dt_t B_t x_t^T,  a_t = -exp(A_log) dt_t,   y_t = S_t^T C_t + D x_t,   out_t = y_t silu(z_t)
// State [head][value dim][n], f32.  The convolution's inputs live in a ring: row p % taps holds the raw x, B, C of position
// p, so a single-token step writes a row that no block of the same step reads, and every block may form the convolution it
// needs by itself.
//
// ssd_step_k: one token, one launch; a block owns 16 value rows of a head, 16 lanes a row.
// ssd_conv_k, ssd_scan_k: several tokens, the recurrence one token after the other with the state in registers.
// ssd_cb_k, ssd_chunk_state_k, ssd_chunk_pass_k, ssd_chunk_out_k: many tokens in chunks of 64 on the fp32 matrix cores.  With
// c_t = sum_{s<=t} a_s inside a chunk that starts from S0:
//     Y = M X + diag(e^{c}) C S0,   M_ts = (C_t . B_s) e^{c_t - c_s} dt_s for s <= t
//     S = e^{c_L} S0 + sum_s e^{c_L - c_s} dt_s B_s x_s^T
// Only S0 depends on the chunk before, and linearly: every chunk's own sum is formed at once, one pass over the chunks, an
// element of the state a thread, turns the sums into the chunks' starting states, and every chunk's read-out is formed at
// once from them.  C B^T is the same for all heads of a group.  c is summed in f64: differences of nearby positions then keep
// their f32 precision whatever decayed before them in the chunk.
#include <algorithm>

#include "it_device.h"
#include "it_float.h"
#include "it_mfma32.h"
#include "it_reduce.h"
#include "kernels_float.h"

namespace itk {
namespace {

constexpr int PR = 16;     // value rows per block
constexpr int TAPS_MAX = 16;
constexpr int N_MAX = 512;

IT_DEV float silu_of(float z, int accurate) { return accurate ? silu_exact(z) : fx_silu(z); }

// ---------------------------------------------------------------- one token
template <int NR>   // state columns a lane holds
__global__ __launch_bounds__(256) void ssd_step_k(SsdP p) {
    __shared__ float bc[2 * N_MAX], xs[PR];
    const int tid = threadIdx.x, l16 = tid & 15, row = tid >> 4;
    const int slices = (p.vdim + PR - 1) / PR, h = blockIdx.x / slices, r0 = (blockIdx.x % slices) * PR;
    const int grp = h / (p.heads / p.groups), inner = p.inner(), nch = p.channels();
    const int pos = p.pos_dyn ? *p.pos_dyn : p.pos;
    const float* raw = p.u + inner;   // this token's x | B | C
    const int pr = r0 + row;
    float* S = p.state + ((int64_t)h * p.vdim + min(pr, p.vdim - 1)) * p.n;
    float st[NR];
#pragma unroll
    for (int i = 0; i < NR; i++) st[i] = l16 + 16 * i < p.n ? S[l16 + 16 * i] : 0.0f;
    // the channels this block needs: its value rows, then the group's B and C
    const int here = pos % p.taps;
    for (int i = tid; i < PR + 2 * p.n; i += 256) {
        const bool is_x = i < PR;
        if (is_x && r0 + i >= p.vdim) {
            xs[i] = 0.0f;
            continue;
        }
        const int k = i - PR;   // B then C
        const int ch = is_x ? h * p.vdim + r0 + i : k < p.n ? inner + grp * p.n + k : inner + (p.groups + grp) * p.n + (k - p.n);
        float acc = p.conv_b[ch];
        for (int t = 0; t < p.taps - 1; t++) {
            const int at = pos - (p.taps - 1) + t;
            if (at >= 0) acc = fmaf(p.conv_w[(int64_t)ch * p.taps + t], p.conv_ring[(int64_t)(at % p.taps) * nch + ch], acc);
        }
        const float now = raw[ch];
        acc = fmaf(p.conv_w[(int64_t)ch * p.taps + p.taps - 1], now, acc);
        p.conv_ring[(int64_t)here * nch + ch] = now;   // (blocks that share a group write the same value)
        const float v = silu_of(acc, p.accurate);
        if (is_x) xs[i] = v;
        else bc[k] = v;
    }
    const float dt = softplus_exact(p.u[inner + nch + h] + p.dt_bias[h]);
    const float decay = expf(-expf(p.a_log[h]) * dt);
    __syncthreads();
    if (pr >= p.vdim) return;
    const float x = xs[row], dx = dt * x;
    float y = 0.0f;
#pragma unroll
    for (int i = 0; i < NR; i++) {
        const int c = l16 + 16 * i;
        if (c < p.n) {
            st[i] = fmaf(dx, bc[c], decay * st[i]);
            y = fmaf(st[i], bc[p.n + c], y);
            S[c] = st[i];
        }
    }
    y = group_sum<16>(y);
    if (l16 == 0) {
        const int j = h * p.vdim + pr;
        p.out[j] = fmaf(p.d[h], x, y) * silu_of(p.u[j], p.accurate);
    }
}

// ---------------------------------------------------------------- several tokens: convolution
constexpr int CT = 8;   // tokens per thread
// V channels a thread; K > 0: the number of taps at compile time
template <int V, int K>
__global__ __launch_bounds__(256) void ssd_conv_k(SsdP p) {
    typedef float fv __attribute__((ext_vector_type(V)));
    const int ch = (blockIdx.x * 256 + threadIdx.x) * V, nch = p.channels(), inner = p.inner(), ud = p.u_dim();
    if (ch >= nch) return;
    const int t0 = blockIdx.y * CT;
    const int taps = K ? K : p.taps;
    auto raw = [&](int t) -> fv {   // token t of this call, or an earlier one
        if (t >= 0) return *(const fv*)(p.u + (int64_t)min(t, p.n_tok - 1) * ud + inner + ch);
        const int at = p.pos + t;
        return at >= 0 ? *(const fv*)(p.conv_ring + (int64_t)(at % taps) * nch + ch) : fv(0.0f);
    };
    fv acc[CT];
    const fv bias = *(const fv*)(p.conv_b + ch);
#pragma unroll
    for (int i = 0; i < CT; i++) acc[i] = bias;
    if constexpr (K > 0) {
        fv in[CT + K - 1];
#pragma unroll
        for (int i = 0; i < CT + K - 1; i++) in[i] = raw(t0 - (K - 1) + i);
#pragma unroll
        for (int k = 0; k < K; k++) {
            fv w;
#pragma unroll
            for (int c = 0; c < V; c++) w[c] = p.conv_w[(int64_t)(ch + c) * K + k];
#pragma unroll
            for (int i = 0; i < CT; i++)
#pragma unroll
                for (int c = 0; c < V; c++) acc[i][c] = fmaf(w[c], in[i + k][c], acc[i][c]);
        }
    } else {
        for (int k = 0; k < taps; k++) {
            fv w;
#pragma unroll
            for (int c = 0; c < V; c++) w[c] = p.conv_w[(int64_t)(ch + c) * taps + k];
#pragma unroll
            for (int i = 0; i < CT; i++) {
                const fv x = raw(t0 + i - (taps - 1) + k);
#pragma unroll
                for (int c = 0; c < V; c++) acc[i][c] = fmaf(w[c], x[c], acc[i][c]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < CT; i++) {
        if (t0 + i >= p.n_tok) continue;
        fv v;
#pragma unroll
        for (int c = 0; c < V; c++) v[c] = silu_of(acc[i][c], p.accurate);
        *(fv*)(p.xbc + (int64_t)(t0 + i) * nch + ch) = v;
    }
}
// after every block of the convolution has read the ring: the call's last inputs take their rows
__global__ __launch_bounds__(256) void ssd_conv_keep_k(SsdP p) {
    const int ch = blockIdx.x * 256 + threadIdx.x, nch = p.channels();
    if (ch >= nch) return;
    for (int t = max(0, p.n_tok - p.taps); t < p.n_tok; t++)
        p.conv_ring[(int64_t)((p.pos + t) % p.taps) * nch + ch] = p.u[(int64_t)t * p.u_dim() + p.inner() + ch];
}

// ---------------------------------------------------------------- several tokens: one after the other
template <int NR>
__global__ __launch_bounds__(256) void ssd_scan_k(SsdP p) {
    const int tid = threadIdx.x, l16 = tid & 15, row = tid >> 4;
    const int slices = (p.vdim + PR - 1) / PR, h = blockIdx.x / slices, pr = (blockIdx.x % slices) * PR + row;
    const int grp = h / (p.heads / p.groups), inner = p.inner(), nch = p.channels(), ud = p.u_dim();
    if (pr >= p.vdim) return;   // (whole groups of 16 lanes)
    const int j = h * p.vdim + pr, ob = inner + grp * p.n, oc = ob + p.groups * p.n;
    float* S = p.state + (int64_t)j * p.n;
    const float a = -expf(p.a_log[h]), bias = p.dt_bias[h], d = p.d[h];
    float st[NR], b[NR], c[NR];
#pragma unroll
    for (int i = 0; i < NR; i++) st[i] = l16 + 16 * i < p.n ? S[l16 + 16 * i] : 0.0f;
    float x = 0, dtr = 0, z = 0;
    auto fetch = [&](int t) __attribute__((always_inline)) {
        const float* q = p.xbc + (int64_t)t * nch;
        x = q[j];
#pragma unroll
        for (int i = 0; i < NR; i++) {
            const bool ok = l16 + 16 * i < p.n;
            b[i] = ok ? q[ob + l16 + 16 * i] : 0.0f;
            c[i] = ok ? q[oc + l16 + 16 * i] : 0.0f;
        }
        dtr = p.u[(int64_t)t * ud + inner + nch + h];
        z = p.u[(int64_t)t * ud + j];
    };
    fetch(0);
    for (int t = 0; t < p.n_tok; t++) {
        const float dt = softplus_exact(dtr + bias), decay = expf(a * dt), dx = dt * x, skip = d * x, zt = z;
        float y = 0.0f;
#pragma unroll
        for (int i = 0; i < NR; i++) {
            st[i] = fmaf(dx, b[i], decay * st[i]);
            y = fmaf(st[i], c[i], y);
        }
        if (t + 1 < p.n_tok) fetch(t + 1);
        y = group_sum<16>(y);
        if (l16 == 0) p.out[(int64_t)t * inner + j] = (y + skip) * silu_of(zt, p.accurate);
    }
#pragma unroll
    for (int i = 0; i < NR; i++)
        if (l16 + 16 * i < p.n) S[l16 + 16 * i] = st[i];
}

// ---------------------------------------------------------------- chunks of 64
constexpr int L = 64;
constexpr int PW = 64;      // value rows of a head per block
constexpr int XS = PW + 4;  // LDS row stride of the inputs
IT_DEV bool rows_vec(const SsdP& p) { return p.n % 4 == 0 && p.inner() % 4 == 0; }

// a call's chunks are taken a stretch at a time (ck0 ..): per stretch
struct ChunkWork {
    float* cb;      // [chunk][group][t][s], tiles on or below the diagonal, zero above it
    float* sums;    // [chunk][head][value row][n]: a chunk's own sum, then its starting state
    float* last;    // [chunk][head]: e^{c_L}
    int ck0, n_ck;
};

// C B^T of one (chunk, group): a wave per 16 x 16 tile
__global__ __launch_bounds__(64) void ssd_cb_k(SsdP p, ChunkWork wk) {
    const int lane = threadIdx.x, m = lane & 15, g = lane >> 4;
    const int rt = blockIdx.z < 1 ? 0 : blockIdx.z < 3 ? 1 : blockIdx.z < 6 ? 2 : 3, ct = blockIdx.z - rt * (rt + 1) / 2;
    const int ck = blockIdx.x, grp = blockIdx.y, t0 = (wk.ck0 + ck) * L, nch = p.channels();
    const int ob = p.inner() + grp * p.n, oc = ob + p.groups * p.n;
    const bool vec = rows_vec(p);
    const float* c = p.xbc + (int64_t)min(t0 + 16 * rt + m, p.n_tok - 1) * nch + oc;
    const float* b = p.xbc + (int64_t)min(t0 + 16 * ct + m, p.n_tok - 1) * nch + ob;
    v4f acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k = 4 * g; k < p.n + 4 * g; k += 16) acc = mfma16(row4(c, k, p.n, vec), row4(b, k, p.n, vec), acc);
    float* out = wk.cb + ((int64_t)ck * p.groups + grp) * L * L;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int t = 16 * rt + 4 * g + i, s = 16 * ct + m;
        out[t * L + s] = s <= t ? acc[i] : 0.0f;
    }
}

// step sizes and decays of a (chunk, head), by the first wave
struct Decays {
    double cum[L];
    float dt[L];
};
IT_DEV void decays_of(const SsdP& p, int t0, int h, Decays& d) {
    const int lane = threadIdx.x, t = t0 + lane;
    const float dt = t < p.n_tok ? softplus_exact(p.u[(int64_t)t * p.u_dim() + p.inner() + p.channels() + h] + p.dt_bias[h]) : 0.0f;
    double x = (double)-expf(p.a_log[h]) * (double)dt;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const double y = __shfl_up(x, off, 64);
        if (lane >= off) x += y;
    }
    d.cum[lane] = x;
    d.dt[lane] = dt;
}
// the chunk's inputs of this block's value rows, each times f(token), to LDS [token][XS]
template <class F> IT_DEV void inputs_of(const SsdP& p, int t0, int h, int r0, float* xs, F f) {
    const int nch = p.channels();
    if (p.vdim % 4 == 0) {   // (then the channels' count and this head's place are too, where rows_vec holds)
        const bool vec = rows_vec(p);
        for (int i = threadIdx.x; i < L * PW / 4; i += 256) {
            const int t = i / (PW / 4), r = i % (PW / 4) * 4;
            const float4 x = t0 + t < p.n_tok ? row4(p.xbc + (int64_t)(t0 + t) * nch + h * p.vdim, r0 + r, p.vdim, vec) : make_float4(0.f, 0.f, 0.f, 0.f);
            const float w = f(t);
            *(float4*)(xs + t * XS + r) = make_float4(x.x * w, x.y * w, x.z * w, x.w * w);
        }
    } else {
        for (int i = threadIdx.x; i < L * PW; i += 256) {
            const int t = i / PW, r = i % PW;
            xs[t * XS + r] = t0 + t < p.n_tok && r0 + r < p.vdim ? p.xbc[(int64_t)(t0 + t) * nch + h * p.vdim + r0 + r] * f(t) : 0.0f;
        }
    }
}

// a chunk's own sum: wave w takes value rows 16 w ..
__global__ __launch_bounds__(256) void ssd_chunk_state_k(SsdP p, ChunkWork wk) {
    extern __shared__ __align__(16) float lds[];
    __shared__ Decays d;
    const int np = (p.n + 15) & ~15, LS = np + 4;
    float *Bs = lds, *Xd = lds + L * LS;
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), m = lane & 15, g = lane >> 4;
    const int slices = (p.vdim + PW - 1) / PW, h = blockIdx.y / slices, r0 = (blockIdx.y % slices) * PW;
    const int ck = blockIdx.x, t0 = (wk.ck0 + ck) * L, nch = p.channels(), grp = h / (p.heads / p.groups);
    const bool vec = rows_vec(p);
    if (w == 0) decays_of(p, t0, h, d);
    for (int i = tid; i < L * (np / 4); i += 256) {
        const int t = i / (np / 4), k = i % (np / 4) * 4;
        *(float4*)(Bs + t * LS + k) = t0 + t < p.n_tok ? row4(p.xbc + (int64_t)(t0 + t) * nch + p.inner() + grp * p.n, k, p.n, vec) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    __syncthreads();
    const double last = d.cum[L - 1];
    inputs_of(p, t0, h, r0, Xd, [&](int t) { return d.dt[t] * expf((float)(last - d.cum[t])); });
    if (tid == 0 && r0 == 0) wk.last[(int64_t)ck * p.heads + h] = expf((float)last);
    __syncthreads();
    if (r0 + 16 * w >= p.vdim) return;
    float a[L / 4];
#pragma unroll
    for (int s = 0; s < L / 4; s++) a[s] = Xd[(4 * s + g) * XS + 16 * w + m];
    float* out = wk.sums + (((int64_t)ck * p.heads + h) * p.vdim + r0 + 16 * w) * p.n;
    for (int c = 0; c < np / 16; c++) {
        v4f acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < L / 4; s++) acc = mfma4(a[s], Bs[(4 * s + g) * LS + 16 * c + m], acc);
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (r0 + 16 * w + 4 * g + i < p.vdim && 16 * c + m < p.n) out[(int64_t)(4 * g + i) * p.n + 16 * c + m] = acc[i];
    }
}

// sums -> starting states, and the state after the stretch
template <int V>   // elements a thread carries (of one head)
__global__ __launch_bounds__(256) void ssd_chunk_pass_k(SsdP p, ChunkWork wk) {
    constexpr int AHEAD = 8;
    const int64_t per_head = (int64_t)p.vdim * p.n, all = per_head * p.heads, e = ((int64_t)blockIdx.x * 256 + threadIdx.x) * V;
    if (e >= all) return;
    const float* last = wk.last + e / per_head;
    typedef float fv __attribute__((ext_vector_type(V)));
    fv run = *(const fv*)(p.state + e);
    float* q = wk.sums + e;
    for (int c0 = 0; c0 < wk.n_ck; c0 += AHEAD) {
        fv v[AHEAD];
        float gl[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; i++)
            if (c0 + i < wk.n_ck) {
                v[i] = *(const fv*)(q + (c0 + i) * all);
                gl[i] = last[(int64_t)(c0 + i) * p.heads];
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

// the read-out: wave w takes tokens 16 w .. of the chunk
__global__ __launch_bounds__(256) void ssd_chunk_out_k(SsdP p, ChunkWork wk) {
    extern __shared__ __align__(16) float lds[];
    __shared__ Decays d;
    const int np = (p.n + 15) & ~15, LS = np + 4;
    float *Ss = lds, *Xd = lds + PW * LS;   // [value row][LS], [token][XS]
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), m = lane & 15, g = lane >> 4;
    const int slices = (p.vdim + PW - 1) / PW, h = blockIdx.y / slices, r0 = (blockIdx.y % slices) * PW;
    const int ck = blockIdx.x, t0 = (wk.ck0 + ck) * L, nch = p.channels(), inner = p.inner(), ud = p.u_dim(), grp = h / (p.heads / p.groups);
    const bool vec = rows_vec(p);
    const int n_tile = (min(PW, p.vdim - r0) + 15) / 16;
    if (w == 0) decays_of(p, t0, h, d);
    const float* s0 = wk.sums + (((int64_t)ck * p.heads + h) * p.vdim + r0) * p.n;
    for (int i = tid; i < PW * (np / 4); i += 256) {
        const int r = i / (np / 4), k = i % (np / 4) * 4;
        *(float4*)(Ss + r * LS + k) = r0 + r < p.vdim ? row4(s0 + (int64_t)r * p.n, k, p.n, p.n % 4 == 0) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    __syncthreads();
    inputs_of(p, t0, h, r0, Xd, [&](int t) { return d.dt[t]; });
    // this lane's row of C and of M while the inputs land
    const int tr = 16 * w + m;
    const float* crow = p.xbc + (int64_t)min(t0 + tr, p.n_tok - 1) * nch + inner + (p.groups + grp) * p.n;
    const float* mrow = wk.cb + (((int64_t)ck * p.groups + grp) * L + tr) * L;
    const double cm = d.cum[tr];
    float4 mv[4];
#pragma unroll
    for (int j = 0; j < 4; j++) {
        mv[j] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (j <= w) {
            const int k = 16 * j + 4 * g;
            const float4 v = *(const float4*)(mrow + k);
            mv[j].x = k <= tr ? v.x * expf((float)(cm - d.cum[k])) : 0.0f;
            mv[j].y = k + 1 <= tr ? v.y * expf((float)(cm - d.cum[k + 1])) : 0.0f;
            mv[j].z = k + 2 <= tr ? v.z * expf((float)(cm - d.cum[k + 2])) : 0.0f;
            mv[j].w = k + 3 <= tr ? v.w * expf((float)(cm - d.cum[k + 3])) : 0.0f;
        }
    }
    __syncthreads();
    v4f y[PW / 16];
#pragma unroll
    for (int x = 0; x < PW / 16; x++) y[x] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
    for (int k = 4 * g; k < np; k += 16) {
        const float4 a = row4(crow, k, p.n, vec);
#pragma unroll
        for (int x = 0; x < PW / 16; x++)
            if (x < n_tile) y[x] = mfma16(a, *(const float4*)(Ss + (16 * x + m) * LS + k), y[x]);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const float gam = expf((float)d.cum[16 * w + 4 * g + i]);
#pragma unroll
        for (int x = 0; x < PW / 16; x++) y[x][i] *= gam;
    }
#pragma unroll
    for (int j = 0; j < 4; j++) {
        if (j > w) continue;
        const float* xk = Xd + (16 * j + 4 * g) * XS + m;
#pragma unroll
        for (int x = 0; x < PW / 16; x++)
            if (x < n_tile) y[x] = mfma16(mv[j], make_float4(xk[16 * x], xk[XS + 16 * x], xk[2 * XS + 16 * x], xk[3 * XS + 16 * x]), y[x]);
    }
    const float D = p.d[h];
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int t = t0 + 16 * w + 4 * g + i;
        if (t >= p.n_tok) continue;
#pragma unroll
        for (int x = 0; x < PW / 16; x++) {
            const int r = r0 + 16 * x + m;
            if (x < n_tile && r < p.vdim) {
                const int j = h * p.vdim + r;
                p.out[(int64_t)t * inner + j] = fmaf(D, p.xbc[(int64_t)t * nch + j], y[x][i]) * silu_of(p.u[(int64_t)t * ud + j], p.accurate);
            }
        }
    }
}

size_t state_lds(int n) { return (size_t)L * (((n + 15) & ~15) + 4 + XS) * sizeof(float); }
size_t out_lds(int n) { return (size_t)(PW * (((n + 15) & ~15) + 4) + L * XS) * sizeof(float); }
// chunks a stretch: its states are about what the last cache level holds
int stretch(const SsdP& p) {
    const int64_t one = (int64_t)p.heads * p.vdim * p.n * sizeof(float);
    return (int)std::min<int64_t>((p.n_tok + L - 1) / L, std::max<int64_t>(8, (128 << 20) / one));
}
template <class F> bool allow_lds(F* fn, size_t lds) {
    if (lds <= 64 * 1024) return true;
    if (hipFuncSetAttribute((const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess) return true;
    (void)hipGetLastError();
    return false;
}

#define IT_BY_N(n, CALL)                    \
    do {                                    \
        if ((n) <= 16) { CALL(1); }         \
        else if ((n) <= 32) { CALL(2); }    \
        else if ((n) <= 64) { CALL(4); }    \
        else if ((n) <= 128) { CALL(8); }   \
        else if ((n) <= 256) { CALL(16); }  \
        else { CALL(32); }                  \
    } while (0)

unsigned blocks(const SsdP& p) { return (unsigned)(p.heads * ((p.vdim + PR - 1) / PR)); }

}  // namespace

bool ssd_takes(const SsdP& p) { return p.n >= 1 && p.n <= N_MAX && p.taps >= 1 && p.taps <= TAPS_MAX && p.vdim >= 1; }

void ssd_step(const SsdP& p, hipStream_t s) {
#define IT_CALL(NR) hipLaunchKernelGGL(ssd_step_k<NR>, dim3(blocks(p)), dim3(256), 0, s, p)
    IT_BY_N(p.n, IT_CALL);
#undef IT_CALL
}
void ssd_conv(const SsdP& p, hipStream_t s) {
    // (whole groups of four channels in every row of the inputs, the ring and the output)
    const bool four = p.channels() % 4 == 0 && p.inner() % 4 == 0 && p.u_dim() % 4 == 0;
    const dim3 grid((p.channels() + (four ? 1023 : 255)) / (four ? 1024 : 256), (p.n_tok + CT - 1) / CT);
#define IT_CALL(V, K) hipLaunchKernelGGL((ssd_conv_k<V, K>), grid, dim3(256), 0, s, p)
    if (!four) IT_CALL(1, 0);
    else if (p.taps == 2) IT_CALL(4, 2);
    else if (p.taps == 3) IT_CALL(4, 3);
    else if (p.taps == 4) IT_CALL(4, 4);
    else IT_CALL(4, 0);
#undef IT_CALL
}
void ssd_conv_keep(const SsdP& p, hipStream_t s) {
    hipLaunchKernelGGL(ssd_conv_keep_k, dim3((p.channels() + 255) / 256), dim3(256), 0, s, p);
}
void ssd_scan(const SsdP& p, hipStream_t s) {
#define IT_CALL(NR) hipLaunchKernelGGL(ssd_scan_k<NR>, dim3(blocks(p)), dim3(256), 0, s, p)
    IT_BY_N(p.n, IT_CALL);
#undef IT_CALL
}

// (the LDS of a CU bounds the state size of the chunked form)
bool ssd_chunk_takes(const SsdP& p) { return p.n_tok >= L && std::max(state_lds(p.n), out_lds(p.n)) <= 156 * 1024; }
size_t ssd_chunk_work_floats(const SsdP& p) {
    return (size_t)stretch(p) * ((size_t)p.groups * L * L + (size_t)p.heads * p.vdim * p.n + p.heads);
}
void ssd_chunk(const SsdP& p, float* work, hipStream_t s) {
    const size_t l1 = state_lds(p.n), l2 = out_lds(p.n);
    if (!allow_lds(ssd_chunk_state_k, l1) || !allow_lds(ssd_chunk_out_k, l2)) {
        ssd_scan(p, s);
        return;
    }
    const int all = (p.n_tok + L - 1) / L, at_once = stretch(p);
    const int64_t elems = (int64_t)p.heads * p.vdim * p.n;
    ChunkWork wk{};
    wk.sums = work;   // (16-byte aligned: first)
    wk.cb = wk.sums + at_once * elems;
    if (elems % 4) wk.cb = work, wk.sums = work + (size_t)at_once * p.groups * L * L;
    wk.last = work + (size_t)at_once * ((size_t)elems + (size_t)p.groups * L * L);
    const dim3 block(256);
    for (wk.ck0 = 0; wk.ck0 < all; wk.ck0 += at_once) {
        wk.n_ck = std::min(at_once, all - wk.ck0);
        const dim3 grid(wk.n_ck, p.heads * ((p.vdim + PW - 1) / PW));
        hipLaunchKernelGGL(ssd_cb_k, dim3(wk.n_ck, p.groups, 10), dim3(64), 0, s, p, wk);
        hipLaunchKernelGGL(ssd_chunk_state_k, grid, block, l1, s, p, wk);
        if ((int64_t)p.vdim * p.n % 4 == 0) hipLaunchKernelGGL(ssd_chunk_pass_k<4>, dim3((unsigned)((elems / 4 + 255) / 256)), block, 0, s, p, wk);
        else hipLaunchKernelGGL(ssd_chunk_pass_k<1>, dim3((unsigned)((elems + 255) / 256)), block, 0, s, p, wk);
        hipLaunchKernelGGL(ssd_chunk_out_k, grid, block, l2, s, p, wk);
    }
}

}  // namespace itk
