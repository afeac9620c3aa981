// The Mamba-2 mixer between its projections (state-space duality):
//     [z | x | B | C | dt] = u;  x, B, C = silu(causal conv + bias);  dt = softplus(dt + bias)
//     S_t = e^{a_t} S_{t-1} + dt_t B_t x_t^T,  a_t = -exp(A_log) dt_t,   y_t = S_t^T C_t + D x_t,   out_t = y_t silu(z_t)
// State [head][value dim][n], f32.  The convolution's inputs live in a ring: row p % taps holds the raw x, B, C of position
// p, so a single-token step writes a row that no block of the same step reads, and every block may form the convolution it
// needs by itself.
//
// ssd_step_k: one token, one launch; a block owns 16 value rows of a head, 16 lanes a row.
// ssd_conv_k, ssd_scan_k: several tokens, the recurrence one token after the other with the state in registers.
// ssd_cb_k, ssd_chunk_k: many tokens in chunks of 64 on the fp32 matrix cores.  With c_t = sum_{s<=t} a_s inside a chunk
// that starts from S0:
//     Y = M X + diag(e^{c}) C S0,   M_ts = (C_t . B_s) e^{c_t - c_s} dt_s for s <= t
//     S = e^{c_L} S0 + sum_s e^{c_L - c_s} dt_s B_s x_s^T
// C B^T does not depend on the head within its group: one launch forms it for every (chunk, group); the second walks the
// chunks, a block per 16 value rows of a head, its slice of S in MFMA accumulators.  c is summed in f64: differences of
// nearby positions then keep their f32 precision whatever decayed before them in the chunk.
#include "it_device.h"
#include "it_float.h"
#include "it_reduce.h"
#include "kernels_float.h"

namespace itk {
namespace {

typedef float v4f __attribute__((ext_vector_type(4)));
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
constexpr int CT = 16;   // tokens per thread
__global__ __launch_bounds__(256) void ssd_conv_k(SsdP p) {
    const int ch = blockIdx.x * 256 + threadIdx.x, nch = p.channels(), inner = p.inner(), ud = p.u_dim();
    if (ch >= nch) return;
    const int t0 = blockIdx.y * CT, t1 = min(p.n_tok, t0 + CT);
    float win[TAPS_MAX], w[TAPS_MAX];
    const int K = p.taps;
#pragma unroll
    for (int k = 0; k < TAPS_MAX; k++)
        if (k < K) w[k] = p.conv_w[(int64_t)ch * K + k];
    auto raw = [&](int t) -> float {   // token t of this call, or an earlier one
        if (t >= 0) return p.u[(int64_t)t * ud + inner + ch];
        const int at = p.pos + t;
        return at >= 0 ? p.conv_ring[(int64_t)(at % K) * nch + ch] : 0.0f;
    };
#pragma unroll
    for (int k = 0; k < TAPS_MAX; k++)
        if (k < K - 1) win[k] = raw(t0 - (K - 1) + k);
    const float bias = p.conv_b[ch];
    for (int t = t0; t < t1; t++) {
        const float now = p.u[(int64_t)t * ud + inner + ch];
        float acc = bias;
#pragma unroll
        for (int k = 0; k < TAPS_MAX; k++)
            if (k < K - 1) acc = fmaf(w[k], win[k], acc);
#pragma unroll
        for (int k = 0; k < TAPS_MAX; k++)
            if (k == K - 1) acc = fmaf(w[k], now, acc);
        p.xbc[(int64_t)t * nch + ch] = silu_of(acc, p.accurate);
#pragma unroll
        for (int k = 0; k < TAPS_MAX - 1; k++)
            if (k < K - 2) win[k] = win[k + 1];
#pragma unroll
        for (int k = 0; k < TAPS_MAX; k++)
            if (k == K - 2) win[k] = now;
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
constexpr int MS = L + 4;   // LDS row stride of the 64 x 64 matrix
// D = A(16 x 4) B(4 x 16) + C: lane l gives A[l % 16][l / 16] and B[l / 16][l % 16], and holds D[4 * (l / 16) + i][l % 16]
IT_DEV v4f mfma4(float a, float b, v4f c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

constexpr int pad4(int n) { return (n + 3) & ~3; }

// C B^T of one (chunk, group): work[chunk][group][t][s], zero above the diagonal
__global__ __launch_bounds__(256) void ssd_cb_k(SsdP p, float* __restrict__ work) {
    extern __shared__ __align__(16) float lds[];
    const int np = pad4(p.n), LS = np + 4;
    float *Bs = lds, *Cs = lds + L * LS;
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), m = lane & 15, g = lane >> 4;
    const int ck = blockIdx.x, grp = blockIdx.y, t0 = ck * L, nch = p.channels();
    const int ob = p.inner() + grp * p.n, oc = ob + p.groups * p.n;
    for (int i = tid; i < L * np; i += 256) {
        const int t = i / np, k = i % np;
        const bool ok = t0 + t < p.n_tok && k < p.n;
        const float* q = p.xbc + (int64_t)(t0 + t) * nch + k;
        Bs[t * LS + k] = ok ? q[ob] : 0.0f;
        Cs[t * LS + k] = ok ? q[oc] : 0.0f;
    }
    __syncthreads();
    float* out = work + ((int64_t)ck * p.groups + grp) * L * L;
    for (int ct = 0; ct < 4; ct++) {
        v4f acc = {0.f, 0.f, 0.f, 0.f};
        if (ct <= w)
            for (int s = 0; s < np / 4; s++) acc = mfma4(Cs[(16 * w + m) * LS + 4 * s + g], Bs[(16 * ct + m) * LS + 4 * s + g], acc);
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = 16 * w + 4 * g + i, s = 16 * ct + m;
            out[t * L + s] = s <= t ? acc[i] : 0.0f;
        }
    }
}

// XT: state column tiles (of 16) a wave holds
template <int XT>
__global__ __launch_bounds__(256) void ssd_chunk_k(SsdP p, const float* __restrict__ cb) {
    extern __shared__ __align__(16) float lds[];
    __shared__ double cum[L];
    __shared__ float dts[L], gam[L], dec[L], glast;
    const int np = (p.n + 15) & ~15, LS = np + 4;
    float *Bs = lds, *Cs = Bs + L * LS, *Ms = Cs + L * LS, *Xs = Ms + L * MS, *Xd = Xs + L * 20, *Ss = Xd + L * 20;   // Ss [16][LS]
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), m = lane & 15, g = lane >> 4;
    // the slices of a head on one die, one behind the other: they share a chunk's B, C and C B^T
    const int slices = (p.vdim + PR - 1) / PR, total = p.heads * slices, per = (total + 7) / 8;
    const int item = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if (item >= total || (int)(blockIdx.x >> 3) >= per) return;
    const int h = item / slices, r0 = (item % slices) * PR;
    const int grp = h / (p.heads / p.groups), inner = p.inner(), nch = p.channels(), ud = p.u_dim();
    const int ob = inner + grp * p.n, oc = ob + p.groups * p.n;
    const float a = -expf(p.a_log[h]), bias = p.dt_bias[h], D = p.d[h];
    const int n_ck = (p.n_tok + L - 1) / L;
    const bool vec = p.n % 4 == 0 && nch % 4 == 0 && inner % 4 == 0;
    v4f st[XT];
#pragma unroll
    for (int x = 0; x < XT; x++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int r = r0 + 4 * g + i, c = 16 * (w + 4 * x) + m;
            st[x][i] = r < p.vdim && c < p.n ? p.state[((int64_t)h * p.vdim + r) * p.n + c] : 0.0f;
        }
    for (int ck = 0; ck < n_ck; ck++) {
        const int t0 = ck * L;
        // operands of the chunk
        if (vec) {
            const int n4 = np / 4;
            for (int i = tid; i < L * n4; i += 256) {
                const int t = i / n4, k = i % n4 * 4;
                const bool ok = t0 + t < p.n_tok && k < p.n;
                const float* q = p.xbc + (int64_t)(t0 + t) * nch + k;
                *(float4*)(Bs + t * LS + k) = ok ? *(const float4*)(q + ob) : make_float4(0.f, 0.f, 0.f, 0.f);
                *(float4*)(Cs + t * LS + k) = ok ? *(const float4*)(q + oc) : make_float4(0.f, 0.f, 0.f, 0.f);
            }
        } else {
            for (int i = tid; i < L * np; i += 256) {
                const int t = i / np, k = i % np;
                const bool ok = t0 + t < p.n_tok && k < p.n;
                const float* q = p.xbc + (int64_t)(t0 + t) * nch + k;
                Bs[t * LS + k] = ok ? q[ob] : 0.0f;
                Cs[t * LS + k] = ok ? q[oc] : 0.0f;
            }
        }
        if (w == 0) {
            const int t = t0 + lane;
            const float dt = t < p.n_tok ? softplus_exact(p.u[(int64_t)t * ud + inner + nch + h] + bias) : 0.0f;
            double x = (double)a * (double)dt;
#pragma unroll
            for (int off = 1; off < 64; off <<= 1) {
                const double y = __shfl_up(x, off, 64);
                if (lane >= off) x += y;
            }
            const double last = __shfl(x, 63, 64);
            cum[lane] = x;
            dts[lane] = dt;
            gam[lane] = expf((float)x);
            dec[lane] = expf((float)(last - x));
            if (lane == 63) glast = expf((float)last);
        }
        // this slice of S0 for the product with C
#pragma unroll
        for (int x = 0; x < XT; x++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int c = 16 * (w + 4 * x) + m;
                if (c < np) Ss[(4 * g + i) * LS + c] = st[x][i];
            }
        __syncthreads();
        const float* cbt = cb + ((int64_t)ck * p.groups + grp) * L * L;
        for (int i = tid; i < L * L / 4; i += 256) {
            const int t = i >> 4, s = (i & 15) * 4;
            const float4 v = *(const float4*)(cbt + t * L + s);
            const double ctm = cum[t];
            float4 r;
            r.x = s <= t ? v.x * __expf((float)(ctm - cum[s])) : 0.0f;
            r.y = s + 1 <= t ? v.y * __expf((float)(ctm - cum[s + 1])) : 0.0f;
            r.z = s + 2 <= t ? v.z * __expf((float)(ctm - cum[s + 2])) : 0.0f;
            r.w = s + 3 <= t ? v.w * __expf((float)(ctm - cum[s + 3])) : 0.0f;
            *(float4*)(Ms + t * MS + s) = r;
        }
        for (int i = tid; i < L * PR; i += 256) {
            const int t = i >> 4, r = i & 15;
            const bool ok = t0 + t < p.n_tok && r0 + r < p.vdim;
            const float x = ok ? p.xbc[(int64_t)(t0 + t) * nch + h * p.vdim + r0 + r] : 0.0f;
            Xs[t * 20 + r] = x;                       // (for the skip)
            Xd[t * 20 + r] = x * dts[t];
        }
        __syncthreads();
        // Y: wave w takes tokens 16 w .. + 15
        v4f y = {0.f, 0.f, 0.f, 0.f};
        for (int s = 0; s < np / 4; s++) y = mfma4(Cs[(16 * w + m) * LS + 4 * s + g], Ss[m * LS + 4 * s + g], y);
#pragma unroll
        for (int i = 0; i < 4; i++) y[i] *= gam[16 * w + 4 * g + i];
        for (int s = 0; s < 4 * (w + 1); s++) y = mfma4(Ms[(16 * w + m) * MS + 4 * s + g], Xd[(4 * s + g) * 20 + m], y);
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int tt = 16 * w + 4 * g + i, t = t0 + tt;
            if (t < p.n_tok && r0 + m < p.vdim) {
                const int j = h * p.vdim + r0 + m;
                p.out[(int64_t)t * inner + j] = fmaf(D, Xs[tt * 20 + m], y[i]) * silu_of(p.u[(int64_t)t * ud + j], p.accurate);
            }
        }
        // S
        const float gl = glast;
#pragma unroll
        for (int x = 0; x < XT; x++) {
            const int c0 = 16 * (w + 4 * x);
            if (c0 < np) {
                v4f s4 = st[x] * gl;
#pragma unroll 4
                for (int s = 0; s < L / 4; s++) {
                    const int t = 4 * s + g;
                    s4 = mfma4(Xd[t * 20 + m] * dec[t], Bs[t * LS + c0 + m], s4);
                }
                st[x] = s4;
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int x = 0; x < XT; x++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int r = r0 + 4 * g + i, c = 16 * (w + 4 * x) + m;
            if (r < p.vdim && c < p.n) p.state[((int64_t)h * p.vdim + r) * p.n + c] = st[x][i];
        }
}

size_t cb_lds(int n) { return (size_t)2 * L * (pad4(n) + 4) * sizeof(float); }
size_t chunk_lds(int n) {
    const int LS = ((n + 15) & ~15) + 4;
    return ((size_t)2 * L * LS + L * MS + 2 * L * 20 + PR * LS) * sizeof(float);
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
    hipLaunchKernelGGL(ssd_conv_k, dim3((p.channels() + 255) / 256, (p.n_tok + CT - 1) / CT), dim3(256), 0, s, p);
}
void ssd_conv_keep(const SsdP& p, hipStream_t s) {
    hipLaunchKernelGGL(ssd_conv_keep_k, dim3((p.channels() + 255) / 256), dim3(256), 0, s, p);
}
void ssd_scan(const SsdP& p, hipStream_t s) {
#define IT_CALL(NR) hipLaunchKernelGGL(ssd_scan_k<NR>, dim3(blocks(p)), dim3(256), 0, s, p)
    IT_BY_N(p.n, IT_CALL);
#undef IT_CALL
}

// the 160 KB of LDS a CU has bound the state size of the chunked form
bool ssd_chunk_takes(const SsdP& p) { return p.n_tok >= L && chunk_lds(p.n) <= 156 * 1024; }
size_t ssd_chunk_work_floats(const SsdP& p) { return (size_t)((p.n_tok + L - 1) / L) * p.groups * L * L; }
void ssd_chunk(const SsdP& p, float* work, hipStream_t s) {
    const size_t l1 = cb_lds(p.n), l2 = chunk_lds(p.n);
    bool ok = allow_lds(ssd_cb_k, l1);
#define IT_ALLOW(X) ok = ok && allow_lds(ssd_chunk_k<X>, l2)
#define IT_CALL(X) hipLaunchKernelGGL(ssd_chunk_k<X>, dim3(((blocks(p) + 7) / 8) * 8), dim3(256), l2, s, p, work)
    if (p.n <= 64) IT_ALLOW(1);
    else if (p.n <= 128) IT_ALLOW(2);
    else IT_ALLOW(4);
    if (!ok) {
        ssd_scan(p, s);
        return;
    }
    hipLaunchKernelGGL(ssd_cb_k, dim3((p.n_tok + L - 1) / L, p.groups), dim3(256), l1, s, p, work);
    if (p.n <= 64) IT_CALL(1);
    else if (p.n <= 128) IT_CALL(2);
    else IT_CALL(4);
#undef IT_CALL
#undef IT_ALLOW
}

}  // namespace itk
