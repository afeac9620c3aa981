// Products of bf16 matrices with a batch of bf16 activations on the matrix cores (f32 sums): the groups and residual
// sums of k_group.hip for many tokens.
//
// A block owns a tile of tokens x matrix rows (256 x 256, or 128 / 64 x 128 where that leaves CUs without one) and walks k in
// slabs of 64, both operands staged in LDS (two buffers, the next slab's loads in flight while this one is multiplied).
// Rows of 64 bf16 are eight 16-byte pieces; piece c of row r sits at c ^ (r & 7), so that the 32 rows an MFMA operand takes
// spread over the banks.  A wave takes 64 rows x 32 to 128 tokens (the more, the fewer LDS reads a product: the large tile
// has three operands for four products) as 32 x 32 tiles of v_mfma_f32_32x32x16_bf16: lane l supplies eight k values of row l % 32 (k group l / 32)
// for A (tokens) and B (matrix rows) and receives column l % 32 (a matrix row) and token rows
// 8 * (i / 4) + 4 * (l / 32) + i % 4, so a store instruction writes 32 consecutive outputs of two tokens.
// A gate / up pair shares a block: its rows are 32 gate rows, the same 32 up rows, and so on, and act(gate) * up is
// formed in the lane that holds both.  A residual sum walks the terms one after the other, adds each one's scaled sums to a
// second set of accumulators, and updates the f32 residual in place.
#include "it_device.h"
#include "it_float.h"
#include "it_rows8.h"
#include "kernels_float.h"

namespace itk {
namespace {

typedef __bf16 b8 __attribute__((ext_vector_type(8)));
typedef float v16f __attribute__((ext_vector_type(16)));
constexpr int BK = 64;

// A block's shape: TM tokens x TN rows over NW waves, each of them 64 rows and what is left of the tokens
template <int TM_, int TN_, int NW_> struct Shape {
    static constexpr int TM = TM_, TN = TN_, NW = NW_, THREADS = 64 * NW;
    static constexpr int WN = TN / 64, WM = NW / WN, MI = TM / (32 * WM);   // waves along rows and tokens; 32-token operands a wave
    static constexpr int RP = THREADS / 8, NA = TM / RP, NB = TN / RP;      // tile rows a staging pass, passes
    static constexpr size_t LDS = (size_t)2 * (TM + TN) * BK * sizeof(uint16_t);
};

IT_DEV uint4 load_piece(const uint16_t* row, int k, int n_in, bool al) {
    if (al) return k < n_in ? *(const uint4*)(row + k) : make_uint4(0, 0, 0, 0);
    uint32_t v[8];
#pragma unroll
    for (int e = 0; e < 8; e++) v[e] = k + e < n_in ? row[k + e] : 0u;
    return make_uint4(v[0] | (v[1] << 16), v[2] | (v[3] << 16), v[4] | (v[5] << 16), v[6] | (v[7] << 16));
}

// acc += A (tokens tok0 ..) B^T (this block's rows) over the whole of k
template <class S, bool AL>
IT_DEV void multiply(const uint16_t* const (&arow)[S::NA], const uint16_t* const (&brow)[S::NB], int n_in, uint16_t* lds,
                     v16f (&acc)[S::MI][2]) {
    constexpr int NA = S::NA, NB = S::NB, MI = S::MI, ABUF = S::TM * BK, BBUF = S::TN * BK;
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = w % S::WM, wn = w / S::WM, r = lane & 31, g = lane >> 5;
    const int srow = tid >> 3, piece = tid & 7;
    uint16_t *As = lds, *Bs = lds + 2 * ABUF;
    const int lda = pad8(n_in);
    uint4 ra[NA], rb[NB];
    auto fetch = [&](int k0) __attribute__((always_inline)) {
        const int k = k0 + piece * 8;
#pragma unroll
        for (int i = 0; i < NA; i++) ra[i] = load_piece(arow[i], k, lda, true);
#pragma unroll
        for (int i = 0; i < NB; i++) rb[i] = load_piece(brow[i], k, n_in, AL);
    };
    auto stash = [&](int buf) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < NA; i++) *(uint4*)(As + buf * ABUF + (srow + S::RP * i) * BK + 8 * (piece ^ (srow & 7))) = ra[i];
#pragma unroll
        for (int i = 0; i < NB; i++) *(uint4*)(Bs + buf * BBUF + (srow + S::RP * i) * BK + 8 * (piece ^ (srow & 7))) = rb[i];
    };
    const int n_slab = (n_in + BK - 1) / BK;
    __syncthreads();   // the tiles of an earlier product are read
    fetch(0);
    stash(0);
    __syncthreads();
    for (int ks = 0; ks < n_slab; ks++) {
        const int cur = ks & 1;
        if (ks + 1 < n_slab) fetch((ks + 1) * BK);
        const uint16_t* a = As + cur * ABUF + (wm * 32 * MI) * BK;
        const uint16_t* b = Bs + cur * BBUF + (wn * 64) * BK;
#pragma unroll
        for (int s = 0; s < BK / 16; s++) {
            const int at = 8 * ((2 * s + g) ^ (r & 7));
            b8 fa[MI], fb[2];
#pragma unroll
            for (int mi = 0; mi < MI; mi++) fa[mi] = *(const b8*)(a + (32 * mi + r) * BK + at);
#pragma unroll
            for (int ni = 0; ni < 2; ni++) fb[ni] = *(const b8*)(b + (32 * ni + r) * BK + at);
#pragma unroll
            for (int mi = 0; mi < MI; mi++)
#pragma unroll
                for (int ni = 0; ni < 2; ni++) acc[mi][ni] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fa[mi], fb[ni], acc[mi][ni], 0, 0, 0);
        }
        if (ks + 1 < n_slab) stash(cur ^ 1);
        __syncthreads();
    }
}

// Tiles are dealt so that each of the eight dies takes a stretch of them (its L2 then holds what neighbours share), and
// inside a stretch four row tiles take turns over the token tiles.
struct Tiles {
    int first[GROUP_MAX + 1];   // row tiles of each matrix
    int rows, toks;             // tiles in all
};
IT_DEV bool tile_of(const Tiles& t, int* row, int* tok) {
    const int total = t.rows * t.toks, per = (total + 7) / 8;
    const int at = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if (at >= total || (int)(blockIdx.x >> 3) >= per) return false;
    const int band = 4 * t.toks, b = at / band, in = at % band;
    const int width = min(4, t.rows - 4 * b);
    *row = 4 * b + in % width;
    *tok = in / width;
    return true;
}

// where column j of a matrix's results goes: one f32 or 16-bit element a token (group_store with everything but the token settled)
struct Dest {
    float* f = nullptr;
    uint16_t* h = nullptr;
    int64_t stride;
    float scale;
    bool bf16;
    IT_DEV Dest(const GroupMat& m, int j) : stride(m.n_out), scale(m.scale), bf16(m.o.half != nullptr) {
        const GroupOut& o = m.o;
        if (o.slab) {
            stride = o.row_stride;
            const int64_t at = (int64_t)(o.row_dyn ? *o.row_dyn : o.row) * stride + (j / o.head_dim) * o.head_stride + j % o.head_dim;
            if (o.slab_f32) f = (float*)o.slab + at;
            else h = (uint16_t*)o.slab + at;
        } else if (o.half) {
            stride = pad8(m.n_out);
            h = o.half + j;
        } else {
            f = o.f32 + j;
        }
    }
    IT_DEV void store(int t, float v) const {
        v *= scale;
        if (f) f[t * stride] = v;
        else h[t * stride] = bf16 ? to_bf16(v) : it_f32_to_f16(v);
    }
};

template <class S, bool AL>
__global__ __launch_bounds__(S::THREADS, 2) void group_gemm_bf16_k(GroupP p, Tiles tl, const uint16_t* __restrict__ x16) {
    extern __shared__ __align__(16) uint16_t glds[];
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = w % S::WM, wn = w / S::WM, r = lane & 31, g = lane >> 5, srow = tid >> 3;
    int rt, tt;
    if (!tile_of(tl, &rt, &tt)) return;
    int mi_ = 0;
    while (mi_ + 1 < p.n_mats && rt >= tl.first[mi_ + 1]) mi_++;
    const GroupMat& m = p.m[mi_];
    const bool pair = m.up != nullptr;
    const int j0 = (rt - tl.first[mi_]) * (pair ? S::TN / 2 : S::TN), tok0 = tt * S::TM;
    const uint16_t *arow[S::NA], *brow[S::NB];
#pragma unroll
    for (int i = 0; i < S::NA; i++) arow[i] = x16 + (int64_t)min(tok0 + srow + S::RP * i, p.n_tok - 1) * pad8(p.n_in);
#pragma unroll
    for (int i = 0; i < S::NB; i++) {
        const int b = srow + S::RP * i, j = pair ? j0 + (b >> 6) * 32 + (b & 31) : j0 + b;
        brow[i] = (const uint16_t*)(pair && (b & 32) ? m.up : m.w) + (int64_t)min(j, m.n_out - 1) * p.n_in;
    }
    v16f acc[S::MI][2];
#pragma unroll
    for (int a = 0; a < S::MI; a++)
#pragma unroll
        for (int b = 0; b < 2; b++)
#pragma unroll
            for (int i = 0; i < 16; i++) acc[a][b][i] = 0.0f;
    multiply<S, AL>(arow, brow, p.n_in, glds, acc);
    const int t0 = tok0 + wm * S::MI * 32 + 4 * g;
    if (pair) {
        const int j = j0 + 32 * wn + r;
        if (j >= m.n_out) return;
        const Dest d(m, j);
#pragma unroll
        for (int mi = 0; mi < S::MI; mi++)
#pragma unroll
            for (int i = 0; i < 16; i++) {
                const int t = t0 + 32 * mi + 8 * (i >> 2) + (i & 3);
                if (t < p.n_tok) d.store(t, act_of(m.act, acc[mi][0][i]) * acc[mi][1][i]);
            }
        return;
    }
#pragma unroll
    for (int ni = 0; ni < 2; ni++) {
        const int j = j0 + 64 * wn + 32 * ni + r;
        if (j >= m.n_out) continue;
        const Dest d(m, j);
#pragma unroll
        for (int mi = 0; mi < S::MI; mi++)
#pragma unroll
            for (int i = 0; i < 16; i++) {
                const int t = t0 + 32 * mi + 8 * (i >> 2) + (i & 3);
                if (t < p.n_tok) d.store(t, acc[mi][ni][i]);
            }
    }
}

struct ResIn {
    const uint16_t* x16[RES_MAX];
};
template <class S, bool AL>
__global__ __launch_bounds__(S::THREADS, 2) void res_gemm_bf16_k(ResP p, Tiles tl, ResIn in) {
    extern __shared__ __align__(16) uint16_t glds[];
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = w % S::WM, wn = w / S::WM, r = lane & 31, g = lane >> 5, srow = tid >> 3;
    int rt, tt;
    if (!tile_of(tl, &rt, &tt)) return;
    const int j0 = rt * S::TN, tok0 = tt * S::TM;
    v16f total[S::MI][2];
#pragma unroll
    for (int a = 0; a < S::MI; a++)
#pragma unroll
        for (int b = 0; b < 2; b++)
#pragma unroll
            for (int i = 0; i < 16; i++) total[a][b][i] = 0.0f;
    for (int k = 0; k < p.n_terms; k++) {
        const ResTerm& q = p.t[k];
        const uint16_t *arow[S::NA], *brow[S::NB];
#pragma unroll
        for (int i = 0; i < S::NA; i++) arow[i] = in.x16[k] + (int64_t)min(tok0 + srow + S::RP * i, p.n_tok - 1) * pad8(q.n_in);
#pragma unroll
        for (int i = 0; i < S::NB; i++) brow[i] = (const uint16_t*)q.w + (int64_t)min(j0 + S::RP * i + srow, p.n_out - 1) * q.n_in;
        v16f acc[S::MI][2];
#pragma unroll
        for (int a = 0; a < S::MI; a++)
#pragma unroll
            for (int b = 0; b < 2; b++)
#pragma unroll
                for (int i = 0; i < 16; i++) acc[a][b][i] = 0.0f;
        multiply<S, AL>(arow, brow, q.n_in, glds, acc);
#pragma unroll
        for (int ni = 0; ni < 2; ni++) {
            const int j = min(j0 + 64 * wn + 32 * ni + r, p.n_out - 1);
            const float sc = q.scale ? q.scale[j] : 1.0f;
#pragma unroll
            for (int mi = 0; mi < S::MI; mi++)
#pragma unroll
                for (int i = 0; i < 16; i++) total[mi][ni][i] = fmaf(acc[mi][ni][i], sc, total[mi][ni][i]);
        }
    }
#pragma unroll
    for (int mi = 0; mi < S::MI; mi++)
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const int t = tok0 + (wm * S::MI + mi) * 32 + 8 * (i >> 2) + 4 * g + (i & 3);
            if (t >= p.n_tok) continue;
#pragma unroll
            for (int ni = 0; ni < 2; ni++) {
                const int j = j0 + 64 * wn + 32 * ni + r;
                if (j >= p.n_out) continue;
                float* x = p.x + (int64_t)t * p.n_out + j;
                *x = p.set ? total[mi][ni][i] : *x + total[mi][ni][i];
            }
        }
}

template <class F> bool allow_lds(F* fn, size_t lds) {
    if (lds <= 64 * 1024) return true;
    if (hipFuncSetAttribute((const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess) return true;
    (void)hipGetLastError();
    return false;
}
typedef Shape<64, 128, 4> Small;
typedef Shape<128, 128, 4> Medium;
typedef Shape<256, 256, 8> Large;
int tiles_of(int n, int per) { return (n + per - 1) / per; }
dim3 grid_of(const Tiles& t) { return dim3((unsigned)(((t.rows * t.toks + 7) / 8) * 8)); }

template <class S> Tiles group_tiles(const GroupP& p) {
    Tiles t{};
    for (int i = 0; i < p.n_mats; i++) t.first[i + 1] = t.first[i] + tiles_of(p.m[i].n_out, p.m[i].up ? S::TN / 2 : S::TN);
    t.rows = t.first[p.n_mats];
    t.toks = tiles_of(p.n_tok, S::TM);
    return t;
}
template <class S> bool group_launch(const GroupP& p, const uint16_t* x16, bool al, hipStream_t s) {
    const Tiles t = group_tiles<S>(p);
    if (!allow_lds(al ? group_gemm_bf16_k<S, true> : group_gemm_bf16_k<S, false>, S::LDS)) return false;
    if (al) hipLaunchKernelGGL((group_gemm_bf16_k<S, true>), grid_of(t), dim3(S::THREADS), S::LDS, s, p, t, x16);
    else hipLaunchKernelGGL((group_gemm_bf16_k<S, false>), grid_of(t), dim3(S::THREADS), S::LDS, s, p, t, x16);
    return true;
}
template <class S> Tiles res_tiles(const ResP& p) {
    Tiles t{};
    t.rows = t.first[1] = tiles_of(p.n_out, S::TN);
    t.toks = tiles_of(p.n_tok, S::TM);
    return t;
}
template <class S> void res_launch(const ResP& p, const ResIn& in, bool al, hipStream_t s) {
    const Tiles t = res_tiles<S>(p);
    if (al) hipLaunchKernelGGL((res_gemm_bf16_k<S, true>), grid_of(t), dim3(S::THREADS), S::LDS, s, p, t, in);
    else hipLaunchKernelGGL((res_gemm_bf16_k<S, false>), grid_of(t), dim3(S::THREADS), S::LDS, s, p, t, in);
}
int count(const Tiles& t) { return t.rows * t.toks; }

}  // namespace

// the largest tiles that still give every CU work
void group_gemm_bf16(const GroupP& p, const uint16_t* x16, hipStream_t s) {
    bool al = p.n_in % 8 == 0;
    for (int i = 0; i < p.n_mats; i++) al = al && aligned16(p.m[i].w) && aligned16(p.m[i].up);
    if (count(group_tiles<Large>(p)) >= 256 && group_launch<Large>(p, x16, al, s)) return;
    if (count(group_tiles<Medium>(p)) >= 512) group_launch<Medium>(p, x16, al, s);
    else group_launch<Small>(p, x16, al, s);
}

void res_gemm_bf16(const ResP& p, const uint16_t* const in16[RES_MAX], hipStream_t s) {
    ResIn in{};
    bool al = true;
    for (int i = 0; i < p.n_terms; i++) {
        in.x16[i] = in16[i];
        al = al && p.t[i].n_in % 8 == 0 && aligned16(p.t[i].w);
    }
    if (count(res_tiles<Medium>(p)) >= 512) res_launch<Medium>(p, in, al, s);
    else res_launch<Small>(p, in, al, s);
}

}  // namespace itk
