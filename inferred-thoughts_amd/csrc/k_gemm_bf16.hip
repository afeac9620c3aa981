// Products of bf16 matrices with a batch of bf16 activations on the matrix cores (f32 sums): the groups and residual
// sums of k_group.hip for many tokens.
//
// A block owns TM tokens x 128 matrix rows and walks k in slabs of 64, both operands staged in LDS (two buffers, the
// next slab's loads in flight while this one is multiplied).  Rows of 64 bf16 are eight 16-byte pieces; piece c of row r
// sits at c ^ (r & 7), so that the 32 rows an MFMA operand takes spread over the banks.  Four waves, each TM/2 tokens
// x 64 rows as 32 x 32 tiles of v_mfma_f32_32x32x16_bf16: lane l supplies eight k values of row l % 32 (k group l / 32)
// for A (tokens) and B (matrix rows) and receives column l % 32 (a matrix row) and token rows
// 8 * (i / 4) + 4 * (l / 32) + i % 4, so a store instruction writes 32 consecutive outputs of two tokens.
// A gate / up pair shares a block: its 128 rows are 32 gate rows, the same 32 up rows, and so on, and silu(gate) * up is
// formed in the lane that holds both.  A residual sum walks the terms one after the other, adds each one's scaled sums to a
// second set of accumulators, and updates the f32 residual in place.
#include "it_device.h"
#include "it_float.h"
#include "kernels_float.h"

namespace itk {
namespace {

typedef __bf16 b8 __attribute__((ext_vector_type(8)));
typedef float v16f __attribute__((ext_vector_type(16)));
constexpr int BK = 64, BN = 128;

IT_DEV uint4 load_piece(const uint16_t* row, int k, int n_in, bool al) {
    if (al) return k < n_in ? *(const uint4*)(row + k) : make_uint4(0, 0, 0, 0);
    uint32_t v[8];
#pragma unroll
    for (int e = 0; e < 8; e++) v[e] = k + e < n_in ? row[k + e] : 0u;
    return make_uint4(v[0] | (v[1] << 16), v[2] | (v[3] << 16), v[4] | (v[5] << 16), v[6] | (v[7] << 16));
}

// acc += A (tokens tok0 ..) B^T (this block's rows) over the whole of k
template <int TM, bool AL>
IT_DEV void multiply(const uint16_t* const (&arow)[TM / 32], const uint16_t* const (&brow)[4], int n_in, uint16_t* lds,
                     v16f (&acc)[TM / 64][2]) {
    constexpr int NA = TM / 32, MI = TM / 64, ABUF = TM * BK, BBUF = BN * BK;
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = w & 1, wn = w >> 1, r = lane & 31, g = lane >> 5;
    const int srow = tid >> 3, piece = tid & 7;
    uint16_t *As = lds, *Bs = lds + 2 * ABUF;
    const int lda = pad8(n_in);
    uint4 ra[NA], rb[4];
    auto fetch = [&](int k0) __attribute__((always_inline)) {
        const int k = k0 + piece * 8;
#pragma unroll
        for (int i = 0; i < NA; i++) ra[i] = load_piece(arow[i], k, lda, true);
#pragma unroll
        for (int i = 0; i < 4; i++) rb[i] = load_piece(brow[i], k, n_in, AL);
    };
    auto stash = [&](int buf) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < NA; i++) *(uint4*)(As + buf * ABUF + (srow + 32 * i) * BK + 8 * (piece ^ (srow & 7))) = ra[i];
#pragma unroll
        for (int i = 0; i < 4; i++) *(uint4*)(Bs + buf * BBUF + (srow + 32 * i) * BK + 8 * (piece ^ (srow & 7))) = rb[i];
    };
    const int n_slab = (n_in + BK - 1) / BK;
    __syncthreads();   // the tiles of an earlier product are read
    fetch(0);
    stash(0);
    __syncthreads();
    for (int ks = 0; ks < n_slab; ks++) {
        const int cur = ks & 1;
        if (ks + 1 < n_slab) fetch((ks + 1) * BK);
        const uint16_t* a = As + cur * ABUF + (wm * (TM / 2)) * BK;
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

template <int TM, bool AL>
__global__ __launch_bounds__(256, 2) void group_gemm_bf16_k(GroupP p, Tiles tl, const uint16_t* __restrict__ x16) {
    extern __shared__ __align__(16) uint16_t glds[];
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = w & 1, wn = w >> 1, r = lane & 31, g = lane >> 5, srow = tid >> 3;
    int rt, tt;
    if (!tile_of(tl, &rt, &tt)) return;
    int mi_ = 0;
    while (mi_ + 1 < p.n_mats && rt >= tl.first[mi_ + 1]) mi_++;
    const GroupMat& m = p.m[mi_];
    const bool pair = m.up != nullptr;
    const int j0 = (rt - tl.first[mi_]) * (pair ? BN / 2 : BN), tok0 = tt * TM;
    const uint16_t *arow[TM / 32], *brow[4];
#pragma unroll
    for (int i = 0; i < TM / 32; i++) arow[i] = x16 + (int64_t)min(tok0 + srow + 32 * i, p.n_tok - 1) * pad8(p.n_in);
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int j = pair ? j0 + (i >> 1) * 32 + srow : j0 + 32 * i + srow;
        brow[i] = (const uint16_t*)(pair && (i & 1) ? m.up : m.w) + (int64_t)min(j, m.n_out - 1) * p.n_in;
    }
    v16f acc[TM / 64][2];
#pragma unroll
    for (int a = 0; a < TM / 64; a++)
#pragma unroll
        for (int b = 0; b < 2; b++)
#pragma unroll
            for (int i = 0; i < 16; i++) acc[a][b][i] = 0.0f;
    multiply<TM, AL>(arow, brow, p.n_in, glds, acc);
#pragma unroll
    for (int mi = 0; mi < TM / 64; mi++) {
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const int t = tok0 + wm * (TM / 2) + 32 * mi + 8 * (i >> 2) + 4 * g + (i & 3);
            if (t >= p.n_tok) continue;
            if (pair) {
                const int j = j0 + 32 * wn + r;
                if (j < m.n_out) group_store(m, t, j, silu_exact(acc[mi][0][i]) * acc[mi][1][i]);
            } else {
#pragma unroll
                for (int ni = 0; ni < 2; ni++) {
                    const int j = j0 + 64 * wn + 32 * ni + r;
                    if (j < m.n_out) group_store(m, t, j, acc[mi][ni][i]);
                }
            }
        }
    }
}

struct ResIn {
    const uint16_t* x16[RES_MAX];
};
template <int TM, bool AL>
__global__ __launch_bounds__(256, 2) void res_gemm_bf16_k(ResP p, Tiles tl, ResIn in) {
    extern __shared__ __align__(16) uint16_t glds[];
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = w & 1, wn = w >> 1, r = lane & 31, g = lane >> 5, srow = tid >> 3;
    int rt, tt;
    if (!tile_of(tl, &rt, &tt)) return;
    const int j0 = rt * BN, tok0 = tt * TM;
    v16f total[TM / 64][2];
#pragma unroll
    for (int a = 0; a < TM / 64; a++)
#pragma unroll
        for (int b = 0; b < 2; b++)
#pragma unroll
            for (int i = 0; i < 16; i++) total[a][b][i] = 0.0f;
    for (int k = 0; k < p.n_terms; k++) {
        const ResTerm& q = p.t[k];
        const uint16_t *arow[TM / 32], *brow[4];
#pragma unroll
        for (int i = 0; i < TM / 32; i++) arow[i] = in.x16[k] + (int64_t)min(tok0 + srow + 32 * i, p.n_tok - 1) * pad8(q.n_in);
#pragma unroll
        for (int i = 0; i < 4; i++) brow[i] = (const uint16_t*)q.w + (int64_t)min(j0 + 32 * i + srow, p.n_out - 1) * q.n_in;
        v16f acc[TM / 64][2];
#pragma unroll
        for (int a = 0; a < TM / 64; a++)
#pragma unroll
            for (int b = 0; b < 2; b++)
#pragma unroll
                for (int i = 0; i < 16; i++) acc[a][b][i] = 0.0f;
        multiply<TM, AL>(arow, brow, q.n_in, glds, acc);
#pragma unroll
        for (int ni = 0; ni < 2; ni++) {
            const int j = min(j0 + 64 * wn + 32 * ni + r, p.n_out - 1);
            const float sc = q.scale ? q.scale[j] : 1.0f;
#pragma unroll
            for (int mi = 0; mi < TM / 64; mi++)
#pragma unroll
                for (int i = 0; i < 16; i++) total[mi][ni][i] = fmaf(acc[mi][ni][i], sc, total[mi][ni][i]);
        }
    }
#pragma unroll
    for (int mi = 0; mi < TM / 64; mi++)
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const int t = tok0 + wm * (TM / 2) + 32 * mi + 8 * (i >> 2) + 4 * g + (i & 3);
            if (t >= p.n_tok) continue;
#pragma unroll
            for (int ni = 0; ni < 2; ni++) {
                const int j = j0 + 64 * wn + 32 * ni + r;
                if (j < p.n_out) p.x[(int64_t)t * p.n_out + j] += total[mi][ni][i];
            }
        }
}

constexpr size_t lds_bytes(int tm) { return (size_t)2 * (tm + BN) * BK * sizeof(uint16_t); }
bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }
// 64 tokens a block where 128 would leave CUs without one
int tokens_per_block(int row_tiles, int n_tok) { return (int64_t)row_tiles * ((n_tok + 127) / 128) < 512 ? 64 : 128; }

}  // namespace

void group_gemm_bf16(const GroupP& p, const uint16_t* x16, hipStream_t s) {
    Tiles t{};
    bool al = p.n_in % 8 == 0;
    for (int i = 0; i < p.n_mats; i++) {
        const int per = p.m[i].up ? BN / 2 : BN;
        t.first[i + 1] = t.first[i] + (p.m[i].n_out + per - 1) / per;
        al = al && aligned16(p.m[i].w) && aligned16(p.m[i].up);
    }
    t.rows = t.first[p.n_mats];
    const int tm = tokens_per_block(t.rows, p.n_tok);
    t.toks = (p.n_tok + tm - 1) / tm;
    const dim3 grid((unsigned)(((t.rows * t.toks + 7) / 8) * 8)), block(256);
    if (tm == 64) {
        if (al) hipLaunchKernelGGL((group_gemm_bf16_k<64, true>), grid, block, lds_bytes(64), s, p, t, x16);
        else hipLaunchKernelGGL((group_gemm_bf16_k<64, false>), grid, block, lds_bytes(64), s, p, t, x16);
    } else {
        if (al) hipLaunchKernelGGL((group_gemm_bf16_k<128, true>), grid, block, lds_bytes(128), s, p, t, x16);
        else hipLaunchKernelGGL((group_gemm_bf16_k<128, false>), grid, block, lds_bytes(128), s, p, t, x16);
    }
}

void res_gemm_bf16(const ResP& p, const uint16_t* const in16[RES_MAX], hipStream_t s) {
    Tiles t{};
    ResIn in{};
    bool al = true;
    for (int i = 0; i < p.n_terms; i++) {
        in.x16[i] = in16[i];
        al = al && p.t[i].n_in % 8 == 0 && aligned16(p.t[i].w);
    }
    t.rows = (p.n_out + BN - 1) / BN;
    t.first[1] = t.rows;
    const int tm = tokens_per_block(t.rows, p.n_tok);
    t.toks = (p.n_tok + tm - 1) / tm;
    const dim3 grid((unsigned)(((t.rows * t.toks + 7) / 8) * 8)), block(256);
    if (tm == 64) {
        if (al) hipLaunchKernelGGL((res_gemm_bf16_k<64, true>), grid, block, lds_bytes(64), s, p, t, in);
        else hipLaunchKernelGGL((res_gemm_bf16_k<64, false>), grid, block, lds_bytes(64), s, p, t, in);
    } else {
        if (al) hipLaunchKernelGGL((res_gemm_bf16_k<128, true>), grid, block, lds_bytes(128), s, p, t, in);
        else hipLaunchKernelGGL((res_gemm_bf16_k<128, false>), grid, block, lds_bytes(128), s, p, t, in);
    }
}

}  // namespace itk
