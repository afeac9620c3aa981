// Launch wrappers of the kernels for models with unquantized (bf16 / f16 / f32) matrices, biased attention and a
// state-space mixer.  Plain device pointers and sizes; `_dyn` pointers name a device int that overrides the scalar
// beside them (what keeps a captured decode graph valid while the position advances).
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "kernels.h"

namespace itk {

constexpr int GROUP_MAX = 6;   // matrices of one group
constexpr int pad8(int n) { return (n + 7) & ~7; }

// Where the rows of one matrix of a group go: f32 [token][n_out], bf16 [token][pad8(n_out)], or a cache slab whose row
// `row + token` holds heads of head_dim elements head_stride apart.
struct GroupOut {
    float* f32;
    uint16_t* half;
    void* slab;
    int slab_f32;               // the slab's elements are f32 instead of f16
    int head_dim, head_stride;
    int64_t row_stride;
    int row;
    const int* row_dyn;
};
struct GroupMat {
    const uint8_t* w;
    const uint8_t* up;          // non-null: the result is act(w x) * (up x)
    int n_out;
    int act;                    // ACT_*
    float scale;
    GroupOut o;
};
enum { ACT_SILU = 0, ACT_RELU = 1 };
// x_new = x + mult * (y / rms(y)) * w: what a sublayer whose output is normed adds to the residual
struct AddNormed {
    const float* y;             // [token][n], or null: nothing to add
    const float* w;             // [n]
    float* x_new;               // [token][n], another buffer than x
    float eps, mult;
};
struct GroupP {
    const float* x;             // [token][n_in]
    AddNormed add;              // what is added to x ahead of the norm
    const float* norm_w;        // RMS norm ahead of the products, or null
    float eps;
    int n_in, n_tok, n_mats, fmt;
    GroupMat m[GROUP_MAX];
};

// x[t][j] += (set: =) sum over the terms of scale[j] * (W norm(in))[j]
struct ResTerm {
    const uint8_t* w;
    const float* in;            // [token][n_in]
    const float* scale;         // [n_out] or null
    const float* norm_w;        // RMS norm of `norm_groups` equal parts ahead of the product, or null
    const float* gate;          // [token][n_in]: the normed input times silu(gate), or null
    int n_in, norm_groups;
    int norm_period;            // elements of norm_w, used again and again along the row: n_in, or a part
    float eps;
};
constexpr int RES_MAX = 2;
struct ResP {
    float* x;
    int n_out, n_tok, n_terms, fmt;
    int set;
    ResTerm t[RES_MAX];
};

// one token: the norm inside the launch, the input in LDS; false: a shape the kernel does not take
bool group_gemv(const GroupP& p, hipStream_t s);
bool group_gemv_takes(const GroupP& p);
bool res_gemv(const ResP& p, hipStream_t s);
bool res_gemv_takes(const ResP& p);
// a few tokens: every weight row read once per eight of them; the inputs are already normed (norm_w is ignored)
void group_rows(const GroupP& p, hipStream_t s);
void res_rows(const ResP& p, hipStream_t s);

// many tokens on the bf16 matrix cores (bf16 matrices only); x16 / in16: bf16 [token][pad8(n_in)], already normed
void group_gemm_bf16(const GroupP& p, const uint16_t* x16, hipStream_t s);
void res_gemm_bf16(const ResP& p, const uint16_t* const in16[RES_MAX], hipStream_t s);

// rows of x in `groups` equal parts, each divided by its own root mean square, times w (null: no norm, a conversion);
// to f32 and / or to bf16 rows of pad8(nd)
void norm_rows(const float* x, const float* w, int groups, float eps, int64_t n_rows, int nd, float* out32, uint16_t* out16,
               hipStream_t s);
// the same with w of `period` elements repeated along the row, and silu(gate) behind it
void norm_gate_rows(const float* x, const float* w, int period, const float* gate, int groups, float eps, int64_t n_rows, int nd,
                    float* out32, uint16_t* out16, hipStream_t s);
// x_new = x + what `add` says; with norm_w also rms(x_new) * norm_w to f32 and / or to bf16 rows of pad8(nd)
void add_norm_rows(const float* x, const AddNormed& add, const float* norm_w, float eps, int64_t n_rows, int nd, float* out32,
                   uint16_t* out16, hipStream_t s);
// a = act(a) * b
void act_mul(float* a, const float* b, int64_t n, int act, hipStream_t s);
// f32 rows of nd from bf16 rows of pad8(nd)
void widen_rows(const uint16_t* in, int64_t n_rows, int nd, float* out, hipStream_t s);
// one matrix's f32 rows to where its GroupOut says (the form with one launch per operation)
void group_scatter(const GroupMat& m, const float* rows, int n_tok, hipStream_t s);
// x += a * sa (+ b * sb), the sum of the two first; scales [nd] or null, b may be null
void scaled_residual(float* x, const float* a, const float* sa, const float* b, const float* sb, int set, int64_t n_rows, int nd, hipStream_t s);
// x[t] += rows[t] (may be null) + 1 * vec: the row first, then the vector (may be null)
void add_rows(float* x, const float* rows, const float* vec, int64_t n_rows, int nd, hipStream_t s);
void gather_rows(const float* src, const int32_t* idx, int n_rows, int nd, float* out, hipStream_t s);

// ---- attention with a distance bias, a sink in the denominator, a query temperature and a value size of its own ----
struct BiasAttnP {
    const float* q;             // [token][n_head * k_dim]
    const void *k, *v;          // slabs: row = position, heads k_stride / v_stride apart
    int kv_f32;
    int n_q, n_pos;
    int k_dim, v_dim, k_stride, v_stride, n_head, n_head_kv;
    float scale;
    const float* slopes;        // [n_head] (device) or null: score -= slope * (i - j)
    int sink;                   // 1: the denominator is e^sinks[head] + sum exp(score)
    const float* sinks;         // [n_head] (device) or null: all 0
    int window;                 // position i sees the keys above i - window; 0: all up to i
    const float* gate;          // [token][n_head]: the output times sigmoid(gate), or null (attend_bias_batch only)
    float temp_coef;            // q *= 1 + coef * ln(floor((p + 1) / every) + 1); 0: none
    int temp_every;
    const int* n_pos_dyn;
};
// any shape, either element type, 32-bit arithmetic; one block per (query, head)
void attend_bias_plain(const BiasAttnP& a, float* out, hipStream_t s);
// f16 slabs on the matrix cores
bool attend_bias_mfma_takes(const BiasAttnP& a);
int attend_bias_splits(int n_pos_max, int n_q);
size_t attend_bias_scratch_floats(const BiasAttnP& a, int n_split);
bool attend_bias_split(const BiasAttnP& a, int n_split, float* scratch, float* out, hipStream_t s);
// many queries; out32 and / or out16 (bf16 rows of pad8(n_head * v_dim))
bool attend_bias_batch(const BiasAttnP& a, float* out32, uint16_t* out16, hipStream_t s);

// ---- Mamba-2 mixer (state-space duality) ----
struct SsdP {
    const float* u;             // [token][z | x | B | C | dt]
    const float *conv_w, *conv_b, *dt_bias, *a_log, *d;
    float* conv_ring;           // [taps][x | B | C]: the raw input of position p in row p % taps
    float* state;               // [heads][vdim][n]
    float* xbc;                 // [token][x | B | C] after conv and silu (not used for one token)
    float* out;                 // [token][heads * vdim]: the read-out times silu(z)
    int heads, vdim, n, groups, taps;
    int n_tok, pos;
    const int* pos_dyn;
    int accurate;               // library exponentials in the short convolution's and the gate's silu
    __host__ __device__ int inner() const { return heads * vdim; }
    __host__ __device__ int channels() const { return inner() + 2 * groups * n; }
    __host__ __device__ int u_dim() const { return inner() + channels() + heads; }
};
bool ssd_takes(const SsdP& p);
void ssd_step(const SsdP& p, hipStream_t s);          // one token
void ssd_conv(const SsdP& p, hipStream_t s);          // several tokens: fills xbc
void ssd_conv_keep(const SsdP& p, hipStream_t s);     // several tokens: the last inputs into the ring
void ssd_scan(const SsdP& p, hipStream_t s);          // several tokens, one after the other
bool ssd_chunk_takes(const SsdP& p);
size_t ssd_chunk_work_floats(const SsdP& p);
void ssd_chunk(const SsdP& p, float* work, hipStream_t s);   // many tokens: chunks of 64 on the fp32 matrix cores


// ---- gated linear attention: a decay per key channel ----
struct GlaP {
    const float *q, *k;         // [token][heads * dim]
    const float* v;             // [token][heads * vdim]
    const float* low;           // [token][rank]: the decay's logit is a2 low + a2_b
    const uint8_t* a2;          // [heads * dim][rank] of type a2_fmt
    int a2_fmt;
    const float* a2_b;
    float inv_tau;
    float* state;               // [heads][vdim][dim]
    float* decay;               // [token][heads * dim] (not used for one token): see gla_decay
    float* out;                 // [token][heads * vdim]
    int heads, dim, vdim, rank, n_tok;
    __host__ __device__ int keys() const { return heads * dim; }
    __host__ __device__ int values() const { return heads * vdim; }
};
bool gla_takes(const GlaP& p);
void gla_step(const GlaP& p, hipStream_t s);          // one token
// several tokens: the decays, or their logarithms summed up over every 16 tokens of the call
void gla_decay(const GlaP& p, int logs, hipStream_t s);
void gla_scan(const GlaP& p, hipStream_t s);          // several tokens, one after the other, from the decays
bool gla_chunk_takes(const GlaP& p);
size_t gla_chunk_work_floats(const GlaP& p);
bool gla_chunk(const GlaP& p, float* work, hipStream_t s);   // many tokens: chunks of 64 on the fp32 matrix cores, from the logarithms

// ---- latent attention: a cache row is [latent | rotated key part], shared by all heads ----
struct LatentP {
    const float* q;             // [token][heads * (dim + rot)]: [unrotated | rotated] a head
    const float* kv;            // [token][rank + rot]: latent before its norm, key part before its rotation; null: rows are there already
    const float* kv_norm;       // [rank]
    float eps;
    const float2* table;        // (cos, sin) of [position][n_rot / 2]
    const uint8_t* uk;          // [heads * dim][rank] of type uk_fmt
    const uint8_t* uv;          // [heads * vdim][rank] of type uv_fmt
    int uk_fmt, uv_fmt;
    void* slab;                 // row = position
    int slab_f32, row_stride;
    const float* gate;          // [token][heads] or null: the output times sigmoid(gate)
    int heads, dim, rot, n_rot, rank, vdim;
    int n_tok, pos;
    const int* n_pos_dyn;       // one token: the context's length (position + 1)
    __host__ __device__ int k_dim() const { return rank + rot; }
};
// queries against the latent itself, [uk^T q | rotated q] of [token][heads]: f32 rows of rank + rot (qa), or f16 rows of kp, times
// scale * log2 e and with zeros behind (q16); and the tokens' cache rows
void latent_prep(const LatentP& p, float* qa, uint16_t* q16, int kp, float scale, hipStream_t s);
// many tokens: their cache rows, and the rotated parts of q in place
void latent_rows(const LatentP& p, float* q, hipStream_t s);
// cache rows `first` .. as bf16 latents of pad8(rank) and as the rotated part of every head's key rows (f16, ks elements a head)
void latent_keys(const LatentP& p, int first, int n_keys, uint16_t* c16, uint16_t* k, int ks, hipStream_t s);
// out [token][heads * vdim] = gate * uv ol, ol [token][heads][rank]
void latent_value(const LatentP& p, const float* ol, float* out, hipStream_t s);
// few queries against rows whose first v_dim elements are the values, one row for all heads, on the f16 matrix cores:
// out [query][head][v_dim]
bool attend_shared_takes(const BiasAttnP& a);
int attend_shared_splits(const BiasAttnP& a, int n_pos_max);
size_t attend_shared_scratch_floats(const BiasAttnP& a, int n_split);
int attend_shared_q_row(const BiasAttnP& a);   // elements of a row of q16
bool attend_shared_split(const BiasAttnP& a, const uint16_t* q16, int n_split, float* scratch, float* out, hipStream_t s);   // (a.q is not read)

}  // namespace itk
