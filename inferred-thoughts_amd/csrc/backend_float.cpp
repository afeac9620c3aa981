// Seam ops of models with unquantized matrices: groups of products behind a norm, residual sums, biased attention, latent
// attention, the Mamba-2 mixer, gated linear attention.  As in backend.cpp, each op checks its shapes on the host before anything is launched, and the first
// error is kept.
#include <algorithm>
#include <climits>
#include <cstring>

#include "backend.h"

using namespace itk;

namespace {
constexpr uint64_t FEW = 16;   // tokens up to which the row kernels are taken

template <class... A>
uint64_t sig_of(const A&... a) {   // FNV-1a over the raw bytes of each argument
    uint64_t h = 0xcbf29ce484222325ull;
    auto mix = [&](const void* p, size_t n) {
        const uint8_t* b = (const uint8_t*)p;
        for (size_t i = 0; i < n; i++) h = (h ^ b[i]) * 0x100000001b3ull;
    };
    (mix(&a, sizeof(a)), ...);
    return h;
}
bool float_type(uint32_t ty) { return ty == IT_F32 || ty == IT_F16 || ty == IT_BF16; }
enum { T_NORM = 0, T_A, T_B, T_HALF0, T_HALF1, T_XBC, T_QA, T_OL, T_LATENT, T_KEYS, T_VALUES };   // tmp_for uses
}  // namespace

void* it_hip::tmp_for(int which, size_t bytes) {
    Tmp& t = tmps[which];
    if (t.bytes < bytes) {
        need_eager("scratch of the unquantized ops has to grow");
        drop_graph();   // a captured graph holds the old buffer
        if (t.p) {
            check(hipStreamSynchronize(stream), "sync before scratch free");
            (void)hipFree(t.p);
            t = Tmp{};
        }
        if (!check(hipMalloc(&t.p, bytes), "hipMalloc(scratch)")) return nullptr;
        t.bytes = bytes;
    }
    return t.p;
}

uint16_t* it_hip::act_half_reserve(Act& a, size_t rows, size_t row) {
    const size_t n = rows * (size_t)pad8((int)row);
    if (a.h_cap < n) {
        need_eager("a bf16 activation buffer has to grow");
        if (a.h16) {
            check(hipStreamSynchronize(stream), "sync before a bf16 form is freed");
            quant_bytes -= a.h_cap * sizeof(uint16_t);
            (void)hipFree(a.h16);
            a.h16 = nullptr;
            a.h_cap = 0;
        }
        if (!check(hipMalloc((void**)&a.h16, n * sizeof(uint16_t)), "hipMalloc(bf16 activations)")) return nullptr;
        a.h_cap = n;
        quant_bytes += n * sizeof(uint16_t);
    }
    // pad elements past a row's end meet zeroed weights only, but must not be NaN
    if (row % 8) fill_zero(a.h16, (int64_t)(n * sizeof(uint16_t)), stream);
    return a.h16;
}
uint16_t* it_hip::act_half_out(const float* host, size_t rows, size_t row) {
    Act* a = act_slot(host, rows * row);
    if (!a) return nullptr;
    uint16_t* h = act_half_reserve(*a, rows, row);
    if (!h) return nullptr;
    a->stale_forms();
    a->dev_current = true;
    a->elided = true;
    a->h_rows = rows;
    a->h_row = row;
    a->h_valid = true;
    return h;
}
void it_hip::act_widen(Act& a) {
    if (a.cap < a.h_rows * a.h_row) return;
    widen_rows(a.h16, (int64_t)a.h_rows, (int)a.h_row, a.dev, stream);
    if (check(hipGetLastError(), "kernel launch")) a.elided = false;
}
const uint16_t* it_hip::act_half_if_valid(const float* host, size_t rows, size_t row) {
    auto it = acts.find(host);
    if (it == acts.end() || !it->second.h_valid || !it->second.dev_current || it->second.h_rows != rows || it->second.h_row != row) return nullptr;
    return it->second.h16;
}

bool it_hip::add_in(const float* x, uint64_t x_len, const it_add_normed& a, uint64_t n_in, AddNormed* out) {
    if (!a.y || !a.norm_w || !a.x_new || a.x_new == x || a.x_new == a.y) {
        fail("add_normed: null argument, or a sum in place");
        return false;
    }
    out->eps = a.eps;
    out->mult = a.mult;
    return (out->w = const_in(a.norm_w, n_in)) && (out->y = act_in(a.y, x_len)) && (out->x_new = act_out(a.x_new, x_len));
}

#define REQUIRE(cond, msg) \
    do {                   \
        if (!(cond)) {     \
            be->fail(msg); \
            return;        \
        }                  \
    } while (0)

extern "C" {

int it_hip_is_f32(const it_hip* be) { return be->f32 ? 1 : 0; }

void it_hip_zero_slab(it_hip* be, const void* host) {
    auto it = be->slabs.find(host);
    if (it == be->slabs.end()) return;
    if (it->second.dev) {
        be->need_eager("a state slab is zeroed");
        fill_zero(it->second.dev, (int64_t)it->second.bytes, be->stream);
        it->second.dev_owned = true;
    } else {
        it->second.dev_owned = false;
    }
}

void it_hip_norm_matmuls(it_hip* be, const float* x, uint64_t x_len, const float* norm_w, uint64_t n_in, float eps,
                         const it_group_mat* mats, uint64_t n_mats) {
    it_hip_add_norm_matmuls(be, x, x_len, nullptr, norm_w, n_in, eps, mats, n_mats);
}

void it_hip_add_norm_matmuls(it_hip* be, const float* x, uint64_t x_len, const it_add_normed* add, const float* norm_w, uint64_t n_in, float eps,
                             const it_group_mat* mats, uint64_t n_mats) {
    if (add && (!be->fuse_enabled || !norm_w)) {   // a launch of its own
        it_hip_add_normed(be, x, x_len, add, n_in);
        x = add->x_new;
        add = nullptr;
    }
    REQUIRE(x && mats && n_mats >= 1 && n_mats <= GROUP_MAX, "norm_matmuls: null argument or too many matrices");
    REQUIRE(n_in > 0 && x_len % n_in == 0, "norm_matmuls: x.len() must be rows of n_in");
    const uint64_t n = x_len / n_in;
    if (n == 0) return;
    REQUIRE(n <= 65535, "norm_matmuls: more than 65535 tokens in one call");
    GroupP p{};
    WView views[GROUP_MAX], ups[GROUP_MAX];
    uint64_t bytes = x_len * 4;
    bool one_fmt = true;
    for (uint64_t i = 0; i < n_mats; i++) {
        const it_group_mat& m = mats[i];
        REQUIRE(m.w.n_in == n_in && float_type(m.w.ty), "norm_matmuls: a matrix of another row length, or a quantized one");
        REQUIRE(m.act == IT_ACT_SILU || m.act == IT_ACT_RELU, "norm_matmuls: unknown activation");
        REQUIRE(!m.up.data || (m.up.n_in == n_in && m.up.n_out == m.w.n_out && m.up.ty == m.w.ty), "norm_matmuls: gate and up differ in shape or type");
        if (m.slab) {
            REQUIRE(m.head_dim > 0 && m.w.n_out % m.head_dim == 0 && m.head_stride >= m.head_dim, "norm_matmuls: rows do not divide into the slab's heads");
            const uint64_t row = m.w.n_out / m.head_dim * m.head_stride;
            REQUIRE((m.slab_row + n) * row <= m.slab_len && m.slab_row + n < (1ull << 31), "norm_matmuls: writes past the end of the slab");
        } else {
            REQUIRE(m.out && m.out_len == n * m.w.n_out, "norm_matmuls: out.len() must be n * n_out");
        }
        if (!be->weights_view(&m.w, "norm_matmuls", &views[i])) return;
        if (m.up.data && !be->weights_view(&m.up, "norm_matmuls(up)", &ups[i])) return;
        one_fmt = one_fmt && views[i].fmt == views[0].fmt;
        bytes += m.w.len + (m.up.data ? m.up.len : 0) + n * m.w.n_out * 4;
    }
    const float* dw = nullptr;
    if (norm_w && !(dw = be->const_in(norm_w, n_in))) return;
    float* dx = be->act_in(x, x_len);
    if (!dx) return;
    const bool fused = be->fuse_enabled && one_fmt;
    p.x = dx;
    if (add && !be->add_in(x, x_len, *add, n_in, &p.add)) return;
    p.norm_w = dw;
    p.eps = eps;
    p.n_in = (int)n_in;
    p.n_tok = (int)n;
    p.n_mats = (int)n_mats;
    p.fmt = views[0].fmt;
    const bool one = fused && group_gemv_takes(p);
    const bool rows = fused && !one && n <= FEW;
    const bool gemm = fused && n > FEW && !be->f32 && p.fmt == W_BF16;
    const bool plain = !one && !rows && !gemm;
    // what the products read when the norm is a launch of its own, and where a product waits for its own scatter
    float *h32 = nullptr, *ta = nullptr, *tb = nullptr;
    uint16_t* h16 = nullptr;
    if (gemm) {
        if (!(h16 = (uint16_t*)be->tmp_for(T_HALF0, n * pad8((int)n_in) * 2))) return;
    } else if (!one && dw) {
        if (!(h32 = (float*)be->tmp_for(T_NORM, x_len * 4))) return;
    }
    if (plain) {
        uint64_t most = 0;
        for (uint64_t i = 0; i < n_mats; i++) most = std::max<uint64_t>(most, mats[i].w.n_out);
        if (!(ta = (float*)be->tmp_for(T_A, n * most * 4)) || !(tb = (float*)be->tmp_for(T_B, n * most * 4))) return;
    }
    for (uint64_t i = 0; i < n_mats; i++) {
        const it_group_mat& m = mats[i];
        GroupMat& g = p.m[i];
        g.w = (const uint8_t*)views[i].q;
        g.up = m.up.data ? (const uint8_t*)ups[i].q : nullptr;
        g.n_out = (int)m.w.n_out;
        g.act = (int)m.act;
        g.scale = m.scale;
        if (m.slab) {
            g.o.slab = be->slab_in(m.slab, m.slab_len * (be->f32 ? 4 : 2), false);
            if (!g.o.slab) return;
            g.o.slab_f32 = be->f32;
            g.o.head_dim = (int)m.head_dim;
            g.o.head_stride = (int)m.head_stride;
            g.o.row_stride = (int64_t)(m.w.n_out / m.head_dim * m.head_stride);
            g.o.row = (int)m.slab_row;
        } else if (gemm && g.up) {   // the product that follows reads bf16 rows
            if (!(g.o.half = be->act_half_out(m.out, n, m.w.n_out))) return;
        } else if (!(g.o.f32 = be->act_out(m.out, m.out_len))) {
            return;
        }
    }
    // (position slots last: nothing below leaves the recorded pass)
    uint64_t sig = sig_of(OP_GROUP, dx, dw, eps, p.n_in, p.n_tok, p.n_mats, p.fmt, h32, h16, ta, tb, p.add.y, p.add.w, p.add.x_new, p.add.eps, p.add.mult);
    for (uint64_t i = 0; i < n_mats; i++) {
        GroupMat& g = p.m[i];
        if (g.o.slab) {
            g.o.row_dyn = be->dyn_slot(g.o.row);
            if (g.o.row_dyn) g.o.row = 0;
        }
        sig = sig_of(sig, g.w, g.up, g.n_out, g.act, g.scale, g.o.f32, g.o.half, g.o.slab, g.o.head_dim, g.o.head_stride, g.o.row_dyn);
    }
    it_hip::OpRec rec;
    rec.id = OP_GROUP;
    be->submit(it_hip::FAM_GROUP, bytes, sig, rec, [=](hipStream_t s) {
        if (one) {
            if (!group_gemv(p, s)) be->fail("norm_matmuls: the one-token kernel could not be launched");
            return;
        }
        GroupP q = p;
        if (gemm) {
            if (p.add.y) add_norm_rows(p.x, p.add, p.norm_w, p.eps, p.n_tok, p.n_in, nullptr, h16, s);
            else norm_rows(p.x, p.norm_w, 1, p.eps, p.n_tok, p.n_in, nullptr, h16, s);
            group_gemm_bf16(q, h16, s);
            return;
        }
        if (p.norm_w) {
            if (p.add.y) add_norm_rows(p.x, p.add, p.norm_w, p.eps, p.n_tok, p.n_in, h32, nullptr, s);
            else norm_rows(p.x, p.norm_w, 1, p.eps, p.n_tok, p.n_in, h32, nullptr, s);
            q.x = h32;
        }
        if (rows) {
            group_rows(q, s);
            return;
        }
        for (int i = 0; i < q.n_mats; i++) {
            const GroupMat& m = q.m[i];
            matmul(WView{m.w, nullptr, views[i].fmt, q.n_in, m.n_out}, q.x, nullptr, nullptr, q.n_tok, ta, 1.0f, 0, s);
            if (m.up) {
                matmul(WView{m.up, nullptr, ups[i].fmt, q.n_in, m.n_out}, q.x, nullptr, nullptr, q.n_tok, tb, 1.0f, 0, s);
                act_mul(ta, tb, (int64_t)q.n_tok * m.n_out, m.act, s);
            }
            group_scatter(m, ta, q.n_tok, s);
        }
    });
}

void it_hip_add_normed(it_hip* be, const float* x, uint64_t x_len, const it_add_normed* add, uint64_t n_in) {
    REQUIRE(x && add && n_in > 0 && x_len % n_in == 0, "add_normed: x.len() must be rows of n_in");
    const uint64_t n = x_len / n_in;
    if (n == 0) return;
    REQUIRE(n < (1ull << 31) && n_in < (1ull << 28), "add_normed: sizes out of range");
    const float* dx = be->act_in(x, x_len);
    AddNormed a{};
    if (!dx || !be->add_in(x, x_len, *add, n_in, &a)) return;
    const int nd = (int)n_in;
    it_hip::OpRec rec;
    rec.id = OP_ADD_NORMED;
    be->submit(it_hip::FAM_NORM, x_len * 12, sig_of(OP_ADD_NORMED, dx, a.y, a.w, a.x_new, a.eps, a.mult, n, nd), rec,
               [=](hipStream_t s) { add_norm_rows(dx, a, nullptr, 0.0f, (int64_t)n, nd, nullptr, nullptr, s); });
}

static void residual_sum(it_hip* be, float* x, uint64_t x_len, const it_res_term* terms, uint64_t n_terms, bool set) {
    REQUIRE(x && terms && n_terms >= 1 && n_terms <= RES_MAX, "matmul_residual: null argument or too many terms");
    const uint64_t nd = terms[0].w.n_out;
    REQUIRE(nd > 0 && x_len % nd == 0, "matmul_residual: x.len() must be rows of n_out");
    const uint64_t n = x_len / nd;
    if (n == 0) return;
    REQUIRE(n <= 65535, "matmul_residual: more than 65535 tokens in one call");
    ResP p{};
    WView views[RES_MAX];
    uint64_t bytes = x_len * 8;
    bool one_fmt = true;
    for (uint64_t i = 0; i < n_terms; i++) {
        const it_res_term& t = terms[i];
        REQUIRE(t.in && t.w.n_out == nd && float_type(t.w.ty), "matmul_residual: a matrix of another row count, or a quantized one");
        REQUIRE(t.in_len == n * t.w.n_in, "matmul_residual: in.len() must be n * n_in");
        REQUIRE(!t.norm_w || (t.norm_groups > 0 && t.w.n_in % t.norm_groups == 0), "matmul_residual: the norm's groups do not divide the row");
        REQUIRE(!t.gate || (t.norm_w && t.gate_len == t.in_len), "matmul_residual: a gate without a norm, or of another size");
        if (!be->weights_view(&t.w, "matmul_residual", &views[i])) return;
        one_fmt = one_fmt && views[i].fmt == views[0].fmt;
        bytes += t.w.len + t.in_len * 4;
        ResTerm& q = p.t[i];
        q.w = (const uint8_t*)views[i].q;
        q.n_in = (int)t.w.n_in;
        q.norm_groups = (int)t.norm_groups;
        q.norm_period = (int)(t.norm_w && t.norm_shared ? t.w.n_in / t.norm_groups : t.w.n_in);
        q.eps = t.eps;
        if (t.scale && !(q.scale = be->const_in(t.scale, nd))) return;
        if (t.norm_w && !(q.norm_w = be->const_in(t.norm_w, (uint64_t)q.norm_period))) return;
    }
    p.n_out = (int)nd;
    p.n_tok = (int)n;
    p.n_terms = (int)n_terms;
    p.set = set;
    p.fmt = views[0].fmt;
    const bool fused = be->fuse_enabled && one_fmt;
    const bool one = fused && res_gemv_takes(p);
    const bool rows = fused && !one && n <= FEW;
    const bool gemm = fused && n > FEW && !be->f32 && p.fmt == W_BF16;
    struct In {
        const uint16_t* ready = nullptr;   // bf16 rows the producer wrote
        uint16_t* h16 = nullptr;
        float* h32 = nullptr;
    } in[RES_MAX];
    float *ta = nullptr, *tb = nullptr;
    if (!one && !gemm && !rows) {
        if (!(ta = (float*)be->tmp_for(T_A, x_len * 4)) || !(tb = (float*)be->tmp_for(T_B, x_len * 4))) return;
    }
    size_t h32_at = 0, h32_need = 0;
    for (uint64_t i = 0; i < n_terms; i++) h32_need += terms[i].norm_w && !one && !gemm ? terms[i].in_len : 0;
    float* h32 = nullptr;
    if (h32_need && !(h32 = (float*)be->tmp_for(T_NORM, h32_need * 4))) return;
    for (uint64_t i = 0; i < n_terms; i++) {
        const it_res_term& t = terms[i];
        if (gemm) {
            if (!t.norm_w) in[i].ready = be->act_half_if_valid(t.in, n, t.w.n_in);
            if (in[i].ready) continue;
            if (!(in[i].h16 = (uint16_t*)be->tmp_for(T_HALF0 + (int)i, n * pad8((int)t.w.n_in) * 2))) return;
        } else if (t.norm_w && !one) {
            in[i].h32 = h32 + h32_at;
            h32_at += t.in_len;
        }
        float* d = be->act_in(t.in, t.in_len);
        if (!d) return;
        p.t[i].in = d;
        if (t.gate && !(p.t[i].gate = be->act_in(t.gate, t.gate_len))) return;
    }
    if (!(p.x = set ? be->act_out(x, x_len) : be->act_inout(x, x_len))) return;
    uint64_t sig = sig_of(OP_RESIDUAL, p.set, p.x, p.n_out, p.n_tok, p.n_terms, p.fmt, ta, tb);
    for (uint64_t i = 0; i < n_terms; i++)
        sig = sig_of(sig, p.t[i].w, p.t[i].in, p.t[i].scale, p.t[i].norm_w, p.t[i].n_in, p.t[i].norm_groups, p.t[i].norm_period, p.t[i].gate, p.t[i].eps, in[i].ready, in[i].h16, in[i].h32);
    it_hip::OpRec rec;
    rec.id = OP_RESIDUAL;
    // the norm as a launch of its own
    auto normed = [](const ResP& p, int i, float* h32, uint16_t* h16, hipStream_t s) {
        const ResTerm& t = p.t[i];
        if (t.norm_w && (t.gate || t.norm_period != t.n_in))
            norm_gate_rows(t.in, t.norm_w, t.norm_period, t.gate, t.norm_groups, t.eps, p.n_tok, t.n_in, h32, h16, s);
        else
            norm_rows(t.in, t.norm_w, t.norm_w ? t.norm_groups : 1, t.eps, p.n_tok, t.n_in, h32, h16, s);
    };
    be->submit(it_hip::FAM_RESIDUAL, bytes, sig, rec, [=](hipStream_t s) {
        if (one) {
            if (!res_gemv(p, s)) be->fail("matmul_residual: the one-token kernel could not be launched");
            return;
        }
        if (gemm) {
            const uint16_t* h[RES_MAX] = {};
            for (int i = 0; i < p.n_terms; i++) {
                h[i] = in[i].ready ? in[i].ready : in[i].h16;
                if (!in[i].ready) normed(p, i, nullptr, in[i].h16, s);
            }
            res_gemm_bf16(p, h, s);
            return;
        }
        ResP q = p;
        for (int i = 0; i < p.n_terms; i++)
            if (in[i].h32) {
                normed(p, i, in[i].h32, nullptr, s);
                q.t[i].in = in[i].h32;
            }
        if (rows) {
            res_rows(q, s);
            return;
        }
        float* to[RES_MAX] = {ta, tb};
        for (int i = 0; i < q.n_terms; i++)
            matmul(WView{q.t[i].w, nullptr, views[i].fmt, q.t[i].n_in, q.n_out}, q.t[i].in, nullptr, nullptr, q.n_tok, to[i], 1.0f, 0, s);
        scaled_residual(q.x, ta, q.t[0].scale, q.n_terms > 1 ? tb : nullptr, q.t[1].scale, q.set, q.n_tok, q.n_out, s);
    });
}
void it_hip_matmul_residual(it_hip* be, float* x, uint64_t x_len, const it_res_term* terms, uint64_t n_terms) {
    residual_sum(be, x, x_len, terms, n_terms, false);
}
void it_hip_matmul_sum(it_hip* be, float* out, uint64_t out_len, const it_res_term* terms, uint64_t n_terms) {
    residual_sum(be, out, out_len, terms, n_terms, true);
}

void it_hip_attend_bias(it_hip* be, const it_attn_bias* a, float* out, uint64_t out_len) {
    REQUIRE(a && a->q && a->k && a->v, "attend_bias: null argument");
    REQUIRE(a->k_dim > 0 && a->v_dim > 0 && a->n_head > 0 && a->n_head_kv > 0 && a->n_head % a->n_head_kv == 0,
            "attend_bias: n_head must be a positive multiple of n_head_kv");
    REQUIRE(a->k_dim <= 4096 && a->v_dim <= 4096, "attend_bias: heads of at most 4096 elements");
    REQUIRE(a->k_stride >= a->k_dim && a->v_stride >= a->v_dim, "attend_bias: head strides smaller than the heads");
    const uint64_t per = a->n_head * a->k_dim;
    REQUIRE(a->q_len % per == 0, "attend_bias: q.len() must be rows of n_head * k_dim");
    const uint64_t n_q = a->q_len / per;
    if (n_q == 0) return;
    REQUIRE(out_len == n_q * a->n_head * a->v_dim, "attend_bias: out.len() must be rows of n_head * v_dim");
    const uint64_t krow = a->n_head_kv * a->k_stride, vrow = a->n_head_kv * a->v_stride;
    REQUIRE(a->n_pos >= n_q && a->n_pos * krow <= a->k_len && a->n_pos * vrow <= a->v_len, "attend_bias: n_pos outside the slabs or smaller than the batch");
    REQUIRE(a->n_pos < (1ull << 24) && n_q * a->n_head < (1ull << 31), "attend_bias: sizes out of range");   // (distances are exact in f32)
    REQUIRE(a->temp_coef == 0.0f || a->temp_every > 0, "attend_bias: temp_every must be positive");
    const uint64_t esz = be->f32 ? 4 : 2;
    BiasAttnP p{};
    p.q = be->act_in(a->q, a->q_len);
    p.k = be->slab_in(a->k, a->k_len * esz, false);
    p.v = be->slab_in(a->v, a->v_len * esz, false);
    if (a->slopes && !(p.slopes = be->const_in(a->slopes, a->n_head))) return;
    if (a->sinks && !(p.sinks = be->const_in(a->sinks, a->n_head))) return;
    if (!p.q || !p.k || !p.v) return;
    p.kv_f32 = be->f32;
    p.n_q = (int)n_q;
    p.n_pos = (int)a->n_pos;
    p.k_dim = (int)a->k_dim; p.v_dim = (int)a->v_dim; p.k_stride = (int)a->k_stride; p.v_stride = (int)a->v_stride;
    p.n_head = (int)a->n_head; p.n_head_kv = (int)a->n_head_kv;
    p.scale = a->scale;
    p.sink = a->sink ? 1 : 0;
    p.window = a->window < (1ull << 24) ? (int)a->window : 0;   // (contexts are shorter)
    p.temp_coef = a->temp_coef;
    p.temp_every = a->temp_every ? (int)std::min<uint32_t>(a->temp_every, INT_MAX) : 1;
    const bool mfma = be->fuse_enabled && attend_bias_mfma_takes(p);
    const bool batch = mfma && n_q > FEW;
    int n_split = 0;
    float* scratch = nullptr;
    if (mfma && !batch) {
        // a graphed pass keeps one launch shape while the context grows: the splits are sized for the whole slab, here too, so
        // that the scratch does not grow in the middle of a capture
        n_split = attend_bias_splits((int)std::min<uint64_t>(a->k_len / krow, INT_MAX), (int)n_q);
        if (!(scratch = be->scratch_f32(attend_bias_scratch_floats(p, n_split)))) return;
    } else if (batch) {
        BiasAttnP one = p;
        one.n_q = 1;
        if (!be->scratch_f32(attend_bias_scratch_floats(one, attend_bias_splits((int)std::min<uint64_t>(a->k_len / krow, INT_MAX), 1)))) return;
    }
    float* d32 = nullptr;
    uint16_t* d16 = nullptr;
    if (batch) d16 = be->act_half_out(out, n_q, a->n_head * a->v_dim);   // the projection that follows reads bf16 rows
    else d32 = be->act_out(out, out_len);
    if (!d32 && !d16) return;
    if (n_q == 1) {
        p.n_pos_dyn = be->dyn_slot(p.n_pos);
        if (p.n_pos_dyn) p.n_pos = 0;
    }
    const uint64_t bytes = a->n_pos * (krow + vrow) * esz + (a->q_len + out_len) * 4;
    it_hip::OpRec rec;
    rec.id = OP_ATTEND_BIAS;
    be->submit(it_hip::FAM_ATTEND, bytes,
               sig_of(OP_ATTEND_BIAS, p.q, p.k, p.v, p.kv_f32, p.n_q, n_q == 1 ? 0 : p.n_pos, p.k_dim, p.v_dim, p.k_stride, p.v_stride, p.n_head,
                      p.n_head_kv, p.scale, p.slopes, p.sink, p.sinks, p.window, p.temp_coef, p.temp_every, p.n_pos_dyn, n_split, scratch, d32, d16),
               rec, [=](hipStream_t s) {
                   bool ok = true;
                   if (batch) ok = attend_bias_batch(p, d32, d16, s);
                   else if (mfma) ok = attend_bias_split(p, n_split, scratch, d32, s);
                   else attend_bias_plain(p, d32, s);
                   if (!ok) be->fail("attend_bias: the matrix-core kernels could not be launched");
               });
}

void it_hip_mamba2(it_hip* be, const it_mamba2* m, const float* u, uint64_t u_len, float* conv_ring, uint64_t ring_len, float* state,
                   uint64_t state_len, float* out, uint64_t out_len) {
    REQUIRE(m && u && conv_ring && state && out && m->conv_w && m->conv_b && m->dt_bias && m->a_log && m->d, "mamba2: null argument");
    REQUIRE(m->heads > 0 && m->vdim > 0 && m->n > 0 && m->groups > 0 && m->taps > 0 && m->heads % m->groups == 0,
            "mamba2: heads must be a positive multiple of groups");
    const uint64_t inner = m->heads * m->vdim, ch = inner + 2 * m->groups * m->n, ud = inner + ch + m->heads;
    REQUIRE(u_len % ud == 0 && ud < (1ull << 28), "mamba2: u.len() must be rows of z, x, B, C and dt");
    const uint64_t n = u_len / ud;
    if (n == 0) return;
    REQUIRE(n <= 65535 && m->pos + n < (1ull << 31), "mamba2: sizes out of range");
    REQUIRE(ring_len == m->taps * ch && state_len == inner * m->n && out_len == n * inner, "mamba2: ring, state or out of another size");
    SsdP p{};
    p.heads = (int)m->heads; p.vdim = (int)m->vdim; p.n = (int)m->n; p.groups = (int)m->groups; p.taps = (int)m->taps;
    p.n_tok = (int)n;
    p.pos = (int)m->pos;
    REQUIRE(ssd_takes(p), "mamba2: a state of at most 512 columns and at most 16 taps");
    p.accurate = be->f32 || !be->fuse_enabled;
    p.u = be->act_in(u, u_len);
    p.conv_w = be->const_in(m->conv_w, ch * m->taps);
    p.conv_b = be->const_in(m->conv_b, ch);
    p.dt_bias = be->const_in(m->dt_bias, m->heads);
    p.a_log = be->const_in(m->a_log, m->heads);
    p.d = be->const_in(m->d, m->heads);
    p.conv_ring = (float*)be->slab_in(conv_ring, ring_len * 4, true);
    p.state = (float*)be->slab_in(state, state_len * 4, true);
    if (!p.u || !p.conv_w || !p.conv_b || !p.dt_bias || !p.a_log || !p.d || !p.conv_ring || !p.state) return;
    const bool step = n == 1;
    const bool chunks = !step && be->fuse_enabled && !be->f32 && ssd_chunk_takes(p);
    float* work = nullptr;
    if (!step && !(p.xbc = (float*)be->tmp_for(T_XBC, n * ch * 4))) return;
    if (chunks && !(work = be->gdn_work_for(ssd_chunk_work_floats(p)))) return;
    if (!(p.out = be->act_out(out, out_len))) return;
    if (step) {
        p.pos_dyn = be->dyn_slot(p.pos);
        if (p.pos_dyn) p.pos = 0;
    }
    it_hip::OpRec rec;
    rec.id = OP_MAMBA2;
    be->submit(it_hip::FAM_SSD, (u_len + out_len + 2 * state_len) * 4 + (step ? 0 : 2 * n * ch * 4),
               sig_of(OP_MAMBA2, p.u, p.conv_w, p.conv_ring, p.state, p.xbc, p.out, work, p.heads, p.vdim, p.n, p.groups, p.taps, p.n_tok, p.pos_dyn,
                      step ? 0 : p.pos),
               rec, [=](hipStream_t s) {
                   if (step) {
                       ssd_step(p, s);
                       return;
                   }
                   ssd_conv(p, s);
                   ssd_conv_keep(p, s);
                   if (chunks) ssd_chunk(p, work, s);
                   else ssd_scan(p, s);
               });
}

void it_hip_gla(it_hip* be, const it_gla* g, float* state, uint64_t state_len, float* out, uint64_t out_len) {
    REQUIRE(g && g->q && g->k && g->v && g->low && g->a2_b && state && out, "gla: null argument");
    const uint64_t nk = g->heads * g->dim, nv = g->heads * g->vdim, rank = g->a2.n_in;
    REQUIRE(g->heads > 0 && g->dim > 0 && g->vdim > 0 && g->heads < (1u << 20) && g->dim <= 4096 && g->vdim < (1u << 20) && nv < (1ull << 28), "gla: sizes out of range");
    REQUIRE(g->q_len % nk == 0, "gla: q.len() must be rows of heads * dim");
    const uint64_t n = g->q_len / nk;
    if (n == 0) return;
    REQUIRE(n <= 65535, "gla: more than 65535 tokens in one call");
    REQUIRE(g->a2.n_out == nk && float_type(g->a2.ty), "gla: the decay's matrix has another row count, or is quantized");
    REQUIRE(g->k_len == n * nk && g->v_len == n * nv && g->low_len == n * rank, "gla: k, v or low of another size");
    REQUIRE(state_len == nv * g->dim && out_len == n * nv, "gla: state or out of another size");
    REQUIRE(g->tau > 0.0f, "gla: tau must be positive");
    GlaP p{};
    p.heads = (int)g->heads; p.dim = (int)g->dim; p.vdim = (int)g->vdim; p.rank = (int)rank; p.n_tok = (int)n;
    REQUIRE(gla_takes(p), "gla: heads of at most 512 key channels and a decay of rank at most 1024");
    WView a2;
    if (!be->weights_view(&g->a2, "gla", &a2)) return;
    p.a2 = (const uint8_t*)a2.q;
    p.a2_fmt = a2.fmt;
    p.inv_tau = 1.0f / g->tau;
    p.a2_b = be->const_in(g->a2_b, nk);
    p.q = be->act_in(g->q, g->q_len);
    p.k = be->act_in(g->k, g->k_len);
    p.v = be->act_in(g->v, g->v_len);
    p.low = be->act_in(g->low, g->low_len);
    p.state = (float*)be->slab_in(state, state_len * 4, true);
    if (!p.a2_b || !p.q || !p.k || !p.v || !p.low || !p.state) return;
    const bool step = n == 1;
    const bool chunks = !step && be->fuse_enabled && !be->f32 && gla_chunk_takes(p);
    float* work = nullptr;
    if (!step && !(p.decay = (float*)be->tmp_for(T_XBC, n * nk * 4))) return;
    if (chunks && !(work = be->gdn_work_for(gla_chunk_work_floats(p)))) return;
    if (!(p.out = be->act_out(out, out_len))) return;
    it_hip::OpRec rec;
    rec.id = OP_GLA;
    be->submit(it_hip::FAM_GLA, (g->q_len + g->k_len + g->v_len + g->low_len + out_len + 2 * state_len) * 4 + g->a2.len,
               sig_of(OP_GLA, p.q, p.k, p.v, p.low, p.a2, p.a2_fmt, p.a2_b, p.inv_tau, p.state, p.decay, p.out, work, p.heads, p.dim, p.vdim, p.rank, p.n_tok),
               rec, [=](hipStream_t s) {
                   if (step) {
                       gla_step(p, s);
                       return;
                   }
                   gla_decay(p, chunks, s);
                   if (!chunks) gla_scan(p, s);
                   else if (!gla_chunk(p, work, s)) be->fail("gla: the chunked kernels could not be launched");
               });
}

void it_hip_attend_latent(it_hip* be, const it_attn_latent* a, float* out, uint64_t out_len) {
    REQUIRE(a && a->q && a->slab && out && (!a->kv || a->kv_norm), "attend_latent: null argument");
    REQUIRE(a->heads > 0 && a->dim > 0 && a->vdim > 0 && a->rank > 0 && a->heads < (1u << 16) && a->dim <= 4096 && a->rot_dim <= 4096 && a->vdim <= 4096 &&
                a->rank <= 4096,
            "attend_latent: sizes out of range");
    REQUIRE(a->rope.dims % 2 == 0 && a->rope.dims <= a->rot_dim, "attend_latent: rotated dimensions must be even and inside the rotated part");
    REQUIRE(a->rope.dims == 0 || a->rope.base > 1.0, "attend_latent: the rotation's base must be above 1");
    REQUIRE(!(a->rope.factor > 0) || (a->rope.original > 0 && a->rope.fast > 0 && a->rope.slow > 0), "attend_latent: incomplete frequency scaling");
    const uint64_t per = a->heads * (a->dim + a->rot_dim), kd = a->rank + a->rot_dim, row = (kd + 7) / 8 * 8;
    REQUIRE(a->q_len % per == 0, "attend_latent: q.len() must be rows of heads * (dim + rot_dim)");
    const uint64_t n = a->q_len / per;
    if (n == 0) return;
    REQUIRE(n <= 65535 && n * a->heads < (1ull << 31), "attend_latent: more than 65535 tokens in one call");
    REQUIRE(!a->kv || a->kv_len == n * kd, "attend_latent: kv.len() must be rows of rank + rot_dim");
    REQUIRE(!a->gate || a->gate_len == n * a->heads, "attend_latent: gate.len() must be rows of heads");
    REQUIRE(out_len == n * a->heads * a->vdim, "attend_latent: out.len() must be rows of heads * vdim");
    const uint64_t cap = a->slab_len / row;
    REQUIRE(a->pos + n <= cap && a->pos + n < (1ull << 24), "attend_latent: positions past the end of the slab");
    REQUIRE(a->uk.n_in == a->rank && a->uk.n_out == a->heads * a->dim && float_type(a->uk.ty) && a->uv.n_in == a->rank &&
                a->uv.n_out == a->heads * a->vdim && float_type(a->uv.ty),
            "attend_latent: uk or uv of another shape, or quantized");
    WView uk, uv;
    if (!be->weights_view(&a->uk, "attend_latent(uk)", &uk) || !be->weights_view(&a->uv, "attend_latent(uv)", &uv)) return;
    LatentP p{};
    p.eps = a->eps;
    p.uk = (const uint8_t*)uk.q; p.uk_fmt = uk.fmt;
    p.uv = (const uint8_t*)uv.q; p.uv_fmt = uv.fmt;
    p.heads = (int)a->heads; p.dim = (int)a->dim; p.rot = (int)a->rot_dim; p.n_rot = (int)a->rope.dims; p.rank = (int)a->rank; p.vdim = (int)a->vdim;
    p.n_tok = (int)n;
    p.pos = (int)a->pos;
    p.row_stride = (int)row;
    p.slab_f32 = be->f32;
    if (a->rope.dims && !(p.table = be->rope_table(a->rope, cap))) return;
    if (a->kv && !(p.kv_norm = be->const_in(a->kv_norm, a->rank))) return;
    if (a->kv && !(p.kv = be->act_in(a->kv, a->kv_len))) return;
    if (a->gate && !(p.gate = be->act_in(a->gate, a->gate_len))) return;
    float* dq = be->act_in(a->q, a->q_len);
    p.q = dq;
    p.slab = be->slab_in(a->slab, a->slab_len * (be->f32 ? 4 : 2), false);
    if (!dq || !p.slab) return;
    BiasAttnP at{};   // the latent's space: one key row for all heads, its first elements the value
    at.k = at.v = p.slab;
    at.kv_f32 = be->f32;
    at.n_q = (int)n;
    at.n_pos = (int)(a->pos + n);
    at.k_dim = (int)kd; at.v_dim = (int)a->rank; at.k_stride = at.v_stride = (int)row;
    at.n_head = (int)a->heads; at.n_head_kv = 1;
    at.scale = a->scale;
    at.sink = a->sinks ? 1 : 0;
    if (a->sinks && !(at.sinks = be->const_in(a->sinks, a->heads))) return;
    at.window = a->window < (1ull << 24) ? (int)a->window : 0;   // (contexts are shorter)
    at.temp_every = 1;

    // keys and values of every head: rows `first` .. of the cache
    const uint64_t first = at.window && a->pos + 1 > a->window ? a->pos + 1 - a->window : 0, n_keys = a->pos + n - first;
    BiasAttnP full = at;
    full.k_dim = (int)(a->dim + a->rot_dim); full.v_dim = (int)a->vdim;
    full.k_stride = pad8(full.k_dim); full.v_stride = pad8(full.v_dim);
    full.n_head_kv = (int)a->heads;
    full.n_pos = (int)n_keys;
    full.gate = p.gate;
    full.q = dq;
    full.k = full.v = nullptr;   // (aligned; set below)
    const bool batch = be->fuse_enabled && n > FEW && uk.fmt == W_BF16 && uv.fmt == W_BF16 && attend_bias_mfma_takes(full);
    const bool split = !batch && be->fuse_enabled && attend_shared_takes(at);
    uint16_t *c16 = nullptr, *d16 = nullptr, *q16 = nullptr;
    int kp = 0;
    float *qa = nullptr, *ol = nullptr, *scratch = nullptr, *d32 = nullptr;
    int n_split = 0;
    if (batch) {
        c16 = (uint16_t*)be->tmp_for(T_LATENT, n_keys * pad8(p.rank) * 2);
        full.k = be->tmp_for(T_KEYS, n_keys * a->heads * full.k_stride * 2);
        full.v = be->tmp_for(T_VALUES, n_keys * a->heads * full.v_stride * 2);
        if (!c16 || !full.k || !full.v || !(d16 = be->act_half_out(out, n, a->heads * a->vdim)) || !(dq = be->act_inout(a->q, a->q_len))) return;
    } else {
        if (!(ol = (float*)be->tmp_for(T_OL, (split ? std::min<uint64_t>(n, FEW) : n) * a->heads * a->rank * 4))) return;
        if (split) {
            kp = attend_shared_q_row(at);
            if (!(q16 = (uint16_t*)be->tmp_for(T_QA, n * a->heads * (uint64_t)kp * 2))) return;
   // (splits for the whole slab: a recorded pass keeps one launch shape)
            n_split = attend_shared_splits(at, (int)std::min<uint64_t>(cap, INT_MAX));
            BiasAttnP few = at;
            few.n_q = (int)std::min<uint64_t>(n, FEW);
            if (!(scratch = be->scratch_f32(attend_shared_scratch_floats(few, n_split)))) return;
        } else if (!(qa = (float*)be->tmp_for(T_QA, n * a->heads * kd * 4))) {
            return;
        }
        if (!(d32 = be->act_out(out, out_len))) return;
    }
    if (n == 1) {
        p.n_pos_dyn = at.n_pos_dyn = be->dyn_slot(at.n_pos);
        if (p.n_pos_dyn) p.pos = at.n_pos = 0;
    }
    const uint64_t esz = be->f32 ? 4 : 2, seen = n_keys * row * esz + a->uk.len + a->uv.len;
    it_hip::OpRec rec;
    rec.id = OP_ATTEND_LATENT;
    be->submit(it_hip::FAM_ATTEND, seen + (a->q_len + out_len) * 4,
               sig_of(OP_ATTEND_LATENT, p.q, p.kv, p.kv_norm, p.eps, p.table, p.uk, p.uk_fmt, p.uv, p.uv_fmt, p.slab, p.slab_f32, p.gate, p.heads, p.dim,
                      p.rot, p.n_rot, p.rank, p.vdim, p.n_tok, n == 1 ? 0 : p.pos, p.n_pos_dyn, at.scale, at.sinks, at.window, c16, full.k, full.v, qa, q16, ol,
                      scratch, n_split, d32, d16),
               rec, [=](hipStream_t s) {
                   bool ok = true;
                   if (batch) {
                       latent_rows(p, dq, s);
                       latent_keys(p, (int)first, (int)n_keys, c16, (uint16_t*)full.k, full.k_stride, s);
                       GroupP g{};
                       g.n_in = p.rank;
                       g.n_tok = (int)n_keys;
                       g.n_mats = 2;
                       g.fmt = W_BF16;
                       auto to = [&](const uint8_t* w, int dim, int stride, const void* slab) {
                           GroupMat m{};
                           m.w = w;
                           m.n_out = p.heads * dim;
                           m.scale = 1.0f;
                           m.o.slab = (void*)slab;
                           m.o.head_dim = dim;
                           m.o.head_stride = stride;
                           m.o.row_stride = (int64_t)p.heads * stride;
                           return m;
                       };
                       g.m[0] = to(p.uk, p.dim, full.k_stride, full.k);
                       g.m[1] = to(p.uv, p.vdim, full.v_stride, full.v);
                       group_gemm_bf16(g, c16, s);
                       ok = attend_bias_batch(full, nullptr, d16, s);
                   } else if (split) {
                       latent_prep(p, nullptr, q16, kp, at.scale, s);
                       const int few = (int)FEW;
                       for (int t0 = 0; t0 < p.n_tok && ok; t0 += few) {
                           LatentP pt = p;
                           BiasAttnP bt = at;
                           bt.n_q = pt.n_tok = std::min(few, p.n_tok - t0);
                           if (!bt.n_pos_dyn) bt.n_pos = p.pos + t0 + bt.n_q;
                           if (p.gate) pt.gate = p.gate + (size_t)t0 * p.heads;
                           ok = attend_shared_split(bt, q16 + (size_t)t0 * p.heads * kp, n_split, scratch, ol, s);
                           if (ok) latent_value(pt, ol, d32 + (size_t)t0 * p.heads * p.vdim, s);
                       }
                   } else {
                       latent_prep(p, qa, nullptr, 0, 1.0f, s);
                       BiasAttnP bt = at;
                       bt.q = qa;
                       attend_bias_plain(bt, ol, s);
                       latent_value(p, ol, d32, s);
                   }
                   if (!ok) be->fail("attend_latent: the matrix-core kernels could not be launched");
               });
}

void it_hip_add_rows(it_hip* be, float* x, uint64_t x_len, const float* rows, const float* vec, uint64_t vec_len) {
    REQUIRE(x && (rows || vec) && vec_len > 0 && x_len % vec_len == 0, "add_rows: x.len() must be rows of vec.len()");
    if (x_len == 0) return;
    const float* dr = nullptr;
    const float* dv = nullptr;
    if (rows && !(dr = be->act_in(rows, x_len))) return;
    if (vec && !(dv = be->const_in(vec, vec_len))) return;
    float* dx = be->act_inout(x, x_len);
    if (!dx) return;
    const int64_t n = (int64_t)(x_len / vec_len);
    const int nd = (int)vec_len;
    it_hip::OpRec rec;
    rec.id = OP_ADD_ROWS;
    be->submit(it_hip::FAM_OTHER, x_len * (dr ? 12 : 8), sig_of(OP_ADD_ROWS, dx, dr, dv, n, nd), rec,
               [=](hipStream_t s) { add_rows(dx, dr, dv, n, nd, s); });
}

void it_hip_gather_rows(it_hip* be, const float* src, uint64_t src_len, uint64_t width, const uint32_t* idx, uint64_t n_rows, float* out,
                        uint64_t out_len) {
    REQUIRE(src && idx && out && width > 0 && src_len % width == 0 && out_len == n_rows * width, "gather_rows: buffers are not whole rows");
    if (n_rows == 0) return;
    REQUIRE(n_rows < (1ull << 31), "gather_rows: too many rows");
    for (uint64_t i = 0; i < n_rows; i++) REQUIRE(idx[i] < src_len / width, "gather_rows: row out of range");
    be->need_eager("a row list is uploaded");
    float* ds = be->act_in(src, src_len);
    int32_t* di = (int32_t*)be->tmp_for(T_A, n_rows * 4);
    float* dout = be->act_out(out, out_len);
    if (!ds || !di || !dout) return;
    if (!be->check(hipMemcpyAsync(di, idx, n_rows * 4, hipMemcpyHostToDevice, be->stream), "upload row list") ||
        !be->check(hipStreamSynchronize(be->stream), "upload row list"))
        return;
    const int nr = (int)n_rows, nd = (int)width;
    it_hip::OpRec rec;
    rec.id = OP_GATHER_ROWS;
    be->submit(it_hip::FAM_OTHER, out_len * 8, sig_of(OP_GATHER_ROWS, ds, di, nr, nd, dout), rec,
               [=](hipStream_t s) { gather_rows(ds, di, nr, nd, dout, s); });
}

}  // extern "C"
#undef REQUIRE
