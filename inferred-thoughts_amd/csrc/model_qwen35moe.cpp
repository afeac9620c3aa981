// The qwen35moe design over the HIP backend: hybrid Gated DeltaNet / attention layers with a routed FFN, driving the
// same C ABI a binding of the reference's `trait Ops` would use.
//
// Mirrors (file:line under /root/reference):
//   Config::from_gguf            src/model/qwen35.rs:333-489
//   tensor views + shape checks  src/model/mod.rs:261-418
//   Qwen35::load, kv_slot, embed src/model/qwen35.rs:755-873
//   Scratch::fit                 src/model/qwen35.rs:673-729 (stable host addresses)
//   forward/attention/gated_delta src/model/qwen35.rs:956-1328
//   moe_batch                    src/model/qwen35.rs:1587-1700
#include <algorithm>
#include <cmath>
#include <cstdio>
#include <cstring>
#include <memory>
#include <string>
#include <vector>

#include "gguf.h"
#include "host_formats.h"
#include "model.h"

namespace {

struct Dims {
    uint64_t n_layer = 0, n_embd = 0, n_vocab = 0, n_head = 0, n_head_kv = 0, head_dim = 0, n_rot = 0;
    uint64_t n_expert = 0, n_used = 0, expert_ff = 0, shared_ff = 0;
    uint64_t d_conv = 0, d_inner = 0, d_state = 0, dt_rank = 0, n_group = 0, interval = 4, nextn = 0;
    float theta = 0, eps = 0;
    uint64_t layers() const { return n_layer - nextn; }
    bool recurrent(uint64_t il) const { return il < layers() && (il + 1) % interval != 0; }
    uint64_t q_gate() const { return head_dim * 2 * n_head; }
    uint64_t q_dim() const { return head_dim * n_head; }
    uint64_t kv_dim() const { return head_dim * n_head_kv; }
    uint64_t dk() const { return d_state; }
    uint64_t dv() const { return d_inner / dt_rank; }
    uint64_t key_dim() const { return dk() * n_group; }
    uint64_t value_dim() const { return dv() * dt_rank; }
    uint64_t conv_dim() const { return 2 * key_dim() + value_dim(); }
    uint64_t ssm_len() const { return dk() * dv() * dt_rank; }
    uint64_t conv_len() const { return (d_conv - 1) * conv_dim(); }
};

struct Block {
    bool recurrent = false;
    std::vector<float> attn_norm, ffn_norm;
    it_weights wq{}, wk{}, wv{}, wo{};
    std::vector<float> q_norm, k_norm;
    it_weights wqkv{}, wgate{}, w_alpha{}, w_beta{}, w_out{};
    std::vector<float> conv1d, ssm_a, dt_bias, ssm_norm;
    it_weights router{}, sh_gate{}, sh_up{}, sh_down{}, sh_gate_inp{};
    it_experts gate{}, up{}, down{};
    float sh_scale[3] = {1, 1, 1};
    bool sh_has[3] = {false, false, false};
};

struct Qwen35 : it_model {
    itg::File file;
    Dims d;
    it_weights tok_embd{}, output{};
    bool has_output_scale = false;
    float output_scale = 1.0f;
    std::vector<float> output_norm;
    std::vector<Block> blocks;
    std::vector<uint64_t> kv_slot;
    uint64_t n_kv_layer = 0;
    const itg::Tensor* need(const std::string& name) {
        const itg::Tensor* t = file.tensor(name);
        if (!t) fail("missing tensor " + name);
        return t;
    }
    static bool shape_is(const std::vector<uint64_t>& got, std::vector<uint64_t> want) {
        auto g = got;
        while (!g.empty() && g.back() == 1) g.pop_back();
        while (!want.empty() && want.back() == 1) want.pop_back();
        return g == want;
    }
    bool shape_err(const std::string& name, const std::vector<uint64_t>& want, const std::vector<uint64_t>& got) {
        std::string m = "tensor " + name + ": expected {";
        for (auto v : want) m += std::to_string(v) + ",";
        m += "} got {";
        for (auto v : got) m += std::to_string(v) + ",";
        return fail(m + "}");
    }
    bool matrix(const std::string& name, uint64_t n_in, uint64_t n_out, it_weights* w) {
        const itg::Tensor* t = need(name);
        if (!t) return false;
        if (!shape_is(t->dims, {n_in, n_out})) return shape_err(name, {n_in, n_out}, t->dims);
        *w = it_weights{file.bytes(*t), itg::type_bytes(t->ty, t->n_elems()), t->ty, 0, n_in, n_out};
        return true;
    }
    bool row_matrix(const std::string& name, uint64_t n_in, it_weights* w) {
        const itg::Tensor* t = need(name);
        if (!t) return false;
        if (!shape_is(t->dims, {n_in})) return shape_err(name, {n_in}, t->dims);
        *w = it_weights{file.bytes(*t), itg::type_bytes(t->ty, n_in), t->ty, 0, n_in, 1};
        return true;
    }
    bool vec(const std::string& name, std::vector<uint64_t> shape, std::vector<float>* out) {
        const itg::Tensor* t = need(name);
        if (!t) return false;
        if (!shape_is(t->dims, shape)) return shape_err(name, shape, t->dims);
        out->resize(t->n_elems());
        if (!ith::dequantize(t->ty, file.bytes(*t), t->n_elems(), out->data()))
            return fail("tensor " + name + ": unsupported type for a vector");
        return true;
    }
    bool experts(const std::string& name, uint64_t n_in, uint64_t n_out, uint64_t n_expert, it_experts* e) {
        const itg::Tensor* t = need(name);
        if (!t) return false;
        if (!shape_is(t->dims, {n_in, n_out, n_expert})) return shape_err(name, {n_in, n_out, n_expert}, t->dims);
        *e = it_experts{file.bytes(*t), itg::type_bytes(t->ty, t->n_elems()), t->ty, 0, n_in, n_out, n_expert, nullptr, 0};
        std::string sn = name;
        size_t at = sn.rfind(".weight");
        if (at != std::string::npos) sn.replace(at, 7, ".scale");
        if (const itg::Tensor* s = file.tensor(sn)) {
            if (!shape_is(s->dims, {n_expert})) return shape_err(sn, {n_expert}, s->dims);
            if (s->ty != IT_F32) return fail("tensor " + sn + ": per-expert scales must be F32");
            e->scale = file.bytes(*s);
            e->scale_len = n_expert * 4;
        }
        return true;
    }
    bool scalar_opt(const std::string& name, bool* has, float* v) {
        *has = false;
        if (!file.tensor(name)) return true;
        std::vector<float> one;
        if (!vec(name, {1}, &one)) return false;
        *has = true;
        *v = one[0];
        return true;
    }

    bool load(const std::string& path_in) {
        path = path_in;
        if (!file.open(path, &err)) return false;
        std::string arch;
        if (!file.get_string("general.architecture", &arch)) return fail("missing general.architecture");
        if (arch != "qwen35moe") return fail("unsupported architecture '" + arch + "' (this backend's loop covers qwen35moe)");
        auto u = [&](const char* k, uint64_t* out) {
            if (file.get_uint(arch + "." + k, out)) return true;
            return fail(std::string("missing key ") + arch + "." + k);
        };
        auto f = [&](const char* k, float* out) {
            if (file.get_float(arch + "." + k, out)) return true;
            return fail(std::string("missing key ") + arch + "." + k);
        };
        uint64_t v_len = 0;
        if (!u("block_count", &d.n_layer) || !u("embedding_length", &d.n_embd) || !u("expert_count", &d.n_expert) ||
            !u("expert_used_count", &d.n_used) || !u("expert_feed_forward_length", &d.expert_ff) ||
            !u("expert_shared_feed_forward_length", &d.shared_ff) || !u("attention.head_count", &d.n_head) ||
            !u("attention.head_count_kv", &d.n_head_kv) || !u("attention.key_length", &d.head_dim) ||
            !u("attention.value_length", &v_len) || !f("rope.freq_base", &d.theta) ||
            !f("attention.layer_norm_rms_epsilon", &d.eps) || !u("rope.dimension_count", &d.n_rot) ||
            !u("ssm.conv_kernel", &d.d_conv) || !u("ssm.inner_size", &d.d_inner) || !u("ssm.state_size", &d.d_state) ||
            !u("ssm.time_step_rank", &d.dt_rank) || !u("ssm.group_count", &d.n_group))
            return false;
        file.get_uint(arch + ".full_attention_interval", &d.interval);
        file.get_uint(arch + ".nextn_predict_layers", &d.nextn);
        const std::vector<int32_t>* sec = file.get_i32_array(arch + ".rope.dimension_sections");
        if (!sec || sec->size() != 4) return fail("rope.dimension_sections: expected an i32 array of 4 entries");
        if (d.n_head_kv == 0 || d.n_head % d.n_head_kv) return fail("GQA grouping: query heads do not divide into kv heads");
        if (v_len != d.head_dim) return fail("head dimension: key_length != value_length");
        if (d.n_used == 0 || d.n_used > d.n_expert) return fail("expert_used_count out of range");
        if (d.dt_rank == 0 || d.d_inner % d.dt_rank) return fail("ssm.inner_size does not divide into value heads");
        if (d.n_group == 0 || d.dt_rank % d.n_group) return fail("delta rule grouping: value heads do not divide into key heads");
        if (d.dv() != d.dk()) return fail("delta rule head dimensions: the recurrence assumes a square state");
        if (d.interval == 0) return fail("full_attention_interval must be non-zero");
        if (d.n_rot > d.head_dim) return fail("rope.dimension_count exceeds head_dim");
        if (d.nextn >= d.n_layer) return fail("nextn_predict_layers exceeds block_count");

        const itg::Tensor* te = need("token_embd.weight");
        if (!te) return false;
        if (te->dims.size() < 2) return fail("token_embd.weight: expected 2 dimensions");
        d.n_vocab = te->dims[1];
        if (!matrix("token_embd.weight", d.n_embd, d.n_vocab, &tok_embd)) return false;
        if (file.tensor("output.weight")) {
            if (!matrix("output.weight", d.n_embd, d.n_vocab, &output)) return false;
            if (!scalar_opt("output.scale", &has_output_scale, &output_scale)) return false;
        } else {
            output = tok_embd;
        }
        blocks.resize(d.layers());
        uint64_t slot = 0;
        for (uint64_t i = 0; i < d.layers(); i++) {
            Block& b = blocks[i];
            auto nm = [&](const char* s) { return "blk." + std::to_string(i) + "." + s; };
            b.recurrent = d.recurrent(i);
            kv_slot.push_back(slot);
            bool ok;
            if (b.recurrent) {
                ok = matrix(nm("attn_qkv.weight"), d.n_embd, d.conv_dim(), &b.wqkv) &&
                     matrix(nm("attn_gate.weight"), d.n_embd, d.value_dim(), &b.wgate) &&
                     vec(nm("ssm_conv1d.weight"), {d.d_conv, d.conv_dim()}, &b.conv1d) &&
                     matrix(nm("ssm_beta.weight"), d.n_embd, d.dt_rank, &b.w_beta) &&
                     matrix(nm("ssm_alpha.weight"), d.n_embd, d.dt_rank, &b.w_alpha) &&
                     vec(nm("ssm_a"), {d.dt_rank}, &b.ssm_a) && vec(nm("ssm_dt.bias"), {d.dt_rank}, &b.dt_bias) &&
                     vec(nm("ssm_norm.weight"), {d.dv()}, &b.ssm_norm) &&
                     matrix(nm("ssm_out.weight"), d.value_dim(), d.n_embd, &b.w_out);
            } else {
                slot++;
                ok = matrix(nm("attn_q.weight"), d.n_embd, d.q_gate(), &b.wq) &&
                     matrix(nm("attn_k.weight"), d.n_embd, d.kv_dim(), &b.wk) &&
                     matrix(nm("attn_v.weight"), d.n_embd, d.kv_dim(), &b.wv) &&
                     matrix(nm("attn_output.weight"), d.q_dim(), d.n_embd, &b.wo) &&
                     vec(nm("attn_q_norm.weight"), {d.head_dim}, &b.q_norm) &&
                     vec(nm("attn_k_norm.weight"), {d.head_dim}, &b.k_norm);
            }
            ok = ok && matrix(nm("ffn_gate_inp.weight"), d.n_embd, d.n_expert, &b.router) &&
                 experts(nm("ffn_gate_exps.weight"), d.n_embd, d.expert_ff, d.n_expert, &b.gate) &&
                 experts(nm("ffn_up_exps.weight"), d.n_embd, d.expert_ff, d.n_expert, &b.up) &&
                 experts(nm("ffn_down_exps.weight"), d.expert_ff, d.n_embd, d.n_expert, &b.down) &&
                 matrix(nm("ffn_gate_shexp.weight"), d.n_embd, d.shared_ff, &b.sh_gate) &&
                 matrix(nm("ffn_up_shexp.weight"), d.n_embd, d.shared_ff, &b.sh_up) &&
                 matrix(nm("ffn_down_shexp.weight"), d.shared_ff, d.n_embd, &b.sh_down) &&
                 row_matrix(nm("ffn_gate_inp_shexp.weight"), d.n_embd, &b.sh_gate_inp) &&
                 scalar_opt(nm("ffn_gate_shexp.scale"), &b.sh_has[0], &b.sh_scale[0]) &&
                 scalar_opt(nm("ffn_up_shexp.scale"), &b.sh_has[1], &b.sh_scale[1]) &&
                 scalar_opt(nm("ffn_down_shexp.scale"), &b.sh_has[2], &b.sh_scale[2]) &&
                 vec(nm("attn_norm.weight"), {d.n_embd}, &b.attn_norm) &&
                 vec(nm("post_attention_norm.weight"), {d.n_embd}, &b.ffn_norm);
            if (!ok) return false;
            // refused at load, not per call (src/ops/mod.rs:29-55)
            char msg[256];
            if (it_hip_check_expert_types(b.gate.ty, b.up.ty, b.down.ty, msg, sizeof msg)) return fail(msg);
        }
        n_kv_layer = slot;
        return vec("output_norm.weight", {d.n_embd}, &output_norm);
    }

    void dims(uint64_t out[10]) const override {
        uint64_t v[10] = {d.layers(), d.n_embd, d.n_vocab, d.n_head, d.n_head_kv, d.head_dim, d.n_expert, d.n_used,
                          d.expert_ff, d.n_rot};
        memcpy(out, v, sizeof v);
    }
    uint64_t vocab() const override { return d.n_vocab; }
    uint64_t width() const override { return d.n_embd; }
    const it_weights& embedding() const override { return tok_embd; }
    uint64_t dense_bytes(const Block& b) const {
        const uint64_t mixer = b.recurrent ? b.wqkv.len + b.wgate.len + b.w_alpha.len + b.w_beta.len + b.w_out.len
                                           : b.wq.len + b.wk.len + b.wv.len + b.wo.len;
        return mixer + b.router.len + b.sh_gate.len + b.sh_up.len + b.sh_down.len + b.sh_gate_inp.len;
    }
    uint64_t decode_weight_bytes() const override {
        uint64_t bytes = output.len;
        for (const Block& b : blocks) bytes += dense_bytes(b) + (b.gate.len + b.up.len + b.down.len) / d.n_expert * d.n_used;
        return bytes;
    }
    void token_macs(uint64_t out[3]) const override {
        uint64_t dense = 0, glu = 0, down = 0;
        auto macs = [](const it_weights& w) { return w.n_in * w.n_out; };
        for (const Block& b : blocks) {
            if (b.recurrent) dense += macs(b.wqkv) + macs(b.wgate) + macs(b.w_alpha) + macs(b.w_beta) + macs(b.w_out);
            else dense += macs(b.wq) + macs(b.wk) + macs(b.wv) + macs(b.wo);
            dense += macs(b.router) + macs(b.sh_gate) + macs(b.sh_up) + macs(b.sh_down) + macs(b.sh_gate_inp);
            glu += d.n_used * (b.gate.n_in * b.gate.n_out + b.up.n_in * b.up.n_out);
            down += d.n_used * b.down.n_in * b.down.n_out;
        }
        out[0] = dense;
        out[1] = glu;
        out[2] = down;
    }
    it_engine* new_engine(it_hip* be, uint64_t n_ctx, uint64_t max_batch) override;
};

constexpr uint64_t PREFETCH_K = 10;  // src/model/qwen4exp.rs:45: how many of the next router's picks a hint guesses
constexpr uint64_t MOE_CHUNK = 512;  // src/model/qwen35.rs:650: the reference's routed-FFN sub-batch; a larger engine batch raises it (new_engine)

struct Qwen35Engine : it_engine {
    Qwen35* m;
    uint64_t moe_chunk = MOE_CHUNK;  // tokens per routed-FFN sub-batch
    HostBuf x, normed, mixed, ffn_out, qg, q, g, k, v, attn, qkv, z, alpha, beta, convo, q_part, k_part, v_part,
        core, router, e_gate, e_up, e_out, e_in, g_all, u_all, o_all, shexp_logit, last, final_norm, picked;

    std::vector<HostBuf*> buffers() override {
        return {&x, &normed, &mixed, &ffn_out, &qg, &q, &g, &k, &v, &attn, &qkv, &z, &alpha, &beta, &convo, &q_part, &k_part, &v_part, &core,
                &router, &e_gate, &e_up, &e_out, &e_in, &g_all, &u_all, &o_all, &shexp_logit, &last, &final_norm, &picked};
    }
    uint64_t slab_len() const { return n_ctx * m->d.kv_dim(); }
    uint16_t* k_slab(uint64_t slot) { return (uint16_t*)cache.k_slab(slot); }
    uint16_t* v_slab(uint64_t slot) { return (uint16_t*)cache.v_slab(slot); }
    float* conv_of(uint64_t il) { return cache.conv_of(il); }
    float* ssm_of(uint64_t il) { return cache.ssm_of(il); }
    int forward(const uint32_t* tokens, uint64_t n, uint64_t start, bool want_logits, uint64_t ring_index) override;
    int forward_rows(const uint32_t* tokens, uint64_t n, uint64_t start, const uint32_t* rows, uint64_t n_rows, float* out) override;
    int layers(const uint32_t* tokens, uint64_t n, uint64_t start, uint64_t ring_index);
};

void fit(Qwen35Engine* e, uint64_t n) {
    const Dims& d = e->m->d;
    e->x.fit(n * d.n_embd, e->be); e->normed.fit(n * d.n_embd, e->be); e->mixed.fit(n * d.n_embd, e->be); e->ffn_out.fit(n * d.n_embd, e->be);
    e->qg.fit(n * d.q_gate(), e->be); e->q.fit(n * d.q_dim(), e->be); e->g.fit(n * d.q_dim(), e->be);
    e->k.fit(n * d.kv_dim(), e->be); e->v.fit(n * d.kv_dim(), e->be); e->attn.fit(n * d.q_dim(), e->be);
    e->qkv.fit(n * d.conv_dim(), e->be); e->z.fit(n * d.value_dim(), e->be); e->alpha.fit(n * d.dt_rank, e->be); e->beta.fit(n * d.dt_rank, e->be);
    e->convo.fit(n * d.conv_dim(), e->be); e->q_part.fit(n * d.key_dim(), e->be); e->k_part.fit(n * d.key_dim(), e->be);
    e->v_part.fit(n * d.value_dim(), e->be); e->core.fit(n * d.value_dim(), e->be);
    uint64_t nt = n < e->moe_chunk ? n : e->moe_chunk;
    uint64_t ff = d.expert_ff > d.shared_ff ? d.expert_ff : d.shared_ff;
    e->router.fit(nt * d.n_expert, e->be); e->e_gate.fit(nt * ff, e->be); e->e_up.fit(nt * ff, e->be); e->e_out.fit(nt * d.n_embd, e->be);
    e->e_in.fit(nt * d.n_embd, e->be); e->g_all.fit(nt * d.n_used * d.expert_ff, e->be); e->u_all.fit(nt * d.n_used * d.expert_ff, e->be);
    e->o_all.fit(nt * d.n_used * d.n_embd, e->be); e->shexp_logit.fit(nt, e->be);
    e->last.fit(d.n_embd, e->be); e->final_norm.fit(d.n_embd, e->be); e->logits.fit(d.n_vocab, e->be);
}

// next_router: the router of the next layer, for a single-token pass.  The reference's qwen35 loop does not hint; its
// qwen4exp loop does (src/model/qwen4exp.rs:1885-1896), between the routing decision and the expert products, and the
// hint changes no value.  The backend acts on it only while part of the expert pool is cold.
void moe_batch(Qwen35Engine* e, const Block& b, uint64_t at, uint64_t n, uint64_t total, const it_weights* next_router) {
    const Dims& d = e->m->d;
    it_hip* be = e->be;
    uint64_t nd = d.n_embd;
    it_hip_gather_chunks(be, e->normed.p(), total * nd, n * nd, n * nd, at, e->e_in.p(), n * nd);
    const float* x = e->e_in.p();
    it_hip_matmul_pair(be, &b.router, &b.sh_gate_inp, x, n * nd, e->router.p(), n * d.n_expert, e->shexp_logit.p(), n);
    it_hip_softmax(be, e->router.p(), n * d.n_expert, d.n_expert);
    it_route route;
    it_hip_route(be, e->router.p(), n * d.n_expert, d.n_expert, d.n_used, &route);
    if (total == 1 && next_router) it_hip_prefetch_hint(be, next_router, x, nd, PREFETCH_K);
    uint64_t pairs = n * d.n_used, ff = pairs * d.expert_ff;
    it_hip_moe_glu(be, &b.gate, &b.up, &route, x, n * nd, e->g_all.p(), ff, e->u_all.p(), ff);
    it_hip_matmul_experts(be, &b.down, &route, e->g_all.p(), ff, e->o_all.p(), pairs * nd);
    uint64_t sff = n * d.shared_ff;
    it_hip_matmul(be, &b.sh_gate, x, n * nd, e->e_gate.p(), sff);
    it_hip_matmul(be, &b.sh_up, x, n * nd, e->e_up.p(), sff);
    if (b.sh_has[1]) it_hip_scale(be, e->e_up.p(), sff, b.sh_scale[1]);
    if (b.sh_has[0]) it_hip_scale(be, e->e_gate.p(), sff, b.sh_scale[0]);
    it_hip_silu_mul(be, e->e_gate.p(), sff, e->e_up.p(), sff);
    it_hip_matmul(be, &b.sh_down, e->e_gate.p(), sff, e->e_out.p(), n * nd);
    if (b.sh_has[2]) it_hip_scale(be, e->e_out.p(), n * nd, b.sh_scale[2]);
    it_hip_moe_finish(be, e->ffn_out.p(), total * nd, at, nd, e->o_all.p(), pairs * nd, &route, e->e_out.p(),
                      n * nd, e->shexp_logit.p(), n, 0);
}

void attention(Qwen35Engine* e, const Block& b, uint64_t il, uint64_t start, uint64_t n) {
    const Dims& d = e->m->d;
    it_hip* be = e->be;
    uint64_t hd = d.head_dim, kd = d.kv_dim(), nd = d.n_embd, qd = d.q_dim();
    it_hip_matmul(be, &b.wq, e->normed.p(), n * nd, e->qg.p(), n * d.q_gate());
    e->tr("Qcur_full", il, e->qg, n * d.q_gate());
    it_hip_gather_chunks(be, e->qg.p(), n * d.q_gate(), hd, 2 * hd, 0, e->q.p(), n * qd);
    it_hip_gather_chunks(be, e->qg.p(), n * d.q_gate(), hd, 2 * hd, hd, e->g.p(), n * qd);
    it_hip_matmul(be, &b.wk, e->normed.p(), n * nd, e->k.p(), n * kd);
    it_hip_matmul(be, &b.wv, e->normed.p(), n * nd, e->v.p(), n * kd);
    it_hip_rms_norm_heads(be, e->q.p(), n * qd, b.q_norm.data(), hd, hd, d.eps);
    e->tr("Qcur_normed", il, e->q, n * qd);
    it_hip_rms_norm_heads(be, e->k.p(), n * kd, b.k_norm.data(), hd, hd, d.eps);
    e->tr("Kcur_normed", il, e->k, n * kd);
    it_hip_rope_neox(be, e->q.p(), n * qd, start, hd, d.n_rot, d.n_head, d.theta);
    e->tr("Qcur", il, e->q, n * qd);
    it_hip_rope_neox(be, e->k.p(), n * kd, start, hd, d.n_rot, d.n_head_kv, d.theta);
    e->tr("Kcur", il, e->k, n * kd);
    uint64_t slot = e->m->kv_slot[il];
    it_hip_kv_write(be, e->k_slab(slot), e->slab_len(), start * kd, e->k.p(), n * kd);
    it_hip_kv_write(be, e->v_slab(slot), e->slab_len(), start * kd, e->v.p(), n * kd);
    it_attn a{e->q.p(), n * qd, e->k_slab(slot), e->v_slab(slot), e->slab_len(), kd, start + n, hd, d.n_head,
              d.n_head_kv, 1.0f / std::sqrt((float)hd)};
    it_hip_attend(be, &a, e->attn.p(), n * qd);
    e->tr("attn_pregate", il, e->attn, n * qd);
    it_hip_sigmoid_mul(be, e->attn.p(), n * qd, e->g.p(), n * qd);
    e->tr("attn_gated", il, e->attn, n * qd);
    it_hip_matmul(be, &b.wo, e->attn.p(), n * qd, e->mixed.p(), n * nd);
    e->tr("attn_output", il, e->mixed, n * nd);
}

void gated_delta(Qwen35Engine* e, const Block& b, uint64_t il, uint64_t n) {
    const Dims& d = e->m->d;
    it_hip* be = e->be;
    uint64_t kdim = d.key_dim(), vdim = d.value_dim(), cdim = d.conv_dim(), nd = d.n_embd, nv = d.dt_rank;
    it_hip_matmul(be, &b.wqkv, e->normed.p(), n * nd, e->qkv.p(), n * cdim);
    e->tr("linear_attn_qkv_mixed", il, e->qkv, n * cdim);
    it_hip_matmul(be, &b.wgate, e->normed.p(), n * nd, e->z.p(), n * vdim);
    e->tr("z", il, e->z, n * vdim);
    it_hip_matmul_pair(be, &b.w_alpha, &b.w_beta, e->normed.p(), n * nd, e->alpha.p(), n * nv, e->beta.p(), n * nv);
    it_hip_ssm_conv(be, e->conv_of(il), d.conv_len(), e->qkv.p(), n * cdim, b.conv1d.data(), b.conv1d.size(), d.d_conv,
                    e->convo.p(), n * cdim);
    e->tr("conv_output_silu", il, e->convo, n * cdim);
    it_hip_gather_chunks(be, e->convo.p(), n * cdim, kdim, cdim, 0, e->q_part.p(), n * kdim);
    it_hip_gather_chunks(be, e->convo.p(), n * cdim, kdim, cdim, kdim, e->k_part.p(), n * kdim);
    it_hip_gather_chunks(be, e->convo.p(), n * cdim, vdim, cdim, 2 * kdim, e->v_part.p(), n * vdim);
    it_hip_l2_norm_heads(be, e->q_part.p(), n * kdim, d.dk(), d.eps);
    it_hip_l2_norm_heads(be, e->k_part.p(), n * kdim, d.dk(), d.eps);
    e->tr("q_conv_predelta", il, e->q_part, n * kdim);
    e->tr("k_conv_predelta", il, e->k_part, n * kdim);
    it_delta dl{e->q_part.p(), e->k_part.p(), e->v_part.p(), e->alpha.p(), e->beta.p(), b.ssm_a.data(),
                b.dt_bias.data(), n, d.dk(), d.dv(), d.n_group, nv};
    it_hip_delta_rule(be, &dl, e->ssm_of(il), d.ssm_len(), e->core.p(), n * vdim);
    e->tr("dnet_out", il, e->core, n * vdim);
    it_hip_rms_norm_heads(be, e->core.p(), n * vdim, b.ssm_norm.data(), d.dv(), d.dv(), d.eps);
    it_hip_silu_mul(be, e->z.p(), n * vdim, e->core.p(), n * vdim);
    e->tr("final_output", il, e->z, n * vdim);
    it_hip_matmul(be, &b.w_out, e->z.p(), n * vdim, e->mixed.p(), n * nd);
    e->tr("linear_attn_out", il, e->mixed, n * nd);
}

// Everything of a pass up to the last layer's residual; the pass stays open
int Qwen35Engine::layers(const uint32_t* tokens, uint64_t n, uint64_t start, uint64_t ring_index) {
    const Dims& d = m->d;
    if (int rc = check_pass(tokens, n, start)) return rc;
    uint64_t nd = d.n_embd;
    it_hip_begin_pass(be, n);
    fit(this, n);
    if (int rc = embed(tokens, n, x.p(), ring_index)) return rc;
    tr("inp_embd", 0, x, n * nd);
    for (uint64_t il = 0; il < d.layers(); il++) {
        const Block& b = m->blocks[il];
        it_hip_rms_norm(be, x.p(), n * nd, b.attn_norm.data(), nd, d.eps, normed.p(), n * nd);
        tr("attn_norm", il, normed, n * nd);
        if (b.recurrent) gated_delta(this, b, il, n);
        else attention(this, b, il, start, n);
        it_hip_add_assign(be, x.p(), n * nd, mixed.p(), n * nd);
        tr("attn_residual", il, x, n * nd);
        it_hip_rms_norm(be, x.p(), n * nd, b.ffn_norm.data(), nd, d.eps, normed.p(), n * nd);
        for (uint64_t t = 0; t < n;) {
            uint64_t take = moe_chunk < n - t ? moe_chunk : n - t;
            moe_batch(this, b, t * nd, take, n, il + 1 < d.layers() ? &m->blocks[il + 1].router : nullptr);
            t += take;
        }
        tr("ffn_moe_out", il, ffn_out, n * nd);
        it_hip_add_assign(be, x.p(), n * nd, ffn_out.p(), n * nd);
        tr("post_ffn", il, x, n * nd);
    }
    len = start + n;
    return 0;
}

int Qwen35Engine::forward(const uint32_t* tokens, uint64_t n, uint64_t start, bool want_logits, uint64_t ring_index) {
    const Dims& d = m->d;
    if (int rc = layers(tokens, n, start, ring_index)) return rc;
    const uint64_t nd = d.n_embd;
    it_hip_gather_chunks(be, x.p(), n * nd, nd, nd, (n - 1) * nd, last.p(), nd);
    it_hip_rms_norm(be, last.p(), nd, m->output_norm.data(), nd, d.eps, final_norm.p(), nd);
    tr("result_norm", 0, final_norm, nd);
    it_hip_matmul(be, &m->output, final_norm.p(), nd, logits.p(), d.n_vocab);
    if (m->has_output_scale) it_hip_scale(be, logits.p(), d.n_vocab, m->output_scale);
    it_hip_end_pass(be);
    if (want_logits) it_hip_host_needs(be, logits.p(), d.n_vocab);
    if (trace) tr("result_output", 0, logits, d.n_vocab);
    return end_pass_check(!tokens);
}

// One row at a time, as the last row of every other pass is formed: a row's logits do not depend on which others are asked for
int Qwen35Engine::forward_rows(const uint32_t* tokens, uint64_t n, uint64_t start, const uint32_t* rows, uint64_t n_rows, float* out) {
    const Dims& d = m->d;
    const uint64_t nd = d.n_embd, nv = d.n_vocab;
    if (int rc = layers(tokens, n, start, 0)) return rc;
    it_hip_end_pass(be);
    picked.fit(nv, be);
    for (uint64_t i = 0; i < n_rows; i++) {
        it_hip_gather_chunks(be, x.p(), n * nd, nd, nd, rows[i] * nd, last.p(), nd);
        it_hip_rms_norm(be, last.p(), nd, m->output_norm.data(), nd, d.eps, final_norm.p(), nd);
        it_hip_matmul(be, &m->output, final_norm.p(), nd, picked.p(), nv);
        if (m->has_output_scale) it_hip_scale(be, picked.p(), nv, m->output_scale);
        it_hip_host_needs(be, picked.p(), nv);
        memcpy(out + i * nv, picked.p(), nv * sizeof(float));
    }
    return end_pass_check(false);
}

it_engine* Qwen35::new_engine(it_hip* be, uint64_t n_ctx, uint64_t max_batch) {
    Qwen35Engine* e = new Qwen35Engine();
    e->m = this;
    // every expert's matrices are read once per routed-FFN sub-batch, so with memory to spare the sub-batch
    // follows the engine batch (the seam carries at most 65535 pairs per call)
    e->moe_chunk = std::max<uint64_t>(MOE_CHUNK, std::min<uint64_t>(max_batch, 65535 / std::max<uint64_t>(1, d.n_used)));
    for (uint64_t s = 0; s < n_kv_layer; s++) e->cache.add_kv(n_ctx * d.kv_dim(), n_ctx * d.kv_dim());
    for (uint64_t il = 0; il < d.layers(); il++) e->cache.add_state(d.conv_len(), d.ssm_len(), d.recurrent(il));
    e->cache.allocate(sizeof(uint16_t));
    // what the reference's CLI tells its device backend before the first pass (src/main.rs:545-560): the permanent
    // weights and the KV cache the expert slab must leave room for, and the size of the expert pool (one read
    // counter per expert matrix)
    uint64_t dense = output.len + tok_embd.len;
    for (const Block& b : blocks) dense += dense_bytes(b);
    // where the experts' bytes can be read from when they are not kept anywhere else (src/main.rs:559-560)
    it_hip_set_model_path(be, path.c_str());
    it_hip_set_map_base(be, (uint64_t)(uintptr_t)file.base());
    it_hip_reserve_for_weights(be, dense);
    it_hip_set_expert_pool(be, d.layers() * 3 * d.n_expert);
    return e;
}

}  // namespace

it_model* open_qwen35moe(const std::string& path, std::string* err) {
    auto m = std::make_unique<Qwen35>();
    if (!m->load(path)) {
        *err = m->err;
        return nullptr;
    }
    return m.release();
}
