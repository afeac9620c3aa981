// The Nubedra design: every sublayer between two norms (x <- x + m norm_b(sublayer(norm(x)))), mixers of two kinds (gated linear
// attention with a decay per key channel; latent attention with a sliding window, a sink, an output gate and scaled rotary
// positions, whose cache rows a later layer may share), feed-forwards with relu, and the embedding table as the output head.
//
// A model is a folder with config.json and model.safetensors; every size and constant comes from there.
#include <cmath>
#include <cstring>
#include <memory>

#include "model_folder.h"

namespace {

struct Gla {
    uint64_t heads = 0, dim = 0, vdim = 0, rank = 0;   // rank: of the decay's matrix, from its tensors
    float tau = 1;
    it_weights q{}, k{}, v{}, g{}, a1{}, a2{};
    std::vector<float> a2_b, norm;
};
struct Latent {
    uint64_t heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0, q_rank = 0, window = 0;
    int64_t kv_from = -1;   // the layer whose cache rows this one reads; -1: its own
    float scale = 0;
    it_rope rope{};
    it_weights dq{}, uq{}, dkv{}, uk{}, uv{}, g{};
    std::vector<float> dq_norm, dkv_norm, sink;
    uint64_t kv_row() const { return kv_rank + rot_dim; }
    uint64_t slab_row() const { return round8(kv_row()); }
};
struct Layer {
    bool latent = false, has_mlp = false;
    Gla r;
    Latent a;
    it_weights o{}, gate{}, up{}, down{};
    uint64_t ff = 0;
    std::vector<float> norm1, norm1b, norm2, norm2b;   // as factors: 1 + what is stored
    uint64_t slot = 0;   // of the cache's slabs (a sharing layer: the other's), or of its states
    uint64_t mixed() const { return latent ? a.heads * a.vdim : r.heads * r.vdim; }
};

bool same_rope(const it_rope& a, const it_rope& b) {
    return a.base == b.base && a.dims == b.dims && a.factor == b.factor && a.original == b.original && a.fast == b.fast && a.slow == b.slow;
}

struct Nubedra : FolderModel {
    float mult = 1, embed_scale = 1;
    std::vector<Layer> layers;
    std::vector<float> final_norm;
    uint64_t n_kv = 0, n_state = 0;

    bool rotation(const itj::Value* mx, const std::string& wm, Latent* a) {
        const itj::Value *rot = mx->get("rot"), *sc = rot ? rot->get("scaling") : nullptr;
        const std::string wr = wm + ".rot", ws = wr + ".scaling";
        if (!real(rot, wr.c_str(), "base", &a->rope.base) || !size(rot, wr.c_str(), "dims", &a->rope.dims)) return false;
        if (a->rope.dims % 2 || a->rope.dims > a->rot_dim || a->rope.base <= 1) return fail("config.json: " + wr + ": odd, or more dimensions than rot_dim, or a base of 1 or less");
        if (!sc || sc->is_null()) return true;
        if (!real(sc, ws.c_str(), "factor", &a->rope.factor) || !real(sc, ws.c_str(), "original", &a->rope.original) ||
            !real(sc, ws.c_str(), "fast", &a->rope.fast) || !real(sc, ws.c_str(), "slow", &a->rope.slow))
            return false;
        return (a->rope.factor > 0 && a->rope.original > 0 && a->rope.fast > 0 && a->rope.slow > 0) || fail("config.json: " + ws + ": values must be positive");
    }
    bool config(const itj::Value& c) {
        if (!size(&c, "", "vocab", &n_vocab) || !size(&c, "", "width", &nd) || !real(c.get("norm"), "norm", "eps", &eps) ||
            !real(&c, "", "residual_mult", &mult) || !real(c.get("embedding"), "embedding", "scale", &embed_scale))
            return false;
        const itj::Value* ls = c.get("layers");
        if (!ls || ls->kind != itj::Value::Array || ls->items.empty()) return fail("config.json: layers is missing or empty");
        layers.resize(ls->items.size());
        for (size_t i = 0; i < layers.size(); i++) {
            const itj::Value &e = ls->items[i], *ty = e.get("type"), *mx = e.get("mixer"), *mlp = e.get("mlp");
            const std::string where = "layers[" + std::to_string(i) + "]", wm = where + ".mixer";
            Layer& l = layers[i];
            if (!ty || ty->kind != itj::Value::String || !mx) return fail("config.json: " + where + " has no type or no mixer");
            if (ty->str == "gla") {
                Gla& r = l.r;
                if (!size(mx, wm.c_str(), "heads", &r.heads) || !size(mx, wm.c_str(), "dim", &r.dim) || !size(mx, wm.c_str(), "vdim", &r.vdim) ||
                    !real(mx, wm.c_str(), "tau", &r.tau))
                    return false;
                if (r.dim > 512 || r.tau <= 0) return fail("config.json: " + wm + ": more than 512 key channels a head, or a tau that is not positive");
                l.slot = n_state++;
            } else if (ty->str == "latent_attention") {
                Latent& a = l.a;
                l.latent = true;
                if (!size(mx, wm.c_str(), "heads", &a.heads) || !size(mx, wm.c_str(), "dim", &a.dim) || !size(mx, wm.c_str(), "rot_dim", &a.rot_dim) ||
                    !size(mx, wm.c_str(), "vdim", &a.vdim) || !size(mx, wm.c_str(), "kv_rank", &a.kv_rank) || !size(mx, wm.c_str(), "q_rank", &a.q_rank) ||
                    !real(mx, wm.c_str(), "scale", &a.scale) || !rotation(mx, wm, &a))
                    return false;
                const itj::Value *mask = mx->get("mask"), *from = mx->get("kv_from");
                if (mask && !mask->is_null() && !size(mask, (wm + ".mask").c_str(), "size", &a.window)) return false;
                if (from && !from->is_null()) {
                    uint64_t j = 0;
                    if (!size(mx, wm.c_str(), "kv_from", &j, 0)) return false;
                    const Layer* o = j < i ? &layers[j] : nullptr;
                    if (!o || !o->latent || o->a.kv_from >= 0) return fail("config.json: " + wm + ".kv_from does not name an earlier layer with a cache of its own");
                    if (o->a.kv_rank != a.kv_rank || o->a.rot_dim != a.rot_dim || !same_rope(o->a.rope, a.rope))
                        return fail("config.json: " + wm + ": the layer that kv_from names has another kv_rank, rot_dim or rotation");
                    a.kv_from = (int64_t)j;
                    l.slot = o->slot;
                } else {
                    l.slot = n_kv++;
                }
            } else {
                return fail("config.json: " + where + ": unknown mixer '" + ty->str + "'");
            }
            if (mlp && !mlp->is_null()) {
                const itj::Value* kind = mlp->get("kind");
                if (!kind || kind->str != "dense") return fail("config.json: " + where + ".mlp: unknown kind");
                l.has_mlp = true;
                if (!size(mlp, (where + ".mlp").c_str(), "ff", &l.ff)) return false;
            }
        }
        return true;
    }

    bool centred(const std::string& name, std::vector<float>* out) {   // stored around zero
        if (!vec(name, {nd}, out)) return false;
        for (float& v : *out) v += 1.0f;
        return true;
    }
    bool load(const std::string& dir) {
        itj::Value c;
        if (!read_config(dir, &c, &err) || !file.open(dir + "/model.safetensors", &err) || !config(c)) return false;
        if (!matrix("embed", n_vocab, nd, &embed_w) || !centred("final.norm", &final_norm)) return false;
        for (size_t i = 0; i < layers.size(); i++) {
            Layer& l = layers[i];
            auto nm = [&](const char* s) { return "l" + std::to_string(i) + "." + s; };
            if (!centred(nm("norm1"), &l.norm1) || !centred(nm("norm1b"), &l.norm1b) || !matrix(nm("mix.o"), nd, l.mixed(), &l.o)) return false;
            if (l.latent) {
                Latent& a = l.a;
                if (!matrix(nm("mix.dq"), a.q_rank, nd, &a.dq) || !vec(nm("mix.dq.norm"), {a.q_rank}, &a.dq_norm) ||
                    !matrix(nm("mix.uq"), a.heads * (a.dim + a.rot_dim), a.q_rank, &a.uq) || !matrix(nm("mix.uk"), a.heads * a.dim, a.kv_rank, &a.uk) ||
                    !matrix(nm("mix.uv"), a.heads * a.vdim, a.kv_rank, &a.uv) || !vec(nm("mix.sink"), {a.heads}, &a.sink) ||
                    !matrix(nm("mix.g"), a.heads, nd, &a.g))
                    return false;
                if (a.kv_from < 0 && (!matrix(nm("mix.dkv"), a.kv_row(), nd, &a.dkv) || !vec(nm("mix.dkv.norm"), {a.kv_rank}, &a.dkv_norm))) return false;
            } else {
                Gla& r = l.r;
                const its::Tensor* a1 = file.tensor(nm("mix.a1"));
                if (a1 && a1->shape.size() == 2) r.rank = a1->shape[0];
                if (!matrix(nm("mix.a1"), r.rank, nd, &r.a1) || !matrix(nm("mix.a2"), r.heads * r.dim, r.rank, &r.a2) ||
                    !vec(nm("mix.a2.b"), {r.heads * r.dim}, &r.a2_b) || !matrix(nm("mix.q"), r.heads * r.dim, nd, &r.q) ||
                    !matrix(nm("mix.k"), r.heads * r.dim, nd, &r.k) || !matrix(nm("mix.v"), r.heads * r.vdim, nd, &r.v) ||
                    !matrix(nm("mix.g"), r.heads * r.vdim, nd, &r.g) || !vec(nm("mix.norm"), {r.vdim}, &r.norm))
                    return false;
                if (r.rank < 1 || r.rank > 1024) return fail("tensor " + nm("mix.a1") + ": a decay of rank 0 or above 1024");
            }
            if (l.has_mlp && (!centred(nm("norm2"), &l.norm2) || !centred(nm("norm2b"), &l.norm2b) || !matrix(nm("mlp.gate"), l.ff, nd, &l.gate) ||
                              !matrix(nm("mlp.up"), l.ff, nd, &l.up) || !matrix(nm("mlp.down"), nd, l.ff, &l.down)))
                return false;
        }
        return true;
    }

    void dims(uint64_t out[10]) const override {   // of the first latent layer where layers may differ
        const Latent none, *a = &none;
        for (const Layer& l : layers)
            if (l.latent) {
                a = &l.a;
                break;
            }
        uint64_t v[10] = {layers.size(), nd, n_vocab, a->heads, a->heads ? 1ull : 0ull, a->dim + a->rot_dim, 0, 0, 0, a->rope.dims};
        memcpy(out, v, sizeof v);
    }
    float embedding_scale() const override { return embed_scale; }
    template <class F> uint64_t over_layers(F per_matrix) const {
        uint64_t n = 0;
        for (const Layer& l : layers) {
            for (const it_weights* w : {&l.o, &l.r.q, &l.r.k, &l.r.v, &l.r.g, &l.r.a1, &l.r.a2, &l.a.dq, &l.a.uq, &l.a.dkv, &l.a.uk, &l.a.uv, &l.a.g, &l.gate,
                                        &l.up, &l.down})
                if (w->data) n += per_matrix(*w);
        }
        return n;
    }
    uint64_t decode_weight_bytes() const override {
        return embed_w.len + over_layers([](const it_weights& w) { return w.len; });
    }
    void token_macs(uint64_t out[3]) const override {
        out[0] = over_layers([](const it_weights& w) { return w.n_in * w.n_out; });
        out[1] = out[2] = 0;
    }
    it_engine* new_engine(it_hip* be, uint64_t n_ctx, uint64_t max_batch) override;
};

struct NubedraEngine : FolderEngine {
    Nubedra* m;
    // the residual stream, in two buffers by turns: a sublayer's normed output is added on the way into the next one's products
    HostBuf xs[2], y, q, k, v, low, g, cq, kv, mixed, ff, shown;
    int cur = 0;
    const std::vector<float>* pending = nullptr;   // the norm of `y`, which is still to be added to xs[cur]
    std::vector<HostBuf*> buffers() override {
        return {&xs[0], &xs[1], &y, &q, &k, &v, &low, &g, &cq, &kv, &mixed, &ff, &shown, &last, &picked};
    }

    void fit(uint64_t n) {
        for (HostBuf* b : {&xs[0], &xs[1], &y}) b->fit(n * m->nd, be);
        for (const Layer& l : m->layers) {
            if (l.latent) {
                const Latent& a = l.a;
                q.fit(n * a.uq.n_out, be);
                cq.fit(n * a.q_rank, be);
                kv.fit(n * a.kv_row(), be);
                g.fit(n * a.heads, be);
            } else {
                const Gla& r = l.r;
                q.fit(n * r.heads * r.dim, be);
                k.fit(n * r.heads * r.dim, be);
                v.fit(n * r.heads * r.vdim, be);
                g.fit(n * r.heads * r.vdim, be);
                low.fit(n * r.rank, be);
            }
            mixed.fit(n * l.mixed(), be);
            if (l.has_mlp) ff.fit(n * l.ff, be);
        }
        logits.fit(m->n_vocab, be);
    }
    it_add_normed addition(HostBuf& to) { return it_add_normed{y.p(), pending->data(), to.p(), m->eps, m->mult}; }

    // the matrices that read norm(x), behind what the sublayer before them left to be added
    void products(const std::vector<float>& norm, uint64_t n, const it_group_mat* mats, uint64_t n_mats) {
        const uint64_t nd = m->nd;
        if (!pending) {
            it_hip_norm_matmuls(be, xs[cur].p(), n * nd, norm.data(), nd, m->eps, mats, n_mats);
            return;
        }
        const it_add_normed add = addition(xs[cur ^ 1]);
        it_hip_add_norm_matmuls(be, xs[cur].p(), n * nd, &add, norm.data(), nd, m->eps, mats, n_mats);
        cur ^= 1;
        pending = nullptr;
    }
    static it_group_mat to_rows(const it_weights& w, HostBuf& b, uint64_t n) {
        it_group_mat g{};
        g.w = w;
        g.out = b.p();
        g.out_len = n * w.n_out;
        g.scale = 1.0f;
        return g;
    }
    void sublayer_out(it_res_term t, uint64_t n, const std::vector<float>& norm) {
        it_hip_matmul_sum(be, y.p(), n * m->nd, &t, 1);
        pending = &norm;
    }

    void layer(const Layer& l, uint64_t start, uint64_t n) {
        it_res_term o{};
        o.w = l.o;
        o.in = mixed.p();
        o.in_len = n * l.mixed();
        if (l.latent) {
            const Latent& a = l.a;
            it_group_mat mats[3] = {to_rows(a.dq, cq, n), to_rows(a.g, g, n), {}};
            if (a.kv_from < 0) mats[2] = to_rows(a.dkv, kv, n);
            products(l.norm1, n, mats, a.kv_from < 0 ? 3 : 2);
            const it_group_mat up = to_rows(a.uq, q, n);
            it_hip_norm_matmuls(be, cq.p(), n * a.q_rank, a.dq_norm.data(), a.q_rank, m->eps, &up, 1);
            it_attn_latent at{};
            at.q = q.p();
            at.q_len = up.out_len;
            if (a.kv_from < 0) {
                at.kv = kv.p();
                at.kv_len = n * a.kv_row();
                at.kv_norm = a.dkv_norm.data();
            }
            at.slab = cache.k_slab(l.slot);
            at.slab_len = n_ctx * a.slab_row();
            at.uk = a.uk;
            at.uv = a.uv;
            at.sinks = a.sink.data();
            at.gate = g.p();
            at.gate_len = n * a.heads;
            at.heads = a.heads; at.dim = a.dim; at.rot_dim = a.rot_dim; at.vdim = a.vdim; at.rank = a.kv_rank;
            at.pos = start;
            at.window = a.window;
            at.scale = a.scale;
            at.eps = m->eps;
            at.rope = a.rope;
            it_hip_attend_latent(be, &at, mixed.p(), n * l.mixed());
        } else {
            const Gla& r = l.r;
            it_group_mat mats[5] = {to_rows(r.q, q, n), to_rows(r.k, k, n), to_rows(r.v, v, n), to_rows(r.g, g, n), to_rows(r.a1, low, n)};
            mats[0].scale = (float)(1.0 / std::sqrt((double)r.dim));
            products(l.norm1, n, mats, 5);
            it_gla ga{};
            ga.q = q.p(); ga.k = k.p(); ga.v = v.p(); ga.low = low.p();
            ga.q_len = mats[0].out_len; ga.k_len = mats[1].out_len; ga.v_len = mats[2].out_len; ga.low_len = mats[4].out_len;
            ga.a2 = r.a2;
            ga.a2_b = r.a2_b.data();
            ga.heads = r.heads; ga.dim = r.dim; ga.vdim = r.vdim;
            ga.tau = r.tau;
            it_hip_gla(be, &ga, cache.ssm_of(l.slot), r.heads * r.vdim * r.dim, mixed.p(), n * l.mixed());
            o.norm_w = r.norm.data();
            o.norm_groups = r.heads;
            o.norm_shared = 1;
            o.eps = m->eps;
            o.gate = g.p();
            o.gate_len = o.in_len;
        }
        sublayer_out(o, n, l.norm1b);
        if (!l.has_mlp) return;
        it_group_mat pair = to_rows(l.gate, ff, n);
        pair.up = l.up;
        pair.act = IT_ACT_RELU;
        products(l.norm2, n, &pair, 1);
        it_res_term d{};
        d.w = l.down;
        d.in = ff.p();
        d.in_len = n * l.ff;
        sublayer_out(d, n, l.norm2b);
    }

    int layers(const uint32_t* tokens, uint64_t n, uint64_t start, uint64_t ring_index) override {
        if (int rc = check_pass(tokens, n, start)) return rc;
        const uint64_t nd = m->nd;
        it_hip_begin_pass(be, n);
        fit(n);
        cur = 0;
        pending = nullptr;
        if (int rc = embed(tokens, n, xs[0].p(), ring_index)) return rc;
        tr("inp_embd", 0, xs[0], n * nd);
        for (uint64_t i = 0; i < m->layers.size(); i++) {
            layer(m->layers[i], start, n);
            if (trace) {   // the sum that the next products will form
                shown.fit(n * nd, be);
                const it_add_normed add = addition(shown);
                it_hip_add_normed(be, xs[cur].p(), n * nd, &add, nd);
                tr("post_layer", i, shown, n * nd);
            }
        }
        if (n > 1) {   // (one token: the head adds it)
            const it_add_normed add = addition(xs[cur ^ 1]);
            it_hip_add_normed(be, xs[cur].p(), n * nd, &add, nd);
            cur ^= 1;
            pending = nullptr;
        }
        len = start + n;
        return 0;
    }
    HostBuf& residual(uint64_t) override { return xs[cur]; }
    it_group_mat head_of(HostBuf& out, uint64_t rows) {
        return to_rows(m->embed_w, out, rows);
    }
    void head(HostBuf& src, uint64_t rows, HostBuf& out) override {
        const it_group_mat h = head_of(out, rows);
        it_hip_norm_matmuls(be, src.p(), rows * m->nd, m->final_norm.data(), m->nd, m->eps, &h, 1);
    }
    void head_of_one() override {
        const it_group_mat h = head_of(logits, 1);
        products(m->final_norm, 1, &h, 1);
    }
};

it_engine* Nubedra::new_engine(it_hip* be, uint64_t n_ctx, uint64_t) {
    NubedraEngine* e = new NubedraEngine();
    e->fm = e->m = this;
    for (const Layer& l : layers) {   // (in the order of their slots)
        if (!l.latent) e->cache.add_state(0, l.r.heads * l.r.vdim * l.r.dim);
        else if (l.a.kv_from < 0) e->cache.add_kv(n_ctx * l.a.slab_row(), 0);   // one row holds what keys and values are made of
    }
    e->cache.allocate(it_hip_is_f32(be) ? 4 : 2);
    return e;
}

}  // namespace

it_model* open_nubedra(const std::string& dir, std::string* err) {
    auto m = std::make_unique<Nubedra>();
    if (!m->load(dir)) {
        *err = m->err;
        return nullptr;
    }
    return m.release();
}
