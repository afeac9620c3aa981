// The Serisun design: parallel layers (one norm feeds the mixer and the feed-forward, each with a scale per channel on its
// way into the residual), mixers of two kinds (attention without rotation: a distance bias per head, a query temperature
// and a sink; Mamba-2), and a stretch of layers that runs several times with the same weights, a cache or state of its
// own per pass, the embedding and a vector per pass added ahead of it.
//
// A model is a folder with config.json and model.safetensors; every size and constant comes from there.
#include <cmath>
#include <cstring>
#include <memory>

#include "model_folder.h"

namespace {

struct Attention {
    uint64_t heads = 0, kv_heads = 0, dim = 0, vdim = 0, temp_every = 0;
    float scale = 0, temp_coef = 0;
    std::vector<float> slopes;
    it_weights q{}, k{}, v{};
    uint64_t k_row() const { return kv_heads * round8(dim); }   // cache row: heads padded to whole 16-byte pieces
    uint64_t v_row() const { return kv_heads * round8(vdim); }
};
struct Mamba2 {
    uint64_t heads = 0, vdim = 0, state = 0, groups = 0, norm_groups = 0, taps = 0;
    it_weights in{};
    std::vector<float> conv, conv_b, dt_bias, a_log, d, norm;
    uint64_t inner() const { return heads * vdim; }
    uint64_t channels() const { return inner() + 2 * groups * state; }
    uint64_t in_dim() const { return inner() + channels() + heads; }
};
struct Layer {
    bool attention = false, has_mlp = false;
    Attention a;
    Mamba2 m;
    it_weights o{}, gate{}, up{}, down{};
    uint64_t ff = 0;
    std::vector<float> norm1, ls1, ls2;
    uint64_t mixed() const { return attention ? a.heads * a.vdim : m.inner(); }
};
// one run of a layer: a looped layer has several, each with a cache or state of its own
struct Run {
    uint64_t layer = 0;
    int64_t opens = -1;   // the number of the pass this run opens
    uint64_t slot = 0;    // of the cache's key / value slabs, or of its states
};

struct Serisun : FolderModel {
    uint64_t passes = 1;   // through the looped layers
    float logit_scale = 1;
    std::vector<Layer> layers;
    std::vector<Run> runs;
    std::vector<float> step, final_norm;   // step: [times][width]
    it_weights head{};

    bool config(const itj::Value& c) {
        if (!size(&c, "", "vocab", &n_vocab) || !size(&c, "", "width", &nd) || !real(c.get("norm"), "norm", "eps", &eps) ||
            !real(&c, "", "logit_scale", &logit_scale))
            return false;
        const itj::Value* ls = c.get("layers");
        if (!ls || ls->kind != itj::Value::Array || ls->items.empty()) return fail("config.json: layers is missing or empty");
        layers.resize(ls->items.size());
        for (size_t i = 0; i < layers.size(); i++) {
            const itj::Value &e = ls->items[i], *ty = e.get("type"), *mx = e.get("mixer"), *mlp = e.get("mlp");
            const std::string where = "layers[" + std::to_string(i) + "]", wm = where + ".mixer";
            Layer& l = layers[i];
            if (!ty || ty->kind != itj::Value::String || !mx) return fail("config.json: " + where + " has no type or no mixer");
            if (ty->str == "attention") {
                Attention& a = l.a;
                l.attention = true;
                if (!size(mx, wm.c_str(), "heads", &a.heads) || !size(mx, wm.c_str(), "kv_heads", &a.kv_heads) || !size(mx, wm.c_str(), "dim", &a.dim) ||
                    !size(mx, wm.c_str(), "vdim", &a.vdim) || !real(mx, wm.c_str(), "scale", &a.scale))
                    return false;
                if (a.heads % a.kv_heads) return fail("config.json: " + wm + ": heads do not divide into kv_heads");
                const itj::Value* t = mx->get("q_temp");
                if (t && !t->is_null() && (!real(t, (wm + ".q_temp").c_str(), "coef", &a.temp_coef) || !size(t, (wm + ".q_temp").c_str(), "every", &a.temp_every)))
                    return false;
                for (uint64_t h = 0; h < a.heads; h++) a.slopes.push_back((float)std::exp2(-8.0 * (double)(h + 1) / (double)a.heads));
            } else if (ty->str == "mamba2") {
                Mamba2& m = l.m;
                if (!size(mx, wm.c_str(), "heads", &m.heads) || !size(mx, wm.c_str(), "vdim", &m.vdim) || !size(mx, wm.c_str(), "state", &m.state) ||
                    !size(mx, wm.c_str(), "groups", &m.groups) || !size(mx, wm.c_str(), "norm_groups", &m.norm_groups) || !size(mx, wm.c_str(), "conv", &m.taps))
                    return false;
                if (m.heads % m.groups) return fail("config.json: " + wm + ": heads do not divide into groups");
                if (m.inner() % m.norm_groups) return fail("config.json: " + wm + ": the inner width does not divide into norm_groups");
                if (m.state > 512 || m.taps > 16) return fail("config.json: " + wm + ": a state of more than 512 columns or more than 16 taps");
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
        // the order of the runs
        uint64_t a = layers.size(), b = layers.size(), times = 1, kv = 0, st = 0;
        const itj::Value* loop = c.get("loop");
        const bool looped = loop && !loop->is_null();
        if (looped) {
            if (!size(loop, "loop", "start", &a, 0) || !size(loop, "loop", "stop", &b) || !size(loop, "loop", "times", &times)) return false;
            if (a >= b || b > layers.size() || times > 4096) return fail("config.json: loop does not name a stretch of the layers");
        }
        passes = times;
        auto add = [&](uint64_t i, int64_t opens) { runs.push_back(Run{i, opens, layers[i].attention ? kv++ : st++}); };
        for (uint64_t i = 0; i < a; i++) add(i, -1);
        for (uint64_t t = 0; looped && t < times; t++)
            for (uint64_t i = a; i < b; i++) add(i, i == a ? (int64_t)t : -1);
        for (uint64_t i = b; i < layers.size(); i++) add(i, -1);
        return !looped || vec("loop.step", {times, nd}, &step);
    }

    bool load(const std::string& dir) {
        itj::Value c;
        if (!read_config(dir, &c, &err) || !file.open(dir + "/model.safetensors", &err) || !config(c)) return false;
        if (!matrix("embed", n_vocab, nd, &embed_w) || !matrix("head", n_vocab, nd, &head) || !vec("final.norm", {nd}, &final_norm)) return false;
        for (size_t i = 0; i < layers.size(); i++) {
            Layer& l = layers[i];
            auto nm = [&](const char* s) { return "l" + std::to_string(i) + "." + s; };
            if (!vec(nm("norm1"), {nd}, &l.norm1) || !vec(nm("ls1"), {nd}, &l.ls1) || !matrix(nm("mix.o"), nd, l.mixed(), &l.o)) return false;
            if (l.attention) {
                Attention& a = l.a;
                if (!matrix(nm("mix.q"), a.heads * a.dim, nd, &a.q) || !matrix(nm("mix.k"), a.kv_heads * a.dim, nd, &a.k) ||
                    !matrix(nm("mix.v"), a.kv_heads * a.vdim, nd, &a.v))
                    return false;
            } else {
                Mamba2& m = l.m;
                if (!matrix(nm("mix.in"), m.in_dim(), nd, &m.in) || !vec(nm("mix.conv"), {m.channels(), m.taps}, &m.conv) ||
                    !vec(nm("mix.conv.b"), {m.channels()}, &m.conv_b) || !vec(nm("mix.dt_bias"), {m.heads}, &m.dt_bias) ||
                    !vec(nm("mix.A_log"), {m.heads}, &m.a_log) || !vec(nm("mix.D"), {m.heads}, &m.d) || !vec(nm("mix.norm"), {m.inner()}, &m.norm))
                    return false;
            }
            if (l.has_mlp && (!matrix(nm("mlp.gate"), l.ff, nd, &l.gate) || !matrix(nm("mlp.up"), l.ff, nd, &l.up) ||
                              !matrix(nm("mlp.down"), nd, l.ff, &l.down) || !vec(nm("ls2"), {nd}, &l.ls2)))
                return false;
        }
        return true;
    }

    void dims(uint64_t out[10]) const override {   // of the first attention layer where layers may differ
        const Attention none, *a = &none;
        for (const Layer& l : layers)
            if (l.attention) {
                a = &l.a;
                break;
            }
        uint64_t v[10] = {layers.size(), nd, n_vocab, a->heads, a->kv_heads, a->dim, 0, 0, 0, 0};
        memcpy(out, v, sizeof v);
    }
    template <class F> uint64_t over_runs(F per_matrix) const {
        uint64_t n = 0;
        for (const Run& r : runs) {
            const Layer& l = layers[r.layer];
            n += per_matrix(l.o) + (l.attention ? per_matrix(l.a.q) + per_matrix(l.a.k) + per_matrix(l.a.v) : per_matrix(l.m.in));
            if (l.has_mlp) n += per_matrix(l.gate) + per_matrix(l.up) + per_matrix(l.down);
        }
        return n;
    }
    uint64_t decode_weight_bytes() const override {
        return head.len + over_runs([](const it_weights& w) { return w.len; });
    }
    void token_macs(uint64_t out[3]) const override {
        out[0] = over_runs([](const it_weights& w) { return w.n_in * w.n_out; });
        out[1] = out[2] = 0;
    }
    it_engine* new_engine(it_hip* be, uint64_t n_ctx, uint64_t max_batch) override;
};

struct SerisunEngine : FolderEngine {
    Serisun* m;
    HostBuf emb, x, q, attn, u, y, ff;
    std::vector<HostBuf*> buffers() override { return {&emb, &x, &q, &attn, &u, &y, &ff, &last, &picked}; }

    void fit(uint64_t n) {
        if (m->passes > 1) emb.fit(n * m->nd, be);
        x.fit(n * m->nd, be);
        for (const Layer& l : m->layers) {
            if (l.attention) {
                q.fit(n * l.a.heads * l.a.dim, be);
                attn.fit(n * l.mixed(), be);
            } else {
                u.fit(n * l.m.in_dim(), be);
                y.fit(n * l.mixed(), be);
            }
            if (l.has_mlp) ff.fit(n * l.ff, be);
        }
        logits.fit(m->n_vocab, be);
    }

    void layer(const Layer& l, const Run& r, uint64_t start, uint64_t n) {
        const uint64_t nd = m->nd;
        it_group_mat mats[5];
        memset(mats, 0, sizeof mats);
        uint64_t k = 0;
        auto to_rows = [&](const it_weights& w, HostBuf& b) -> it_group_mat& {
            it_group_mat& g = mats[k++];
            g.w = w;
            g.out = b.p();
            g.out_len = n * w.n_out;
            g.scale = 1.0f;
            return g;
        };
        auto to_slab = [&](const it_weights& w, void* slab, uint64_t slab_len, uint64_t head_dim) {
            it_group_mat& g = mats[k++];
            g.w = w;
            g.slab = slab;
            g.slab_len = slab_len;
            g.slab_row = start;
            g.head_dim = head_dim;
            g.head_stride = round8(head_dim);
            g.scale = 1.0f;
        };
        // one norm for both sublayers, and every matrix that reads it
        if (l.attention) {
            to_rows(l.a.q, q);
            to_slab(l.a.k, cache.k_slab(r.slot), n_ctx * l.a.k_row(), l.a.dim);
            to_slab(l.a.v, cache.v_slab(r.slot), n_ctx * l.a.v_row(), l.a.vdim);
        } else {
            to_rows(l.m.in, u);
        }
        if (l.has_mlp) to_rows(l.gate, ff).up = l.up;
        it_hip_norm_matmuls(be, x.p(), n * nd, l.norm1.data(), nd, m->eps, mats, k);

        it_res_term terms[2];
        memset(terms, 0, sizeof terms);
        it_res_term& o = terms[0];
        o.w = l.o;
        o.in_len = n * l.mixed();
        o.scale = l.ls1.data();
        if (l.attention) {
            const Attention& a = l.a;
            it_attn_bias at{q.p(), n * a.heads * a.dim, cache.k_slab(r.slot), cache.v_slab(r.slot), n_ctx * a.k_row(), n_ctx * a.v_row(),
                            start + n, a.dim, a.vdim, round8(a.dim), round8(a.vdim), a.heads, a.kv_heads, a.scale, 1, a.slopes.data(),
                            a.temp_coef, (uint32_t)a.temp_every, nullptr, 0};
            it_hip_attend_bias(be, &at, attn.p(), n * l.mixed());
            o.in = attn.p();
        } else {
            const Mamba2& s = l.m;
            it_mamba2 mm{s.conv.data(), s.conv_b.data(), s.dt_bias.data(), s.a_log.data(), s.d.data(), s.heads, s.vdim, s.state, s.groups, s.taps, start};
            it_hip_mamba2(be, &mm, u.p(), n * s.in_dim(), cache.conv_of(r.slot), s.taps * s.channels(), cache.ssm_of(r.slot), s.inner() * s.state,
                          y.p(), n * s.inner());
            o.in = y.p();
            o.norm_w = s.norm.data();
            o.norm_groups = s.norm_groups;
            o.eps = m->eps;
        }
        if (l.has_mlp) {
            it_res_term& d = terms[1];
            d.w = l.down;
            d.in = ff.p();
            d.in_len = n * l.ff;
            d.scale = l.ls2.data();
        }
        it_hip_matmul_residual(be, x.p(), n * nd, terms, l.has_mlp ? 2 : 1);
    }

    int layers(const uint32_t* tokens, uint64_t n, uint64_t start, uint64_t ring_index) override {
        if (int rc = check_pass(tokens, n, start)) return rc;
        const uint64_t nd = m->nd;
        it_hip_begin_pass(be, n);
        fit(n);
        // the embedding is kept beside the residual where a later pass of the loop adds it again
        if (int rc = embed(tokens, n, m->passes > 1 ? emb.p() : x.p(), ring_index)) return rc;
        if (m->passes > 1) it_hip_gather_chunks(be, emb.p(), n * nd, n * nd, n * nd, 0, x.p(), n * nd);
        tr("inp_embd", 0, x, n * nd);
        for (uint64_t i = 0; i < m->runs.size(); i++) {
            const Run& r = m->runs[i];
            if (r.opens >= 0) it_hip_add_rows(be, x.p(), n * nd, r.opens > 0 ? emb.p() : nullptr, m->step.data() + (uint64_t)r.opens * nd, nd);
            layer(m->layers[r.layer], r, start, n);
            tr("post_layer", i, x, n * nd);
        }
        len = start + n;
        return 0;
    }
    HostBuf& residual(uint64_t) override { return x; }
    void head(HostBuf& src, uint64_t rows, HostBuf& out) override {
        it_group_mat g;
        memset(&g, 0, sizeof g);
        g.w = m->head;
        g.out = out.p();
        g.out_len = rows * m->n_vocab;
        g.scale = m->logit_scale;
        it_hip_norm_matmuls(be, src.p(), rows * m->nd, m->final_norm.data(), m->nd, m->eps, &g, 1);
    }

};

it_engine* Serisun::new_engine(it_hip* be, uint64_t n_ctx, uint64_t) {
    SerisunEngine* e = new SerisunEngine();
    e->fm = e->m = this;
    for (const Run& r : runs) {
        const Layer& l = layers[r.layer];
        if (l.attention) e->cache.add_kv(n_ctx * l.a.k_row(), n_ctx * l.a.v_row());
        else e->cache.add_state(l.m.taps * l.m.channels(), l.m.inner() * l.m.state);
    }
    e->cache.allocate(it_hip_is_f32(be) ? 4 : 2);
    return e;
}

}  // namespace

it_model* open_serisun(const std::string& dir, std::string* err) {
    auto m = std::make_unique<Serisun>();
    if (!m->load(dir)) {
        *err = m->err;
        return nullptr;
    }
    return m.release();
}
