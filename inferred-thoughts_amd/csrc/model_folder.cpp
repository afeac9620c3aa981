#include "model_folder.h"

#include <cmath>
#include <cstring>
#include <fstream>
#include <sstream>

#include "host_formats.h"

bool read_config(const std::string& dir, itj::Value* out, std::string* err) {
    std::ifstream f(dir + "/config.json", std::ios::binary);
    if (!f) {
        *err = dir + "/config.json: cannot be read";
        return false;
    }
    std::stringstream s;
    s << f.rdbuf();
    const std::string text = s.str();
    std::string why;
    if (itj::parse(text.data(), text.size(), out, &why)) return true;
    *err = dir + "/config.json: " + why;
    return false;
}
bool config_architecture(const std::string& dir, std::string* name, std::string* err) {
    itj::Value c;
    if (!read_config(dir, &c, err)) return false;
    const itj::Value* a = c.get("architecture");
    if (!a || a->kind != itj::Value::String) {
        *err = dir + "/config.json: no architecture";
        return false;
    }
    *name = a->str;
    return true;
}

bool FolderModel::size(const itj::Value* o, const char* where, const char* key, uint64_t* out, uint64_t least) {
    const itj::Value* v = o ? o->get(key) : nullptr;
    if (!v || v->kind != itj::Value::Number || v->num < (double)least || v->num > 1e9 || v->num != std::floor(v->num))
        return fail(std::string("config.json: ") + where + "." + key + " is missing or not a whole number in range");
    *out = (uint64_t)v->num;
    return true;
}
bool FolderModel::real(const itj::Value* o, const char* where, const char* key, double* out) {
    const itj::Value* v = o ? o->get(key) : nullptr;
    if (!v || v->kind != itj::Value::Number) return fail(std::string("config.json: ") + where + "." + key + " is missing or not a number");
    *out = v->num;
    return true;
}
bool FolderModel::real(const itj::Value* o, const char* where, const char* key, float* out) {
    double v = 0;
    if (!real(o, where, key, &v)) return false;
    *out = (float)v;
    return true;
}
const its::Tensor* FolderModel::need(const std::string& name, const std::vector<uint64_t>& shape) {
    const its::Tensor* t = file.tensor(name);
    if (!t) {
        fail("missing tensor " + name);
        return nullptr;
    }
    if (t->shape != shape) {
        std::string m = "tensor " + name + ": expected [";
        for (auto v : shape) m += std::to_string(v) + ",";
        m += "] got [";
        for (auto v : t->shape) m += std::to_string(v) + ",";
        fail(m + "]");
        return nullptr;
    }
    return t;
}
bool FolderModel::matrix(const std::string& name, uint64_t n_out, uint64_t n_in, it_weights* w) {
    const its::Tensor* t = need(name, {n_out, n_in});
    if (!t) return false;
    *w = it_weights{t->data, t->bytes, t->ty, 0, n_in, n_out};
    return true;
}
bool FolderModel::vec(const std::string& name, const std::vector<uint64_t>& shape, std::vector<float>* out) {
    const its::Tensor* t = need(name, shape);
    if (!t) return false;
    out->resize(t->n_elems());
    return ith::dequantize(t->ty, t->data, t->n_elems(), out->data()) || fail("tensor " + name + ": unsupported type for a vector");
}

int FolderEngine::forward(const uint32_t* tokens, uint64_t n, uint64_t start, bool want_logits, uint64_t ring_index) {
    if (int rc = layers(tokens, n, start, ring_index)) return rc;
    if (n == 1) {
        head_of_one();
    } else {
        last.fit(fm->nd, be);
        it_hip_gather_chunks(be, residual(n).p(), n * fm->nd, fm->nd, fm->nd, (n - 1) * fm->nd, last.p(), fm->nd);
        head(last, 1, logits);
    }
    it_hip_end_pass(be);
    if (want_logits) it_hip_host_needs(be, logits.p(), fm->n_vocab);
    if (trace) tr("result_output", 0, logits, fm->n_vocab);
    return end_pass_check(!tokens);
}
int FolderEngine::forward_rows(const uint32_t* tokens, uint64_t n, uint64_t start, const uint32_t* rows, uint64_t n_rows, float* out) {
    const uint64_t nv = fm->n_vocab, nd = fm->nd;
    if (n == 1) {   // the same pass whether its logits are wanted or not: one recorded graph serves both
        if (int rc = forward(tokens, 1, start, n_rows > 0, 0)) return rc;
        if (n_rows) memcpy(out, logits.p(), nv * sizeof(float));
        return 0;
    }
    if (int rc = layers(tokens, n, start, 0)) return rc;
    it_hip_end_pass(be);
    const uint64_t most = std::max<uint64_t>(1, std::min<uint64_t>(256, (64ull << 20) / nv));   // rows whose logits are held at a time
    for (uint64_t at = 0; at < n_rows; at += most) {
        const uint64_t k = std::min(most, n_rows - at);
        last.fit(k * nd, be);
        picked.fit(k * nv, be);
        it_hip_gather_rows(be, residual(n).p(), n * nd, nd, rows + at, k, last.p(), k * nd);
        head(last, k, picked);
        it_hip_host_needs(be, picked.p(), k * nv);
        memcpy(out + at * nv, picked.p(), k * nv * sizeof(float));
    }
    return end_pass_check(false);
}
