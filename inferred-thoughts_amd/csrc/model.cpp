// The registry of model designs and the engine above a pass: chunked prefill, greedy generation, checkpoints.
//
// Mirrors (file:line under /root/reference):
//   Model registry by architecture name  src/model/mod.rs:261-418
//   Engine run/prefill/generate          src/engine/mod.rs:310-437
//   Engine reset/checkpoint/rewind       src/engine/mod.rs:223-306
#include "model.h"

#include <sys/stat.h>

#include <algorithm>
#include <cstdio>
#include <cstring>
#include <memory>

#include "gguf.h"
#include "host_formats.h"

namespace {

// A design is opened by the name its files give it: general.architecture of a GGUF file, "architecture" of a folder's
// config.json (the design reads and checks the name itself)
struct Design {
    const char* name;
    bool folder;   // config.json + model.safetensors instead of one GGUF file
    it_model* (*open)(const std::string& path, std::string* err);
};
const Design DESIGNS[] = {
    {"qwen35moe", false, open_qwen35moe},
    {"Serisun", true, open_serisun},
    {"Nubedra", true, open_nubedra},
};

it_model* open_model(const std::string& path, std::string* err) {
    struct stat st;
    if (stat(path.c_str(), &st)) {
        *err = path + ": no such file or folder";
        return nullptr;
    }
    const bool folder = S_ISDIR(st.st_mode);
    std::string name;
    if (folder) {
        if (!config_architecture(path, &name, err)) return nullptr;
    } else {
        itg::File f;
        if (!f.open(path, err)) return nullptr;
        if (!f.get_string("general.architecture", &name)) {
            *err = "missing general.architecture";
            return nullptr;
        }
    }
    std::string known;
    for (const Design& d : DESIGNS) {
        if (d.folder == folder && name == d.name) {
            it_model* m = d.open(path, err);
            if (m) m->path = path;
            return m;
        }
        known += std::string(known.empty() ? "" : ", ") + d.name;
    }
    *err = "unsupported architecture '" + name + "' (this backend's loop covers " + known + ")";
    return nullptr;
}

uint32_t host_argmax(const float* l, uint64_t n) {  // src/profile.rs:192-213
    uint64_t best = 0;
    for (uint64_t i = 1; i < n; i++)
        if (l[i] > l[best]) best = i;
    return (uint32_t)best;
}
}  // namespace

int it_engine::check_pass(const uint32_t* tokens, uint64_t n, uint64_t start) {
    if (n == 0) { err = "forward: no tokens supplied"; return -1; }
    if (start + n > n_ctx) { err = "context overflow: position " + std::to_string(start + n - 1) + " with n_ctx " + std::to_string(n_ctx); return -2; }
    for (uint64_t t = 0; tokens && t < n; t++)
        if (tokens[t] >= model->vocab()) { err = "token id " + std::to_string(tokens[t]) + " outside the vocabulary"; return -3; }
    return 0;
}

int it_engine::embed(const uint32_t* tokens, uint64_t n, float* x, uint64_t ring_index) {
    const it_weights& w = model->embedding();
    const uint64_t nd = w.n_in;
    const float scale = model->embedding_scale();
    if (tokens) {
        uint64_t row_bytes = itg::type_bytes(w.ty, nd);
        for (uint64_t t = 0; t < n; t++) ith::dequantize(w.ty, w.data + tokens[t] * row_bytes, nd, x + t * nd);
        if (scale != 1.0f)
            for (uint64_t i = 0; i < n * nd; i++) x[i] *= scale;
        it_hip_host_wrote(be, x, n * nd);
    } else if (!it_hip_embed_argmax(be, &w, logits.p(), model->vocab(), x, nd, ring_index)) {
        it_hip_end_pass(be);
        err = "the embedding table's type has no device form";
        return -4;
    } else if (scale != 1.0f) {
        it_hip_scale(be, x, nd, scale);
    }
    return 0;
}

int it_engine::end_pass_check(bool device_fed) {
    // a device-fed pass does not wait for the device: only an error already recorded is looked at,
    // and the caller polls once, with a wait, after its last pass
    if (device_fed && !it_hip_has_error(be)) return 0;
    char msg[512];
    if (it_hip_take_error(be, msg, sizeof msg)) {
        err = msg;
        return -10;
    }
    return 0;
}

extern "C" {

it_model* it_model_open(const char* path, char* err, size_t err_len) {
    std::string why;
    it_model* m = open_model(path ? path : "", &why);
    if (!m && err && err_len) snprintf(err, err_len, "%s", why.c_str());
    return m;
}
void it_model_close(it_model* m) { delete m; }
void it_model_dims(const it_model* m, uint64_t out[10]) { m->dims(out); }
uint64_t it_model_decode_weight_bytes(const it_model* m) { return m->decode_weight_bytes(); }
void it_model_token_macs(const it_model* m, uint64_t out[3]) { m->token_macs(out); }

it_engine* it_engine_new(it_model* m, it_hip* be, uint64_t n_ctx, uint64_t max_batch) {
    if (!m || !be || n_ctx == 0) return nullptr;
    if (!max_batch) max_batch = 512;  // DEFAULT_MAX_BATCH, src/engine/mod.rs:87
    it_engine* e = m->new_engine(be, n_ctx, max_batch);
    e->model = m;
    e->be = be;
    e->n_ctx = n_ctx;
    e->max_batch = max_batch;
    e->kv_reserved = e->cache.bytes();
    it_hip_reserve_for_kv(be, e->kv_reserved);
    return e;
}
void it_engine_free(it_engine* e) {
    if (!e) return;
    // the host buffers are about to be freed: drop the device copies keyed on them
    auto bufs = e->buffers();
    bufs.push_back(&e->logits);
    for (HostBuf* b : bufs)
        if (!b->v.empty()) it_hip_release(e->be, b->p());
    e->cache.release(e->be);
    // the reserve is additive (placement.rs:341-343): give this engine's share back (unsigned wrap-around subtracts)
    it_hip_reserve_for_kv(e->be, (uint64_t)0 - e->kv_reserved);
    delete e;
}

// Engine::reset, src/engine/mod.rs:296-306
void it_engine_reset(it_engine* e) {
    e->len = 0;
    e->cache.zero(e->be);
}
// Engine::checkpoint / restore / rewind, src/engine/mod.rs:223-294.  The device owns the recurrent state once it has
// touched it: a checkpoint brings every layer's slabs home through read_state first, a restore writes the host slabs
// and tells the backend to forget its copies.  The KV needs no stored copy: positions past `pos` are no longer part of
// the sequence and the next pass overwrites them.
void it_engine_state_sizes(const it_engine* e, uint64_t out[2]) {
    out[0] = e->cache.conv.size();
    out[1] = e->cache.ssm.size();
}
uint64_t it_engine_checkpoint(it_engine* e, float* conv_out, float* ssm_out) {
    e->cache.bring_home(e->be);
    if (conv_out) memcpy(conv_out, e->cache.conv.data(), e->cache.conv.size() * sizeof(float));
    if (ssm_out) memcpy(ssm_out, e->cache.ssm.data(), e->cache.ssm.size() * sizeof(float));
    return e->len;
}
int it_engine_restore(it_engine* e, uint64_t pos, const float* conv_in, const float* ssm_in) {
    if (pos > e->n_ctx) {
        e->err = "checkpoint stands at " + std::to_string(pos) + " positions, context is " + std::to_string(e->n_ctx);
        return -1;
    }
    if (!conv_in || !ssm_in) {
        e->err = "restore: null state";
        return -2;
    }
    e->len = pos;
    memcpy(e->cache.conv.data(), conv_in, e->cache.conv.size() * sizeof(float));
    memcpy(e->cache.ssm.data(), ssm_in, e->cache.ssm.size() * sizeof(float));
    it_hip_forget_state(e->be);  // after both halves
    return 0;
}
int it_engine_rewind(it_engine* e, uint64_t len) {
    if (e->cache.recurrent()) return 0;  // a recurrent state is not a log: it cannot drop tokens
    if (len > e->len) return 0;
    e->len = len;
    return 1;
}
void it_engine_set_trace(it_engine* e, it_trace_fn fn, void* user) {
    e->trace = fn;
    e->trace_user = user;
}
uint64_t it_engine_pos(const it_engine* e) { return e->len; }
const char* it_engine_last_error(it_engine* e) { return e->err.c_str(); }

int it_engine_forward(it_engine* e, const uint32_t* tokens, uint64_t n, float* logits) {
    int rc = e->forward(tokens, n, e->len, logits != nullptr);
    if (rc == 0 && logits) memcpy(logits, e->logits.p(), e->model->vocab() * 4);
    return rc;
}

int it_engine_prefill(it_engine* e, const uint32_t* tokens, uint64_t n, float* logits) {
    for (uint64_t at = 0; at < n; at += e->max_batch) {
        uint64_t take = e->max_batch < n - at ? e->max_batch : n - at;
        bool last = at + take >= n;
        int rc = e->forward(tokens + at, take, e->len, last && logits != nullptr);
        if (rc) return rc;
    }
    if (logits) memcpy(logits, e->logits.p(), e->model->vocab() * 4);
    return 0;
}

int it_engine_forward_rows(it_engine* e, const uint32_t* tokens, uint64_t n, const uint32_t* rows, uint64_t n_rows, float* out) {
    for (uint64_t i = 0; i < n_rows; i++)
        if (!rows || rows[i] >= n || (i && rows[i] <= rows[i - 1])) {
            e->err = "forward_rows: the rows must ascend and lie inside the tokens";
            return -5;
        }
    if (n_rows && !out) {
        e->err = "forward_rows: null output";
        return -6;
    }
    uint64_t r = 0;
    std::vector<uint32_t> here;
    for (uint64_t at = 0; at < n || at == 0; at += e->max_batch) {
        const uint64_t take = std::min(e->max_batch, n - at);
        here.clear();
        const uint64_t r0 = r;
        for (; r < n_rows && rows[r] < at + take; r++) here.push_back((uint32_t)(rows[r] - at));
        if (int rc = e->forward_rows(tokens + at, take, e->len, here.data(), here.size(), out ? out + r0 * e->model->vocab() : nullptr)) return rc;
    }
    return 0;
}

int64_t it_engine_generate(it_engine* e, const uint32_t* prompt, uint64_t n_prompt, uint64_t max_new,
                           uint32_t* out_ids, float* last_logits) {
    uint64_t nv = e->model->vocab();
    for (uint64_t at = 0; at < n_prompt; at += e->max_batch) {
        uint64_t take = e->max_batch < n_prompt - at ? e->max_batch : n_prompt - at;
        int rc = e->forward(prompt + at, take, e->len, at + take >= n_prompt);
        if (rc) return rc;
    }
    uint64_t produced = 0;
    for (uint64_t i = 0; i < max_new; i++) {
        uint64_t pos = e->len;
        uint32_t next = host_argmax(e->logits.p(), nv);
        out_ids[produced++] = next;
        if (produced == max_new) break;
        if (pos + 1 >= e->n_ctx) break;
        int rc = e->forward(&next, 1, e->len, true);
        if (rc) return rc;
    }
    if (last_logits) memcpy(last_logits, e->logits.p(), nv * 4);
    return (int64_t)produced;
}

// Greedy decoding with the token fed back on the device: passes are issued back to back and the
// host waits once, at the end, to read the ids.  Falls back to a host round trip per token when
// the embedding table has no device form.
int64_t it_engine_decode_greedy(it_engine* e, uint64_t n, uint32_t* out_ids) {
    uint64_t nv = e->model->vocab();
    uint64_t produced = 0;
    const uint32_t ty = e->model->embedding().ty;
    const bool on_device = ty == IT_Q8_0 || ty == IT_F16 || ty == IT_BF16 || ty == IT_F32;
    if (on_device) {
        const uint64_t first = e->ring_next;
        for (uint64_t i = 0; i < n && i < 65536; i++) {
            if (e->len + 1 > e->n_ctx) break;
            int rc = e->forward(nullptr, 1, e->len, false, e->ring_next);
            if (rc) return rc;
            e->ring_next++;
            produced++;
        }
        if (produced && out_ids) {
            it_hip_read_tokens(e->be, first, produced, out_ids);
            char msg[512];
            if (it_hip_take_error(e->be, msg, sizeof msg)) {
                e->err = msg;
                return -10;
            }
        }
        return (int64_t)produced;
    }
    for (uint64_t i = 0; i < n; i++) {
        if (e->len + 1 > e->n_ctx) break;
        uint32_t next = it_hip_argmax(e->be, e->logits.p(), nv);
        if (out_ids) out_ids[produced] = next;
        produced++;
        int rc = e->forward(&next, 1, e->len, false);
        if (rc) return rc;
    }
    return (int64_t)produced;
}

const float* it_engine_ssm_state(it_engine* e, uint64_t layer, uint64_t* len) {
    *len = e->cache.states[layer].ssm_len;
    it_hip_read_state(e->be, e->cache.ssm_of(layer), *len);
    return e->cache.ssm_of(layer);
}
const float* it_engine_conv_state(it_engine* e, uint64_t layer, uint64_t* len) {
    *len = e->cache.states[layer].conv_len;
    it_hip_read_state(e->be, e->cache.conv_of(layer), *len);
    return e->cache.conv_of(layer);
}
// (a cache of 32-bit elements shows as pairs of 16-bit words)
const uint16_t* it_engine_k_slab(it_engine* e, uint64_t slot, uint64_t* len) {
    *len = e->cache.kvs[slot].k_len * (e->cache.elem / 2);
    it_hip_read_kv(e->be, (uint16_t*)e->cache.k_slab(slot), *len);
    return (const uint16_t*)e->cache.k_slab(slot);
}
const uint16_t* it_engine_v_slab(it_engine* e, uint64_t slot, uint64_t* len) {
    *len = e->cache.kvs[slot].v_len * (e->cache.elem / 2);
    it_hip_read_kv(e->be, (uint16_t*)e->cache.v_slab(slot), *len);
    return (const uint16_t*)e->cache.v_slab(slot);
}

}  // extern "C"
