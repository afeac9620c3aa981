// What every model design of the framework provides, and the engine around it: a model knows its weights and sizes, an
// engine runs passes of one sequence over a SeqCache.  model.cpp holds the registry and everything above a pass
// (chunked prefill, greedy generation, checkpoints); a design is one file with a model and an engine class.
#pragma once
#include <cstdint>
#include <string>
#include <vector>

#include "../../include/inferred_hip.h"
#include "cache.h"

// A host buffer whose address never changes once it has reached its largest size
// (/root/reference src/model/qwen35.rs:572-583, 653-673).
struct HostBuf {
    std::vector<float> v;
    // Growing moves the buffer: the backend's mirror and quantized copy are keyed on the OLD address and would
    // otherwise leak, or be inherited by whatever the allocator places there next.
    void fit(uint64_t n, it_hip* be) {
        if (v.size() >= n) return;
        if (!v.empty() && n > v.capacity()) it_hip_release(be, v.data());
        v.resize(n, 0.0f);
    }
    float* p() { return v.data(); }
};

struct it_model {
    std::string path, err;
    virtual ~it_model() = default;
    virtual void dims(uint64_t out[10]) const = 0;
    virtual uint64_t vocab() const = 0;
    virtual uint64_t width() const = 0;
    virtual uint64_t decode_weight_bytes() const = 0;
    virtual void token_macs(uint64_t out[3]) const = 0;
    virtual const it_weights& embedding() const = 0;
    virtual float embedding_scale() const { return 1.0f; }
    virtual it_engine* new_engine(it_hip* be, uint64_t n_ctx, uint64_t max_batch) = 0;

    bool fail(const std::string& m) {
        if (err.empty()) err = m;
        return false;
    }
};

struct it_engine {
    it_model* model = nullptr;
    it_hip* be = nullptr;
    uint64_t n_ctx = 0, max_batch = 0;
    uint64_t len = 0;
    uint64_t ring_next = 0;  // next slot of the backend's device token ring this engine files into
    SeqCache cache;
    it_trace_fn trace = nullptr;
    void* trace_user = nullptr;
    std::string err;
    uint64_t kv_reserved = 0;  // bytes this engine asked the backend to keep free of the expert slab
    HostBuf logits;            // of the last token of the last pass that formed any

    virtual ~it_engine() = default;
    // One pass over n tokens from position `start`.  `tokens == nullptr` is the greedy feedback pass: one token, chosen
    // on the device as the arg-max of the previous pass's logits and embedded there (its id lands at `ring_index` of the
    // device ring).  The last token's logits go to `logits` and come home when want_logits is set.
    virtual int forward(const uint32_t* tokens, uint64_t n, uint64_t start, bool want_logits, uint64_t ring_index = 0) = 0;
    // The same for logits of the rows `rows` of the pass (none: n_rows = 0), copied to out [n_rows][vocab]
    virtual int forward_rows(const uint32_t* tokens, uint64_t n, uint64_t start, const uint32_t* rows, uint64_t n_rows, float* out) = 0;
    virtual std::vector<HostBuf*> buffers() = 0;   // every activation buffer besides `logits`

    void tr(const char* name, uint64_t il, HostBuf& b, uint64_t n) {
        if (!trace) return;
        it_hip_host_needs(be, b.p(), n);
        trace(trace_user, name, (uint32_t)il, b.p(), n);
    }
    int check_pass(const uint32_t* tokens, uint64_t n, uint64_t start);   // 0, or the error of a pass that cannot run
    int embed(const uint32_t* tokens, uint64_t n, float* x, uint64_t ring_index);   // 0, or an error (the pass is ended)
    int end_pass_check(bool device_fed);
};

// The designs: each opens what its file format's architecture name says
it_model* open_qwen35moe(const std::string& path, std::string* err);
it_model* open_serisun(const std::string& dir, std::string* err);
it_model* open_nubedra(const std::string& dir, std::string* err);
// "architecture" of a folder's config.json
bool config_architecture(const std::string& dir, std::string* name, std::string* err);
