// What the designs share whose models are folders (config.json, model.safetensors; matrices not quantized): reading both files,
// and an engine's pass around its layers.
#pragma once
#include <string>
#include <vector>

#include "json.h"
#include "model.h"
#include "safetensors.h"

// rows of a cache slab, or of its heads, are padded to whole 16-byte pieces
inline uint64_t round8(uint64_t n) { return (n + 7) / 8 * 8; }

bool read_config(const std::string& dir, itj::Value* out, std::string* err);

struct FolderModel : it_model {
    its::File file;
    uint64_t n_vocab = 0, nd = 0;
    float eps = 0;
    it_weights embed_w{};

    uint64_t vocab() const override { return n_vocab; }
    uint64_t width() const override { return nd; }
    const it_weights& embedding() const override { return embed_w; }

    // config.json: false, with the reason in err, where a value is missing or of another kind
    bool size(const itj::Value* o, const char* where, const char* key, uint64_t* out, uint64_t least = 1);
    bool real(const itj::Value* o, const char* where, const char* key, float* out);
    bool real(const itj::Value* o, const char* where, const char* key, double* out);
    // tensors: checked against the shape the configuration asks for
    const its::Tensor* need(const std::string& name, const std::vector<uint64_t>& shape);
    bool matrix(const std::string& name, uint64_t n_out, uint64_t n_in, it_weights* w);
    bool vec(const std::string& name, const std::vector<uint64_t>& shape, std::vector<float>* out);
};

struct FolderEngine : it_engine {
    FolderModel* fm = nullptr;
    HostBuf last, picked;
    // everything of a pass up to the last layer; the pass stays open
    virtual int layers(const uint32_t* tokens, uint64_t n, uint64_t start, uint64_t ring_index) = 0;
    // the residual stream that the last pass of n tokens left, complete
    virtual HostBuf& residual(uint64_t n) = 0;
    // the final norm and the head over `rows` rows of `src`; over a pass of one token straight from what its layers left
    virtual void head(HostBuf& src, uint64_t rows, HostBuf& out) = 0;
    virtual void head_of_one() { head(residual(1), 1, logits); }

    int forward(const uint32_t* tokens, uint64_t n, uint64_t start, bool want_logits, uint64_t ring_index) override;
    int forward_rows(const uint32_t* tokens, uint64_t n, uint64_t start, const uint32_t* rows, uint64_t n_rows, float* out) override;
};
