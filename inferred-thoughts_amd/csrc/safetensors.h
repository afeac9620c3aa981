// Memory-mapped safetensors reader: an 8-byte little-endian header length, a JSON header (name -> dtype, shape,
// data_offsets), then the data.
#pragma once
#include <cstdint>
#include <string>
#include <unordered_map>
#include <vector>

namespace its {

struct Tensor {
    uint32_t ty = 0;               // the library's type codes (IT_F32, IT_F16, IT_BF16)
    std::vector<uint64_t> shape;   // as written: [out, in]
    const uint8_t* data = nullptr;
    uint64_t bytes = 0;
    uint64_t n_elems() const {
        uint64_t n = 1;
        for (auto d : shape) n *= d;
        return n;
    }
};

class File {
  public:
    File() = default;
    File(const File&) = delete;
    File& operator=(const File&) = delete;
    ~File();
    bool open(const std::string& path, std::string* err);
    const Tensor* tensor(const std::string& name) const {
        auto it = tensors_.find(name);
        return it == tensors_.end() ? nullptr : &it->second;
    }

  private:
    const uint8_t* base_ = nullptr;
    size_t size_ = 0;
    std::unordered_map<std::string, Tensor> tensors_;
};

}  // namespace its
