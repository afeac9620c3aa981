#include "safetensors.h"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cmath>
#include <cstring>

#include "../../include/inferred_hip.h"
#include "json.h"

namespace its {

File::~File() {
    if (base_) munmap((void*)base_, size_);
}

bool File::open(const std::string& path, std::string* err) {
    auto bad = [&](const std::string& m) {
        if (err) *err = path + ": " + m;
        return false;
    };
    const int fd = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) return bad(strerror(errno));
    struct stat st;
    if (fstat(fd, &st) || st.st_size < 8) {
        ::close(fd);
        return bad("too short to be a safetensors file");
    }
    size_ = (size_t)st.st_size;
    void* m = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
    ::close(fd);
    if (m == MAP_FAILED) {
        size_ = 0;
        return bad("cannot be mapped");
    }
    base_ = (const uint8_t*)m;
    uint64_t n = 0;
    memcpy(&n, base_, 8);
    if (n > size_ - 8) return bad("header longer than the file");
    itj::Value head;
    std::string why;
    if (!itj::parse((const char*)base_ + 8, n, &head, &why)) return bad("header: " + why);
    if (head.kind != itj::Value::Object) return bad("header is not an object");
    const uint64_t room = size_ - 8 - n;
    auto whole = [](const itj::Value& v, uint64_t* out) {
        if (v.kind != itj::Value::Number || v.num < 0 || v.num > 9007199254740992.0 || v.num != std::floor(v.num)) return false;
        *out = (uint64_t)v.num;
        return true;
    };
    for (const auto& kv : head.members) {
        if (kv.first == "__metadata__") continue;
        const itj::Value *ty = kv.second.get("dtype"), *shape = kv.second.get("shape"), *at = kv.second.get("data_offsets");
        if (!ty || !shape || !at || ty->kind != itj::Value::String || shape->kind != itj::Value::Array || at->items.size() != 2)
            return bad("tensor " + kv.first + ": incomplete entry");
        Tensor t;
        uint64_t esz = 4;
        if (ty->str == "BF16") { t.ty = IT_BF16; esz = 2; }
        else if (ty->str == "F16") { t.ty = IT_F16; esz = 2; }
        else if (ty->str == "F32") t.ty = IT_F32;
        else continue;   // a type no matrix of this library has: the loader reports the tensor missing if it needs it
        uint64_t count = 1, from = 0, to = 0;
        for (const auto& d : shape->items) {
            uint64_t v = 0;
            if (!whole(d, &v) || __builtin_mul_overflow(count, v, &count)) return bad("tensor " + kv.first + ": bad shape");
            t.shape.push_back(v);
        }
        if (!whole(at->items[0], &from) || !whole(at->items[1], &to) || from > to || to > room || count > room || to - from != count * esz)
            return bad("tensor " + kv.first + ": its bytes do not fit its shape or the file");
        t.data = base_ + 8 + n + from;
        t.bytes = to - from;
        tensors_.emplace(kv.first, std::move(t));
    }
    return true;
}

}  // namespace its
