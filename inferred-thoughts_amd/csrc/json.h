// A small JSON reader for model configurations: the whole document as a tree, numbers as doubles.
#pragma once
#include <cstdint>
#include <map>
#include <string>
#include <vector>

namespace itj {

struct Value {
    enum Kind { Null, Bool, Number, String, Array, Object } kind = Null;
    bool b = false;
    double num = 0;
    std::string str;
    std::vector<Value> items;
    std::map<std::string, Value> members;
    const Value* get(const std::string& key) const {   // null: not an object, or no such member
        if (kind != Object) return nullptr;
        auto it = members.find(key);
        return it == members.end() ? nullptr : &it->second;
    }
    bool is_null() const { return kind == Null; }
};

// false with the place and reason in *err
bool parse(const char* text, size_t len, Value* out, std::string* err);

}  // namespace itj
