// What one sequence keeps between passes: key / value slabs per attention layer run and recurrent state (a convolution
// window and a state matrix) per recurrent layer run, of any sizes.  The host copies name the device's: the device owns
// a slab once it has touched it (KvCache / RecurrentState, /root/reference src/cache/mod.rs:33-65, 215-252,
// src/cache/recurrent.rs:31-142).
#pragma once
#include <algorithm>
#include <cstdint>
#include <cstring>
#include <vector>

#include "../../include/inferred_hip.h"

struct SeqCache {
    struct Kv {
        uint64_t k_at, k_len, v_at, v_len;   // elements
    };
    struct State {
        uint64_t conv_at, conv_len, ssm_at, ssm_len;   // floats
        bool live;                                     // false: the layer at this index is not recurrent
    };
    uint64_t elem = 2;   // bytes of a key or value element
    std::vector<uint8_t> k, v;
    std::vector<float> conv, ssm;
    std::vector<Kv> kvs;
    std::vector<State> states;

    uint64_t add_kv(uint64_t k_len, uint64_t v_len) {
        Kv s{kvs.empty() ? 0 : kvs.back().k_at + kvs.back().k_len, k_len, kvs.empty() ? 0 : kvs.back().v_at + kvs.back().v_len, v_len};
        kvs.push_back(s);
        return kvs.size() - 1;
    }
    uint64_t add_state(uint64_t conv_len, uint64_t ssm_len, bool live = true) {
        State s{states.empty() ? 0 : states.back().conv_at + states.back().conv_len, conv_len,
                states.empty() ? 0 : states.back().ssm_at + states.back().ssm_len, ssm_len, live};
        states.push_back(s);
        return states.size() - 1;
    }
    void allocate(uint64_t element_bytes) {   // once every slab is known: the addresses never change afterwards
        elem = element_bytes;
        if (!kvs.empty()) {
            k.assign((kvs.back().k_at + kvs.back().k_len) * elem, 0);
            v.assign((kvs.back().v_at + kvs.back().v_len) * elem, 0);
        }
        if (!states.empty()) {
            conv.assign(states.back().conv_at + states.back().conv_len, 0.0f);
            ssm.assign(states.back().ssm_at + states.back().ssm_len, 0.0f);
        }
    }
    void* k_slab(uint64_t slot) { return k.data() + kvs[slot].k_at * elem; }
    void* v_slab(uint64_t slot) { return v.data() + kvs[slot].v_at * elem; }
    float* conv_of(uint64_t i) { return conv.data() + states[i].conv_at; }
    float* ssm_of(uint64_t i) { return ssm.data() + states[i].ssm_at; }
    uint64_t bytes() const { return k.size() + v.size() + (conv.size() + ssm.size()) * sizeof(float); }
    bool recurrent() const {
        for (const State& s : states)
            if (s.live) return true;
        return false;
    }
    // a new sequence: states start from zero; old keys and values are past its end and get overwritten
    void zero(it_hip* be) {
        std::fill(conv.begin(), conv.end(), 0.0f);
        std::fill(ssm.begin(), ssm.end(), 0.0f);
        for (uint64_t i = 0; i < states.size(); i++) {
            if (!states[i].live) continue;
            it_hip_zero_slab(be, conv_of(i));
            it_hip_zero_slab(be, ssm_of(i));
        }
    }
    void bring_home(it_hip* be) {
        for (uint64_t i = 0; i < states.size(); i++) {
            if (!states[i].live) continue;
            it_hip_read_state(be, conv_of(i), states[i].conv_len);
            it_hip_read_state(be, ssm_of(i), states[i].ssm_len);
        }
    }
    void release(it_hip* be) {
        for (uint64_t s = 0; s < kvs.size(); s++) {
            it_hip_release(be, k_slab(s));
            it_hip_release(be, v_slab(s));
        }
        for (uint64_t i = 0; i < states.size(); i++) {
            if (!states[i].live) continue;
            it_hip_release(be, conv_of(i));
            it_hip_release(be, ssm_of(i));
        }
    }
};
