// The open model folder behind include/wick_safetensors.h, as C++ host code sees it.  Not installed.
#pragma once

#include <string>
#include <unordered_map>
#include <vector>

#include "../../include/wick_safetensors.h"
#include "json.h"

struct wick_safetensors {
    struct Tensor {
        std::string name;
        int dtype = 0;
        std::vector<uint64_t> shape;
        const uint8_t* data = nullptr;
        size_t nbytes = 0;
    };
    std::string config_text, architecture;
    wick_rocm::Json config;
    const uint8_t* map = nullptr;
    size_t map_bytes = 0;
    std::vector<Tensor> tensors;
    std::unordered_map<std::string, size_t> index;

    ~wick_safetensors();
    const Tensor* find(const std::string& name) const {
        const auto it = index.find(name);
        return it == index.end() ? nullptr : &tensors[it->second];
    }
};
