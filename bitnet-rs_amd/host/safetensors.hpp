// safetensors.hpp -- reader of the safetensors container: an 8-byte little-endian header length, a JSON header
// (name -> dtype, shape, data_offsets), the data.  The file is mapped; every tensor's byte range is checked against its shape.
#pragma once

#include <cstddef>
#include <cstdint>
#include <cstring>
#include <map>
#include <string>
#include <vector>

namespace bitnet_host {

inline float bf16_value(uint16_t h) {
    const uint32_t u = (uint32_t)h << 16;
    float v;
    memcpy(&v, &u, 4);
    return v;
}

struct SafeTensor {
    std::string dtype;
    std::vector<uint64_t> shape;
    const uint8_t *data = nullptr;
    size_t bytes = 0;
    uint64_t elements() const {
        uint64_t n = 1;
        for (uint64_t d : shape) n *= d;
        return n;
    }
};

class SafeTensors {
  public:
    SafeTensors() = default;
    ~SafeTensors();
    SafeTensors(const SafeTensors &) = delete;
    SafeTensors &operator=(const SafeTensors &) = delete;
    bool open(const std::string &path, std::string &err);
    const SafeTensor *find(const std::string &name) const;
    // a bf16 matrix of exactly this shape, or null with err set
    const uint16_t *matrix(const std::string &name, size_t rows, size_t cols, std::string &err) const;
    // a bf16 or f32 vector of exactly n elements as f32
    bool vector(const std::string &name, size_t n, std::vector<float> &out, std::string &err) const;

  private:
    const uint8_t *map_ = nullptr;
    size_t len_ = 0;
    std::map<std::string, SafeTensor> tensors_;
};

}  // namespace bitnet_host
