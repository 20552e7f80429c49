// safetensors container (read only): an 8-byte little-endian header length, a JSON object
// name -> {dtype, shape, data_offsets}, then the data.  Mapped, not copied.
#pragma once
#include <cstdint>
#include <map>
#include <memory>
#include <string>
#include <vector>

namespace cera {

struct SafeTensor {
    std::string dtype;              // "BF16", "F32", "I32", ...
    std::vector<uint64_t> shape;    // row-major
    const void* data = nullptr;
    uint64_t nbytes = 0;
    uint64_t elements() const {
        uint64_t n = 1;
        for (uint64_t d : shape) n *= d;
        return n;
    }
};

class SafeTensors {
public:
    // nullptr + *err on any malformed input (offsets outside the file, sizes that do not fit the shape)
    static std::unique_ptr<SafeTensors> open(const std::string& path, std::string* err);
    ~SafeTensors();
    SafeTensors(const SafeTensors&) = delete;
    SafeTensors& operator=(const SafeTensors&) = delete;
    const SafeTensor* find(const std::string& name) const;
    const std::map<std::string, SafeTensor>& tensors() const { return tensors_; }

private:
    SafeTensors() = default;
    void* map_ = nullptr;
    uint64_t size_ = 0;
    std::map<std::string, SafeTensor> tensors_;
};

}  // namespace cera
