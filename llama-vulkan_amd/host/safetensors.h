// safetensors.h — a safetensors file, mapped read-only: a 64-bit little-endian header length, that many bytes of JSON
// (name -> dtype, shape, data_offsets), then the tensors' bytes.
#pragma once

#include <cstddef>
#include <string>
#include <vector>

#include "types.h"

struct safetensors_entry {
    std::string name, dtype;
    std::vector<u64> shape;
    u64 offset, size;          // from the start of the mapping
};

class safetensors_file {
public:
    explicit safetensors_file(const std::string &path);
    ~safetensors_file();
    safetensors_file(const safetensors_file &) = delete;
    safetensors_file &operator=(const safetensors_file &) = delete;

    [[nodiscard]] bool is_open() const { return problem.empty(); }
    [[nodiscard]] const std::string &error() const { return problem; }
    [[nodiscard]] const u8 *data() const { return mapping; }
    [[nodiscard]] std::size_t data_size() const { return mapping_size; }
    [[nodiscard]] const std::vector<safetensors_entry> &entries() const { return table; }

private:
    void parse();

    u8 *mapping = nullptr;
    std::size_t mapping_size = 0;
    std::vector<safetensors_entry> table;
    std::string problem;
};
