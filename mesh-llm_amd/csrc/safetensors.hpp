// Bounded safetensors reader: an 8-byte little-endian header length, that many bytes of JSON (name -> dtype, shape,
// data_offsets), then the data.  Tensor bytes are mapped, never copied.
#pragma once

#include <cstdint>
#include <map>
#include <string>
#include <vector>

namespace mesh {

struct SafeTensor {
    std::string dtype;               // "BF16", "F32", "I32", ...
    std::vector<uint64_t> shape;     // outermost first; a scalar has none
    uint64_t begin = 0, nbytes = 0;  // within the data section
    uint64_t elems() const { uint64_t n = 1; for (uint64_t d : shape) n *= d; return n; }
};

class SafetensorsFile {
  public:
    SafetensorsFile() = default;
    ~SafetensorsFile();
    SafetensorsFile(const SafetensorsFile &) = delete;
    SafetensorsFile &operator=(const SafetensorsFile &) = delete;

    // 0 or a negative mesh_status (message in mesh_last_error).  Every entry has been checked against the file's size.
    int open(const char *path);
    const SafeTensor *find(const std::string &name) const;
    const uint8_t *data(const SafeTensor &t) const { return map_ + data_ + t.begin; }
    const std::map<std::string, SafeTensor> &tensors() const { return tensors_; }
    uint64_t file_size() const { return size_; }
    uint64_t data_offset() const { return data_; }

  private:
    int fd_ = -1;
    const uint8_t *map_ = nullptr;
    uint64_t size_ = 0, data_ = 0;
    std::map<std::string, SafeTensor> tensors_;
};

}  // namespace mesh
