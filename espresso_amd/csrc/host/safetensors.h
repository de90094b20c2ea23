// Reader of .safetensors files: an 8-byte little-endian header length, that many bytes of JSON (tensor name -> dtype, shape,
// data_offsets), then the data.  The file is memory-mapped; tensors are views into the mapping.
#pragma once

#include <cstdint>
#include <map>
#include <memory>
#include <string>
#include <vector>

namespace esp {

struct TensorView {
    std::string dtype;              // "BF16", "F16", "F32", "I32", ...
    std::vector<int64_t> shape;
    const uint8_t *data = nullptr;
    size_t bytes = 0;
    size_t elements() const;
};
size_t safetensors_dtype_bytes(const std::string &dtype);   // 0 for an unknown type

class SafetensorsFile {
  public:
    ~SafetensorsFile();
    SafetensorsFile(const SafetensorsFile &) = delete;
    SafetensorsFile &operator=(const SafetensorsFile &) = delete;
    // Checks that every tensor lies inside the file and that its byte range fits its shape and type.
    static bool open(const std::string &path, std::unique_ptr<SafetensorsFile> *out, std::string *error);
    const TensorView *find(const std::string &name) const;
    const std::map<std::string, TensorView> &tensors() const { return tensors_; }

  private:
    SafetensorsFile() = default;
    void *map_ = nullptr;
    size_t map_bytes_ = 0;
    std::map<std::string, TensorView> tensors_;
};

}  // namespace esp
