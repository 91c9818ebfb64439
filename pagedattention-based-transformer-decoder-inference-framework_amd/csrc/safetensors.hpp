// Read-only view of a safetensors file (memory-mapped).
#pragma once

#include <cstdint>
#include <map>
#include <string>
#include <vector>

namespace llm {

struct TensorView {
  const uint8_t* data = nullptr;
  size_t bytes = 0;
  std::string dtype;           // "BF16", "F32", "I32", ...
  std::vector<int64_t> shape;
};

class SafeTensors {
 public:
  SafeTensors() = default;
  ~SafeTensors();
  SafeTensors(const SafeTensors&) = delete;
  SafeTensors& operator=(const SafeTensors&) = delete;
  // Map the file and check every tensor's range and size; an llm_status.
  int open(const std::string& path);
  // The tensor `name` of exactly this shape; an llm_status.
  int get(const std::string& name, const std::vector<int64_t>& shape, TensorView* out) const;
  // Its values: the bits of a BF16 tensor, or a BF16 / F32 tensor as floats.
  int get_bf16(const std::string& name, const std::vector<int64_t>& shape,
               std::vector<uint16_t>* out) const;
  int get_f32(const std::string& name, const std::vector<int64_t>& shape,
              std::vector<float>* out) const;
  bool has(const std::string& name) const { return tensors_.count(name) != 0; }

 private:
  std::map<std::string, TensorView> tensors_;
  void* map_ = nullptr;
  size_t size_ = 0;
};

}  // namespace llm
