// safetensors reader: an 8-byte little-endian header length, a JSON header
// (name -> dtype, shape, data_offsets), then the data.
#include "safetensors.hpp"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cstring>

#include "common.hpp"
#include "json.hpp"

namespace llm {

SafeTensors::~SafeTensors() {
  if (map_) munmap(map_, size_);
}

static size_t dtype_bytes(const std::string& d) {
  if (d == "BF16" || d == "F16" || d == "I16" || d == "U16") return 2;
  if (d == "F32" || d == "I32" || d == "U32") return 4;
  if (d == "F64" || d == "I64" || d == "U64") return 8;
  if (d == "I8" || d == "U8" || d == "BOOL") return 1;
  return 0;
}

int SafeTensors::open(const std::string& path) {
  const int fd = ::open(path.c_str(), O_RDONLY);
  if (fd < 0) return fail(LLM_ERR_IO, "cannot open weight file: " + path);
  struct stat sb;
  if (fstat(fd, &sb) != 0 || sb.st_size < 8) {
    ::close(fd);
    return fail(LLM_ERR_IO, path + ": not a safetensors file");
  }
  size_ = (size_t)sb.st_size;
  map_ = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
  ::close(fd);
  if (map_ == MAP_FAILED) {
    map_ = nullptr;
    return fail(LLM_ERR_IO, "cannot map weight file: " + path);
  }
  const uint8_t* base = static_cast<const uint8_t*>(map_);
  uint64_t hlen = 0;
  std::memcpy(&hlen, base, 8);
  Json head;
  if (hlen > size_ - 8 ||
      !JsonReader(reinterpret_cast<const char*>(base + 8), (size_t)hlen).parse(head) ||
      !head.is_object())
    return fail(LLM_ERR_IO, path + ": bad safetensors header");
  const size_t data = 8 + (size_t)hlen, room = size_ - data;
  for (const auto& kv : head.obj) {
    if (kv.first == "__metadata__") continue;
    const Json& off = kv.second["data_offsets"];
    const Json& shp = kv.second["shape"];
    TensorView t;
    t.dtype = kv.second["dtype"].str;
    size_t n = 1;
    for (const Json& s : shp.arr) {
      if (s.num < 0 || (s.num > 0 && n > size_ / (size_t)s.num))
        return fail(LLM_ERR_IO, path + ": bad shape of tensor " + kv.first);
      t.shape.push_back((int64_t)s.num);
      n *= (size_t)s.num;
    }
    const size_t es = dtype_bytes(t.dtype);
    if (!shp.is_array() || !off.is_array() || off.arr.size() != 2 || es == 0 ||
        off.arr[0].num < 0 || off.arr[1].num < off.arr[0].num || off.arr[1].num > (double)room ||
        (size_t)off.arr[1].num - (size_t)off.arr[0].num != n * es)
      return fail(LLM_ERR_IO, path + ": bad entry of tensor " + kv.first);
    t.data = base + data + (size_t)off.arr[0].num;
    t.bytes = n * es;
    tensors_[kv.first] = t;
  }
  return LLM_OK;
}

static std::string shape_str(const std::vector<int64_t>& s) {
  std::string o = "[";
  for (size_t i = 0; i < s.size(); ++i) o += (i ? ", " : "") + std::to_string(s[i]);
  return o + "]";
}

int SafeTensors::get(const std::string& name, const std::vector<int64_t>& shape,
                     TensorView* out) const {
  const auto it = tensors_.find(name);
  if (it == tensors_.end()) return fail(LLM_ERR_IO, "weights: missing tensor " + name);
  if (it->second.shape != shape)
    return fail(LLM_ERR_IO, "weights: " + name + " has shape " + shape_str(it->second.shape) +
                                ", expected " + shape_str(shape));
  *out = it->second;
  return LLM_OK;
}

int SafeTensors::get_bf16(const std::string& name, const std::vector<int64_t>& shape,
                          std::vector<uint16_t>* out) const {
  TensorView t;
  if (int rc = get(name, shape, &t)) return rc;
  if (t.dtype != "BF16") return fail(LLM_ERR_IO, "weights: " + name + " is " + t.dtype + ", expected BF16");
  out->resize(t.bytes / 2);
  std::memcpy(out->data(), t.data, t.bytes);
  return LLM_OK;
}

int SafeTensors::get_f32(const std::string& name, const std::vector<int64_t>& shape,
                         std::vector<float>* out) const {
  TensorView t;
  if (int rc = get(name, shape, &t)) return rc;
  if (t.dtype == "F32") {
    out->resize(t.bytes / 4);
    std::memcpy(out->data(), t.data, t.bytes);
    return LLM_OK;
  }
  if (t.dtype != "BF16") return fail(LLM_ERR_IO, "weights: " + name + " is " + t.dtype);
  out->resize(t.bytes / 2);
  for (size_t i = 0; i < out->size(); ++i) {
    uint16_t h;
    std::memcpy(&h, t.data + 2 * i, 2);
    const uint32_t u = (uint32_t)h << 16;
    std::memcpy(&(*out)[i], &u, 4);
  }
  return LLM_OK;
}

}  // namespace llm
