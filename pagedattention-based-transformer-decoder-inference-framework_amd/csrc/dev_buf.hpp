// Owned device memory of the runtimes.
#pragma once

#include <hip/hip_runtime.h>

#include <string>

#include "common.hpp"

namespace llm {

template <typename T>
struct DevBuf {
  T* p = nullptr;
  size_t n = 0;
  DevBuf() = default;
  DevBuf(const DevBuf&) = delete;
  DevBuf& operator=(const DevBuf&) = delete;
  ~DevBuf() { if (p) (void)hipFree(p); }
  int alloc(size_t count) {
    if (p) { (void)hipFree(p); p = nullptr; }
    n = count;
    if (count == 0) return LLM_OK;
    if (hipMalloc(&p, count * sizeof(T)) != hipSuccess) {
      (void)hipGetLastError();
      return fail(LLM_ERR_OOM, "decoder: device allocation of " + std::to_string(count * sizeof(T)) +
                                   " bytes failed");
    }
    return LLM_OK;
  }
};

#define RET_IF(x) do { int _rc = (x); if (_rc) return _rc; } while (0)

}  // namespace llm
