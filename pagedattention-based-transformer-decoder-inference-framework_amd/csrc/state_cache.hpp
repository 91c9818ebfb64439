// Recurrent state of a layer run, per sequence slot: fp32 state and the last
// inputs of its convolution.  A sequence at position 0 starts from zeros without
// reading either, so a slot that is used again needs no clearing.
#pragma once

#include <algorithm>

#include "dev_buf.hpp"

namespace llm {

struct StateCache {
  int slots = 0, state = 0, ldc = 0, taps = 0;
  DevBuf<float> s;          // [slots][state][ldc]
  DevBuf<uint8_t> history;  // [slots][taps - 1][ldc] in the element type, oldest first

  int init(int slots_, int state_, int ldc_, int taps_, int elem_size) {
    slots = slots_; state = state_; ldc = ldc_; taps = taps_;
    RET_IF(s.alloc((size_t)slots * state * ldc));
    RET_IF(history.alloc((size_t)slots * std::max(taps - 1, 1) * ldc * elem_size));
    LLM_HIP_RET(hipMemset(s.p, 0, s.n * sizeof(float)));
    LLM_HIP_RET(hipMemset(history.p, 0, history.n));
    LLM_HIP_RET(hipDeviceSynchronize());
    return LLM_OK;
  }
};

}  // namespace llm
