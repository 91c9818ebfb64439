// RMS norms around a layer's sublayers (csrc/rms_norm.hip).
#pragma once

#include <hip/hip_runtime.h>

#include <cstddef>
#include <cstdint>

#include "llm_decoder.h"

namespace llm {

// One launch between two sublayers, per token row m:
//   x  = E[tok]                                   (embed 1: the model's start)
//   x += rms(sublayer output) * w_post            (w_post set)
//   x += E[tok]                                   (embed 2: a repeated pass starts)
//   h  = rms(x) * w_pre                           (w_pre set)
// y_scale (a layer scale) multiplies the sublayer output element by element after
// its norm.  emb_scale multiplies E[tok].
//
// With several residual streams (streams > 0) x holds x_1 .. x_s per token and
// the sum becomes
//   x_t = sum_s hc_mix[s][t] x_s + hc_out[t] y,   u = sum_t hc_in[t] x_t
// where u takes the place of x in the norm.  hc_mix and hc_out belong to the
// sublayer that left y, hc_in to the one that comes next (NULL: ones).  The
// embedding starts every stream.
// The sublayer output is y's row m, or the sum of its parts rows m * parts ..
// + parts - 1 and, with `shared`, row M * parts + m (the expert outputs).
// All in fp32; h in the model's element type.
struct NormStep {
  float* x = nullptr;       // [M][max(streams, 1)][ldx] residual, columns past `width` zero
  int ldx = 0, width = 0, M = 0;
  float eps = 0.f;
  int embed = 0;
  const uint16_t* emb = nullptr;  // bf16 [vocab][ldx]
  const int32_t* tok = nullptr;
  float emb_scale = 1.f;
  const float* w_post = nullptr;  // [ldx]
  const float* y_scale = nullptr; // [ldx]
  const float* y = nullptr;       // NULL: no sublayer output to add
  int ldy = 0, parts = 1, shared = 0;
  const float* w_pre = nullptr;   // [ldx]
  void* h = nullptr;
  int ldh = 0;
  // rows (optional): only these rows of x, h row i = row rows[i]; M = their
  // number, M_y the tokens y was written for
  const int32_t* rows = nullptr;
  int M_y = 0;
  int streams = 0;                // 0: one residual, no mixing
  const float* hc_mix = nullptr;  // [streams][streams], from first
  const float* hc_out = nullptr;  // [streams]
  const float* hc_in = nullptr;   // [streams]
  float* u = nullptr;             // [M][ldx] (streams only, optional): u itself
};
constexpr int kMaxStreams = 16;
hipError_t rms_norm_step(int dtype, const NormStep& a, hipStream_t st);

// turn[m][i] = mul * (cos, sin)(pos[m] * freq[i])
hipError_t rope_turns(const int32_t* pos, int M, const float* freq, int half, float mul,
                      float2* turn, hipStream_t st);

}  // namespace llm
