// Expert routing (csrc/moe.hip).
#pragma once

#include <hip/hip_runtime.h>

#include <cstdint>

#include "mm.hpp"

namespace llm {

// scores s = sigmoid(z); the `top` experts with the largest s + correction
// (ties: the lower index); weights s * scale, not renormalised.
struct RouteArgs {
  const float* z = nullptr;           // [M][ldz] router logits
  int ldz = 0, M = 0, experts = 0, top = 0;
  const float* correction = nullptr;  // [experts] or NULL
  float scale = 1.f;
  bool shared = false;                // tiles of the shared expert (group `experts`) follow
  int tile_rows = 16;
  int32_t* choice = nullptr;          // [M * top] scratch: chosen experts
  float* weight = nullptr;            // [M * top]
  int32_t* perm = nullptr;            // [M * top] sorted assignment -> token * top + choice
  MmTile* tiles = nullptr;            // [route_max_tiles]
  int32_t* n_tiles = nullptr;
};
constexpr int kMaxExperts = 512;
int route_max_tiles(int M, int top, int experts, bool shared, int tile_rows);
hipError_t route(const RouteArgs& a, hipStream_t st);

}  // namespace llm
