// Paged latent attention (csrc/paged_latent.hip): one row per token in the
// cache -- a normed latent and a rotated key part -- serves every head as key
// and, its latent part, as value.  Queries come already multiplied into the
// latent space, so a token's heads are rows against one key/value head.
#pragma once

#include <hip/hip_runtime.h>

#include "mm.hpp"
#include "paged_gqa.hpp"

namespace llm {

// Cached row: latent [0, rank), turned key part at latent_rot_at(rank), zeros up
// to latent_row(rank, rot).
__host__ __device__ inline int latent_rot_at(int rank) { return (rank + 7) / 8 * 8; }
inline int latent_row(int rank, int rot) { return (latent_rot_at(rank) + rot + 31) / 32 * 32; }
constexpr int kLatentMaxRank = 512, kLatentMaxRow = 576;

// GqaArgs with G = 1, Dp = latent_row, Dv = rank; v_pool unused.  tile_rows: 16,
// 32 or 64.
hipError_t latent_attention(int dtype, const GqaArgs& a, int tile_rows, hipStream_t st);

// down's rows -> cache pages: the latent normed with w, the key part turned.
struct LatentAppend {
  int M = 0, rank = 0, rot = 0;
  const float* down = nullptr;    // [M][ldd]: latent, key part at rot_at
  int ldd = 0, rot_at = 0;
  const float* w = nullptr;       // [rank]
  float eps = 0.f;
  const float2* turn = nullptr;   // [M][rot / 2]
  MmPageRows page;                // where the rows go (pool is written)
};
hipError_t latent_append(int dtype, const LatentAppend& a, hipStream_t st);

// The turned key part of M cached rows (src) into the expanded keys of every
// head: page (slot, head, tile) of `table` takes it at column `at`.
struct LatentSpread {
  int M = 0, H = 0, rot = 0, src_at = 0;
  MmPageRows src;
  const int32_t* slot = nullptr;   // [M] page-table row of the expanded keys
  const int32_t* table = nullptr;  // [slots][H][max_tiles]
  int max_tiles = 0, num_pages = 0;
  void* k_pool = nullptr;          // page: [kPageTokens][Dp]
  size_t page_stride = 0;
  int Dp = 0, at = 0;
};
hipError_t latent_spread(int dtype, const LatentSpread& a, hipStream_t st);

}  // namespace llm
