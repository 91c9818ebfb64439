// Paged grouped-query attention of a mixed batch (csrc/paged_gqa.hip): prompt
// portions and single decoded tokens in one launch, key and value sizes of
// their own, an optional sink per head.
#pragma once

#include <hip/hip_runtime.h>

#include <cstdint>

#include "llm_decoder.h"

namespace llm {

// One workgroup row tile: the queries of one sequence's new tokens, flattened
// per key/value head as rows (token, head of the group), row = token * R + r.
// It covers rows row0 .. row0 + tile_rows - 1 (of nrows) against the keys of
// pages [page0, page1).
struct GqaItem {
  int32_t tok0;   // batch row of the sequence's first new token
  int32_t slot;   // page-table row
  int32_t p0;     // its position
  int32_t row0, nrows;
  int32_t page0, page1;
  int32_t part;   // partial state index, or -1: the only split, writes `out`
};
// The splits of one row tile: parts part0 .. part0 + nsplit - 1.
struct GqaMerge {
  int32_t tok0, row0, nrows, part0, nsplit;
};

struct GqaArgs {
  const void* q = nullptr;  // [tokens][H][Dp]
  void* out = nullptr;      // [tokens][ldo], head h's values at h * Dv
  int ldo = 0;
  int ldh = 0;              // elements between the heads of out (0: Dv)
  const void* k_pool = nullptr;  // page [64][Dp]
  const void* v_pool = nullptr;  // page [Dvp][64] (mm.hpp v_page_slot)
  size_t page_stride = 0;        // bytes
  const int32_t* table = nullptr;  // [slots][G][max_tiles]
  int max_tiles = 0, num_pages = 0;
  int H = 0, G = 0, Dp = 0, Dv = 0, Dvp = 0;
  float scale = 1.f;
  const float* sink = nullptr;   // [H] or NULL
  const GqaItem* items = nullptr;
  int n_items = 0;
  const GqaMerge* merges = nullptr;
  int n_merges = 0;
  float* part_o = nullptr;   // [part][G][tile_rows][gqa_part_dim]
  float* part_ml = nullptr;  // [part][G][tile_rows][2]
};
constexpr int kGqaMaxDim = 256;
constexpr int kGqaSmallRows = 64;  // sequences up to this many rows take tiles of 16
// Rows per tile for sequences that bring `rows` rows per key/value head.
int gqa_tile_rows(int dtype, int Dp, int Dvp, int rows);
inline int gqa_part_dim(int Dv) { return (Dv + 15) / 16 * 16; }
// One launch; every item was cut for tile_rows.
hipError_t gqa_attention(int dtype, const GqaArgs& a, int tile_rows, hipStream_t st);
// The merges of a launch that left partial states (gqa_attention does its own).
constexpr int kGqaMaxMergeDim = 512;
hipError_t gqa_merge(int dtype, const GqaArgs& a, int tile_rows, hipStream_t st);

}  // namespace llm
