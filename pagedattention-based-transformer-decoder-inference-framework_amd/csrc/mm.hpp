// Matrix products of the layer-stack models (csrc/mm.hip): C = A . W^T in bf16
// or fp32 with fp32 accumulation, W packed once at load time, and the work that
// follows each product in its epilogue.
#pragma once

#include <hip/hip_runtime.h>

#include <cstddef>
#include <cstdint>

#include "llm_decoder.h"

namespace llm {

// Element type of activations and packed weights: LLM_BF16 or LLM_F32.
inline int mm_elem_size(int dtype) { return dtype == LLM_F32 ? 4 : 2; }
inline int mm_kstep(int dtype) { return dtype == LLM_F32 ? 16 : 32; }
// Activation rows are padded with zeros to whole k-steps of either type.
inline int mm_pad(int k) { return (k + 31) / 32 * 32; }

// Packed weights: for every (16 output columns, k-step) one 1 KiB block, lane
// l's 16 bytes holding W[n0 + (l & 15)][k0 + (l >> 4) * (kstep / 4) ...].
size_t mm_packed_bytes(int dtype, int N, int K);
// src: bf16 [rows][K] row-major on the device; packed column n takes source
// row row_map[n] (NULL: n; -1: zeros).
hipError_t mm_pack(int dtype, const uint16_t* src, const int32_t* row_map, int N, int K, void* dst,
                   hipStream_t st);

// Projection epilogue of an attention layer: columns are the query heads, then
// the key heads, then the value heads.  Query and key columns are stored with
// rotation partners side by side (columns 2i and 2i + 1 of a head are
// dimensions i and i + rot / 2), turned by the row's angle, and the keys and
// values go straight into the row's cache page.
struct MmQkv {
  const int32_t* pos = nullptr;   // [M]
  const int32_t* slot = nullptr;  // [M] page-table row
  const float2* turn = nullptr;   // [M][rot / 2] (cos, sin); unused when rot == 0
  int rot = 0;
  int H = 0, G = 0, D = 0, Dv = 0;
  int Dp = 0, Dvp = 0;            // row lengths in the pages
  void* q = nullptr;              // [M][H][Dp]
  const int32_t* table = nullptr; // [slots][G][max_tiles] of the layer
  int slots = 0, max_tiles = 0, num_pages = 0;
  void* k_pool = nullptr;         // page: [kPageTokens][Dp]
  void* v_pool = nullptr;         // page: [Dvp][kPageTokens], keys ordered by v_page_slot
  size_t page_stride = 0;         // bytes
};

constexpr int kPageTokens = 64;
// Place of a token inside a row of its V page.  The second attention product
// takes keys in groups: with bf16 a lane's 8 operands are keys 4g..4g+3 and
// 16+4g..16+4g+3 of a 32-key block, so those lie together.
__host__ __device__ __forceinline__ int v_page_slot(int t, bool bf16) {
  return bf16 ? (t & 32) + 8 * ((t & 15) >> 2) + 4 * ((t >> 4) & 1) + (t & 3) : t;
}

// y = g sigmoid(alpha g) (u + up_bias), g = min(gate, limit), u = clamp(up, +-limit)
struct GluParams {
  float limit = 0.f, alpha = 1.f, up_bias = 0.f;
};

// A group of a grouped product: expert g of a layer, or its shared expert.
struct MmGroup {
  const void* w_in = nullptr;   // gate and up rows interleaved, N = 2 ff
  const void* w_out = nullptr;  // N = width, K = ff
  int n_in = 0, ks_in = 0, n_out = 0, ks_out = 0;
  GluParams glu;
};
struct MmTile {
  int group, row0, rows, pad;
};
// Rows of a grouped product.  Routed rows (groups < n_routed) are the sorted
// assignments s: perm[s] = token * top + choice.  Shared rows are the tokens.
struct MmGrouped {
  const MmGroup* groups = nullptr;  // [n_routed + shared], device
  const MmTile* tiles = nullptr;    // device list
  const int32_t* n_tiles = nullptr;
  const int32_t* perm = nullptr;
  const float* weight = nullptr;    // [M * top], by token * top + choice
  int n_routed = 0, top = 0, M = 0;
  int max_tiles = 0;                // grid bound
  int tile_rows = 16;               // 16, 64 or 128: rows of a tile list entry
  int max_n = 0;                    // widest group's columns
  int min_ks = 0;
  const void* h = nullptr;          // [M][ldh] tokens' rows
  int ldh = 0;
  void* act = nullptr;              // [M * top][lda] routed activations
  int lda = 0;
  void* act_shared = nullptr;       // [M][lds]
  int lds = 0;
  float* out = nullptr;             // [M * top + M][ldo]: choices, then the shared rows
  int ldo = 0;
};

struct MmArgs {
  const void* A = nullptr;  // [M][lda], zero-padded to whole k-steps
  int lda = 0;
  const void* W = nullptr;
  int M = 0, N = 0, K = 0;
  int w_nt = 0;             // weights streamed once per step (not kept in cache)
  float* C = nullptr;       // [M][ldc]
  int ldc = 0;
  float softcap = 0.f;      // C = softcap tanh(C / softcap) when set
};

// Columns [0, n_t) go to `t` in the element type, the others to `f` in fp32
// (from its column 0).  n_t and the row lengths are even; an odd N may write its
// padding column.
struct MmSplit {
  void* t = nullptr;
  int ldt = 0, n_t = 0;
  float* f = nullptr;
  int ldf = 0;
};

// The input product of a layer with a short causal convolution, for rows that
// are one token each: columns [0, channels) pass the convolution of the row's
// slot and silu into `x`, and shift its history; columns from `gate` on go to z.
constexpr int kMmConvTaps = 4;  // most taps this epilogue takes
struct MmConv {
  int channels = 0, gate = 0, taps = 0;
  const int32_t* pos = nullptr;   // [M]
  const int32_t* slot = nullptr;  // [M]
  const float* w = nullptr;       // [taps][ldw], the last tap is the current token's
  const float* bias = nullptr;    // [ldw]
  int ldw = 0;
  void* history = nullptr;        // [slots][taps - 1][ldw], oldest first
  void* x = nullptr;
  int ldx = 0;
  void* z = nullptr;
  int ldz = 0;
};

// Projections of a latent-attention layer: H heads of D + rot query columns (D
// and rot even; partners of a rotation are columns 2i and 2i + 1), then the
// latent and the shared key part in fp32 (not turned).  Queries go to `q`; their
// turned part also behind the latent part of `q_lat`.
struct MmLatent {
  const float2* turn = nullptr;   // [M][rot / 2]
  int H = 0, D = 0, rot = 0;
  void* q = nullptr;              // [M][H][ldq]: D, then rot
  int ldq = 0;
  void* q_lat = nullptr;          // [M][H][ld_lat], turned part at `lat_rot`
  int ld_lat = 0, lat_rot = 0;
  float* down = nullptr;          // [M][ldd]
  int ldd = 0;
};

// One product per head: A and C move by a_head / c_head elements, W by w_head
// bytes.  With `rows` only these rows of A and C take part (M: their number).
struct MmHeads {
  int heads = 1;
  size_t a_head = 0, w_head = 0;
  void* C = nullptr;
  int ldc = 0, c_head = 0;
  const int32_t* rows = nullptr;
};

// Rows of A taken from cache pages: row m is token pos[m] of page-table row
// slot[m] (MmArgs::A and lda unused).
struct MmPageRows {
  const int32_t* pos = nullptr;
  const int32_t* slot = nullptr;
  const int32_t* table = nullptr;  // [slots][max_tiles]
  int max_tiles = 0, num_pages = 0;
  const void* pool = nullptr;      // page: [kPageTokens][row]
  size_t page_stride = 0;          // bytes
  int row = 0;                     // elements
};

hipError_t mm(int dtype, const MmArgs& a, hipStream_t st);
hipError_t mm_split(int dtype, const MmArgs& a, const MmSplit& e, hipStream_t st);
// W holds gate and up rows interleaved (N = 2 ff); act [M][ld] = glu
hipError_t mm_glu(int dtype, const MmArgs& a, const GluParams& p, void* act, int ld, hipStream_t st);
// C = softplus(A . W^T + bias), bias padded to an even length
hipError_t mm_softplus(int dtype, const MmArgs& a, const float* bias, hipStream_t st);
hipError_t mm_conv(int dtype, const MmArgs& a, const MmConv& e, hipStream_t st);
hipError_t mm_latent(int dtype, const MmArgs& a, const MmLatent& e, hipStream_t st);
hipError_t mm_heads(int dtype, const MmArgs& a, const MmHeads& e, hipStream_t st);
// keys and values (no queries, e.H = 0, not turned) of the rows of cache pages,
// into the pages of e
hipError_t mm_expand(int dtype, const MmArgs& a, const MmPageRows& r, const MmQkv& e, hipStream_t st);
hipError_t mm_qkv(int dtype, const MmArgs& a, const MmQkv& e, hipStream_t st);
// act = glu(h . w_in^T) of every group's rows
hipError_t mm_grouped_in(int dtype, const MmGrouped& g, int w_nt, hipStream_t st);
// out = weight * (act . w_out^T)
hipError_t mm_grouped_out(int dtype, const MmGrouped& g, int w_nt, hipStream_t st);
// Rows per tile mm_grouped_* wants for M tokens (the routing kernel builds the list).
int mm_group_tile_rows(int M, int top, int experts);

}  // namespace llm
