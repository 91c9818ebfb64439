// Expert routing: choose each token's experts from the router logits, sort the
// assignments by expert, cut every expert's rows into the tiles of the grouped
// products.  Few tokens: one launch of one workgroup; many: the choice runs one
// wave per token over the chip, and one workgroup sorts.
#include "common.hpp"
#include "moe.hpp"

#include <algorithm>

namespace llm {
namespace {

constexpr int kSortThreads = 1024;
constexpr int kFusedTokens = 16;  // a token per wave of the one workgroup
constexpr int kFusedTop = 32;

// One wave: token m's choices.  Lane l holds LE experts: l, l + 64, ...
template <int LE>
__device__ __forceinline__ void choose(const RouteArgs& a, int m, int32_t* choice) {
  const int lane = lane_id();
  float s[LE], key[LE];
#pragma unroll
  for (int j = 0; j < LE; ++j) {
    const int e = lane + 64 * j;
    s[j] = 0.f;
    key[j] = -INFINITY;
    if (e < a.experts) {
      s[j] = 1.f / (1.f + expf(-a.z[(size_t)m * a.ldz + e]));
      key[j] = s[j] + (a.correction ? a.correction[e] : 0.f);
    }
  }
  for (int k = 0; k < a.top; ++k) {
    float best = key[0];
#pragma unroll
    for (int j = 1; j < LE; ++j) best = fmaxf(best, key[j]);
    best = wave_max_dpp(best);
    // the lowest expert that has it (scores that are not numbers match nothing:
    // any valid expert then)
    int be = k;
    float bs = 0.f;
#pragma unroll
    for (int j = LE - 1; j >= 0; --j) {
      const unsigned long long hit = __ballot(key[j] == best);
      if (hit) {
        const int l = __ffsll(hit) - 1;
        be = l + 64 * j;
        bs = __shfl(s[j], l, 64);
      }
    }
    if (be >= a.experts) be = k;
    if (lane == 0) {
      choice[(size_t)m * a.top + k] = be;
      a.weight[(size_t)m * a.top + k] = bs * a.scale;
    }
#pragma unroll
    for (int j = 0; j < LE; ++j)
      if (be == lane + 64 * j) key[j] = -INFINITY;
  }
}

// One workgroup: counts per expert, their starts, the tile list, the order.
__device__ __forceinline__ void sort_assignments(const RouteArgs& a, const int32_t* choice, int* cnt,
                                                 int* start, int* tile0) {
  const int n = a.M * a.top, E = a.experts;
  for (int e = threadIdx.x; e < E; e += kSortThreads) cnt[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < n; i += kSortThreads) atomicAdd(&cnt[choice[i]], 1);
  __syncthreads();
  if (threadIdx.x < 64) {  // exclusive sums of rows and tiles, 64 experts at a time
    int rows = 0, tiles = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + threadIdx.x;
      const int c = e < E ? cnt[e] : 0, t = (c + a.tile_rows - 1) / a.tile_rows;
      int cs = c, ts = t;
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const int oc = __shfl_up(cs, off, 64), ot = __shfl_up(ts, off, 64);
        if ((int)threadIdx.x >= off) { cs += oc; ts += ot; }
      }
      if (e < E) {
        start[e] = rows + cs - c;
        tile0[e] = tiles + ts - t;
      }
      rows += __shfl(cs, 63, 64);
      tiles += __shfl(ts, 63, 64);
    }
    if (threadIdx.x == 0) tile0[E] = tiles;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += kSortThreads) {
    const int c = cnt[e];
    for (int r = 0, t = tile0[e]; r < c; r += a.tile_rows, ++t)
      a.tiles[t] = MmTile{e, start[e] + r, min(a.tile_rows, c - r), 0};
  }
  const int ts = a.shared ? (a.M + a.tile_rows - 1) / a.tile_rows : 0;
  for (int t = threadIdx.x; t < ts; t += kSortThreads)
    a.tiles[tile0[E] + t] =
        MmTile{E, t * a.tile_rows, min(a.tile_rows, a.M - t * a.tile_rows), 0};
  if (threadIdx.x == 0) *a.n_tiles = tile0[E] + ts;
  __syncthreads();  // cnt becomes the cursor
  for (int e = threadIdx.x; e < E; e += kSortThreads) cnt[e] = start[e];
  __syncthreads();
  for (int i = threadIdx.x; i < n; i += kSortThreads) {
    const int at = atomicAdd(&cnt[choice[i]], 1);
    a.perm[at] = i;
  }
}

template <int LE>
__global__ __launch_bounds__(kSortThreads) void route_small_kernel(RouteArgs a) {
  __shared__ int cnt[kMaxExperts], start[kMaxExperts], tile0[kMaxExperts + 1];
  __shared__ int32_t choice[kFusedTokens * kFusedTop];
  const int m = wave_id_uniform();
  if (m < a.M) choose<LE>(a, m, choice);
  __syncthreads();
  sort_assignments(a, choice, cnt, start, tile0);
}

template <int LE>
__global__ __launch_bounds__(256) void route_choose_kernel(RouteArgs a) {
  const int m = blockIdx.x * 4 + wave_id_uniform();
  if (m < a.M) choose<LE>(a, m, a.choice);
}

__global__ __launch_bounds__(kSortThreads) void route_sort_kernel(RouteArgs a) {
  __shared__ int cnt[kMaxExperts], start[kMaxExperts], tile0[kMaxExperts + 1];
  sort_assignments(a, a.choice, cnt, start, tile0);
}

}  // namespace

int route_max_tiles(int M, int top, int experts, bool shared, int tile_rows) {
  const int n = M * top;
  // every expert rounds up at most once
  const int routed = std::min(n, std::min(n, experts) + n / tile_rows);
  return routed + (shared ? (M + tile_rows - 1) / tile_rows : 0);
}

template <int LE>
static hipError_t route_le(const RouteArgs& a, hipStream_t st) {
  if (a.M <= kFusedTokens && a.top <= kFusedTop) {
    hipLaunchKernelGGL(route_small_kernel<LE>, dim3(1), dim3(kSortThreads), 0, st, a);
    return hipGetLastError();
  }
  hipLaunchKernelGGL(route_choose_kernel<LE>, dim3((a.M + 3) / 4), dim3(256), 0, st, a);
  if (hipError_t e = hipGetLastError()) return e;
  hipLaunchKernelGGL(route_sort_kernel, dim3(1), dim3(kSortThreads), 0, st, a);
  return hipGetLastError();
}

hipError_t route(const RouteArgs& a, hipStream_t st) {
  if (a.M <= 0) return hipSuccess;
  if (a.experts <= 64) return route_le<1>(a, st);
  if (a.experts <= 128) return route_le<2>(a, st);
  return a.experts <= 256 ? route_le<4>(a, st) : route_le<kMaxExperts / 64>(a, st);
}

}  // namespace llm
