// Matrix products of the layer-stack models on gfx950 MFMA.
//
//   bf16: v_mfma_f32_16x16x32_bf16      fp32: v_mfma_f32_16x16x4_f32
//
// One kernel, three shapes.  A wave owns MT x NT tiles of 16 x 16 outputs and
// streams A fragments (row-major rows, 64 bytes per row and k-step) and packed
// W fragments (1 KiB blocks) straight into registers, double-buffered.
//   decode rows    MT = rows / 16, 8 waves split K and add through LDS: every
//                  weight byte of the product is in flight at once
//   prompt rows    4 waves in a 2 x 2 square of MT x NT tiles
//   grouped rows   a tile list (built by the routing kernel) names the group
//                  and rows of each block of the grid
// A and W share the k order inside a fragment, so the sum is exact whatever the
// hardware's own order; C: column = lane & 15, row = 4 (lane >> 4) + reg.
//
// Epilogues work on column pairs (2i, 2i + 1), which sit in neighbouring lanes:
// rotation partners and (gate, up) pairs are packed side by side, so a pair is
// one DPP move away and no product needs a second launch to finish it.
#include "common.hpp"
#include "mm.hpp"

#include <algorithm>

namespace llm {
namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

enum Epi { kStore, kQkv, kGroupIn, kGroupOut };

template <typename T>
struct Kind;
template <>
struct Kind<__bf16> {
  static constexpr bool BF16 = true;
  static __device__ __forceinline__ f32x4 mma(u32x4 a, u32x4 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a),
                                                   __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
  }
};
template <>
struct Kind<float> {
  static constexpr bool BF16 = false;
  static __device__ __forceinline__ f32x4 mma(u32x4 a, u32x4 b, f32x4 c) {
    const f32x4 x = __builtin_bit_cast(f32x4, a), y = __builtin_bit_cast(f32x4, b);
#pragma unroll
    for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[j], y[j], c, 0, 0, 0);
    return c;
  }
};

struct KernelArgs {
  MmArgs a;
  int KS;
  MmQkv q;
  MmGrouped g;
};

__device__ __forceinline__ float glu(float gate, float up, const GluParams& p) {
  const float g = fminf(gate, p.limit);
  const float u = fminf(fmaxf(up, -p.limit), p.limit);
  return g / (1.f + expf(-p.alpha * g)) * (u + p.up_bias);
}

template <typename T>
__device__ __forceinline__ void put_pair(T* p, float v0, float v1) {
  typedef T pair_t __attribute__((ext_vector_type(2)));
  pair_t v;
  v[0] = (T)v0;
  v[1] = (T)v1;
  *reinterpret_cast<pair_t*>(p) = v;
}

template <typename T>
__device__ __forceinline__ void emit_qkv(const MmQkv& e, int m, int n, float v0, float v1) {
  const int nq = e.H * e.D, nk = e.G * e.D;
  const int pos = e.pos[m];
  if (n < nq + nk) {
    const bool key = n >= nq;
    const int nn = key ? n - nq : n;
    const int head = nn / e.D, d = nn - head * e.D;
    if (d < e.rot) {
      const float2 cs = e.turn[(size_t)m * (e.rot >> 1) + (d >> 1)];
      const float u = v0, v = v1;
      v0 = u * cs.x - v * cs.y;
      v1 = v * cs.x + u * cs.y;
    }
    if (!key) {
      put_pair(static_cast<T*>(e.q) + ((size_t)m * e.H + head) * e.Dp + d, v0, v1);
      return;
    }
    const int tile = pos / kPageTokens;
    if (tile >= e.max_tiles) return;
    const int page = e.table[((size_t)e.slot[m] * e.G + head) * e.max_tiles + tile];
    if (page < 0 || page >= e.num_pages) return;
    T* row = reinterpret_cast<T*>(static_cast<char*>(e.k_pool) + (size_t)page * e.page_stride);
    put_pair(row + (size_t)(pos % kPageTokens) * e.Dp + d, v0, v1);
    return;
  }
  const int tile = pos / kPageTokens;
  if (tile >= e.max_tiles) return;
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int nv = n + j - nq - nk;
    const int head = nv / e.Dv, d = nv - head * e.Dv;
    if (head >= e.G) return;  // the pair's second half past the last column
    const int page = e.table[((size_t)e.slot[m] * e.G + head) * e.max_tiles + tile];
    if (page < 0 || page >= e.num_pages) continue;
    T* row = reinterpret_cast<T*>(static_cast<char*>(e.v_pool) + (size_t)page * e.page_stride);
    row[(size_t)d * kPageTokens + v_page_slot(pos % kPageTokens, Kind<T>::BF16)] =
        (T)(j ? v1 : v0);
  }
}

// WM x WN waves tile the block, WK waves split K.
template <typename T, int EPI, int MT, int NT, int WM, int WN, int WK>
__global__ __launch_bounds__(64 * WM * WN * WK) void mm_kernel(KernelArgs p) {
  constexpr bool GROUP = EPI == kGroupIn || EPI == kGroupOut;
  constexpr int U = MT * NT >= 16 ? 1 : MT * NT >= 4 ? 2 : 4;  // k-steps per load batch
  const int lane = lane_id();
  const int w = wave_id_uniform();
  const int wk = w % WK, wn = (w / WK) % WN, wm = w / (WK * WN);

  const T* A = static_cast<const T*>(p.a.A);
  const char* W = static_cast<const char*>(p.a.W);
  int lda = p.a.lda, M = p.a.M, N = p.a.N, KS = p.KS;
  int mb = (int)blockIdx.y * 16 * MT * WM;
  bool shared = false;
  GluParams gp;
  if constexpr (GROUP) {
    if ((int)blockIdx.y >= *p.g.n_tiles) return;
    const MmTile t = p.g.tiles[blockIdx.y];
    const MmGroup g = p.g.groups[t.group];
    shared = t.group >= p.g.n_routed;
    mb = t.row0;
    M = t.row0 + t.rows;
    if constexpr (EPI == kGroupIn) {
      A = static_cast<const T*>(p.g.h);
      lda = p.g.ldh;
      W = static_cast<const char*>(g.w_in);
      N = g.n_in;
      KS = g.ks_in;
      gp = g.glu;
    } else {
      A = static_cast<const T*>(shared ? p.g.act_shared : p.g.act);
      lda = shared ? p.g.lds : p.g.lda;
      W = static_cast<const char*>(g.w_out);
      N = g.n_out;
      KS = g.ks_out;
    }
  }
  const int ntiles = (N + 15) >> 4;
  if ((int)blockIdx.x * WN * NT >= ntiles) return;  // (the whole block: groups differ in width)
  const int nt0 = ((int)blockIdx.x * WN + wn) * NT;
  const int m0 = mb + wm * 16 * MT;

  const char* ap[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    int m = min(m0 + 16 * i + (lane & 15), M - 1);
    if constexpr (EPI == kGroupIn) {
      if (!shared) m = p.g.perm[m] / p.g.top;
    }
    ap[i] = reinterpret_cast<const char*>(A + (size_t)m * lda) + 16 * (lane >> 4);
  }
  const char* bp[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j)
    bp[j] = W + (size_t)min(nt0 + j, ntiles - 1) * KS * 1024 + lane * 16;

  f32x4 acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};

  const int ks0 = wk * KS / WK, ks1 = (wk + 1) * KS / WK;
  struct Batch {
    u32x4 a[U][MT], b[U][NT];
  };
  const bool nt_load = p.a.w_nt;
  auto load = [&](Batch& x, int ks) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = ks + u;
      if (k < ks1) {
#pragma unroll
        for (int j = 0; j < NT; ++j) {
          const u32x4* src = reinterpret_cast<const u32x4*>(bp[j] + (size_t)k * 1024);
          x.b[u][j] = nt_load ? __builtin_nontemporal_load(src) : *src;
        }
#pragma unroll
        for (int i = 0; i < MT; ++i)
          x.a[u][i] = *reinterpret_cast<const u32x4*>(ap[i] + (size_t)k * 64);
      } else {
#pragma unroll
        for (int j = 0; j < NT; ++j) x.b[u][j] = u32x4{0u, 0u, 0u, 0u};
#pragma unroll
        for (int i = 0; i < MT; ++i) x.a[u][i] = u32x4{0u, 0u, 0u, 0u};
      }
    }
  };
  auto mul = [&](const Batch& x) {
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int i = 0; i < MT; ++i)
#pragma unroll
        for (int j = 0; j < NT; ++j) acc[i][j] = Kind<T>::mma(x.a[u][i], x.b[u][j], acc[i][j]);
  };
  if (ks0 < ks1) {
    Batch x, y;
    load(x, ks0);
    for (int ks = ks0;;) {
      if (ks + U < ks1) load(y, ks + U);
      mul(x);
      ks += U;
      if (ks >= ks1) break;
      if (ks + U < ks1) load(x, ks + U);
      mul(y);
      ks += U;
      if (ks >= ks1) break;
    }
  }

  // one 16 x 16 tile of finished sums -> the epilogue, a column pair per lane
  auto emit = [&](f32x4 c, int i, int j) {
    f32x4 o;
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] = mov_dpp<0xB1>(c[r]);  // the neighbouring column
    const bool odd = lane & 1;
    const int n = (nt0 + j) * 16 + (lane & 14);
#pragma unroll
    for (int r = 0; r < 2; ++r) {
      const float v0 = odd ? o[2 + r] : c[r], v1 = odd ? c[2 + r] : o[r];
      const int m = m0 + 16 * i + 4 * (lane >> 4) + (odd ? 2 : 0) + r;
      if (m >= M || n >= N) continue;
      if constexpr (EPI == kStore) {
        float* d = p.a.C + (size_t)m * p.a.ldc + n;
        d[0] = v0;
        if (n + 1 < N) d[1] = v1;
      } else if constexpr (EPI == kQkv) {
        emit_qkv<T>(p.q, m, n, v0, v1);
      } else if constexpr (EPI == kGroupIn) {
        T* d = static_cast<T*>(shared ? p.g.act_shared : p.g.act);
        d[(size_t)m * (shared ? p.g.lds : p.g.lda) + (n >> 1)] = (T)glu(v0, v1, gp);
      } else {
        const int row = shared ? p.g.M * p.g.top + m : p.g.perm[m];
        const float s = shared ? 1.f : p.g.weight[row];
        float* d = p.g.out + (size_t)row * p.g.ldo + n;
        d[0] = s * v0;
        if (n + 1 < N) d[1] = s * v1;
      }
    }
  };

  if constexpr (WK == 1) {
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < NT; ++j) emit(acc[i][j], i, j);
  } else {
    static_assert(WM == 1 && WN == 1, "k-split blocks hold one tile square");
    __shared__ f32x4 red[WK][MT * NT][64];
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < NT; ++j) red[wk][i * NT + j][lane] = acc[i][j];
    __syncthreads();
    for (int t = w; t < MT * NT; t += WK) {
      f32x4 s = red[0][t][lane];
#pragma unroll
      for (int k = 1; k < WK; ++k) s += red[k][t][lane];
      emit(s, t / NT, t % NT);
    }
  }
}

template <typename T>
__global__ void mm_pack_kernel(const uint16_t* __restrict__ src, const int32_t* __restrict__ map,
                               int N, int K, int KS, size_t chunks, u32x4* __restrict__ dst) {
  constexpr int E = 16 / sizeof(T);
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= chunks) return;
  const int lane = idx & 63;
  const size_t blk = idx >> 6;
  const int ks = (int)(blk % KS);
  const int n = (int)(blk / KS) * 16 + (lane & 15);
  const int row = n < N ? (map ? map[n] : n) : -1;
  const int k0 = ks * 4 * E + (lane >> 4) * E;
  T v[E];
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const uint16_t h = row >= 0 && k0 + e < K ? src[(size_t)row * K + k0 + e] : (uint16_t)0;
    if constexpr (sizeof(T) == 2)
      v[e] = __builtin_bit_cast(T, h);
    else
      v[e] = __builtin_bit_cast(T, (uint32_t)h << 16);
  }
  u32x4 o;
  __builtin_memcpy(&o, v, 16);
  dst[idx] = o;
}

template <typename T, int EPI, int MT, int NT, int WM, int WN, int WK>
hipError_t go(const KernelArgs& p, int rows_blocks, int N, hipStream_t st) {
  const int ntiles = (N + 15) / 16;
  const dim3 grid((ntiles + WN * NT - 1) / (WN * NT), rows_blocks);
  hipLaunchKernelGGL((mm_kernel<T, EPI, MT, NT, WM, WN, WK>), grid, dim3(64 * WM * WN * WK), 0, st,
                     p);
  return hipGetLastError();
}

template <typename T, int EPI>
hipError_t launch(const KernelArgs& p, hipStream_t st) {
  const int M = p.a.M, N = p.a.N;
  const int ntiles = (N + 15) / 16;
  if (M <= 64) {
    // two column tiles per block once one per block already fills the chip
    if (M <= 16) return go<T, EPI, 1, 1, 1, 1, 8>(p, 1, N, st);
    if (M <= 32)
      return ntiles >= 512 ? go<T, EPI, 2, 2, 1, 1, 8>(p, 1, N, st)
                           : go<T, EPI, 2, 1, 1, 1, 8>(p, 1, N, st);
    return ntiles >= 512 ? go<T, EPI, 4, 2, 1, 1, 8>(p, 1, N, st)
                         : go<T, EPI, 2, 1, 1, 1, 8>(p, (M + 31) / 32, N, st);
  }
  const int big = ((M + 127) / 128) * ((ntiles + 7) / 8);
  if (big >= 256) return go<T, EPI, 4, 4, 2, 2, 1>(p, (M + 127) / 128, N, st);
  const int mid = ((M + 63) / 64) * ((ntiles + 3) / 4);
  if (mid >= 192) return go<T, EPI, 2, 2, 2, 2, 1>(p, (M + 63) / 64, N, st);
  return go<T, EPI, 2, 2, 1, 1, 8>(p, (M + 31) / 32, N, st);
}

template <typename T, int EPI>
hipError_t launch_grouped(const MmGrouped& g, int w_nt, hipStream_t st) {
  KernelArgs p{};
  p.g = g;
  p.a.w_nt = w_nt;
  if (g.tile_rows == 16) {
    // few k-steps per wave are not worth eight of them
    if (g.min_ks >= 16) return go<T, EPI, 1, 1, 1, 1, 8>(p, g.max_tiles, g.max_n, st);
    return go<T, EPI, 1, 1, 1, 1, 4>(p, g.max_tiles, g.max_n, st);
  }
  return go<T, EPI, 4, 2, 1, 4, 1>(p, g.max_tiles, g.max_n, st);
}

}  // namespace

size_t mm_packed_bytes(int dtype, int N, int K) {
  const int ks = mm_kstep(dtype);
  return (size_t)((N + 15) / 16) * ((K + ks - 1) / ks) * 1024;
}

hipError_t mm_pack(int dtype, const uint16_t* src, const int32_t* row_map, int N, int K, void* dst,
                   hipStream_t st) {
  const int ks = mm_kstep(dtype), KS = (K + ks - 1) / ks;
  const size_t chunks = (size_t)((N + 15) / 16) * KS * 64;
  const dim3 grid((unsigned)((chunks + 255) / 256));
  if (dtype == LLM_F32)
    hipLaunchKernelGGL(mm_pack_kernel<float>, grid, dim3(256), 0, st, src, row_map, N, K, KS,
                       chunks, static_cast<u32x4*>(dst));
  else
    hipLaunchKernelGGL(mm_pack_kernel<__bf16>, grid, dim3(256), 0, st, src, row_map, N, K, KS,
                       chunks, static_cast<u32x4*>(dst));
  return hipGetLastError();
}

static KernelArgs plain_args(int dtype, const MmArgs& a) {
  KernelArgs p{};
  p.a = a;
  p.KS = (a.K + mm_kstep(dtype) - 1) / mm_kstep(dtype);
  return p;
}

hipError_t mm(int dtype, const MmArgs& a, hipStream_t st) {
  const KernelArgs p = plain_args(dtype, a);
  return dtype == LLM_F32 ? launch<float, kStore>(p, st) : launch<__bf16, kStore>(p, st);
}

hipError_t mm_qkv(int dtype, const MmArgs& a, const MmQkv& e, hipStream_t st) {
  KernelArgs p = plain_args(dtype, a);
  p.q = e;
  return dtype == LLM_F32 ? launch<float, kQkv>(p, st) : launch<__bf16, kQkv>(p, st);
}

int mm_group_tile_rows(int M, int top, int experts) {
  return (long long)M * top >= 24LL * experts && M > 64 ? 64 : 16;
}

hipError_t mm_grouped_in(int dtype, const MmGrouped& g, int w_nt, hipStream_t st) {
  return dtype == LLM_F32 ? launch_grouped<float, kGroupIn>(g, w_nt, st)
                          : launch_grouped<__bf16, kGroupIn>(g, w_nt, st);
}

hipError_t mm_grouped_out(int dtype, const MmGrouped& g, int w_nt, hipStream_t st) {
  return dtype == LLM_F32 ? launch_grouped<float, kGroupOut>(g, w_nt, st)
                          : launch_grouped<__bf16, kGroupOut>(g, w_nt, st);
}

}  // namespace llm
