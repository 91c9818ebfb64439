// Kernels of the layer-stack models' matrix products on gfx950 MFMA; mm.hip and
// mm_mix.hip instantiate them per epilogue.
//
//   bf16: v_mfma_f32_16x16x32_bf16      fp32: v_mfma_f32_16x16x4_f32
//
// Two kernels.  Decode rows stream: a block owns 16 MT rows x 16 NT columns, its
// 8 waves split K and load A (row-major rows, 64 bytes per row and k-step) and W
// (packed 1 KiB fragments) straight into registers, so every weight byte of the
// product is in flight at once.  Prompt rows go through LDS in 128 x 128 (or 64 x
// 128) blocks, both operands loaded from memory into LDS in fragment order.
// Grouped rows take either form; a tile list (built by the routing kernel) names
// the group and rows of each row of the grid.
// A and W share the k order inside a fragment, so the sum is exact whatever the
// hardware's own order; C: column = lane & 15, row = 4 (lane >> 4) + reg.
//
// Epilogues work on column pairs (2i, 2i + 1), which sit in neighbouring lanes:
// rotation partners and (gate, up) pairs are packed side by side, so a pair is
// one DPP move away and no product needs a second launch to finish it.
#pragma once

#include <algorithm>

#include "common.hpp"
#include "mm.hpp"

namespace llm {
namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

enum Epi {
  kStore, kQkv, kGroupIn, kGroupOut,                                    // mm.hip
  kSplit, kGlu, kSoftplus, kConv, kLatent, kHeads, kExpand              // mm_mix.hip
};

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
  MmSplit split;
  MmConv conv;
  MmLatent lat;
  MmHeads heads;
  MmPageRows page_rows;
  GluParams glu;
  const float* bias;
};

__device__ __forceinline__ float glu(float gate, float up, const GluParams& p) {
  const float g = fminf(gate, p.limit);
  const float u = fminf(fmaxf(up, -p.limit), p.limit);
  return g / (1.f + expf(-p.alpha * g)) * (u + p.up_bias);
}

// log(1 + e^v) = max(v, 0) + log1p(e), e = e^-|v|; log1p(e) = 2 atanh(s) with
// s = e / (2 + e) <= 1/3, whose series needs no case for small or large v
__device__ __forceinline__ float softplus(float v) {
  const float a = -fabsf(v), t = a * kLog2e;
  const float lo = fmaf(a, kLog2e, -t);  // what rounding took from the exponent
  const float p = __builtin_amdgcn_exp2f(t);
  const float e = fmaf(p, lo * 0.6931472f, p);
  const float s = e * __builtin_amdgcn_rcpf(2.f + e), q = s * s;
  float r = 1.f / 15.f;
  r = fmaf(r, q, 1.f / 13.f);
  r = fmaf(r, q, 1.f / 11.f);
  r = fmaf(r, q, 1.f / 9.f);
  r = fmaf(r, q, 1.f / 7.f);
  r = fmaf(r, q, 1.f / 5.f);
  r = fmaf(r, q, 1.f / 3.f);
  r = fmaf(r, q, 1.f);
  return fmaxf(v, 0.f) + 2.f * s * r;
}

template <typename T>
__device__ __forceinline__ void put_pair(T* p, float v0, float v1) {
  typedef T pair_t __attribute__((ext_vector_type(2)));
  pair_t v;
  v[0] = (T)v0;
  v[1] = (T)v1;
  *reinterpret_cast<pair_t*>(p) = v;
}

// What a block of rows and columns works on: set once from the launch arguments
// or the tile list.
template <typename T>
struct Block {
  const T* A = nullptr;
  const char* W = nullptr;
  int lda = 0, M = 0, N = 0, KS = 0, m0 = 0;
  bool shared = false;
  GluParams glu;
};

template <typename T, int EPI>
__device__ __forceinline__ Block<T> block_of(const KernelArgs& p, int row_blocks) {
  Block<T> b;
  if constexpr (EPI == kGroupIn || EPI == kGroupOut) {
    const MmTile t = p.g.tiles[blockIdx.y];
    const MmGroup g = p.g.groups[t.group];
    b.shared = t.group >= p.g.n_routed;
    b.m0 = t.row0;
    b.M = t.row0 + t.rows;
    if constexpr (EPI == kGroupIn) {
      b.A = static_cast<const T*>(p.g.h);
      b.lda = p.g.ldh;
      b.W = static_cast<const char*>(g.w_in);
      b.N = g.n_in;
      b.KS = g.ks_in;
      b.glu = g.glu;
    } else {
      b.A = static_cast<const T*>(b.shared ? p.g.act_shared : p.g.act);
      b.lda = b.shared ? p.g.lds : p.g.lda;
      b.W = static_cast<const char*>(g.w_out);
      b.N = g.n_out;
      b.KS = g.ks_out;
    }
  } else {
    b.A = static_cast<const T*>(p.a.A);
    b.W = static_cast<const char*>(p.a.W);
    b.lda = p.a.lda;
    b.M = p.a.M;
    b.N = p.a.N;
    b.KS = p.KS;
    b.m0 = (int)blockIdx.y * row_blocks;
    b.glu = p.glu;
    if constexpr (EPI == kHeads) {
      b.A += blockIdx.z * p.heads.a_head;
      b.W += blockIdx.z * p.heads.w_head;
    }
  }
  return b;
}

// This lane's 16 bytes of the first k-step of row m's fragments.
template <typename T, int EPI>
__device__ __forceinline__ const char* a_lane(const KernelArgs& p, const Block<T>& b, int m) {
  m = min(m, b.M - 1);
  if constexpr (EPI == kGroupIn) {
    if (!b.shared) m = p.g.perm[m] / p.g.top;
  }
  if constexpr (EPI == kHeads) {
    if (p.heads.rows) m = p.heads.rows[m];
  }
  if constexpr (EPI == kExpand) {
    const MmPageRows& r = p.page_rows;
    const int pos = r.pos[m];
    int page = r.table[(size_t)r.slot[m] * r.max_tiles + min(pos / kPageTokens, r.max_tiles - 1)];
    page = min(max(page, 0), r.num_pages - 1);
    return static_cast<const char*>(r.pool) + (size_t)page * r.page_stride +
           (size_t)(pos % kPageTokens) * r.row * sizeof(T) + 16 * (lane_id() >> 4);
  }
  return reinterpret_cast<const char*>(b.A + (size_t)m * b.lda) + 16 * (lane_id() >> 4);
}

template <int EPI>
struct History {};
template <>
struct History<kConv> {  // of the pair's two channels: earlier inputs, taps, bias
  float v[2][kMmConvTaps - 1], w[2][kMmConvTaps], bias[2];
};

// What an epilogue needs of a row, and of a column pair (n, n + 1): found once
// per row and column of a block's tiles.
template <int EPI>
struct RowOf {
  static constexpr bool PAGED = EPI == kQkv || EPI == kExpand;
  int m = -1;             // -1: no such row
  int at = 0, entry = 0;  // paged: place in the page, page-table entry of head 0 (-1: none)
  int pos = 0;

  __device__ __forceinline__ RowOf() {}
  template <typename T>
  __device__ __forceinline__ RowOf(const KernelArgs& p, const Block<T>& b, int row) {
    if (row >= b.M) return;
    m = row;
    if constexpr (PAGED) {
      const MmQkv& e = p.q;
      pos = e.pos[m];
      const int tile = pos / kPageTokens;
      at = pos % kPageTokens;
      entry = tile < e.max_tiles ? e.slot[m] * e.G * e.max_tiles + tile : -1;
    }
  }
};
template <int EPI>
struct ColOf {
  int n = -1;  // -1: no such column
  int part = 0, head = 0, d = 0;

  __device__ __forceinline__ ColOf() {}
  template <typename T>
  __device__ __forceinline__ ColOf(const KernelArgs& p, const Block<T>& b, int col) {
    if (col >= b.N) return;
    n = col;
    if constexpr (RowOf<EPI>::PAGED) {  // query, key, value
      const MmQkv& e = p.q;
      const int nq = e.H * e.D, nk = e.G * e.D;
      part = n < nq ? 0 : n < nq + nk ? 1 : 2;
      const int i = n - (part == 0 ? 0 : part == 1 ? nq : nq + nk), size = part == 2 ? e.Dv : e.D;
      head = i / size;
      d = i - head * size;
    } else if constexpr (EPI == kLatent) {  // query, projected down
      const MmLatent& e = p.lat;
      const int hd = e.D + e.rot;
      part = n >= e.H * hd;
      if (part) {
        d = n - e.H * hd;
      } else {
        head = n / hd;
        d = n - head * hd;
      }
    }
  }
};

template <typename T>
__device__ __forceinline__ T* page_at(const MmQkv& e, void* pool, int entry, int head) {
  const int page = e.table[(size_t)entry + (size_t)head * e.max_tiles];
  return page >= 0 && page < e.num_pages
             ? reinterpret_cast<T*>(static_cast<char*>(pool) + (size_t)page * e.page_stride)
             : nullptr;
}

// Where a column pair of a row goes, and what it still needs: found before the
// sums are there, so the loads behind it (page, angle, assignment) overlap the
// weight stream.
template <typename T, int EPI>
struct Target {
  History<EPI> past;
  void* p0 = nullptr;  // NULL: nothing to write
  void* p1 = nullptr;  // the second column's place where it is not next to the first
  float cs = 1.f, sn = 0.f;  // rotation; kGroupOut: cs is the weight

  __device__ __forceinline__ void find(const KernelArgs& p, const Block<T>& b, const RowOf<EPI>& r,
                                       const ColOf<EPI>& c) {
    const int m = r.m, n = c.n;
    if (m < 0 || n < 0) return;
    if constexpr (EPI == kStore) {
      float* d = p.a.C + (size_t)m * p.a.ldc + n;
      p0 = d;
      p1 = n + 1 < b.N ? d + 1 : nullptr;
    } else if constexpr (EPI == kGroupIn) {
      T* d = static_cast<T*>(b.shared ? p.g.act_shared : p.g.act);
      p0 = d + (size_t)m * (b.shared ? p.g.lds : p.g.lda) + (n >> 1);
    } else if constexpr (EPI == kGroupOut) {
      const int row = b.shared ? p.g.M * p.g.top + m : p.g.perm[m];
      if (!b.shared) cs = p.g.weight[row];
      float* d = p.g.out + (size_t)row * p.g.ldo + n;
      p0 = d;
      p1 = n + 1 < b.N ? d + 1 : nullptr;
    } else if constexpr (EPI == kSplit) {
      const MmSplit& e = p.split;
      if (n < e.n_t) p0 = static_cast<T*>(e.t) + (size_t)m * e.ldt + n;
      else p0 = e.f + (size_t)m * e.ldf + (n - e.n_t);
    } else if constexpr (EPI == kGlu) {
      p0 = static_cast<T*>(p.split.t) + (size_t)m * p.split.ldt + (n >> 1);
    } else if constexpr (EPI == kSoftplus) {
      p0 = p.a.C + (size_t)m * p.a.ldc + n;
      cs = p.bias[n];
      sn = p.bias[n + 1];
    } else if constexpr (EPI == kHeads) {
      const MmHeads& e = p.heads;
      const int row = e.rows ? e.rows[m] : m;
      T* d = static_cast<T*>(e.C) + (size_t)row * e.ldc + (size_t)blockIdx.z * e.c_head + n;
      p0 = d;
      p1 = n + 1 < b.N ? d + 1 : nullptr;
    } else if constexpr (EPI == kLatent) {
      const MmLatent& e = p.lat;
      const bool turned = !c.part && c.d >= e.D;
      T* q = static_cast<T*>(e.q) + ((size_t)m * e.H + c.head) * e.ldq + c.d;
      float* down = e.down + (size_t)m * e.ldd + c.d;
      p0 = c.part ? static_cast<void*>(down) : static_cast<void*>(q);
      if (turned) {
        const float2 t = e.turn[(size_t)m * (e.rot >> 1) + ((c.d - e.D) >> 1)];
        cs = t.x;
        sn = t.y;
        p1 = static_cast<T*>(e.q_lat) + ((size_t)m * e.H + c.head) * e.ld_lat + e.lat_rot + (c.d - e.D);
      }
    } else if constexpr (EPI == kConv) {
      const MmConv& e = p.conv;
      if (n >= e.gate) {
        p0 = static_cast<T*>(e.z) + (size_t)m * e.ldz + (n - e.gate);
        return;
      }
      p0 = static_cast<T*>(e.x) + (size_t)m * e.ldx + n;
      T* h = static_cast<T*>(e.history) + (size_t)e.slot[m] * (e.taps - 1) * e.ldw + n;
      p1 = h;
      const int pos = e.pos[m];
#pragma unroll
      for (int k = 0; k < kMmConvTaps; ++k) {
        float2 w = {0.f, 0.f};
        if (k < e.taps) w = *reinterpret_cast<const float2*>(e.w + (size_t)k * e.ldw + n);
        past.w[0][k] = w.x;
        past.w[1][k] = w.y;
        if (k == kMmConvTaps - 1) break;
#pragma unroll
        for (int j = 0; j < 2; ++j)
          past.v[j][k] = k < e.taps - 1 && pos >= e.taps - 1 - k ? (float)h[(size_t)k * e.ldw + j] : 0.f;
      }
      past.bias[0] = e.bias[n];
      past.bias[1] = e.bias[n + 1];
    } else {
      const MmQkv& e = p.q;
      if (c.part == 0) {
        turn(e, m, c.d);
        p0 = static_cast<T*>(e.q) + ((size_t)m * e.H + c.head) * e.Dp + c.d;
        return;
      }
      if (r.entry < 0) return;
      if (c.part == 1) {
        turn(e, m, c.d);
        T* page = page_at<T>(e, e.k_pool, r.entry, c.head);
        if (page) p0 = page + (size_t)r.at * e.Dp + c.d;
        return;
      }
      const int slot = v_page_slot(r.at, Kind<T>::BF16);
      T* page = page_at<T>(e, e.v_pool, r.entry, c.head);
      if (page) p0 = page + (size_t)c.d * kPageTokens + slot;
      if (c.d + 1 < e.Dv) {
        if (page) p1 = page + (size_t)(c.d + 1) * kPageTokens + slot;
      } else if (c.head + 1 < e.G) {  // (not the second half of the last pair)
        page = page_at<T>(e, e.v_pool, r.entry, c.head + 1);
        if (page) p1 = page + slot;
      }
    }
  }

  __device__ __forceinline__ void put(const KernelArgs& p, const Block<T>& b, int n, float v0,
                                      float v1) const {
    if constexpr (EPI == kStore || EPI == kGroupOut) {
      if constexpr (EPI == kGroupOut) {
        v0 *= cs;
        v1 *= cs;
      } else if (p.a.softcap > 0.f) {
        v0 = p.a.softcap * tanhf(v0 / p.a.softcap);
        v1 = p.a.softcap * tanhf(v1 / p.a.softcap);
      }
      if (p0) *static_cast<float*>(p0) = v0;
      if (p1) *static_cast<float*>(p1) = v1;
    } else if constexpr (EPI == kGroupIn || EPI == kGlu) {
      if (p0) *static_cast<T*>(p0) = (T)glu(v0, v1, b.glu);
    } else if constexpr (EPI == kSplit) {
      if (!p0) return;
      if (n < p.split.n_t) put_pair(static_cast<T*>(p0), v0, v1);
      else put_pair(static_cast<float*>(p0), v0, v1);
    } else if constexpr (EPI == kSoftplus) {
      if (p0) put_pair(static_cast<float*>(p0), softplus(v0 + cs), softplus(v1 + sn));
    } else if constexpr (EPI == kHeads) {
      if (p0) *static_cast<T*>(p0) = (T)v0;
      if (p1) *static_cast<T*>(p1) = (T)v1;
    } else if constexpr (EPI == kLatent) {
      if (!p0) return;
      if (n >= p.lat.H * (p.lat.D + p.lat.rot)) {
        put_pair(static_cast<float*>(p0), v0, v1);
      } else {
        const float t0 = v0 * cs - v1 * sn, t1 = v1 * cs + v0 * sn;
        put_pair(static_cast<T*>(p0), t0, t1);
        if (p1) put_pair(static_cast<T*>(p1), t0, t1);
      }
    } else if constexpr (EPI == kConv) {
      if (!p0) return;
      if (!p1) {
        put_pair(static_cast<T*>(p0), v0, v1);
        return;
      }
      const MmConv& e = p.conv;
      const float now[2] = {(float)(T)v0, (float)(T)v1};
      float o[2];
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        float s = past.bias[j];
#pragma unroll
        for (int k = 0; k < kMmConvTaps; ++k) {
          if (k < e.taps - 1 && k < kMmConvTaps - 1) s += past.v[j][k] * past.w[j][k];
          if (k == e.taps - 1) s += now[j] * past.w[j][k];
        }
        o[j] = s / (1.f + expf(-s));
      }
      put_pair(static_cast<T*>(p0), o[0], o[1]);
      T* h = static_cast<T*>(p1);
#pragma unroll
      for (int k = 0; k < kMmConvTaps - 1; ++k) {
        if (k + 2 < e.taps && k + 2 < kMmConvTaps)
          put_pair(h + (size_t)k * e.ldw, past.v[0][k + 1], past.v[1][k + 1]);
        else if (k + 2 == e.taps)
          put_pair(h + (size_t)k * e.ldw, now[0], now[1]);
      }
    } else {
      if (n < (p.q.H + p.q.G) * p.q.D) {
        if (p0) put_pair(static_cast<T*>(p0), v0 * cs - v1 * sn, v1 * cs + v0 * sn);
      } else {
        if (p0) *static_cast<T*>(p0) = (T)v0;
        if (p1) *static_cast<T*>(p1) = (T)v1;
      }
    }
  }

 private:
  __device__ __forceinline__ void turn(const MmQkv& e, int m, int d) {
    if (d >= e.rot) return;
    const float2 t = e.turn[(size_t)m * (e.rot >> 1) + (d >> 1)];
    cs = t.x;
    sn = t.y;
  }
};

// A column of 16 x 16 tiles of finished sums (tile i's rows m0 + 16 i .., columns
// n0 ..) -> the epilogue, a column pair per lane.  Every lane of the wave takes
// part; rows are what row_of() found for this lane.
template <typename T, int EPI, int MT>
struct TileRows {
  RowOf<EPI> r[MT][2];
  __device__ __forceinline__ TileRows(const KernelArgs& p, const Block<T>& b, int m0) {
    const int lane = lane_id(), first = m0 + 4 * (lane >> 4) + (lane & 1 ? 2 : 0);
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int k = 0; k < 2; ++k) r[i][k] = RowOf<EPI>(p, b, first + 16 * i + k);
  }
};

template <typename T, int EPI, int MT, int NT>
__device__ __forceinline__ void emit_column(const KernelArgs& p, const Block<T>& b,
                                            const TileRows<T, EPI, MT>& rows, const f32x4 (&acc)[MT][NT],
                                            int j, int m0, int n0) {
  const int lane = lane_id();
  const bool odd = lane & 1;
  if constexpr (RowOf<EPI>::PAGED) {
    // values lie token by token: a lane's four rows of its own column are one
    // store where they are tokens 4 t .. 4 t + 3 of a sequence
    if (n0 >= (p.q.H + p.q.G) * p.q.D) {
      typedef T quad_t __attribute__((ext_vector_type(4)));
      const ColOf<EPI> col(p, b, n0 + (lane & 15));
#pragma unroll
      for (int i = 0; i < MT; ++i) {
        const int m = m0 + 16 * i + 4 * (lane >> 4);
        const RowOf<EPI> lo(p, b, m), hi(p, b, m + 3);
        if (lo.m < 0 || col.n < 0) continue;
        if (hi.m >= 0 && (lo.at & 3) == 0 && hi.pos == lo.pos + 3 && hi.entry == lo.entry) {
          if (lo.entry < 0) continue;
          T* page = page_at<T>(p.q, p.q.v_pool, lo.entry, col.head);
          if (!page) continue;
          quad_t v;
#pragma unroll
          for (int r = 0; r < 4; ++r) v[r] = (T)acc[i][j][r];
          *reinterpret_cast<quad_t*>(page + (size_t)col.d * kPageTokens +
                                     v_page_slot(lo.at, Kind<T>::BF16)) = v;
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const RowOf<EPI> row(p, b, m + r);
            if (row.m < 0 || row.entry < 0) continue;
            T* page = page_at<T>(p.q, p.q.v_pool, row.entry, col.head);
            if (page)
              page[(size_t)col.d * kPageTokens + v_page_slot(row.at, Kind<T>::BF16)] = (T)acc[i][j][r];
          }
        }
      }
      return;
    }
  }
  const int n = n0 + (lane & 14);
  const ColOf<EPI> col(p, b, n);
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const f32x4 c = acc[i][j];
    f32x4 o;
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] = mov_dpp<0xB1>(c[r]);  // the neighbouring column
#pragma unroll
    for (int r = 0; r < 2; ++r) {
      Target<T, EPI> t;
      t.find(p, b, rows.r[i][r], col);
      t.put(p, b, n, odd ? o[2 + r] : c[r], odd ? c[2 + r] : o[r]);
    }
  }
}

// Decode rows (and short grouped tiles): a block owns 16 MT rows x 16 NT columns
// and its WK waves split K, adding through LDS in a fixed order.
template <typename T, int EPI, int MT, int NT, int WK>
__global__ __launch_bounds__(64 * WK, MT * NT == 1 ? 4 : 2) void mm_stream_kernel(KernelArgs p) {
  if constexpr (EPI == kGroupIn || EPI == kGroupOut)
    if ((int)blockIdx.y >= *p.g.n_tiles) return;
  constexpr int U = MT * NT >= 4 ? 2 : 4;  // k-steps per load batch
  const int lane = lane_id();
  const int w = wave_id_uniform();
  const Block<T> b = block_of<T, EPI>(p, 16 * MT);
  const int ntiles = (b.N + 15) >> 4;
  const int nt0 = (int)blockIdx.x * NT;
  if (nt0 >= ntiles) return;  // (groups differ in width)

  const char* ap[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) ap[i] = a_lane<T, EPI>(p, b, b.m0 + 16 * i + (lane & 15));
  const char* bp[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j)
    bp[j] = b.W + (size_t)min(nt0 + j, ntiles - 1) * b.KS * 1024 + lane * 16;

  f32x4 acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};

  // Neighbouring blocks start at different k ranges, so they do not all pull
  // the same A lines at once.
  const int wr = (w + (int)blockIdx.x) % WK;
  const int ks0 = wr * b.KS / WK, ks1 = (wr + 1) * b.KS / WK;
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
  // thread t finishes column pairs t, t + THREADS, ...: 8 pairs a row, 128 a tile
  constexpr int PAIRS = MT * NT * 128, THREADS = 64 * WK, EPT = (PAIRS + THREADS - 1) / THREADS;
  __shared__ float red[WK][MT * NT][4][64];
  Target<T, EPI> target[EPT];
  Batch x, y;
  if (ks0 < ks1) load(x, ks0);
#pragma unroll
  for (int e = 0; e < EPT; ++e) {
    const int pr = threadIdx.x + e * THREADS, t = pr >> 7;
    if (pr < PAIRS)
      target[e].find(p, b, RowOf<EPI>(p, b, b.m0 + 16 * (t / NT) + ((pr >> 3) & 15)),
                     ColOf<EPI>(p, b, (nt0 + t % NT) * 16 + (pr & 7) * 2));
  }
  if (ks0 < ks1) {
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

#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) red[wr][i * NT + j][r][lane] = acc[i][j][r];
  __syncthreads();
#pragma unroll
  for (int e = 0; e < EPT; ++e) {
    const int pr = threadIdx.x + e * THREADS;
    if (pr >= PAIRS) break;
    const int t = pr >> 7, row = (pr >> 3) & 15, col = (pr & 7) * 2;
    float2 s = {0.f, 0.f};
#pragma unroll
    for (int k = 0; k < WK; ++k) {
      const float2 v = *reinterpret_cast<const float2*>(&red[k][t][row & 3][(row >> 2) * 16 + col]);
      s.x += v.x;
      s.y += v.y;
    }
    target[e].put(p, b, (nt0 + t % NT) * 16 + col, s.x, s.y);
  }
}

// Prompt rows: a block of 16 MB rows x 128 columns, 4 waves as WM x (4 / WM).
// Fragments go from memory straight into LDS (A gathered row by row, W linear),
// two k-steps per stage, the next stage in flight while one is multiplied.
template <typename T, int EPI, int MB, int WM>
__global__ __launch_bounds__(256, 2) void mm_block_kernel(KernelArgs p) {
  if constexpr (EPI == kGroupIn || EPI == kGroupOut)
    if ((int)blockIdx.y >= *p.g.n_tiles) return;
  constexpr int NB = 8, WN = 4 / WM, MT = MB / WM, NT = NB / WN;
  constexpr int AW = MB / 4, BW = NB / 4;  // row / column tiles a wave loads
  __shared__ u32x4 sa[2][2][MB][64];       // [stage][k-step][tile][lane]
  __shared__ u32x4 sb[2][2][NB][64];
  const int lane = lane_id();
  const int w = wave_id_uniform();
  const Block<T> b = block_of<T, EPI>(p, 16 * MB);
  const int ntiles = (b.N + 15) >> 4;
  const int nt0 = (int)blockIdx.x * NB;
  if (nt0 >= ntiles) return;

  const char* ap[AW];
#pragma unroll
  for (int i = 0; i < AW; ++i)
    ap[i] = a_lane<T, EPI>(p, b, b.m0 + 16 * (w * AW + i) + (lane & 15));
  const char* bp[BW];
#pragma unroll
  for (int j = 0; j < BW; ++j)
    bp[j] = b.W + (size_t)min(nt0 + w * BW + j, ntiles - 1) * b.KS * 1024 + lane * 16;
  auto issue = [&](int st, int ks) {
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      if (ks + u >= b.KS) break;
#pragma unroll
      for (int i = 0; i < AW; ++i) load_to_lds(ap[i] + (size_t)(ks + u) * 64, sa[st][u][w * AW + i]);
#pragma unroll
      for (int j = 0; j < BW; ++j)
        load_to_lds(bp[j] + (size_t)(ks + u) * 1024, sb[st][u][w * BW + j]);
    }
  };
  const int wm = w / WN, wn = w % WN;
  f32x4 acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  auto mul = [&](int st, int u) {
    u32x4 a[MT], c[NT];
#pragma unroll
    for (int i = 0; i < MT; ++i) a[i] = sa[st][u][wm * MT + i][lane];
#pragma unroll
    for (int j = 0; j < NT; ++j) c[j] = sb[st][u][wn * NT + j][lane];
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < NT; ++j) acc[i][j] = Kind<T>::mma(a[i], c[j], acc[i][j]);
  };
  issue(0, 0);
  int st = 0;
  for (int ks = 0; ks < b.KS; ks += 2, st ^= 1) {
    wait_lds_loads();
    __syncthreads();  // stage st has landed, stage st ^ 1 is read out
    if (ks + 2 < b.KS) issue(st ^ 1, ks + 2);
    mul(st, 0);
    if (ks + 1 < b.KS) mul(st, 1);
  }
  const int m0 = b.m0 + 16 * wm * MT;
  const TileRows<T, EPI, MT> rows(p, b, m0);
#pragma unroll
  for (int j = 0; j < NT; ++j) emit_column(p, b, rows, acc, j, m0, (nt0 + wn * NT + j) * 16);
}

template <int EPI>
int heads_of(const KernelArgs& p) {
  return EPI == kHeads ? p.heads.heads : 1;
}

template <typename T, int EPI, int MT, int NT, int WK = 8>
hipError_t stream(const KernelArgs& p, int row_blocks, int N, hipStream_t st) {
  const dim3 grid(((N + 15) / 16 + NT - 1) / NT, row_blocks, heads_of<EPI>(p));
  hipLaunchKernelGGL((mm_stream_kernel<T, EPI, MT, NT, WK>), grid, dim3(64 * WK), 0, st, p);
  return hipGetLastError();
}

template <typename T, int EPI, int MB, int WM>
hipError_t blocks(const KernelArgs& p, int row_blocks, int N, hipStream_t st) {
  const dim3 grid((N + 127) / 128, row_blocks, heads_of<EPI>(p));
  hipLaunchKernelGGL((mm_block_kernel<T, EPI, MB, WM>), grid, dim3(256), 0, st, p);
  return hipGetLastError();
}

template <typename T, int EPI>
hipError_t launch(const KernelArgs& p, hipStream_t st) {
  const int M = p.a.M, N = p.a.N;
  const int ntiles = (N + 15) / 16;
  if (M <= 16) return stream<T, EPI, 1, 1>(p, 1, N, st);
  if (M <= 64) {
    // The form with the fewest rounds of workgroups over the chip, a round priced
    // by its column tiles and the rows it reads: 64 x 12288 x 2048 17.4 us as 4 x 3
    // tiles (one round) against 25.9 as 4 x 2, 64 x 8192 14.5 as 4 x 2 against 16.1.
    struct Form {
      int mt, nt;
      float rows;
      hipError_t (*go)(const KernelArgs&, int, int, hipStream_t);
    };
    static constexpr Form forms[] = {{1, 1, 0.5f, stream<T, EPI, 1, 1>}, {1, 2, 0.5f, stream<T, EPI, 1, 2>},
                                     {2, 2, 1.5f, stream<T, EPI, 2, 2>}, {2, 3, 1.5f, stream<T, EPI, 2, 3>},
                                     {4, 2, 3.f, stream<T, EPI, 4, 2>},  {4, 3, 3.f, stream<T, EPI, 4, 3>}};
    const Form* best = nullptr;
    int row_blocks = 0;
    float least = 0.f;
    for (const Form& f : forms) {
      const int rb = (M + 16 * f.mt - 1) / (16 * f.mt);
      const int groups = (ntiles + f.nt - 1) / f.nt * rb * heads_of<EPI>(p);
      const float cost = (float)((groups + 255) / 256) * ((float)f.nt + f.rows);
      if (best && cost >= least) continue;
      best = &f;
      least = cost;
      row_blocks = rb;
    }
    return best->go(p, row_blocks, N, st);
  }
  if constexpr (EPI == kSplit) {
    // narrow products: all columns in two blocks, so a row is read twice
    if (ntiles <= 10 && (M + 31) / 32 * 2 < 1024) return stream<T, EPI, 2, 5>(p, (M + 31) / 32, N, st);
  }
  // prompt rows: blocks once there are enough of them, else 32-row streams
  const int n128 = (N + 127) / 128 * heads_of<EPI>(p);
  if ((M + 127) / 128 * n128 >= 256) return blocks<T, EPI, 8, 2>(p, (M + 127) / 128, N, st);
  if ((M + 63) / 64 * n128 >= 128) return blocks<T, EPI, 4, 1>(p, (M + 63) / 64, N, st);
  return stream<T, EPI, 2, 1>(p, (M + 31) / 32, N, st);
}

template <typename T, int EPI>
hipError_t launch_grouped(const MmGrouped& g, int w_nt, hipStream_t st) {
  KernelArgs p{};
  p.g = g;
  p.a.w_nt = w_nt;
  if (g.tile_rows == 128) return blocks<T, EPI, 8, 2>(p, g.max_tiles, g.max_n, st);
  if (g.tile_rows == 64) return blocks<T, EPI, 4, 1>(p, g.max_tiles, g.max_n, st);
  // few k-steps per wave are not worth eight of them
  return g.min_ks >= 16 ? stream<T, EPI, 1, 1>(p, g.max_tiles, g.max_n, st)
                        : stream<T, EPI, 1, 1, 4>(p, g.max_tiles, g.max_n, st);
}

}  // namespace
}  // namespace llm
