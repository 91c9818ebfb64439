// Paged grouped-query attention on MFMA for a mixed batch.
//
// A workgroup takes one row tile (the group's heads of consecutive tokens,
// flattened as rows) of one key/value head.  Per block of KEYS keys (32 in
// bf16, 16 in fp32):
//   S^T[keys][rows] = K . Q^T,     O^T[Dv][rows] += V^T . P^T
// Keys are the MFMA row index of S^T, so a lane holds 4 keys per tile of ONE
// row and its P values are already the B operand of the second product; the V
// page is kept transposed ([d][token]) in exactly the key order of that
// operand, so K, V and Q fragments all come from memory as 16 bytes per lane.
//
//   few rows   gqa_split_kernel: a tile of 16 rows; the 4 waves take the key
//              blocks in turn, fragments straight to registers, one block
//              ahead, and are merged through LDS.  A decoded token of a group of
//              8 heads is 8 rows: its K and V are read once for the group.
//   many rows  gqa_rows_kernel: every wave owns 16 MT rows; the workgroup loads
//              each page into LDS once, in fragment order, one stage ahead.
//
// The probabilities stay fp32 up to the product: in bf16 they enter it as
// hi + lo halves.  Scores, maxima and sums are fp32 in log2 units.  A sink is
// one more term of the denominator, added where the row is finished.
#include "common.hpp"
#include "mm.hpp"
#include "paged_gqa.hpp"

#include <algorithm>

namespace llm {
namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
constexpr int kWaves = 4;

template <typename T>
struct Att;
template <>
struct Att<__bf16> {
  static constexpr int KSTEP = 32, KT = 2;  // dims per product step, 16-key tiles per block
};
template <>
struct Att<float> {
  static constexpr int KSTEP = 16, KT = 1;
};

template <typename T>
__device__ __forceinline__ f32x4 dot_step(u32x4 a, u32x4 b, f32x4 c) {
  if constexpr (sizeof(T) == 2) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a),
                                                   __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
  } else {
    const f32x4 x = __builtin_bit_cast(f32x4, a), y = __builtin_bit_cast(f32x4, b);
#pragma unroll
    for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[j], y[j], c, 0, 0, 0);
    return c;
  }
}

// The rows one wave works on.  CK, CV: largest Dp and Dvp of the class.
template <typename T, int CK, int CV, int MT>
struct Rows {
  static constexpr int KSTEP = Att<T>::KSTEP, KT = Att<T>::KT, KEYS = 16 * KT;
  static constexpr int NK = CK / KSTEP, ND = CV / 16;
  u32x4 q[MT][NK];
  f32x4 o[ND][MT];
  float m[MT], l[MT];
  int pos[MT];  // the row's position (-1: no row)

  // rows first .. first + 16 MT - 1 of the item's tile, of which `rows` exist
  __device__ __forceinline__ void init(const GqaArgs& a, const GqaItem& it, int kvh, int first,
                                       int rows) {
    const int g = lane_id() >> 4, c = lane_id() & 15, R = a.H / a.G;
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      const int rr = first + 16 * t + c;
      const bool ok = rr < rows;
      const int row = it.row0 + rr, tok = row / R;
      pos[t] = ok ? it.p0 + tok : -1;
      const T* qp = static_cast<const T*>(a.q) +
                    ((size_t)(it.tok0 + tok) * a.H + kvh * R + (row - tok * R)) * a.Dp;
#pragma unroll
      for (int k = 0; k < NK; ++k) {
        const int d = k * KSTEP + g * (KSTEP / 4);
        q[t][k] = ok && d < a.Dp ? *reinterpret_cast<const u32x4*>(qp + d) : u32x4{0u, 0u, 0u, 0u};
      }
      m[t] = kNegSentinel;
      l[t] = 0.f;
#pragma unroll
      for (int n = 0; n < ND; ++n) o[n][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
  }

  // One block of KEYS keys from position key0: kf(u, k) and vf(n) give its
  // fragments; mask: some row ends inside it.
  template <typename KF, typename VF>
  __device__ __forceinline__ void attend(const GqaArgs& a, int key0, bool mask, float scale2, KF kf,
                                         VF vf) {
    const int g = lane_id() >> 4;
    f32x4 s[MT][KT];
#pragma unroll
    for (int u = 0; u < KT; ++u) {
#pragma unroll
      for (int t = 0; t < MT; ++t) s[t][u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < NK; ++k)
        if (k * KSTEP < a.Dp) {
          const u32x4 x = kf(u, k);
#pragma unroll
          for (int t = 0; t < MT; ++t) s[t][u] = dot_step<T>(x, q[t][k], s[t][u]);
        }
    }
    u32x4 hi[MT], lo[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      float mloc = kNegSentinel;
#pragma unroll
      for (int u = 0; u < KT; ++u) {
        s[t][u] *= scale2;
        if (mask) {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (key0 + 16 * u + 4 * g + r > pos[t]) s[t][u][r] = 2.f * kNegSentinel;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) mloc = fmaxf(mloc, s[t][u][r]);
      }
      mloc = fmaxf(mloc, __shfl_xor(mloc, 16, 64));
      mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
      if (__any(mloc > m[t])) {
        const float mnew = fmaxf(m[t], mloc);  // >= the sentinel: masked scores stay far below
        const float corr = __builtin_amdgcn_exp2f(m[t] - mnew);
        l[t] *= corr;
#pragma unroll
        for (int n = 0; n < ND; ++n)
          if (16 * n < a.Dvp) o[n][t] *= corr;
        m[t] = mnew;
      }
#pragma unroll
      for (int u = 0; u < KT; ++u)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          s[t][u][r] = __builtin_amdgcn_exp2f(s[t][u][r] - m[t]);
          l[t] += s[t][u][r];
        }
      if constexpr (sizeof(T) == 2) {
        bf16x8 h, w;
#pragma unroll
        for (int u = 0; u < KT; ++u)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            h[4 * u + r] = (__bf16)s[t][u][r];
            w[4 * u + r] = (__bf16)(s[t][u][r] - (float)h[4 * u + r]);
          }
        hi[t] = __builtin_bit_cast(u32x4, h);
        lo[t] = __builtin_bit_cast(u32x4, w);
      } else {
        hi[t] = __builtin_bit_cast(u32x4, s[t][0]);
      }
    }
#pragma unroll
    for (int n = 0; n < ND; ++n)
      if (16 * n < a.Dvp) {
        const u32x4 x = vf(n);
#pragma unroll
        for (int t = 0; t < MT; ++t) {
          o[n][t] = dot_step<T>(x, hi[t], o[n][t]);
          if constexpr (sizeof(T) == 2) o[n][t] = dot_step<T>(x, lo[t], o[n][t]);
        }
      }
  }

  // the 4 lanes of a row hold sums over their own keys
  __device__ __forceinline__ void join_lanes() {
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      l[t] += __shfl_xor(l[t], 16, 64);
      l[t] += __shfl_xor(l[t], 32, 64);
    }
  }

  // finished row -> out, or a split's state -> the part buffers
  __device__ __forceinline__ void write(const GqaArgs& a, const GqaItem& it, int kvh, int first,
                                        int rows, int tile_rows) {
    const int g = lane_id() >> 4, c = lane_id() & 15, R = a.H / a.G;
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      const int rr = first + 16 * t + c;
      if (rr >= rows) continue;
      const int row = it.row0 + rr;
      if (it.part >= 0) {
        const size_t base = ((size_t)it.part * a.G + kvh) * tile_rows + rr;
        float* dst = a.part_o + base * ((a.Dv + 15) / 16 * 16);
#pragma unroll
        for (int n = 0; n < ND; ++n)
          if (16 * n < a.Dv) *reinterpret_cast<f32x4*>(dst + 16 * n + 4 * g) = o[n][t];
        if (g == 0) *reinterpret_cast<float2*>(a.part_ml + base * 2) = float2{m[t], l[t]};
        continue;
      }
      const int tok = row / R, head = kvh * R + (row - tok * R);
      float den = l[t], f = 1.f;
      if (a.sink) {
        const float s2 = a.sink[head] * kLog2e, m2 = fmaxf(m[t], s2);
        f = __builtin_amdgcn_exp2f(m[t] - m2);
        den = l[t] * f + __builtin_amdgcn_exp2f(s2 - m2);
      }
      f /= den;
      T* dst = static_cast<T*>(a.out) + (size_t)(it.tok0 + tok) * a.ldo +
             (size_t)head * (a.ldh ? a.ldh : a.Dv);
#pragma unroll
      for (int n = 0; n < ND; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (16 * n + 4 * g + r < a.Dv) dst[16 * n + 4 * g + r] = (T)(o[n][t][r] * f);
    }
  }
};

__device__ __forceinline__ int page_at(const GqaArgs& a, const int32_t* pt, int tile, bool ok) {
  int p = ok && tile < a.max_tiles ? pt[tile] : -1;
  p = p < a.num_pages ? p : -1;
  return __builtin_amdgcn_readfirstlane(p);
}

template <typename T, int C>
__global__ __launch_bounds__(64 * kWaves, C < 256 ? 2 : 1) void gqa_split_kernel(GqaArgs a) {
  using RowsT = Rows<T, C, C, 1>;
  constexpr int KSTEP = RowsT::KSTEP, KT = RowsT::KT, KEYS = RowsT::KEYS;
  constexpr int NK = RowsT::NK, ND = RowsT::ND;
  constexpr int BPP = kPageTokens / KEYS;
  constexpr bool DOUBLE = C < 256;
  __shared__ float ml[kWaves][16][2];
  __shared__ f32x4 ox[2][ND][64];

  const int lane = lane_id(), w = wave_id_uniform();
  const int g = lane >> 4, c = lane & 15;
  const GqaItem it = a.items[blockIdx.x];
  const int kvh = blockIdx.y, R = a.H / a.G;
  const int32_t* pt = a.table + ((size_t)it.slot * a.G + kvh) * a.max_tiles;
  const int rows = min(16, it.nrows - it.row0);
  const int first_pos = it.p0 + it.row0 / R;
  const int last_pos = it.p0 + (it.row0 + rows - 1) / R;
  // key blocks of the item, taken in turn by the waves
  const int b0 = it.page0 * BPP, b1 = min(it.page1 * BPP, last_pos / KEYS + 1);

  struct Block {
    u32x4 k[KT][NK], v[ND];
  };
  auto page_of = [&](int b) { return page_at(a, pt, b / BPP, b < b1); };
  auto load = [&](Block& x, int b, int page) {
    if (page < 0) return;
    const int off = b % BPP * KEYS;
    const T* kp = reinterpret_cast<const T*>(static_cast<const char*>(a.k_pool) +
                                             (size_t)page * a.page_stride) +
                  (size_t)(off + c) * a.Dp;
    const T* vp = reinterpret_cast<const T*>(static_cast<const char*>(a.v_pool) +
                                             (size_t)page * a.page_stride) +
                  off + g * (KEYS / 4);
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      const int d = k * KSTEP + g * (KSTEP / 4);
      if (k * KSTEP < a.Dp) {
#pragma unroll
        for (int t = 0; t < KT; ++t)
          x.k[t][k] = d < a.Dp ? *reinterpret_cast<const u32x4*>(kp + (size_t)16 * t * a.Dp + d)
                               : u32x4{0u, 0u, 0u, 0u};
      }
    }
#pragma unroll
    for (int n = 0; n < ND; ++n) {
      if (16 * n < a.Dvp)
        x.v[n] = 16 * n + c < a.Dvp
                     ? *reinterpret_cast<const u32x4*>(vp + (size_t)(16 * n + c) * kPageTokens)
                     : u32x4{0u, 0u, 0u, 0u};
    }
  };
  const float scale2 = a.scale * kLog2e;
  RowsT row;
  Block x, y;
  int b = b0 + w;
  int page = page_of(b), next = page_of(b + kWaves);
  load(x, b, page);
  row.init(a, it, kvh, 0, rows);
  auto work = [&](const Block& blk, int bb) {
    row.attend(
        a, bb * KEYS, bb * KEYS + KEYS - 1 > first_pos, scale2,
        [&](int u, int k) { return blk.k[u][k]; }, [&](int d) { return blk.v[d]; });
  };
  if constexpr (DOUBLE) {
    while (b < b1) {
      const int after = page_of(b + 2 * kWaves);
      load(y, b + kWaves, next);
      if (page >= 0) work(x, b);
      b += kWaves;
      if (b >= b1) break;
      const int after2 = page_of(b + 2 * kWaves);
      load(x, b + kWaves, after);
      if (next >= 0) work(y, b);
      b += kWaves;
      page = after;
      next = after2;
    }
  } else {
    while (b < b1) {
      if (page >= 0) work(x, b);
      b += kWaves;
      const int after = page_of(b + kWaves);
      load(x, b, next);
      page = next;
      next = after;
    }
  }

  row.join_lanes();
  if (g == 0) {
    ml[w][c][0] = row.m[0];
    ml[w][c][1] = row.l[0];
  }
  __syncthreads();
  float M = kNegSentinel, L = 0.f;
#pragma unroll
  for (int i = 0; i < kWaves; ++i) M = fmaxf(M, ml[i][c][0]);
#pragma unroll
  for (int i = 0; i < kWaves; ++i) L += ml[i][c][1] * __builtin_amdgcn_exp2f(ml[i][c][0] - M);
  const float f = __builtin_amdgcn_exp2f(row.m[0] - M);
#pragma unroll
  for (int n = 0; n < ND; ++n) row.o[n][0] *= f;
  // waves 2, 3 -> 0, 1, then 1 -> 0
#pragma unroll
  for (int half = kWaves / 2; half >= 1; half >>= 1) {
    if (w >= half && w < 2 * half) {
#pragma unroll
      for (int n = 0; n < ND; ++n) ox[w - half][n][lane] = row.o[n][0];
    }
    __syncthreads();
    if (w < half) {
#pragma unroll
      for (int n = 0; n < ND; ++n) row.o[n][0] += ox[w][n][lane];
    }
    if (half > 1) __syncthreads();
  }
  if (w != 0) return;
  row.m[0] = M;
  row.l[0] = L;
  row.write(a, it, kvh, 0, rows, 16);
}

// Keys a stage of the row kernel holds: 32 KiB of K and V fragments at most.
template <typename T, int CK, int CV>
constexpr int stage_keys() {
  int n = kPageTokens;
  while (n * (CK + CV) * (int)sizeof(T) > 32768) n /= 2;
  return n;
}

template <typename T, int CK, int CV, int MT>
__global__ __launch_bounds__(64 * kWaves, 2) void gqa_rows_kernel(GqaArgs a) {
  using RowsT = Rows<T, CK, CV, MT>;
  constexpr int KSTEP = RowsT::KSTEP, KT = RowsT::KT, KEYS = RowsT::KEYS;
  constexpr int NK = RowsT::NK, ND = RowsT::ND;
  constexpr int SK = stage_keys<T, CK, CV>(), SPP = kPageTokens / SK;
  constexpr int FK = SK / 16 * NK, FV = SK / KEYS * ND, FW = (FK + FV) / kWaves;
  constexpr int TR = 16 * MT * kWaves;
  static_assert(SK % KEYS == 0 && (FK + FV) % kWaves == 0, "whole fragments per wave");
  __shared__ u32x4 lds[2][FK + FV][64];

  const int lane = lane_id(), w = wave_id_uniform();
  const int g = lane >> 4, c = lane & 15;
  const GqaItem it = a.items[blockIdx.x];
  const int kvh = blockIdx.y, R = a.H / a.G;
  const int32_t* pt = a.table + ((size_t)it.slot * a.G + kvh) * a.max_tiles;
  const int rows = min(TR, it.nrows - it.row0);
  const int wrow = 16 * MT * w;  // this wave's first row of the tile
  const int first_pos = it.p0 + (it.row0 + wrow) / R;
  const int wave_last = wrow < rows ? it.p0 + (it.row0 + min(wrow + 16 * MT, rows) - 1) / R : -1;
  const int last_pos = it.p0 + (it.row0 + rows - 1) / R;
  const int s0 = it.page0 * SPP, s1 = min(it.page1 * SPP, last_pos / SK + 1);

  // fragment f of a stage: K (16-key tile f / NK, step f % NK), then V (block,
  // 16-dim tile).  Lanes past a row's end read its start: their products meet
  // zeros (K) or columns nobody writes (V).
  auto issue = [&](int buf, int s, int page) {
    if (page < 0) return;
    const int off = s % SPP * SK;
    const T* kp = reinterpret_cast<const T*>(static_cast<const char*>(a.k_pool) +
                                             (size_t)page * a.page_stride) +
                  (size_t)(off + c) * a.Dp;
    const T* vp = reinterpret_cast<const T*>(static_cast<const char*>(a.v_pool) +
                                             (size_t)page * a.page_stride) +
                  off + g * (KEYS / 4);
#pragma unroll
    for (int i = 0; i < FW; ++i) {
      const int f = w * FW + i;
      if (f < FK) {
        const int t = f / NK, k = f % NK, d = k * KSTEP + g * (KSTEP / 4);
        if (k * KSTEP < a.Dp)
          load_to_lds(kp + (size_t)16 * t * a.Dp + (d < a.Dp ? d : 0), lds[buf][f]);
      } else {
        const int kb = (f - FK) / ND, n = (f - FK) % ND;
        if (16 * n < a.Dvp)
          load_to_lds(vp + kb * KEYS + (size_t)min(16 * n + c, a.Dvp - 1) * kPageTokens,
                      lds[buf][f]);
      }
    }
  };
  const float scale2 = a.scale * kLog2e;
  RowsT row;
  auto page_of = [&](int s) { return page_at(a, pt, s / SPP, s < s1); };
  int page = page_of(s0), next = page_of(s0 + 1), buf = 0;
  issue(0, s0, page);
  row.init(a, it, kvh, wrow, rows);
  for (int s = s0; s < s1; ++s, buf ^= 1) {
    const int after = page_of(s + 2);
    wait_lds_loads();
    __syncthreads();  // stage s has landed, the other buffer is read out
    issue(buf ^ 1, s + 1, next);
    if (page >= 0) {
#pragma unroll
      for (int kb = 0; kb < SK / KEYS; ++kb) {
        const int key0 = s * SK + kb * KEYS;
        if (key0 > wave_last) break;
        row.attend(
            a, key0, key0 + KEYS - 1 > first_pos, scale2,
            [&](int u, int k) { return lds[buf][(kb * KT + u) * NK + k][lane]; },
            [&](int n) { return lds[buf][FK + kb * ND + n][lane]; });
      }
    }
    page = next;
    next = after;
  }
  row.join_lanes();
  row.write(a, it, kvh, wrow, rows, TR);
}

// One wave per row of a split tile.
template <typename T, int MAXD>
__global__ __launch_bounds__(256) void gqa_merge_kernel(GqaArgs a, int TR) {
  const GqaMerge it = a.merges[blockIdx.x];
  const int kvh = blockIdx.y, R = a.H / a.G, lane = lane_id();
  const int rows = min(TR, it.nrows - it.row0);
  const int pd = (a.Dv + 15) / 16 * 16;
  for (int rr = blockIdx.z * 4 + wave_id_uniform(); rr < rows; rr += 4 * (int)gridDim.z) {
    const int row = it.row0 + rr, tok = row / R, head = kvh * R + (row - tok * R);
    // lane s holds split s's state (nsplit <= 64)
    const bool mine = lane < it.nsplit;
    const size_t base = ((size_t)(it.part0 + (mine ? lane : 0)) * a.G + kvh) * TR + rr;
    const float2 st = *reinterpret_cast<const float2*>(a.part_ml + base * 2);
    float m = wave_max(mine ? st.x : kNegSentinel);
    const float s2 = a.sink ? a.sink[head] * kLog2e : kNegSentinel;
    m = fmaxf(m, s2);
    const float wgt = mine ? __builtin_amdgcn_exp2f(st.x - m) : 0.f;
    float den = wave_sum(mine ? st.y * wgt : 0.f);
    if (a.sink) den += __builtin_amdgcn_exp2f(s2 - m);
    float acc[MAXD / 64] = {};
    constexpr int U = 8;  // splits in flight
    for (int k = 0; k < it.nsplit; k += U) {
      float v[U][MAXD / 64];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int sp = min(k + u, it.nsplit - 1);
        const float* src = a.part_o + (((size_t)(it.part0 + sp) * a.G + kvh) * TR + rr) * pd;
#pragma unroll
        for (int j = 0; j < MAXD / 64; ++j)
          if (lane + 64 * j < a.Dv) v[u][j] = src[lane + 64 * j];
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const float ws = k + u < it.nsplit ? __shfl(wgt, k + u, 64) : 0.f;
#pragma unroll
        for (int j = 0; j < MAXD / 64; ++j)
          if (lane + 64 * j < a.Dv) acc[j] += ws * v[u][j];
      }
    }
    T* dst = static_cast<T*>(a.out) + (size_t)(it.tok0 + tok) * a.ldo +
             (size_t)head * (a.ldh ? a.ldh : a.Dv);
#pragma unroll
    for (int j = 0; j < MAXD / 64; ++j)
      if (lane + 64 * j < a.Dv) dst[lane + 64 * j] = (T)(acc[j] / den);
  }
}

template <typename T>
hipError_t merge(const GqaArgs& a, int tile_rows, hipStream_t st) {
  if (a.n_merges <= 0) return hipSuccess;
  const dim3 grid(a.n_merges, a.G, std::min(tile_rows / 4, 8));
  if (a.Dv <= kGqaMaxDim)
    hipLaunchKernelGGL((gqa_merge_kernel<T, kGqaMaxDim>), grid, dim3(256), 0, st, a, tile_rows);
  else
    hipLaunchKernelGGL((gqa_merge_kernel<T, kGqaMaxMergeDim>), grid, dim3(256), 0, st, a, tile_rows);
  return hipGetLastError();
}

template <typename T, int C>
hipError_t split(const GqaArgs& a, hipStream_t st) {
  hipLaunchKernelGGL((gqa_split_kernel<T, C>), dim3(a.n_items, a.G), dim3(64 * kWaves), 0, st, a);
  if (hipError_t e = hipGetLastError()) return e;
  return merge<T>(a, 16, st);
}

template <typename T, int CK, int CV, int MT>
hipError_t rows(const GqaArgs& a, hipStream_t st) {
  hipLaunchKernelGGL((gqa_rows_kernel<T, CK, CV, MT>), dim3(a.n_items, a.G), dim3(64 * kWaves), 0, st, a);
  if (hipError_t e = hipGetLastError()) return e;
  return merge<T>(a, 16 * MT * kWaves, st);
}

template <typename T>
hipError_t launch(const GqaArgs& a, int tile_rows, hipStream_t st) {
  const int d = std::max(a.Dp, a.Dvp);
  if (tile_rows == 16)
    return d <= 64 ? split<T, 64>(a, st) : d <= 128 ? split<T, 128>(a, st) : split<T, 256>(a, st);
  if constexpr (sizeof(T) == 2) {
    if (tile_rows == 128) {
      if (d <= 64) return rows<T, 64, 64, 2>(a, st);
      return d <= 128 ? rows<T, 128, 128, 2>(a, st) : rows<T, 192, 128, 2>(a, st);
    }
  }
  if (d <= 64) return rows<T, 64, 64, 1>(a, st);
  return d <= 128 ? rows<T, 128, 128, 1>(a, st) : rows<T, 256, 256, 1>(a, st);
}

}  // namespace

int gqa_tile_rows(int dtype, int Dp, int Dvp, int rows) {
  if (rows <= kGqaSmallRows) return 16;
  return dtype == LLM_BF16 && Dp <= 192 && Dvp <= 128 ? 128 : 64;
}

hipError_t gqa_merge(int dtype, const GqaArgs& a, int tile_rows, hipStream_t st) {
  return dtype == LLM_F32 ? merge<float>(a, tile_rows, st) : merge<__bf16>(a, tile_rows, st);
}

hipError_t gqa_attention(int dtype, const GqaArgs& a, int tile_rows, hipStream_t st) {
  if (a.n_items <= 0) return hipSuccess;
  return dtype == LLM_F32 ? launch<float>(a, tile_rows, st) : launch<__bf16>(a, tile_rows, st);
}

}  // namespace llm
