// Paged grouped-query attention on MFMA for a mixed batch.
//
// A workgroup takes one row tile (16 MT rows: the group's heads of consecutive
// tokens) and one key/value head; its 4 waves take the key blocks of the
// tile's pages in turn, each with its own online softmax, and are merged
// through LDS.  Per block of KEYS keys (32 in bf16, 16 in fp32):
//   S^T[keys][rows] = K . Q^T,     O^T[Dv][rows] += V^T . P^T
// Keys are the MFMA row index of S^T, so a lane holds 4 keys per tile of ONE
// row and its P values are already the B operand of the second product; the V
// page is kept transposed ([d][token]) in exactly the key order of that
// operand, so K, V and Q fragments all come straight from memory with 16-byte
// loads and nothing is staged.  A decoded token of a group of 8 heads is a tile
// of 8 rows: its K and V are read once for the whole group.
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

// C: largest Dp / Dvp of the class (64, 128 or 256)
template <typename T, int C, int MT>
__global__ __launch_bounds__(64 * kWaves, C < 256 ? 2 : 1) void gqa_kernel(GqaArgs a) {
  constexpr int KSTEP = Att<T>::KSTEP, KT = Att<T>::KT, KEYS = 16 * KT;
  constexpr int NK = C / KSTEP, ND = C / 16;
  constexpr int BPP = kPageTokens / KEYS;
  constexpr bool DOUBLE = C < 256;
  constexpr int TR = 16 * MT;
  __shared__ float ml[kWaves][TR][2];
  __shared__ f32x4 ox[2][MT * ND][64];

  const int lane = lane_id(), w = wave_id_uniform();
  const int g = lane >> 4, c = lane & 15;
  const GqaItem it = a.items[blockIdx.x];
  const int kvh = blockIdx.y;
  const int R = a.H / a.G;
  const int32_t* pt = a.table + ((size_t)it.slot * a.G + kvh) * a.max_tiles;

  const int rows = min(TR, it.nrows - it.row0);
  const int first_pos = it.p0 + it.row0 / R;
  const int last_pos = it.p0 + (it.row0 + rows - 1) / R;
  const int b0 = it.page0 * BPP, b1 = min(it.page1 * BPP, last_pos / KEYS + 1);

  int qpos[MT];
  u32x4 qf[MT][NK];
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int rr = 16 * t + c;
    const int row = it.row0 + rr;
    const bool ok = rr < rows;
    const int tok = row / R;
    qpos[t] = ok ? it.p0 + tok : -1;
    const T* qp = static_cast<const T*>(a.q) +
                  ((size_t)(it.tok0 + tok) * a.H + kvh * R + (row - tok * R)) * a.Dp;
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      const int d = k * KSTEP + g * (KSTEP / 4);
      qf[t][k] = ok && d < a.Dp ? *reinterpret_cast<const u32x4*>(qp + d) : u32x4{0u, 0u, 0u, 0u};
    }
  }

  f32x4 o[ND][MT];
#pragma unroll
  for (int n = 0; n < ND; ++n)
#pragma unroll
    for (int t = 0; t < MT; ++t) o[n][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  float mrun[MT], lrun[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) mrun[t] = kNegSentinel, lrun[t] = 0.f;

  struct Block {
    u32x4 k[KT][NK], v[ND];
  };
  auto page_of = [&](int b) {
    const int tile = b / BPP;
    int p = b < b1 && tile < a.max_tiles ? pt[tile] : -1;
    p = p < a.num_pages ? p : -1;
    return __builtin_amdgcn_readfirstlane(p);
  };
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
  auto work = [&](const Block& x, int b) {
    const bool mask = b * KEYS + KEYS - 1 > first_pos;
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      f32x4 s[KT];
      float mloc = kNegSentinel;
#pragma unroll
      for (int u = 0; u < KT; ++u) {
        s[u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < NK; ++k)
          if (k * KSTEP < a.Dp) s[u] = dot_step<T>(x.k[u][k], qf[t][k], s[u]);
        s[u] *= scale2;
        if (mask) {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (b * KEYS + 16 * u + 4 * g + r > qpos[t]) s[u][r] = 2.f * kNegSentinel;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) mloc = fmaxf(mloc, s[u][r]);
      }
      mloc = fmaxf(mloc, __shfl_xor(mloc, 16, 64));
      mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
      const float mnew = fmaxf(mrun[t], mloc);  // >= the sentinel: masked scores stay far below
      if (__any(mnew > mrun[t])) {
        const float corr = __builtin_amdgcn_exp2f(mrun[t] - mnew);
        lrun[t] *= corr;
#pragma unroll
        for (int n = 0; n < ND; ++n)
          if (16 * n < a.Dvp) o[n][t] *= corr;
        mrun[t] = mnew;
      }
      f32x4 p[KT];
#pragma unroll
      for (int u = 0; u < KT; ++u)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          p[u][r] = __builtin_amdgcn_exp2f(s[u][r] - mrun[t]);
          lrun[t] += p[u][r];
        }
      if constexpr (sizeof(T) == 2) {
        bf16x8 hi, lo;
#pragma unroll
        for (int u = 0; u < KT; ++u)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const __bf16 h = (__bf16)p[u][r];
            hi[4 * u + r] = h;
            lo[4 * u + r] = (__bf16)(p[u][r] - (float)h);
          }
#pragma unroll
        for (int n = 0; n < ND; ++n)
          if (16 * n < a.Dvp) {
            o[n][t] = dot_step<T>(x.v[n], __builtin_bit_cast(u32x4, hi), o[n][t]);
            o[n][t] = dot_step<T>(x.v[n], __builtin_bit_cast(u32x4, lo), o[n][t]);
          }
      } else {
#pragma unroll
        for (int n = 0; n < ND; ++n)
          if (16 * n < a.Dvp) o[n][t] = dot_step<T>(x.v[n], __builtin_bit_cast(u32x4, p[0]), o[n][t]);
      }
    }
  };

  {
    Block x, y;
    int b = b0 + w;
    int page = page_of(b), next = page_of(b + kWaves);
    if constexpr (DOUBLE) {
      load(x, b, page);
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
      for (; b < b1; b += kWaves) {
        load(x, b, page);
        const int after = page_of(b + 2 * kWaves);
        if (page >= 0) work(x, b);
        page = next;
        next = after;
      }
    }
  }

  // the 4 lanes of a row hold sums over their own keys
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    lrun[t] += __shfl_xor(lrun[t], 16, 64);
    lrun[t] += __shfl_xor(lrun[t], 32, 64);
    if (g == 0) {
      ml[w][16 * t + c][0] = mrun[t];
      ml[w][16 * t + c][1] = lrun[t];
    }
  }
  __syncthreads();
  float M[MT], L[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    M[t] = kNegSentinel;
#pragma unroll
    for (int i = 0; i < kWaves; ++i) M[t] = fmaxf(M[t], ml[i][16 * t + c][0]);
    L[t] = 0.f;
#pragma unroll
    for (int i = 0; i < kWaves; ++i)
      L[t] += ml[i][16 * t + c][1] * __builtin_amdgcn_exp2f(ml[i][16 * t + c][0] - M[t]);
    const float f = __builtin_amdgcn_exp2f(mrun[t] - M[t]);
#pragma unroll
    for (int n = 0; n < ND; ++n) o[n][t] *= f;
  }
  // waves 2, 3 -> 0, 1, then 1 -> 0
  for (int half = kWaves / 2; half >= 1; half >>= 1) {
    if (w >= half && w < 2 * half) {
#pragma unroll
      for (int n = 0; n < ND; ++n)
#pragma unroll
        for (int t = 0; t < MT; ++t) ox[w - half][n * MT + t][lane] = o[n][t];
    }
    __syncthreads();
    if (w < half) {
#pragma unroll
      for (int n = 0; n < ND; ++n)
#pragma unroll
        for (int t = 0; t < MT; ++t) o[n][t] += ox[w][n * MT + t][lane];
    }
    __syncthreads();
  }
  if (w != 0) return;

#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int rr = 16 * t + c;
    if (rr >= rows) continue;
    const int row = it.row0 + rr;
    if (it.part >= 0) {
      const size_t base = ((size_t)it.part * a.G + kvh) * TR + rr;
      float* dst = a.part_o + base * ((a.Dv + 15) / 16 * 16);
#pragma unroll
      for (int n = 0; n < ND; ++n)
        if (16 * n < a.Dv) *reinterpret_cast<f32x4*>(dst + 16 * n + 4 * g) = o[n][t];
      if (g == 0) *reinterpret_cast<float2*>(a.part_ml + base * 2) = float2{M[t], L[t]};
      continue;
    }
    const int tok = row / R, head = kvh * R + (row - tok * R);
    float den = L[t], f = 1.f;
    if (a.sink) {
      const float s2 = a.sink[head] * kLog2e, m2 = fmaxf(M[t], s2);
      f = __builtin_amdgcn_exp2f(M[t] - m2);
      den = L[t] * f + __builtin_amdgcn_exp2f(s2 - m2);
    }
    f /= den;
    T* dst = static_cast<T*>(a.out) + (size_t)(it.tok0 + tok) * a.ldo + (size_t)head * a.Dv;
#pragma unroll
    for (int n = 0; n < ND; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (16 * n + 4 * g + r < a.Dv) dst[16 * n + 4 * g + r] = (T)(o[n][t][r] * f);
  }
}

// One wave per row of a split tile.
template <typename T>
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
    float acc[kGqaMaxDim / 64] = {};
    for (int s = 0; s < it.nsplit; ++s) {
      const float ws = __shfl(wgt, s, 64);
      const float* src = a.part_o + (((size_t)(it.part0 + s) * a.G + kvh) * TR + rr) * pd;
#pragma unroll
      for (int j = 0; j < kGqaMaxDim / 64; ++j)
        if (lane + 64 * j < a.Dv) acc[j] += ws * src[lane + 64 * j];
    }
    T* dst = static_cast<T*>(a.out) + (size_t)(it.tok0 + tok) * a.ldo + (size_t)head * a.Dv;
#pragma unroll
    for (int j = 0; j < kGqaMaxDim / 64; ++j)
      if (lane + 64 * j < a.Dv) dst[lane + 64 * j] = (T)(acc[j] / den);
  }
}

template <typename T, int C, int MT>
hipError_t go(const GqaArgs& a, hipStream_t st) {
  hipLaunchKernelGGL((gqa_kernel<T, C, MT>), dim3(a.n_items, a.G), dim3(64 * kWaves), 0, st, a);
  if (hipError_t e = hipGetLastError()) return e;
  if (a.n_merges > 0) {
    hipLaunchKernelGGL(gqa_merge_kernel<T>, dim3(a.n_merges, a.G, MT == 1 ? 2 : 4), dim3(256), 0, st,
                       a, 16 * MT);
    return hipGetLastError();
  }
  return hipSuccess;
}

inline int dim_class(int Dp, int Dvp) {
  const int d = std::max(Dp, Dvp);
  return d <= 64 ? 64 : d <= 128 ? 128 : 256;
}

}  // namespace

int gqa_tile_rows(int dtype, int Dp, int Dvp, int rows) {
  if (rows <= 16) return 16;
  const int c = dim_class(Dp, Dvp);
  if (c == 64) return dtype == LLM_F32 ? 32 : 64;
  if (c == 128 && dtype != LLM_F32) return 32;
  return 16;
}

hipError_t gqa_attention(int dtype, const GqaArgs& a, int tile_rows, hipStream_t st) {
  if (a.n_items <= 0) return hipSuccess;
  const int c = dim_class(a.Dp, a.Dvp);
  if (dtype == LLM_F32) {
    if (c == 64) return tile_rows == 32 ? go<float, 64, 2>(a, st) : go<float, 64, 1>(a, st);
    return c == 128 ? go<float, 128, 1>(a, st) : go<float, 256, 1>(a, st);
  }
  if (c == 64) return tile_rows == 64 ? go<__bf16, 64, 4>(a, st) : go<__bf16, 64, 1>(a, st);
  if (c == 128) return tile_rows == 32 ? go<__bf16, 128, 2>(a, st) : go<__bf16, 128, 1>(a, st);
  return go<__bf16, 256, 1>(a, st);
}

}  // namespace llm
