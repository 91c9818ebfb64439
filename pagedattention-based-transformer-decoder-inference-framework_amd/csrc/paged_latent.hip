// Paged latent attention on MFMA for a mixed batch.
//
// A workgroup takes one tile of 16 MT rows (the heads of consecutive tokens) and
// a range of pages.  Every stage of SK cached rows is loaded into LDS once and
// used twice:
//   S^T[keys][rows] = C . Q^T       the 4 waves share the (row tile, key tile)s
//   O^T[rank][rows] += C^T . P^T    every wave owns a quarter of the latent
// The scores pass through LDS as finished 16 x 16 tiles in lane order, so each
// wave finds the probabilities of all rows as operands of its second product
// (keys are the MFMA row index of S^T) and keeps its own copy of the running
// maximum and sum.  C^T operands: transposed LDS reads in bf16, single floats in
// fp32.  Row r's 16-byte chunks are rotated by r in LDS, which spreads both
// access patterns over the banks.
//
// Scores, maxima, sums and probabilities are fp32 in log2 units; in bf16 the
// probabilities enter the second product as hi + lo halves.
#include "common.hpp"
#include "paged_latent.hpp"

#include <algorithm>

namespace llm {
namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));
constexpr int kWaves = 4;

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

__device__ __forceinline__ int wrap(int v, int n) { return v >= n ? v - n : v; }

// NK: most k-steps of a row, NDW: most 16-wide latent tiles of a wave
template <typename T, int NK, int NDW, int MT, int SK>
__global__ __launch_bounds__(64 * kWaves, sizeof(T) == 2 && NK * MT < 72 ? 2 : 1) void latent_kernel(GqaArgs a) {
  constexpr bool BF16 = sizeof(T) == 2;
  constexpr int KSTEP = BF16 ? 32 : 16, KT = BF16 ? 2 : 1;  // 16-key tiles per step of product 2
  // product 1: a row tile's NG waves share the key tiles, and where there are fewer
  // of those, the row's k-steps (PARTS sums, added where they are read)
  constexpr int KTS = SK / 16, NG = kWaves / MT;
  constexpr int PARTS = NG > KTS ? NG / KTS : 1, UG = NG / PARTS, UW = KTS / UG, NKP = NK / PARTS;
  static_assert(UG * PARTS == NG && UW * UG == KTS && NKP * PARTS == NK, "even shares");
  constexpr int SPP = kPageTokens / SK, FILL = (SK * 4 * NK + 255) / 256;
  __shared__ u32x4 stage[2][SK * 4 * NK];
  __shared__ f32x4 score[MT][KTS][PARTS][64];

  const int lane = lane_id(), w = wave_id_uniform();
  const int g = lane >> 4, c = lane & 15;
  const GqaItem it = a.items[blockIdx.x];
  const int R = a.H;
  const int32_t* pt = a.table + (size_t)it.slot * a.max_tiles;
  const int rows = min(16 * MT, it.nrows - it.row0);
  const int first_pos = it.p0 + it.row0 / R;
  const int last_pos = it.p0 + (it.row0 + rows - 1) / R;
  const int s0 = it.page0 * SPP, s1 = min(it.page1 * SPP, last_pos / SK + 1);
  const int cpr = a.Dp * (int)sizeof(T) / 16;  // 16-byte chunks per row

  // chunk i of this lane: place (256 i + 64 w + lane) of a stage
  int from[FILL];
#pragma unroll
  for (int i = 0; i < FILL; ++i) {
    const int q = (kWaves * i + w) * 64 + lane, key = q / cpr, at = q - key * cpr;
    from[i] = (key * cpr + wrap(at + cpr - key % cpr, cpr)) * 16;
  }
  auto issue = [&](int buf, int s, int page) {
    if (page < 0) return;
    const char* src = static_cast<const char*>(a.k_pool) + (size_t)page * a.page_stride +
                      (size_t)(s % SPP) * SK * cpr * 16;
#pragma unroll
    for (int i = 0; i < FILL; ++i) {
      const int q0 = (kWaves * i + w) * 64;
      if (q0 < SK * cpr) load_to_lds(src + from[i], &stage[buf][q0]);
    }
  };
  // a stage's page: looked up a stage before it is asked for
  auto lookup = [&](int s) { return pt[min(s / SPP, a.max_tiles - 1)]; };
  auto page_of = [&](int s, int found) {
    const int p = s < s1 && s / SPP < a.max_tiles && found < a.num_pages ? found : -1;
    return __builtin_amdgcn_readfirstlane(p);
  };
  int page = page_of(s0, lookup(s0)), next = page_of(s0 + 1, lookup(s0 + 1)), buf = 0;
  issue(0, s0, page);

  // this wave's row tile, key tiles u0, u0 + UG, ... and k-steps k1 ..
  const int t1 = w % MT, u0 = w / MT % UG, part = w / MT / UG, k1 = part * NKP;
  u32x4 q[NKP];
  {
    const int rr = 16 * t1 + c;
    const bool ok = rr < rows;
    const int row = it.row0 + (ok ? rr : 0), tok = row / R;
    const T* qp = static_cast<const T*>(a.q) +
                  ((size_t)(it.tok0 + tok) * R + (row - tok * R)) * a.Dp + g * (KSTEP / 4);
#pragma unroll
    for (int k = 0; k < NKP; ++k)  // (steps past the row meet zeros)
      q[k] = ok && (k1 + k) * KSTEP < a.Dp
                 ? *reinterpret_cast<const u32x4*>(qp + (k1 + k) * KSTEP)
                 : u32x4{0u, 0u, 0u, 0u};
  }
  int turn1[UW];  // rotation of the key this lane reads in product 1
#pragma unroll
  for (int i = 0; i < UW; ++i) turn1[i] = (16 * (u0 + UG * i) + c) % cpr;
  int turn2[KTS][BF16 ? 1 : 4];  // and in product 2
#pragma unroll
  for (int u = 0; u < KTS; ++u) {
    if constexpr (BF16) turn2[u][0] = (16 * u + 4 * g + (c >> 2)) % cpr;
    else
#pragma unroll
      for (int j = 0; j < 4; ++j) turn2[u][j] = (16 * u + 4 * g + j) % cpr;
  }
  int pos[MT];
  float m[MT], l[MT];
  f32x4 o[NDW][MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int rr = 16 * t + c;
    pos[t] = rr < rows ? it.p0 + (it.row0 + rr) / R : -1;
    m[t] = kNegSentinel;
    l[t] = 0.f;
#pragma unroll
    for (int n = 0; n < NDW; ++n) o[n][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float scale2 = a.scale * kLog2e;
  const int last_tile = (a.Dv + 15) / 16 - 1;

  for (int s = s0; s < s1; ++s, buf ^= 1) {
    wait_lds_loads();
    __syncthreads();  // stage s has landed, the other buffer and the scores are read out
    issue(buf ^ 1, s + 1, next);
    const int found = lookup(s + 2);
    const u32x4* st = stage[buf];
    if (MT == 1 || 16 * t1 < rows) {
#pragma unroll
      for (int i = 0; i < UW; ++i) {
        const int u = u0 + UG * i;
        f32x4 d0 = {0.f, 0.f, 0.f, 0.f}, d1 = d0;
        const u32x4* row = st + (16 * u + c) * cpr;
        u32x4 x[NKP];
#pragma unroll
        for (int k = 0; k < NKP; ++k)
          x[k] = row[wrap(min(4 * (k1 + k) + g, cpr - 1) + turn1[i], cpr)];
#pragma unroll
        for (int k = 0; k < NKP; ++k) {
          if (k & 1) d1 = dot_step<T>(x[k], q[k], d1);
          else d0 = dot_step<T>(x[k], q[k], d0);
        }
        score[t1][u][part][lane] = d0 + d1;
      }
    }
    __syncthreads();
    if (page >= 0) {
      const int key0 = s * SK;
      const bool mask = key0 + SK - 1 > first_pos;
      u32x4 hi[MT][KTS / KT], lo[MT][KTS / KT];
#pragma unroll
      for (int t = 0; t < MT; ++t) {
        if (t > 0 && 16 * t >= rows) break;
        f32x4 x[KTS];
        float mloc = kNegSentinel;
#pragma unroll
        for (int u = 0; u < KTS; ++u) {
          x[u] = score[t][u][0][lane];
#pragma unroll
          for (int i = 1; i < PARTS; ++i) x[u] += score[t][u][i][lane];
          x[u] *= scale2;
          if (mask || 16 * t + 16 > rows) {
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (key0 + 16 * u + 4 * g + r > pos[t]) x[u][r] = 2.f * kNegSentinel;
          }
#pragma unroll
          for (int r = 0; r < 4; ++r) mloc = fmaxf(mloc, x[u][r]);
        }
        mloc = fmaxf(mloc, __shfl_xor(mloc, 16, 64));
        mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
        if (__any(mloc > m[t])) {
          const float mnew = fmaxf(m[t], mloc);
          const float corr = __builtin_amdgcn_exp2f(m[t] - mnew);
          l[t] *= corr;
#pragma unroll
          for (int n = 0; n < NDW; ++n) o[n][t] *= corr;
          m[t] = mnew;
        }
#pragma unroll
        for (int u = 0; u < KTS; ++u)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            x[u][r] = __builtin_amdgcn_exp2f(x[u][r] - m[t]);
            l[t] += x[u][r];
          }
#pragma unroll
        for (int b = 0; b < KTS / KT; ++b) {
          if constexpr (BF16) {
            bf16x8 h, e;
#pragma unroll
            for (int j = 0; j < 8; ++j) {
              const float v = x[2 * b + j / 4][j % 4];
              h[j] = (__bf16)v;
              e[j] = (__bf16)(v - (float)h[j]);
            }
            hi[t][b] = __builtin_bit_cast(u32x4, h);
            lo[t][b] = __builtin_bit_cast(u32x4, e);
          } else {
            hi[t][b] = __builtin_bit_cast(u32x4, x[b]);
          }
        }
      }
#pragma unroll
      for (int b = 0; b < KTS / KT; ++b) {
        u32x4 v[NDW];
#pragma unroll
        for (int n = 0; n < NDW; ++n) {
          // (tiles past the latent repeat the last one, nobody reads their sums)
          const int tile = min(w + kWaves * n, last_tile);
          if constexpr (BF16) {
            // lane 4 q + p of 16 addresses key 4 g + q, dims 4 p ..; it gets keys
            // 4 g .. 4 g + 3 of dim `lane`
            const int ch = 2 * tile + ((c & 3) >> 1);
            s16x4 half[2];
#pragma unroll
            for (int j = 0; j < 2; ++j) {
              const int u = 2 * b + j, key = 16 * u + 4 * g + (c >> 2);
              const char* at = reinterpret_cast<const char*>(
                                   st + key * cpr + wrap(ch + turn2[u][0], cpr)) + (c & 1) * 8;
              half[j] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                  (__attribute__((address_space(3))) s16x4*)at);
            }
            v[n] = __builtin_bit_cast(u32x4, s16x8{half[0][0], half[0][1], half[0][2], half[0][3],
                                                   half[1][0], half[1][1], half[1][2], half[1][3]});
          } else {
            const int d = 16 * tile + c;
            f32x4 f;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
              const int key = 16 * b + 4 * g + j;
              f[j] = reinterpret_cast<const float*>(
                  st + key * cpr + wrap((d >> 2) + turn2[b][j], cpr))[d & 3];
            }
            v[n] = __builtin_bit_cast(u32x4, f);
          }
        }
#pragma unroll
        for (int t = 0; t < MT; ++t) {
          if (t > 0 && 16 * t >= rows) break;
#pragma unroll
          for (int n = 0; n < NDW; ++n) {
            o[n][t] = dot_step<T>(v[n], hi[t][b], o[n][t]);
            if constexpr (BF16) o[n][t] = dot_step<T>(v[n], lo[t][b], o[n][t]);
          }
        }
      }
    }
    page = next;
    next = page_of(s + 2, found);
  }

#pragma unroll
  for (int t = 0; t < MT; ++t) {
    l[t] += __shfl_xor(l[t], 16, 64);
    l[t] += __shfl_xor(l[t], 32, 64);
    const int rr = 16 * t + c;
    if (rr >= rows) continue;
    const int row = it.row0 + rr;
    if (it.part >= 0) {
      const size_t base = (size_t)it.part * 16 * MT + rr;
      float* dst = a.part_o + base * ((a.Dv + 15) / 16 * 16);
#pragma unroll
      for (int n = 0; n < NDW; ++n) {
        const int d = 16 * (w + kWaves * n);
        if (d < a.Dv) *reinterpret_cast<f32x4*>(dst + d + 4 * g) = o[n][t];
      }
      if (w == 0 && g == 0) *reinterpret_cast<float2*>(a.part_ml + base * 2) = float2{m[t], l[t]};
      continue;
    }
    const int tok = row / R, head = row - tok * R;
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
    for (int n = 0; n < NDW; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * (w + kWaves * n) + 4 * g + r;
        if (d < a.Dv) dst[d] = (T)(o[n][t][r] * f);
      }
  }
}

template <typename T, int NK, int NDW, int MT, int SK>
hipError_t go(const GqaArgs& a, hipStream_t st) {
  hipLaunchKernelGGL((latent_kernel<T, NK, NDW, MT, SK>), dim3(a.n_items), dim3(64 * kWaves), 0, st, a);
  if (hipError_t e = hipGetLastError()) return e;
  return gqa_merge(sizeof(T) == 2 ? LLM_BF16 : LLM_F32, a, 16 * MT, st);
}

// classes by row length and rank: two workgroups' stages fit a CU's LDS
template <typename T, int MT>
hipError_t go(const GqaArgs& a, hipStream_t st) {
  constexpr int F = 4 / sizeof(T);  // 2: bf16, 1: fp32
  constexpr int E = 2 / F;          // k-steps of a 32-element row piece
  if (a.Dp <= 128 && a.Dv <= 128) return go<T, 4 * E, 2, MT, 64>(a, st);
  if (a.Dp <= 320 && a.Dv <= 256) return go<T, 10 * E, 4, MT, 16 * F>(a, st);
  if (a.Dp <= kLatentMaxRow && a.Dv <= kLatentMaxRank) return go<T, 18 * E, 8, MT, 16 * F>(a, st);
  return hipErrorInvalidValue;
}

template <typename T>
hipError_t go(const GqaArgs& a, int tile_rows, hipStream_t st) {
  if (tile_rows == 16) return go<T, 1>(a, st);
  if (tile_rows == 32) return go<T, 2>(a, st);
  return tile_rows == 64 ? go<T, 4>(a, st) : hipErrorInvalidValue;
}

// ------------------------------------------------------------- cache rows
template <typename T>
__device__ __forceinline__ T* row_of(const MmPageRows& r, int pos, int slot) {
  const int tile = pos / kPageTokens;
  const int page = tile < r.max_tiles ? r.table[(size_t)slot * r.max_tiles + tile] : -1;
  if (page < 0 || page >= r.num_pages) return nullptr;
  return reinterpret_cast<T*>(static_cast<char*>(const_cast<void*>(r.pool)) +
                              (size_t)page * r.page_stride) +
         (size_t)(pos % kPageTokens) * r.row;
}

// a wave per token
template <typename T>
__global__ __launch_bounds__(64) void append_kernel(LatentAppend a) {
  constexpr int NV = kLatentMaxRank / 64;
  const int mrow = blockIdx.x, lane = lane_id();
  const float* src = a.down + (size_t)mrow * a.ldd;
  const int pos = a.page.pos[mrow], slot = a.page.slot[mrow];
  // everything that does not hang on the page is on its way before it is known
  float v[NV], w[NV], ss = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int d = min(lane + 64 * j, a.rank - 1);
    v[j] = src[d];
    w[j] = a.w[d];
  }
  const int pairs = a.rot / 2;
  float2 t = {1.f, 0.f}, k = {0.f, 0.f};
  if (lane < pairs) {
    t = a.turn[(size_t)mrow * pairs + lane];
    k = *reinterpret_cast<const float2*>(src + a.rot_at + 2 * lane);
  }
  T* dst = row_of<T>(a.page, pos, slot);
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    if (lane + 64 * j >= a.rank) v[j] = 0.f;
    ss += v[j] * v[j];
  }
  const float r = 1.f / sqrtf(wave_sum(ss) / (float)a.rank + a.eps);
  if (!dst) return;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int d = lane + 64 * j;
    if (d < a.rank) dst[d] = (T)(v[j] * r * w[j]);
  }
  T* rot = dst + latent_rot_at(a.rank);
  for (int i = lane; i < pairs; i += 64) {
    if (i != lane) {
      t = a.turn[(size_t)mrow * pairs + i];
      k = *reinterpret_cast<const float2*>(src + a.rot_at + 2 * i);
    }
    rot[2 * i] = (T)(k.x * t.x - k.y * t.y);
    rot[2 * i + 1] = (T)(k.y * t.x + k.x * t.y);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void spread_kernel(LatentSpread a) {
  const int m = blockIdx.x;
  const int pos = a.src.pos[m];
  const T* src = row_of<T>(a.src, pos, a.src.slot[m]);
  const int tile = pos / kPageTokens;
  if (!src || tile >= a.max_tiles) return;
  for (int i = threadIdx.x; i < a.H * a.rot; i += 256) {
    const int h = i / a.rot, d = i - h * a.rot;
    const int page = a.table[((size_t)a.slot[m] * a.H + h) * a.max_tiles + tile];
    if (page < 0 || page >= a.num_pages) continue;
    reinterpret_cast<T*>(static_cast<char*>(a.k_pool) + (size_t)page * a.page_stride)
        [(size_t)(pos % kPageTokens) * a.Dp + a.at + d] = src[a.src_at + d];
  }
}

}  // namespace

hipError_t latent_attention(int dtype, const GqaArgs& a, int tile_rows, hipStream_t st) {
  if (a.n_items <= 0) return hipSuccess;
  return dtype == LLM_F32 ? go<float>(a, tile_rows, st) : go<__bf16>(a, tile_rows, st);
}

hipError_t latent_append(int dtype, const LatentAppend& a, hipStream_t st) {
  if (a.M <= 0) return hipSuccess;
  if (dtype == LLM_F32) hipLaunchKernelGGL(append_kernel<float>, dim3(a.M), dim3(64), 0, st, a);
  else hipLaunchKernelGGL(append_kernel<__bf16>, dim3(a.M), dim3(64), 0, st, a);
  return hipGetLastError();
}

hipError_t latent_spread(int dtype, const LatentSpread& a, hipStream_t st) {
  if (a.M <= 0) return hipSuccess;
  if (dtype == LLM_F32) hipLaunchKernelGGL(spread_kernel<float>, dim3(a.M), dim3(256), 0, st, a);
  else hipLaunchKernelGGL(spread_kernel<__bf16>, dim3(a.M), dim3(256), 0, st, a);
  return hipGetLastError();
}

}  // namespace llm
