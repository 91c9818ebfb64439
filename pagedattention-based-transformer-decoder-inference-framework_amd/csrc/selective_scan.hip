// Causal convolution and selective scan on gfx950.
//
// Lanes are channels, so x, dt, z, the state ([state][channel]) and the output
// are contiguous across a wave, and B and C are the same for all lanes: they are
// staged in LDS once per chunk and read as broadcasts.  A lane keeps up to 32
// states of its channel in registers; wider states are spread over SP lanes.
#include "common.hpp"
#include "selective_scan.hpp"

#include <algorithm>

namespace llm {
namespace {

constexpr int kThreads = 256;

constexpr int chunk_of(int padded_state) { return std::min(64, 4096 / padded_state); }

// within 3 ulp: exp2 and the reciprocal are the hardware's
__device__ __forceinline__ float silu(float v) {
  return v * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-kLog2e * v));
}

enum Pass { kEmit, kChunk };

template <typename T, int NS, int SP, int PASS>
__global__ __launch_bounds__(kThreads) void scan_kernel(ScanArgs a, const ScanItem* __restrict__ items) {
  constexpr int NP = NS * SP, CH = chunk_of(NP), LC = 64 / SP, U = 4;
  constexpr int COLS = PASS == kEmit ? 2 : 1;
  __shared__ __align__(16) float bc[CH][COLS * NP];
  const ScanItem it = items[blockIdx.x];
  const int lane = lane_id(), sp = lane / LC, n0 = sp * NS;
  const int ch = ((int)blockIdx.y * (kThreads / 64) + wave_id_uniform()) * LC + lane % LC;
  const bool ok = ch < a.inner;
  const int c = ok ? ch : a.inner - 1;
  const int n = min(it.n, CH);

  struct Rows {
    float x[U], dt[U], z[U];
  };
  auto load = [&](Rows& r, int t0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const size_t m = (size_t)(it.tok0 + min(t0 + u, n - 1));
      r.x[u] = (float)static_cast<const T*>(a.x)[m * a.ldx + c];
      r.dt[u] = a.dt[m * a.ldt + c];
      if constexpr (PASS == kEmit) r.z[u] = (float)static_cast<const T*>(a.z)[m * a.ldz + c];
    }
  };
  Rows r0, r1;
  load(r0, 0);

  float S[NS], A[NS];
  const bool carried = PASS == kEmit && it.part >= 0;
  const bool slot_state = PASS == kEmit ? it.part < 0 : it.last != 0;
  const float* from = carried ? a.carry + (size_t)it.part * a.state * a.ldc
                              : a.slots + (size_t)it.slot * a.state * a.ldc;
  const bool zero = !carried && !(slot_state && it.p0 > 0);
#pragma unroll
  for (int k = 0; k < NS; ++k) {
    const bool in = n0 + k < a.state;
    const size_t at = (size_t)(in ? n0 + k : 0) * a.ldc + c;
    A[k] = in ? a.A[at] : 0.f;
    S[k] = in && !zero ? from[at] : 0.f;
  }
  for (int i = threadIdx.x; i < n * COLS * NP; i += kThreads) {
    const int t = i / (COLS * NP), j = i % (COLS * NP), k = j % NP;
    bc[t][j] = k < a.state ? a.bc[(size_t)(it.tok0 + t) * a.ldb + (j < NP ? 0 : a.c_at) + k] : 0.f;
  }
  const float D = PASS == kEmit ? a.D[c] : 0.f;
  __syncthreads();

  float sum = 0.f;
  auto work = [&](const Rows& r, int t0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int t = t0 + u;
      if (t >= n) break;
      const float dt = r.dt[u], dx = dt * r.x[u];
      const f32x4* b = reinterpret_cast<const f32x4*>(&bc[t][n0]);
      const f32x4* cc = reinterpret_cast<const f32x4*>(&bc[t][(COLS - 1) * NP + n0]);
      float y[2] = {0.f, 0.f};
#pragma unroll
      for (int q = 0; q < NS / 4; ++q) {
        const f32x4 bq = b[q];
        f32x4 cq = {0.f, 0.f, 0.f, 0.f};
        if constexpr (PASS == kEmit) cq = cc[q];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int k = 4 * q + e;
          S[k] = __builtin_amdgcn_exp2f(dt * A[k]) * S[k] + dx * bq[e];
          if constexpr (PASS == kEmit) y[e & 1] += S[k] * cq[e];
        }
      }
      if constexpr (PASS == kEmit) {
        float v = y[0] + y[1];
#pragma unroll
        for (int off = LC; off < 64; off *= 2) v += __shfl_xor(v, off, 64);
        v = (v + D * r.x[u]) * silu(r.z[u]);
        if (ok && sp == 0) static_cast<T*>(a.out)[(size_t)(it.tok0 + t) * a.ldo + c] = (T)v;
      } else {
        sum += dt;
      }
    }
  };
  for (int t = 0;;) {
    if (t + U < n) load(r1, t + U);
    work(r0, t);
    t += U;
    if (t >= n) break;
    if (t + U < n) load(r0, t + U);
    work(r1, t);
    t += U;
    if (t >= n) break;
  }

  if (!ok) return;
  if constexpr (PASS == kChunk) {
    float* dst = a.carry + (size_t)it.part * a.state * a.ldc;
#pragma unroll
    for (int k = 0; k < NS; ++k)
      if (n0 + k < a.state) dst[(size_t)(n0 + k) * a.ldc + c] = S[k];
    if (sp == 0) a.sum_dt[(size_t)it.part * a.ldc + c] = sum;
  } else if (it.last) {
    float* dst = a.slots + (size_t)it.slot * a.state * a.ldc;
#pragma unroll
    for (int k = 0; k < NS; ++k)
      if (n0 + k < a.state) dst[(size_t)(n0 + k) * a.ldc + c] = S[k];
    if (sp == 0 && a.taps > 1) {
      // oldest first: entry j is read (from a later place) before it is written
      T* h = static_cast<T*>(a.history) + (size_t)it.slot * (a.taps - 1) * a.ldc + c;
      for (int j = 0; j < a.taps - 1; ++j) {
        const int off = it.seq_n - (a.taps - 1) + j;
        T v = (T)0.f;
        if (off >= 0) v = static_cast<const T*>(a.raw)[(size_t)(it.seq0 + off) * a.ld_raw + c];
        else if (it.p0 + off >= 0) v = h[(size_t)(it.seq_n + j) * a.ldc];
        h[(size_t)j * a.ldc] = v;
      }
    }
  }
}

// One lane per (channel, state): the chunks' end states become true ones.
__global__ __launch_bounds__(kThreads) void scan_carry_kernel(ScanArgs a,
                                                              const ScanCarry* __restrict__ seqs) {
  const ScanCarry s = seqs[blockIdx.x];
  const int c = (int)blockIdx.y * kThreads + threadIdx.x, n = blockIdx.z;
  if (c >= a.inner) return;
  const float A = a.A[(size_t)n * a.ldc + c];
  const size_t step = (size_t)a.state * a.ldc;
  float* p = a.carry + (size_t)s.part0 * step + (size_t)n * a.ldc + c;
  const float* d = a.sum_dt + (size_t)s.part0 * a.ldc + c;
  float S = p[0];
  constexpr int U = 8;  // parts in flight
  for (int k = 1; k < s.n; k += U) {
    float v[U], w[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int i = min(k + u, s.n - 1);
      v[u] = p[(size_t)i * step];
      w[u] = d[(size_t)i * a.ldc];
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (k + u < s.n) {
        S = __builtin_amdgcn_exp2f(w[u] * A) * S + v[u];
        p[(size_t)(k + u) * step] = S;
      }
  }
}

// Four channels per lane, RB rows.  TAPS (0: any number): blocks whose rows and
// their past are one sequence's rows of this batch, nearly all of a prompt, read
// each row once.
template <typename T, int TAPS>
__global__ __launch_bounds__(kThreads) void conv_kernel(ConvArgs a) {
  typedef T quad_t __attribute__((ext_vector_type(4)));
  constexpr int RB = 8;
  const int c = 4 * ((int)blockIdx.y * kThreads + threadIdx.x);
  if (c >= a.channels) return;
  const int m0 = (int)blockIdx.x * RB;
  const f32x4 bias = *reinterpret_cast<const f32x4*>(a.bias + c);
  f32x4 acc[RB];
#pragma unroll
  for (int r = 0; r < RB; ++r) acc[r] = bias;
  bool plain = false;
  if constexpr (TAPS > 0) {
    plain = m0 + RB <= a.M && a.seq0[min(m0 + RB, a.M) - 1] <= m0 - (TAPS - 1);
    if (plain) {
      quad_t v[RB + TAPS - 1];
      const T* src = static_cast<const T*>(a.in) + (size_t)(m0 - (TAPS - 1)) * a.ld_in + c;
#pragma unroll
      for (int r = 0; r < RB + TAPS - 1; ++r)
        v[r] = *reinterpret_cast<const quad_t*>(src + (size_t)r * a.ld_in);
#pragma unroll
      for (int k = 0; k < TAPS; ++k) {
        const f32x4 w = *reinterpret_cast<const f32x4*>(a.w + (size_t)k * a.ldc + c);
#pragma unroll
        for (int r = 0; r < RB; ++r)
#pragma unroll
          for (int e = 0; e < 4; ++e) acc[r][e] += w[e] * (float)v[r + k][e];
      }
    }
  }
  if (!plain) {
    for (int k = 0; k < a.taps; ++k) {
      const f32x4 w = *reinterpret_cast<const f32x4*>(a.w + (size_t)k * a.ldc + c);
      const int back = a.taps - 1 - k;
#pragma unroll
      for (int r = 0; r < RB; ++r) {
        const int m = m0 + r;
        if (m >= a.M) break;
        const T* src = nullptr;
        if (m - back >= a.seq0[m])
          src = static_cast<const T*>(a.in) + (size_t)(m - back) * a.ld_in + c;
        else if (a.pos[m] >= back)  // entry taps - 1 is the portion's first row
          src = static_cast<const T*>(a.history) +
                ((size_t)a.slot[m] * (a.taps - 1) + (m - back - a.seq0[m] + a.taps - 1)) * a.ldc + c;
        if (!src) continue;
        const quad_t v = *reinterpret_cast<const quad_t*>(src);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[r][e] += w[e] * (float)v[e];
      }
    }
  }
#pragma unroll
  for (int r = 0; r < RB; ++r) {
    if (m0 + r >= a.M) break;
    quad_t v;
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = (T)silu(acc[r][e]);
    *reinterpret_cast<quad_t*>(static_cast<T*>(a.x) + (size_t)(m0 + r) * a.ldx + c) = v;
  }
}

template <typename T>
hipError_t conv(const ConvArgs& a, hipStream_t st) {
  const dim3 grid((a.M + 7) / 8, (a.channels + 4 * kThreads - 1) / (4 * kThreads));
#define LLM_CONV_GO(TAPS) \
  hipLaunchKernelGGL((conv_kernel<T, TAPS>), grid, dim3(kThreads), 0, st, a)
  switch (a.taps) {
    case 2: LLM_CONV_GO(2); break;
    case 3: LLM_CONV_GO(3); break;
    case 4: LLM_CONV_GO(4); break;
    default: LLM_CONV_GO(0);
  }
#undef LLM_CONV_GO
  return hipGetLastError();
}

template <typename T, int NS, int SP, int PASS>
hipError_t launch(const ScanArgs& a, const ScanItem* items, int n, hipStream_t st) {
  const int per_block = kThreads / SP;
  hipLaunchKernelGGL((scan_kernel<T, NS, SP, PASS>), dim3(n, (a.inner + per_block - 1) / per_block),
                     dim3(kThreads), 0, st, a, items);
  return hipGetLastError();
}

template <typename T, int PASS>
hipError_t launch(const ScanArgs& a, const ScanItem* items, int n, hipStream_t st) {
  if (a.state <= 8) return launch<T, 8, 1, PASS>(a, items, n, st);
  if (a.state <= 16) return launch<T, 16, 1, PASS>(a, items, n, st);
  if (a.state <= 32) return launch<T, 32, 1, PASS>(a, items, n, st);
  if (a.state <= 64) return launch<T, 32, 2, PASS>(a, items, n, st);
  if (a.state <= 128) return launch<T, 32, 4, PASS>(a, items, n, st);
  return a.state <= kMaxScanState ? launch<T, 32, 8, PASS>(a, items, n, st) : hipErrorInvalidValue;
}

template <int PASS>
hipError_t launch(int dtype, const ScanArgs& a, const ScanItem* items, int n, hipStream_t st) {
  if (n <= 0) return hipSuccess;
  return dtype == LLM_F32 ? launch<float, PASS>(a, items, n, st)
                          : launch<__bf16, PASS>(a, items, n, st);
}

}  // namespace

int scan_chunk(int state) {
  int p = 8;
  while (p < state) p *= 2;
  return chunk_of(p);
}

hipError_t scan(int dtype, const ScanArgs& a, const ScanItem* items, int n, hipStream_t st) {
  return launch<kEmit>(dtype, a, items, n, st);
}

hipError_t scan_chunks(int dtype, const ScanArgs& a, const ScanItem* items, int n, hipStream_t st) {
  return launch<kChunk>(dtype, a, items, n, st);
}

hipError_t scan_carry(const ScanArgs& a, const ScanCarry* seqs, int n, hipStream_t st) {
  if (n <= 0) return hipSuccess;
  hipLaunchKernelGGL(scan_carry_kernel, dim3(n, (a.inner + kThreads - 1) / kThreads, a.state),
                     dim3(kThreads), 0, st, a, seqs);
  return hipGetLastError();
}

hipError_t causal_conv(int dtype, const ConvArgs& a, hipStream_t st) {
  if (a.M <= 0) return hipSuccess;
  return dtype == LLM_F32 ? conv<float>(a, st) : conv<__bf16>(a, st);
}

}  // namespace llm
