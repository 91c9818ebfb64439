// The residual stream (or streams) between sublayers: add the sublayer output,
// normed or scaled, add the embedding where a repeated pass starts, norm for the
// next sublayer -- one launch, the row in registers.  Also the rotation angles
// of a step.
#include "common.hpp"
#include "rms_norm.hpp"

namespace llm {
namespace {

typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));

template <int THREADS>
__device__ __forceinline__ float row_sum(float v, float* sh) {
  v = wave_sum(v);
  if constexpr (THREADS == 64) return v;
  __syncthreads();  // sh free again
  if (lane_id() == 0) sh[wave_id_uniform()] = v;
  __syncthreads();
  float s = sh[0];
#pragma unroll
  for (int i = 1; i < THREADS / 64; ++i) s += sh[i];
  return s;
}

__device__ __forceinline__ float square_sum(f32x4 v) {
  return v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
}

// THREADS lanes per row, NV float4 per lane; SM: most streams (0: one residual)
template <typename T, int THREADS, int NV, int SM>
__global__ __launch_bounds__(THREADS) void norm_step_kernel(NormStep a) {
  constexpr int SN = SM > 0 ? SM : 1;
  __shared__ float sh[THREADS / 64];
  __shared__ float coef[SN * SN + 2 * SN];  // mix, out, in
  const int i = blockIdx.x;
  const int m = a.rows ? a.rows[i] : i;
  const int nv = a.ldx >> 2;
  float* xr = a.x + (size_t)m * (SM > 0 ? a.streams : 1) * a.ldx;
  f32x4 x[NV];
  // up to 4 streams fly with the other loads; more are read where they are mixed
  constexpr bool EARLY = SM > 0 && SM <= 4 && NV * SM <= 16;
  f32x4 early[EARLY ? NV : 1][SN];
  auto embed_at = [&](int c) {
    const uint2 e = *reinterpret_cast<const uint2*>(a.emb + (size_t)a.tok[m] * a.ldx + 4 * c);
    return f32x4{__builtin_bit_cast(float, e.x << 16), __builtin_bit_cast(float, e.x & 0xFFFF0000u),
                 __builtin_bit_cast(float, e.y << 16),
                 __builtin_bit_cast(float, e.y & 0xFFFF0000u)} * a.emb_scale;
  };
  if constexpr (SM == 0) {
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = threadIdx.x + j * THREADS;
      x[j] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (c < nv) x[j] = a.embed == 1 ? embed_at(c) : *reinterpret_cast<const f32x4*>(xr + 4 * c);
    }
  } else {
    const int S = a.streams;
    if constexpr (EARLY) {
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int c = min((int)threadIdx.x + j * THREADS, nv - 1);
#pragma unroll
        for (int s = 0; s < SN; ++s)
          early[j][s] = a.embed == 1 ? embed_at(c)
                                     : *reinterpret_cast<const f32x4*>(
                                           xr + (size_t)min(s, S - 1) * a.ldx + 4 * c);
      }
    }
    for (int k = threadIdx.x; k < S * S + 2 * S; k += THREADS) {
      float v = 1.f;  // hc_in
      if (k < S * S) v = a.y ? a.hc_mix[k] : k / S == k % S ? 1.f : 0.f;
      else if (k < S * S + S) v = a.y ? a.hc_out[k - S * S] : 0.f;
      else if (a.hc_in) v = a.hc_in[k - S * S - S];
      coef[k] = v;
    }
  }
  const float inv_w = 1.f / (float)a.width;
  // the norm weights fly while the rows are summed
  f32x4 wpost[NV], wpre[NV], scale[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = threadIdx.x + j * THREADS;
    wpost[j] = wpre[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    scale[j] = f32x4{1.f, 1.f, 1.f, 1.f};
    if (c < nv && a.y_scale) scale[j] = *reinterpret_cast<const f32x4*>(a.y_scale + 4 * c);
    if (c < nv && a.w_post) wpost[j] = *reinterpret_cast<const f32x4*>(a.w_post + 4 * c);
    if (c < nv && a.w_pre) wpre[j] = *reinterpret_cast<const f32x4*>(a.w_pre + 4 * c);
  }
  f32x4 y[NV];
  if (a.y) {
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = threadIdx.x + j * THREADS;
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
      if (c < nv) {
        const float* y0 = a.y + (size_t)m * a.parts * a.ldy + 4 * c;
        if (a.shared)
          s = *reinterpret_cast<const f32x4*>(a.y + ((size_t)a.M_y * a.parts + m) * a.ldy + 4 * c);
        for (int q = 0; q < a.parts; q += 4) {  // four parts' loads in flight
          f32x4 v[4];
#pragma unroll
          for (int u = 0; u < 4; ++u)
            v[u] = *reinterpret_cast<const f32x4*>(y0 + (size_t)min(q + u, a.parts - 1) * a.ldy);
#pragma unroll
          for (int u = 0; u < 4; ++u)
            if (q + u < a.parts) s += v[u];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (4 * c + e >= a.width) s[e] = 0.f;
      }
      y[j] = s;
      ss += square_sum(s);
    }
    if (a.w_post) {
      const float r = 1.f / sqrtf(row_sum<THREADS>(ss, sh) * inv_w + a.eps);
#pragma unroll
      for (int j = 0; j < NV; ++j) y[j] = y[j] * r * wpost[j];
    }
    if (a.y_scale) {
#pragma unroll
      for (int j = 0; j < NV; ++j) y[j] *= scale[j];
    }
  } else {
#pragma unroll
    for (int j = 0; j < NV; ++j) y[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  if constexpr (SM == 0) {
    if (a.y) {
#pragma unroll
      for (int j = 0; j < NV; ++j) x[j] += y[j];
    }
    if (a.embed == 2) {
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int c = threadIdx.x + j * THREADS;
        if (c < nv) x[j] += embed_at(c);
      }
    }
    if ((a.y || a.embed) && !a.rows) {
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int c = threadIdx.x + j * THREADS;
        if (c < nv) *reinterpret_cast<f32x4*>(xr + 4 * c) = x[j];
      }
    }
  } else {
    // x[j] becomes u; the streams themselves pass through
    __syncthreads();  // coef
    const int S = a.streams;
    const float *mix = coef, *out = coef + S * S, *in = out + S;
    const bool store = (a.y || a.embed) && !a.rows;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = threadIdx.x + j * THREADS;
      x[j] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (c >= nv) continue;
      f32x4 old[SN];
      const f32x4 e = a.embed ? embed_at(c) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < SN; ++s)
        if constexpr (EARLY) old[s] = early[j][s];
        else if (s < S)
          old[s] = a.embed == 1 ? e : *reinterpret_cast<const f32x4*>(xr + (size_t)s * a.ldx + 4 * c);
#pragma unroll SN <= 4 ? SN : 1
      for (int t = 0; t < SN; ++t) {
        if (t >= S) break;
        f32x4 v = out[t] * y[j];
#pragma unroll
        for (int s = 0; s < SN; ++s)
          if (s < S) v += mix[s * S + t] * old[s];
        if (a.embed == 2) v += e;
        if (store) *reinterpret_cast<f32x4*>(xr + (size_t)t * a.ldx + 4 * c) = v;
        x[j] += in[t] * v;
      }
      if (a.u) *reinterpret_cast<f32x4*>(a.u + (size_t)i * a.ldx + 4 * c) = x[j];
    }
  }
  if (!a.w_pre) return;
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) ss += square_sum(x[j]);
  const float r = 1.f / sqrtf(row_sum<THREADS>(ss, sh) * inv_w + a.eps);
  T* hr = static_cast<T*>(a.h) + (size_t)i * a.ldh;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = threadIdx.x + j * THREADS;
    if (c >= nv) continue;
    const f32x4 o = x[j] * r * wpre[j];
    if constexpr (sizeof(T) == 2)
      *reinterpret_cast<bf16x4*>(hr + 4 * c) =
          bf16x4{(__bf16)o[0], (__bf16)o[1], (__bf16)o[2], (__bf16)o[3]};
    else
      *reinterpret_cast<f32x4*>(hr + 4 * c) = o;
  }
}

template <typename T, int SM>
hipError_t launch_norm(const NormStep& a, hipStream_t st) {
  const dim3 grid(a.M);
  const int nv = a.ldx >> 2;
#define LLM_NORM_GO(TH, NV)                                                           \
  hipLaunchKernelGGL((norm_step_kernel<T, TH, NV, SM>), grid, dim3(TH), 0, st, a);    \
  return hipGetLastError()
  if (SM > 0 && a.M <= 256 && nv > 64) {  // few rows of several streams: a lane per column
    if (nv <= 256) { LLM_NORM_GO(256, 1); }
    if (nv <= 512) { LLM_NORM_GO(512, 1); }
    if (nv <= 1024) { LLM_NORM_GO(1024, 1); }
  }
  if (nv <= 64) { LLM_NORM_GO(64, 1); }
  if (nv <= 128) { LLM_NORM_GO(64, 2); }
  if (nv <= 256) { LLM_NORM_GO(256, 1); }
  if (nv <= 512) { LLM_NORM_GO(256, 2); }
  if (nv <= 1024) { LLM_NORM_GO(256, 4); }
  if (nv <= 2048) { LLM_NORM_GO(256, 8); }
#undef LLM_NORM_GO
  return hipErrorInvalidValue;
}

template <typename T>
hipError_t launch_norm(const NormStep& a, hipStream_t st) {
  if (a.streams == 0) return launch_norm<T, 0>(a, st);
  if (a.streams <= 4) return launch_norm<T, 4>(a, st);
  return a.streams <= kMaxStreams ? launch_norm<T, kMaxStreams>(a, st) : hipErrorInvalidValue;
}

__global__ void rope_turns_kernel(const int32_t* __restrict__ pos, int M,
                                  const float* __restrict__ freq, int half, float mul,
                                  float2* __restrict__ turn) {
  const int idx = blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= M * half) return;
  const float a = (float)pos[idx / half] * freq[idx % half];
  float s, c;
  sincosf(a, &s, &c);
  turn[idx] = float2{c * mul, s * mul};
}

}  // namespace

hipError_t rms_norm_step(int dtype, const NormStep& a, hipStream_t st) {
  if (a.M <= 0) return hipSuccess;
  return dtype == LLM_F32 ? launch_norm<float>(a, st) : launch_norm<__bf16>(a, st);
}

hipError_t rope_turns(const int32_t* pos, int M, const float* freq, int half, float mul,
                      float2* turn, hipStream_t st) {
  if (M <= 0 || half <= 0) return hipSuccess;
  hipLaunchKernelGGL(rope_turns_kernel, dim3((M * half + 255) / 256), dim3(256), 0, st, pos, M,
                     freq, half, mul, turn);
  return hipGetLastError();
}

}  // namespace llm
