// Matrix products of the layer-stack models: packing, plain products, the
// grouped-query projections and the grouped (expert) products.  The kernels are
// in mm_impl.hpp; mm_mix.hip has the epilogues of the other mixers.
#include "mm_impl.hpp"

namespace llm {
namespace {

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
  const long long rows = (long long)M * top / experts;  // of an expert, on average
  return M <= 64 || rows < 24 ? 16 : rows < 192 ? 64 : 128;
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
