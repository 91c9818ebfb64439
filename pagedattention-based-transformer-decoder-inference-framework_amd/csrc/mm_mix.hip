// Matrix products of the layer-stack models whose epilogues belong to the dense
// feed-forward, latent attention and the selective scan (kernels: mm_impl.hpp).
#include "mm_impl.hpp"

namespace llm {
namespace {

KernelArgs plain_args(int dtype, const MmArgs& a) {
  KernelArgs p{};
  p.a = a;
  p.KS = (a.K + mm_kstep(dtype) - 1) / mm_kstep(dtype);
  return p;
}

template <int EPI>
hipError_t go(int dtype, const KernelArgs& p, hipStream_t st) {
  return dtype == LLM_F32 ? launch<float, EPI>(p, st) : launch<__bf16, EPI>(p, st);
}

}  // namespace

hipError_t mm_split(int dtype, const MmArgs& a, const MmSplit& e, hipStream_t st) {
  KernelArgs p = plain_args(dtype, a);
  p.split = e;
  return go<kSplit>(dtype, p, st);
}

hipError_t mm_glu(int dtype, const MmArgs& a, const GluParams& g, void* act, int ld, hipStream_t st) {
  KernelArgs p = plain_args(dtype, a);
  p.glu = g;
  p.split.t = act;
  p.split.ldt = ld;
  return go<kGlu>(dtype, p, st);
}

hipError_t mm_softplus(int dtype, const MmArgs& a, const float* bias, hipStream_t st) {
  KernelArgs p = plain_args(dtype, a);
  p.bias = bias;
  return go<kSoftplus>(dtype, p, st);
}

hipError_t mm_conv(int dtype, const MmArgs& a, const MmConv& e, hipStream_t st) {
  if (e.taps < 1 || e.taps > kMmConvTaps) return hipErrorInvalidValue;
  KernelArgs p = plain_args(dtype, a);
  p.conv = e;
  return go<kConv>(dtype, p, st);
}

hipError_t mm_latent(int dtype, const MmArgs& a, const MmLatent& e, hipStream_t st) {
  KernelArgs p = plain_args(dtype, a);
  p.lat = e;
  return go<kLatent>(dtype, p, st);
}

hipError_t mm_heads(int dtype, const MmArgs& a, const MmHeads& e, hipStream_t st) {
  if (a.M <= 0) return hipSuccess;
  KernelArgs p = plain_args(dtype, a);
  p.heads = e;
  return go<kHeads>(dtype, p, st);
}

hipError_t mm_expand(int dtype, const MmArgs& a, const MmPageRows& r, const MmQkv& e,
                     hipStream_t st) {
  KernelArgs p = plain_args(dtype, a);
  p.page_rows = r;
  p.q = e;
  return go<kExpand>(dtype, p, st);
}

}  // namespace llm
