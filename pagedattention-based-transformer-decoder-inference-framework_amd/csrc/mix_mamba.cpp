// The selective scan in the layer-stack model.
//
//   x | z product -> causal convolution, silu -> product of x to (dt | B | C) ->
//   dt product, softplus -> [prompt portions: chunk end states, carried over the
//   chunks] -> scan, gate -> o product
//
// Where every entry of the step is a single token the convolution is the first
// product's epilogue.
#include <algorithm>
#include <cmath>

#include "common.hpp"
#include "layer_stack_impl.hpp"

namespace llm {

int LayerStack::init_mamba(Layer& l) {
  const MambaSpec& m = l.s.mamba;
  const int ldc = mm_pad(m.inner);
  const int chunk = scan_chunk(m.state);
  int k = 0;
  for (; k < (int)scans_.size(); ++k)
    if (scans_[k].chunk == chunk) break;
  if (k == (int)scans_.size()) {
    scans_.emplace_back();
    scans_.back().chunk = chunk;
  }
  l.scan = k;
  ld_xz_ = std::max(ld_xz_, 2 * ldc);
  ld_inner_ = std::max(ld_inner_, ldc);
  ld_low_ = std::max(ld_low_, mm_pad(m.dt_rank));
  ld_bc_ = std::max(ld_bc_, 2 * up(m.state, 2));
  carry_floats_ = std::max(carry_floats_, (size_t)m.state * ldc);
  return LLM_OK;
}

int LayerStack::load_mamba(const SafeTensors& f, const std::string& mix, Layer& l) {
  const MambaSpec& m = l.s.mamba;
  const int ldc = mm_pad(m.inner), low = up(m.dt_rank, 2), state = up(m.state, 2);
  std::vector<int32_t> map;
  for (int part = 0; part < 2; ++part)  // x | z, each padded with zero columns
    for (int c = 0; c < ldc; ++c) map.push_back(c < m.inner ? part * m.inner + c : -1);
  RET_IF(load_packed(f, {{mix + "in", 2 * m.inner}}, cfg_.width, &map, l.in));
  map.clear();
  for (int n = 0; n < low; ++n) map.push_back(n < m.dt_rank ? n : -1);
  for (int part = 0; part < 2; ++part)
    for (int n = 0; n < state; ++n)
      map.push_back(n < m.state ? m.dt_rank + part * m.state + n : -1);
  RET_IF(load_packed(f, {{mix + "x", m.dt_rank + 2 * m.state}}, m.inner, &map, l.x));
  RET_IF(load_packed(f, {{mix + "dt", m.inner}}, m.dt_rank, nullptr, l.dt));
  RET_IF(load_packed(f, {{mix + "o", cfg_.width}}, m.inner, nullptr, l.o));
  RET_IF(load_vector(f, mix + "conv.b", m.inner, ldc, l.conv_bias));
  RET_IF(load_vector(f, mix + "dt.b", m.inner, ldc, l.dt_bias));
  RET_IF(load_vector(f, mix + "D", m.inner, ldc, l.D));
  std::vector<float> v, t((size_t)m.taps * ldc, 0.f);
  RET_IF(f.get_f32(mix + "conv", {m.inner, m.taps}, &v));
  for (int c = 0; c < m.inner; ++c)
    for (int k = 0; k < m.taps; ++k) t[(size_t)k * ldc + c] = v[(size_t)c * m.taps + k];
  RET_IF(upload_vec(l.conv, t));
  // A = -exp(A_log), kept as A log2(e) for exp2
  RET_IF(f.get_f32(mix + "A_log", {m.inner, m.state}, &v));
  t.assign((size_t)m.state * ldc, 0.f);
  for (int c = 0; c < m.inner; ++c)
    for (int n = 0; n < m.state; ++n)
      t[(size_t)n * ldc + c] = (float)(-std::exp((double)v[(size_t)c * m.state + n]) * M_LOG2E);
  return upload_vec(l.A, t);
}

void LayerStack::plan_scan(const std::vector<StepSeq>& batch, ScanPlan& p,
                           std::vector<ScanItem>& items, std::vector<ScanItem>& chunks,
                           std::vector<ScanCarry>& carry) {
  p.parts = 0;
  int seq0 = 0;
  for (const StepSeq& s : batch) {
    const int n = (s.n + p.chunk - 1) / p.chunk;
    for (int k = 0; k < n; ++k) {
      ScanItem it;
      it.tok0 = seq0 + k * p.chunk;
      it.n = std::min(p.chunk, s.n - k * p.chunk);
      it.seq0 = seq0;
      it.seq_n = s.n;
      it.slot = s.slot;
      it.p0 = s.p0;
      it.part = k > 0 ? p.parts + k - 1 : -1;
      it.last = k == n - 1;
      items.push_back(it);
      if (k == n - 1) continue;
      it.part = p.parts + k;
      it.last = k == 0;
      chunks.push_back(it);
    }
    if (n > 2) carry.push_back(ScanCarry{p.parts, n - 1});
    p.parts += n - 1;
    seq0 += s.n;
  }
  p.n_items = (int)items.size();
  p.n_chunks = (int)chunks.size();
  p.n_carry = (int)carry.size();
}

int LayerStack::mamba(const Layer& l, const Run& r, int M, hipStream_t st) {
  const MambaSpec& m = l.s.mamba;
  const int ldc = mm_pad(m.inner), low = up(m.dt_rank, 2), state = up(m.state, 2);
  const int ld_low = mm_pad(m.dt_rank);
  const bool fused = single_ && m.taps <= kMmConvTaps;
  uint8_t* z = xz_.p + (size_t)ldc * es_;  // z half of a row

  MmArgs a;
  a.A = h_.p;
  a.lda = ldx_;
  a.W = l.in.p;
  a.M = M;
  a.N = 2 * ldc;
  a.K = cfg_.width;
  a.w_nt = w_nt_;
  if (fused) {
    MmConv c;
    c.channels = m.inner;
    c.gate = ldc;
    c.taps = m.taps;
    c.pos = meta<int32_t>(at_pos_);
    c.slot = meta<int32_t>(at_slot_);
    c.w = l.conv.p;
    c.bias = l.conv_bias.p;
    c.ldw = ldc;
    c.history = r.state->history.p;
    c.x = xc_.p;
    c.ldx = ldc;
    c.z = z;
    c.ldz = 2 * ldc;
    LLM_HIP_RET(mm_conv(dt_, a, c, st));
  } else {
    MmSplit s;
    s.t = xz_.p;
    s.ldt = s.n_t = 2 * ldc;
    LLM_HIP_RET(mm_split(dt_, a, s, st));
    ConvArgs c;
    c.M = M;
    c.channels = m.inner;
    c.taps = m.taps;
    c.ldc = ldc;
    c.pos = meta<int32_t>(at_pos_);
    c.slot = meta<int32_t>(at_slot_);
    c.seq0 = meta<int32_t>(at_seq0_);
    c.in = xz_.p;
    c.ld_in = 2 * ldc;
    c.w = l.conv.p;
    c.bias = l.conv_bias.p;
    c.history = r.state->history.p;
    c.x = xc_.p;
    c.ldx = ldc;
    LLM_HIP_RET(causal_conv(dt_, c, st));
  }

  a.A = xc_.p;
  a.lda = ldc;
  a.W = l.x.p;
  a.N = low + 2 * state;
  a.K = m.inner;
  MmSplit s;
  s.t = low_.p;
  s.ldt = ld_low;
  s.n_t = low;
  s.f = bc_.p;
  s.ldf = 2 * state;
  LLM_HIP_RET(mm_split(dt_, a, s, st));

  a.A = low_.p;
  a.lda = ld_low;
  a.W = l.dt.p;
  a.N = m.inner;
  a.K = m.dt_rank;
  a.C = dtv_.p;
  a.ldc = ldc;
  LLM_HIP_RET(mm_softplus(dt_, a, l.dt_bias.p, st));

  const ScanPlan& p = scans_[l.scan];
  ScanArgs c;
  c.inner = m.inner;
  c.state = m.state;
  c.ldc = ldc;
  c.x = xc_.p;
  c.ldx = ldc;
  c.dt = dtv_.p;
  c.ldt = ldc;
  c.z = z;
  c.ldz = 2 * ldc;
  c.bc = bc_.p;
  c.ldb = 2 * state;
  c.c_at = state;
  c.A = l.A.p;
  c.D = l.D.p;
  c.out = gated_.p;
  c.ldo = ldc;
  c.slots = r.state->s.p;
  if (!fused) {
    c.taps = m.taps;
    c.raw = xz_.p;
    c.ld_raw = 2 * ldc;
    c.history = r.state->history.p;
  }
  c.carry = carry_.p;
  c.sum_dt = sum_dt_.p;
  LLM_HIP_RET(scan_chunks(dt_, c, meta<ScanItem>(p.chunks_at), p.n_chunks, st));
  LLM_HIP_RET(scan_carry(c, meta<ScanCarry>(p.carry_at), p.n_carry, st));
  LLM_HIP_RET(scan(dt_, c, meta<ScanItem>(p.items_at), p.n_items, st));
  return out_product(l, gated_.p, ldc, m.inner, M, st);
}

}  // namespace llm
