// The layer-stack model: weights, cache geometry and the step.
//
// One step runs every entry of a mixed batch (prompt portions beside single
// decoded tokens) as one list of token rows:
//   angles | embed + norm -> per layer run { mixer -> add + norm -> feed-forward
//   -> add + norm } -> norm of the wanted rows -> head product
// where a mixer is one of
//   attention: q|k|v product, rotation, append to the pages -> paged attention ->
//     o product
//   latent attention (mix_latent.cpp), selective scan (mix_mamba.cpp)
// and the feed-forward a gated pair of products, dense or of routed experts.
// Everything a step depends on besides the weights is in one device block
// (tokens, positions, slots, attention items, wanted rows) written by one copy,
// so a decode step's launches are captured into a hipGraph per shape and
// replayed.
//
// The cache: layers of one head geometry share a KvCache; each run of a layer is
// a cache layer of its own (or has a StateCache of its own), so a repeated layer
// keeps one cache or state per pass.
#include "layer_stack_impl.hpp"

#include <algorithm>
#include <cmath>
#include <cstring>
#include <mutex>

#include "common.hpp"
#include "paged_latent.hpp"

namespace llm {

std::vector<float> rope_frequencies(const RopeSpec& r, float* mul) {
  std::vector<float> f((size_t)r.dims / 2);
  *mul = 1.f;
  double lo = 0, hi = 0;
  if (r.yarn) {
    // the pair that turns t times within the original context
    const auto pair_at = [&](double t) {
      return r.dims * std::log(r.original / (2.0 * M_PI * t)) / (2.0 * std::log(r.base));
    };
    lo = std::max(std::floor(pair_at(r.fast)), 0.0);
    hi = std::min(std::ceil(pair_at(r.slow)), (double)(r.dims - 1));
    *mul = (float)(0.1 * std::log(r.factor) + 1.0);
  }
  for (size_t i = 0; i < f.size(); ++i) {
    const double w = std::pow(r.base, -2.0 * (double)i / r.dims);
    double ramp = 0.0;
    if (r.yarn) ramp = std::min(std::max(((double)i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
    f[i] = (float)(w / r.factor * ramp + w * (1.0 - ramp));
  }
  return f;
}

namespace {

constexpr int kDefaultStepTokens = 2048;
constexpr int kMaxSplits = 64;
constexpr int kTargetGroups = 512;   // workgroups an attention launch is split up to: 2 per CU
constexpr int kMinSplitPages = 4;    // a page per wave
constexpr int kMinLatentPages = 3;   // 16 rows x 4096 keys: 3 30.4 us, 4 35.3, 2 30.3 and a longer merge
constexpr size_t kMaxGraphs = 256;   // decode shapes kept captured
constexpr size_t kKeepBytes = (size_t)192 << 20;  // weights up to this stay in the Infinity Cache

int check_config(const LayerStackConfig& c, const ModelOptions& o) {
  LLM_REQUIRE(o.dtype == LLM_BF16 || o.dtype == LLM_F32, "model: dtype must be bfloat16 or float32");
  LLM_REQUIRE(o.max_seqs >= 1 && o.max_tokens >= 1, "model: max_seqs and max_tokens must be positive");
  LLM_REQUIRE(c.vocab > 0 && c.width > 0 && c.width <= 8192 && !c.layers.empty(),
              "config: vocab, width (<= 8192) and layers must be positive");
  LLM_REQUIRE(c.loop_times >= 1 && c.loop_start >= 0 && c.loop_start <= c.loop_stop &&
                  c.loop_stop <= (int)c.layers.size(),
              "config: bad loop");
  LLM_REQUIRE(c.streams >= 0 && c.streams <= kMaxStreams, "config: streams must be at most " +
                                                              std::to_string(kMaxStreams));
  const auto rope_ok = [](const RopeSpec& r) {
    return r.dims >= 0 && r.dims % 2 == 0 && (r.dims == 0 || r.base > 1.0);
  };
  for (size_t i = 0; i < c.layers.size(); ++i) {
    const LayerSpec& l = c.layers[i];
    const std::string at = "config: layer " + std::to_string(i) + ": ";
    if (l.mixer == Mixer::kAttention) {
      const AttentionSpec& a = l.attn;
      LLM_REQUIRE(a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0,
                  at + "heads must be a multiple of kv_heads");
      LLM_REQUIRE(a.dim > 0 && a.vdim > 0 && a.dim <= kGqaMaxDim && a.vdim <= kGqaMaxDim &&
                      a.dim % 2 == 0,
                  at + "head sizes must be in [1, 256] and dim even");
      LLM_REQUIRE(rope_ok(a.rope) && a.rope.dims <= a.dim,
                  at + "rot.dims must be even and at most dim, rot.base > 1");
    } else if (l.mixer == Mixer::kLatent) {
      const LatentSpec& a = l.latent;
      LLM_REQUIRE(a.heads > 0 && a.dim > 0 && a.vdim > 0 && a.rank > 0,
                  at + "heads, dim, vdim and kv_rank must be positive");
      LLM_REQUIRE(rope_ok(a.rope), at + "rot_dim must be even, rot.base > 1");
      LLM_REQUIRE(a.rank <= kLatentMaxRank && latent_row(a.rank, a.rot_dim) <= kLatentMaxRow,
                  at + "kv_rank is at most 512, with rot_dim at most 576");
    } else {
      const MambaSpec& m = l.mamba;
      LLM_REQUIRE(m.inner > 0 && m.dt_rank > 0 && m.taps > 0 && m.state > 0 && m.state <= kMaxScanState,
                  at + "inner, dt_rank and conv must be positive, state in [1, 256]");
    }
    if (!l.has_mlp) continue;
    if (l.dense) {
      LLM_REQUIRE(l.ffn.ff >= 1, at + "mlp.ff must be positive");
      continue;
    }
    const MoeSpec& m = l.moe;
    LLM_REQUIRE(m.experts >= 1 && m.experts <= kMaxExperts && m.top >= 1 && m.top <= m.experts &&
                    m.expert.ff >= 1 && (!m.has_shared || m.shared.ff >= 1),
                at + "bad expert sizes");
  }
  return LLM_OK;
}

}  // namespace

int LayerStack::init(const LayerStackConfig& cfg, const std::string& dir, const ModelOptions& opt) {
  RET_IF(check_config(cfg, opt));
  cfg_ = cfg;
  opt_ = opt;
  dt_ = opt.dtype;
  es_ = mm_elem_size(dt_);
  ldx_ = mm_pad(cfg.width);
  cap_ = opt.max_step_tokens > 0 ? opt.max_step_tokens : kDefaultStepTokens;
  pool_pages_ = (opt.max_tokens + kPageTokens - 1) / kPageTokens;
  const long long len = opt.max_seq_len > 0 ? std::min<long long>(opt.max_seq_len, opt.max_tokens)
                                            : opt.max_tokens;
  LLM_REQUIRE(pool_pages_ * kPageTokens < (1LL << 30), "model: max_tokens too large");
  max_len_ = up((int)len, kPageTokens);
  use_graph_ = env_int("LLM_GRAPH", 1) != 0;

  for (const LayerSpec& s : cfg.layers) {
    auto l = std::make_unique<Layer>();
    l->s = s;
    if (s.mixer == Mixer::kLatent) {
      RET_IF(init_latent(*l));
    } else if (s.mixer == Mixer::kMamba) {
      RET_IF(init_mamba(*l));
    } else {
      const AttentionSpec& a = s.attn;
      l->geo = find_geometry(false, a.kv_heads, a.dim, a.vdim);
      const Geometry& geo = *geos_[l->geo];
      RET_IF(find_rope(a.rope, &l->rope));
      auto p = std::make_unique<Plan>();
      p->R = a.heads / a.kv_heads;
      p->G = a.kv_heads;
      p->big_tile = gqa_tile_rows(dt_, geo.Dp, geo.Dvp, 1 << 20);
      p->max_pd = gqa_part_dim(a.vdim);
      l->plan = add_plan(std::move(p));
      ld_q_ = std::max(ld_q_, a.heads * geo.Dp);
      ld_att_ = std::max(ld_att_, mm_pad(a.heads * a.vdim));
    }
    if (s.has_mlp && s.dense) {
      ld_act_ = std::max(ld_act_, mm_pad(s.ffn.ff));
    } else if (s.has_mlp) {
      max_top_ = std::max(max_top_, s.moe.top);
      max_e_ = std::max(max_e_, s.moe.experts);
      ld_act_ = std::max(ld_act_, mm_pad(s.moe.expert.ff));
      if (s.moe.has_shared) ld_shared_ = std::max(ld_shared_, mm_pad(s.moe.shared.ff));
    }
    layers_.push_back(std::move(l));
  }
  for (int i = 0; i < cfg.loop_start; ++i) RET_IF(add_run(i, false));
  for (int p = 0; p < cfg.loop_times; ++p)
    for (int i = cfg.loop_start; i < cfg.loop_stop; ++i) RET_IF(add_run(i, p > 0 && i == cfg.loop_start));
  for (int i = cfg.loop_stop; i < (int)layers_.size(); ++i) RET_IF(add_run(i, false));

  for (auto& g : geos_) {
    if (g->layers == 0) continue;
    RET_IF(g->kv.init(g->layers, opt.max_seqs, g->G, g->Dp, kPageTokens, max_len_ / kPageTokens,
                      pool_pages_ * g->layers * g->G, dt_, g->latent ? -1 : g->Dvp));
    RET_IF(g->kv.zero_pools(nullptr));
  }
  LLM_HIP_RET(hipEventCreateWithFlags(&meta_done_, hipEventDisableTiming));
  LLM_HIP_RET(hipStreamCreateWithFlags(&cap_stream_, hipStreamNonBlocking));
  RET_IF(load(dir));
  w_nt_ = weight_bytes_ > kKeepBytes;
  return LLM_OK;
}

int LayerStack::find_rope(const RopeSpec& spec, int* index) {
  *index = -1;
  if (spec.dims == 0) return LLM_OK;
  int r = 0;
  for (; r < (int)ropes_.size(); ++r)
    if (ropes_[r]->spec == spec) break;
  if (r == (int)ropes_.size()) {
    auto n = std::make_unique<Rope>();
    n->spec = spec;
    RET_IF(upload_vec(n->freq, rope_frequencies(spec, &n->mul)));
    ropes_.push_back(std::move(n));
  }
  *index = r;
  return LLM_OK;
}

int LayerStack::find_geometry(bool latent, int G, int D, int Dv) {
  for (size_t g = 0; g < geos_.size(); ++g)
    if (geos_[g]->latent == latent && geos_[g]->G == G && geos_[g]->D == D && geos_[g]->Dv == Dv)
      return (int)g;
  auto n = std::make_unique<Geometry>();
  n->latent = latent;
  n->G = G;
  n->D = D;
  n->Dv = Dv;
  n->Dp = latent ? latent_row(D, Dv) : up(D, 8);
  n->Dvp = latent ? 0 : up(Dv, 8);
  geos_.push_back(std::move(n));
  return (int)geos_.size() - 1;
}

int LayerStack::add_plan(std::unique_ptr<Plan> p) {
  size_t k = 0;
  for (; k < plans_.size(); ++k)
    if (plans_[k]->same(*p)) break;
  const int pd = p->max_pd;
  if (k == plans_.size()) plans_.push_back(std::move(p));
  plans_[k]->max_pd = std::max(plans_[k]->max_pd, pd);
  return (int)k;
}

int LayerStack::add_run(int layer, bool again) {
  const Layer& l = *layers_[layer];
  Run r;
  r.layer = layer;
  r.again = again;
  if (l.geo >= 0) r.cache_layer = geos_[l.geo]->layers++;
  if (l.s.mixer == Mixer::kMamba) {
    const MambaSpec& m = l.s.mamba;
    r.state = std::make_unique<StateCache>();
    RET_IF(r.state->init(opt_.max_seqs, m.state, mm_pad(m.inner), m.taps, es_));
  }
  runs_.push_back(std::move(r));
  return LLM_OK;
}

// ---------------------------------------------------------------------------
// weights
// ---------------------------------------------------------------------------

// Pack the rows of one or more [rows][K] tensors, stacked and then reordered by
// `map` (packed column n takes stacked row map[n], zeros where it is -1).
int LayerStack::pack_rows(const SafeTensors& f,
                          const std::vector<std::pair<std::string, int>>& parts, int K,
                          const std::vector<int32_t>* map, uint8_t* dst) {
  int N = 0;
  for (const auto& p : parts) N += p.second;
  const size_t need = (size_t)N * K * 2;
  if (staging_.n < need) RET_IF(staging_.alloc(need));
  size_t at = 0;
  for (const auto& p : parts) {
    TensorView t;
    RET_IF(f.get(p.first, {p.second, K}, &t));
    if (t.dtype != "BF16")
      return fail(LLM_ERR_IO, "weights: " + p.first + " is " + t.dtype + ", expected BF16");
    LLM_HIP_RET(hipMemcpy(staging_.p + at, t.data, t.bytes, hipMemcpyHostToDevice));
    at += t.bytes;
  }
  if (map) {
    N = (int)map->size();
    RET_IF(upload_vec(map_, *map));
  }
  LLM_HIP_RET(mm_pack(dt_, reinterpret_cast<const uint16_t*>(staging_.p), map ? map_.p : nullptr, N,
                      K, dst, nullptr));
  LLM_HIP_RET(hipStreamSynchronize(nullptr));  // staging and map are used again
  weight_bytes_ += mm_packed_bytes(dt_, N, K);
  return LLM_OK;
}

int LayerStack::pack_host(const std::vector<uint16_t>& rows, int K, const std::vector<int32_t>* map,
                          uint8_t* dst) {
  const size_t need = rows.size() * 2;
  if (staging_.n < need) RET_IF(staging_.alloc(need));
  LLM_HIP_RET(hipMemcpy(staging_.p, rows.data(), need, hipMemcpyHostToDevice));
  const int N = map ? (int)map->size() : (int)(rows.size() / K);
  if (map) RET_IF(upload_vec(map_, *map));
  LLM_HIP_RET(mm_pack(dt_, reinterpret_cast<const uint16_t*>(staging_.p), map ? map_.p : nullptr, N,
                      K, dst, nullptr));
  LLM_HIP_RET(hipStreamSynchronize(nullptr));
  weight_bytes_ += mm_packed_bytes(dt_, N, K);
  return LLM_OK;
}

int LayerStack::load_packed(const SafeTensors& f,
                            const std::vector<std::pair<std::string, int>>& parts, int K,
                            const std::vector<int32_t>* map, DevBuf<uint8_t>& b) {
  int N = 0;
  for (const auto& p : parts) N += p.second;
  RET_IF(b.alloc(mm_packed_bytes(dt_, map ? (int)map->size() : N, K)));
  return pack_rows(f, parts, K, map, b.p);
}

int LayerStack::load_vector(const SafeTensors& f, const std::string& name, int n, int padded,
                            DevBuf<float>& b) {
  std::vector<float> v;
  RET_IF(f.get_f32(name, {n}, &v));
  v.resize(padded, 0.f);
  return upload_vec(b, v);
}

int LayerStack::load_hyper(const SafeTensors& f, const std::string& name, Hyper& h) {
  const int S = cfg_.streams;
  std::vector<float> v;
  RET_IF(load_vector(f, name + ".in", S, S, h.in));
  RET_IF(load_vector(f, name + ".out", S, S, h.out));
  RET_IF(f.get_f32(name + ".mix", {S, S}, &v));
  return upload_vec(h.mix, v);
}

// column 2i: gate i, 2i + 1: up i
static std::vector<int32_t> gate_up_rows(int ff) {
  std::vector<int32_t> v((size_t)2 * ff);
  for (int n = 0; n < 2 * ff; ++n) v[n] = (n & 1) * ff + n / 2;
  return v;
}

int LayerStack::load(const std::string& dir) {
  SafeTensors f;
  RET_IF(f.open(dir + "/model.safetensors"));
  const int W = cfg_.width;
  {
    std::vector<uint16_t> e;
    RET_IF(f.get_bf16("embed", {cfg_.vocab, W}, &e));
    std::vector<uint16_t> p((size_t)cfg_.vocab * ldx_, 0);
    for (int v = 0; v < cfg_.vocab; ++v)
      std::memcpy(&p[(size_t)v * ldx_], &e[(size_t)v * W], (size_t)W * 2);
    RET_IF(upload_vec(emb_, p));
  }
  for (size_t i = 0; i < layers_.size(); ++i) {
    Layer& l = *layers_[i];
    const std::string at = "l" + std::to_string(i) + ".", mix = at + "mix.", ml = at + "mlp.";
    RET_IF(load_vector(f, at + "norm1", W, ldx_, l.norm1));
    if (cfg_.post_norm) RET_IF(load_vector(f, at + "norm1b", W, ldx_, l.norm1b));
    if (cfg_.layer_scale) RET_IF(load_vector(f, at + "ls1", W, ldx_, l.ls1));
    if (cfg_.streams > 0) RET_IF(load_hyper(f, at + "hc1", l.hc1));
    switch (l.s.mixer) {
      case Mixer::kAttention: RET_IF(load_attention(f, mix, l)); break;
      case Mixer::kLatent: RET_IF(load_latent(f, mix, l)); break;
      case Mixer::kMamba: RET_IF(load_mamba(f, mix, l)); break;
    }
    if (!l.s.has_mlp) continue;
    RET_IF(load_vector(f, at + "norm2", W, ldx_, l.norm2));
    if (cfg_.post_norm) RET_IF(load_vector(f, at + "norm2b", W, ldx_, l.norm2b));
    if (cfg_.layer_scale) RET_IF(load_vector(f, at + "ls2", W, ldx_, l.ls2));
    if (cfg_.streams > 0) RET_IF(load_hyper(f, at + "hc2", l.hc2));
    if (l.s.dense) {
      const int ff = l.s.ffn.ff;
      const std::vector<int32_t> pairs = gate_up_rows(ff);
      RET_IF(load_packed(f, {{ml + "gate", ff}, {ml + "up", ff}}, W, &pairs, l.ffn_in));
      RET_IF(load_packed(f, {{ml + "down", W}}, ff, nullptr, l.ffn_out));
    } else {
      RET_IF(load_moe(f, ml, l));
    }
  }
  RET_IF(load_vector(f, "final.norm", W, ldx_, final_norm_));
  RET_IF(load_packed(f, {{"head", cfg_.vocab}}, W, nullptr, head_));
  RET_IF(staging_.alloc(0));
  RET_IF(map_.alloc(0));
  return LLM_OK;
}

int LayerStack::load_attention(const SafeTensors& f, const std::string& mix, Layer& l) {
  const AttentionSpec& a = l.s.attn;
  // q | k | v with rotation partners side by side
  const int nq = a.heads * a.dim, nk = a.kv_heads * a.dim, nv = a.kv_heads * a.vdim;
  l.n_qkv = nq + nk + nv;
  std::vector<int32_t> map((size_t)l.n_qkv);
  const int half = a.rope.dims / 2;
  for (int n = 0; n < l.n_qkv; ++n) {
    const int d = n % a.dim;
    map[n] = n < nq + nk && d < a.rope.dims ? n - d + d / 2 + (d & 1) * half : n;
  }
  RET_IF(load_packed(f, {{mix + "q", nq}, {mix + "k", nk}, {mix + "v", nv}}, cfg_.width, &map, l.qkv));
  RET_IF(load_packed(f, {{mix + "o", cfg_.width}}, a.heads * a.vdim, nullptr, l.o));
  if (a.sink) RET_IF(load_vector(f, mix + "sink", a.heads, a.heads, l.sink));
  return LLM_OK;
}

int LayerStack::load_moe(const SafeTensors& f, const std::string& ml, Layer& l) {
  const MoeSpec& m = l.s.moe;
  const int W = cfg_.width;
  RET_IF(load_packed(f, {{ml + "router", m.experts}}, W, nullptr, l.router));
  RET_IF(load_vector(f, ml + "correction", m.experts, m.experts, l.correction));
  const auto describe = [&](const ExpertSpec& e, const uint8_t* in, const uint8_t* out) {
    MmGroup g;
    g.w_in = in;
    g.w_out = out;
    g.n_in = 2 * e.ff;
    g.ks_in = (W + mm_kstep(dt_) - 1) / mm_kstep(dt_);
    g.n_out = W;
    g.ks_out = (e.ff + mm_kstep(dt_) - 1) / mm_kstep(dt_);
    g.glu = e.glu;
    return g;
  };
  std::vector<MmGroup> groups;
  const int ff = m.expert.ff;
  const size_t b_in = mm_packed_bytes(dt_, 2 * ff, W), b_out = mm_packed_bytes(dt_, W, ff);
  RET_IF(l.experts_in.alloc(b_in * m.experts));
  RET_IF(l.experts_out.alloc(b_out * m.experts));
  const std::vector<int32_t> pairs = gate_up_rows(ff);
  for (int e = 0; e < m.experts; ++e) {
    const std::string ex = ml + "e" + std::to_string(e) + ".";
    uint8_t *in = l.experts_in.p + b_in * e, *out = l.experts_out.p + b_out * e;
    RET_IF(pack_rows(f, {{ex + "gate", ff}, {ex + "up", ff}}, W, &pairs, in));
    RET_IF(pack_rows(f, {{ex + "down", W}}, ff, nullptr, out));
    groups.push_back(describe(m.expert, in, out));
  }
  if (m.has_shared) {
    const int sf = m.shared.ff;
    const std::vector<int32_t> sp = gate_up_rows(sf);
    RET_IF(load_packed(f, {{ml + "shared.gate", sf}, {ml + "shared.up", sf}}, W, &sp, l.shared_in));
    RET_IF(load_packed(f, {{ml + "shared.down", W}}, sf, nullptr, l.shared_out));
    groups.push_back(describe(m.shared, l.shared_in.p, l.shared_out.p));
  }
  return upload_vec(l.groups, groups);
}

// ---------------------------------------------------------------------------
// step
// ---------------------------------------------------------------------------
int LayerStack::ensure_rows(int M) {
  if (M <= rows_) return LLM_OK;
  int n = 64;
  while (n < M) n *= 2;
  n = std::max(M, std::min(n, cap_));
  LLM_HIP_RET(hipDeviceSynchronize());
  clear_graphs();
  rows_ = 0;
  RET_IF(alloc_zero(x_, (size_t)n * std::max(cfg_.streams, 1) * ldx_));
  RET_IF(alloc_zero(h_, (size_t)n * ldx_ * es_));
  // (a product may read whole k-steps past the last row's end)
  const size_t slack = (size_t)64 * es_;
  RET_IF(alloc_zero(q_, (size_t)n * ld_q_ * es_ + slack));
  RET_IF(alloc_zero(att_, (size_t)n * ld_att_ * es_));
  RET_IF(alloc_zero(y_, (size_t)n * (max_top_ + 1) * ldx_));
  RET_IF(alloc_zero(act_, (size_t)n * std::max(max_top_, 1) * ld_act_ * es_));
  RET_IF(alloc_zero(q_lat_, (size_t)n * ld_qlat_ * es_ + slack));
  RET_IF(alloc_zero(o_lat_, (size_t)n * ld_olat_ * es_ + slack));
  RET_IF(alloc_zero(down_, (size_t)n * ld_down_));
  RET_IF(alloc_zero(xz_, (size_t)n * ld_xz_ * es_));
  RET_IF(alloc_zero(xc_, (size_t)n * ld_inner_ * es_));
  RET_IF(alloc_zero(gated_, (size_t)n * ld_inner_ * es_));
  RET_IF(alloc_zero(dtv_, (size_t)n * ld_inner_));
  RET_IF(alloc_zero(low_, (size_t)n * ld_low_ * es_));
  RET_IF(alloc_zero(bc_, (size_t)n * ld_bc_));
  if (max_top_ > 0) {
    RET_IF(alloc_zero(z_, (size_t)n * max_e_));
    RET_IF(alloc_zero(act_shared_, (size_t)n * ld_shared_ * es_));
    RET_IF(alloc_zero(weight_, (size_t)n * max_top_));
    RET_IF(alloc_zero(choice_, (size_t)n * max_top_));
    RET_IF(alloc_zero(perm_, (size_t)n * max_top_));
    RET_IF(alloc_zero(tiles_, (size_t)route_max_tiles(n, max_top_, kMaxExperts, true, 16)));
    RET_IF(alloc_zero(n_tiles_, 1));
  }
  for (auto& r : ropes_) RET_IF(alloc_zero(r->turn, (size_t)n * (r->spec.dims / 2)));
  LLM_HIP_RET(hipDeviceSynchronize());
  rows_ = n;
  return LLM_OK;
}

// The row tiles of one attention launch: the plan's sequences that bring few rows
// per key/value head (big false) or many, split over their pages until the launch
// holds about kTargetGroups workgroups; long tiles first.
void LayerStack::cut(const std::vector<StepSeq>& batch, Plan& p, bool big,
                     std::vector<GqaItem>& items, std::vector<GqaMerge>& merges, Launch& l) {
  l = Launch();
  l.tile_rows = big ? p.big_tile : p.small_tile;
  const auto mine = [&](const StepSeq& s) {
    return s.n >= p.min_n && s.n <= p.max_n && ((s.n * p.R > p.small_max) == big);
  };
  long long tiles = 0;
  int max_pages = 1, tok0 = 0, entry = 0;
  for (const StepSeq& s : batch) {
    if (!mine(s)) continue;
    const int rows = s.n * p.R;
    tiles += (rows + l.tile_rows - 1) / l.tile_rows;
    max_pages = std::max(max_pages, (s.p0 + s.n - 1) / kPageTokens + 1);
  }
  if (tiles == 0) return;
  const int want = (int)std::min<long long>(std::max<long long>(kTargetGroups / (tiles * p.G), 1), kMaxSplits);
  // single tokens share one split count, so a decode step keeps its launch
  // shape (and graph) while contexts grow
  const int least = p.latent ? kMinLatentPages : kMinSplitPages;
  const int common = std::min(want, (max_pages + least - 1) / least);
  for (const StepSeq& s : batch) {
    const int rows = s.n * p.R;
    const int t0 = tok0;
    tok0 += s.n;
    const int slot = p.expand ? entry : s.slot;  // expanded keys have a table of their own
    entry += s.n >= p.min_n && s.n <= p.max_n;
    if (!mine(s)) continue;
    for (int r0 = 0; r0 < rows; r0 += l.tile_rows) {
      const int last = s.p0 + (std::min(r0 + l.tile_rows, rows) - 1) / p.R;
      const int pages = last / kPageTokens + 1;
      const int ns = big ? std::min(want, (pages + least - 1) / least) : common;
      for (int k = 0; k < ns; ++k)
        items.push_back(GqaItem{t0, slot, s.p0, r0, rows, (int)((long long)pages * k / ns),
                                (int)((long long)pages * (k + 1) / ns), ns > 1 ? l.parts + k : -1});
      l.n_items += ns;
      if (ns > 1) {
        merges.push_back(GqaMerge{t0, r0, rows, l.parts, ns});
        l.n_merges += 1;
        l.parts += ns;
      }
    }
  }
  if (big)
    std::stable_sort(items.begin(), items.end(), [](const GqaItem& x, const GqaItem& y) {
      return x.page1 - x.page0 > y.page1 - y.page0;
    });
}

int LayerStack::build_meta(const std::vector<StepSeq>& batch, int M, int n_want, hipStream_t st) {
  // pieces of the block besides the token rows, in their places
  std::vector<std::pair<size_t, std::vector<uint8_t>>> pieces;
  size_t at = 0, part_o = 0, part_ml = 0;
  const auto take = [&](size_t bytes) {
    const size_t a = at;
    at += (bytes + 15) / 16 * 16;
    return a;
  };
  const auto place = [&](const auto& v) {
    const size_t bytes = v.size() * sizeof(v[0]), a = take(bytes);
    if (bytes) {
      const uint8_t* b = reinterpret_cast<const uint8_t*>(v.data());
      pieces.emplace_back(a, std::vector<uint8_t>(b, b + bytes));
    }
    return a;
  };
  at_tok_ = take((size_t)M * 4);
  at_pos_ = take((size_t)M * 4);
  at_slot_ = take((size_t)M * 4);
  at_seq0_ = take((size_t)M * 4);
  at_want_ = take((size_t)n_want * 4);
  for (auto& pp : plans_) {
    Plan& p = *pp;
    for (int b = 0; b < 2; ++b) {
      Launch& l = b ? p.big : p.small;
      std::vector<GqaItem> items;
      std::vector<GqaMerge> merges;
      cut(batch, p, b != 0, items, merges, l);
      l.items_at = place(items);
      l.merges_at = place(merges);
      const size_t rows = (size_t)l.parts * p.G * l.tile_rows;
      part_o = std::max(part_o, rows * p.max_pd);
      part_ml = std::max(part_ml, rows * 2);
    }
    if (p.latent) {
      std::vector<int32_t> rows;
      int m = 0;
      for (const StepSeq& s : batch) {
        for (int i = 0; i < s.n; ++i)
          if (s.n >= p.min_n && s.n <= p.max_n) rows.push_back(m + i);
        m += s.n;
      }
      p.n_rows = (int)rows.size();
      p.rows_at = place(rows);
    }
    if (p.expand) {
      std::vector<int32_t> pos, slot, entry, table;
      plan_expansion(batch, p, pos, slot, entry, table);
      p.x_pos = place(pos);
      p.x_slot = place(slot);
      p.x_entry = place(entry);
      p.x_table = place(table);
      const size_t bytes = (size_t)p.x_pages * kPageTokens * (p.Dp + p.Dvp) * es_;
      if (bytes > p.pool.n) {
        LLM_HIP_RET(hipDeviceSynchronize());
        RET_IF(alloc_zero(p.pool, bytes + bytes / 4));  // (zeros: padding of the rows)
        LLM_HIP_RET(hipDeviceSynchronize());
      }
    }
  }
  size_t parts = 0;
  for (ScanPlan& p : scans_) {
    std::vector<ScanItem> items, chunks;
    std::vector<ScanCarry> carry;
    plan_scan(batch, p, items, chunks, carry);
    p.items_at = place(items);
    p.chunks_at = place(chunks);
    p.carry_at = place(carry);
    parts = std::max(parts, (size_t)p.parts);
  }
  if (part_o > part_o_.n || part_ml > part_ml_.n || at > meta_cap_ ||
      parts * carry_floats_ > carry_.n) {
    LLM_HIP_RET(hipDeviceSynchronize());
    clear_graphs();
    if (part_o > part_o_.n) RET_IF(part_o_.alloc(part_o * 2));
    if (part_ml > part_ml_.n) RET_IF(part_ml_.alloc(part_ml * 2));
    if (parts * carry_floats_ > carry_.n) {
      RET_IF(carry_.alloc(parts * carry_floats_));
      RET_IF(sum_dt_.alloc(parts * ld_inner_));
    }
    if (at > meta_cap_) {
      if (h_meta_) LLM_HIP_RET(hipHostFree(h_meta_));
      h_meta_ = nullptr;
      meta_cap_ = 0;
      const size_t cap = std::max<size_t>(at * 2, 1 << 16);
      RET_IF(meta_.alloc(cap));
      LLM_HIP_RET(hipHostMalloc(reinterpret_cast<void**>(&h_meta_), cap, hipHostMallocDefault));
      meta_cap_ = cap;
    }
  }
  LLM_HIP_RET(hipEventSynchronize(meta_done_));  // the previous step's copy
  int32_t* tok = reinterpret_cast<int32_t*>(h_meta_ + at_tok_);
  int32_t* pos = reinterpret_cast<int32_t*>(h_meta_ + at_pos_);
  int32_t* slot = reinterpret_cast<int32_t*>(h_meta_ + at_slot_);
  int32_t* seq0 = reinterpret_cast<int32_t*>(h_meta_ + at_seq0_);
  int32_t* want = reinterpret_cast<int32_t*>(h_meta_ + at_want_);
  int m = 0, w = 0;
  for (const StepSeq& s : batch) {
    const int first = m;
    for (int i = 0; i < s.n_want; ++i) want[w++] = m + s.want[i];
    for (int i = 0; i < s.n; ++i, ++m) {
      tok[m] = s.tokens[i];
      pos[m] = s.p0 + i;
      slot[m] = s.slot;
      seq0[m] = first;
    }
  }
  for (const auto& p : pieces) std::memcpy(h_meta_ + p.first, p.second.data(), p.second.size());
  LLM_HIP_RET(hipMemcpyAsync(meta_.p, h_meta_, at, hipMemcpyHostToDevice, st));
  LLM_HIP_RET(hipEventRecord(meta_done_, st));
  return LLM_OK;
}

int LayerStack::attention(const Layer& l, const Run& r, int M, hipStream_t st) {
  const AttentionSpec& a = l.s.attn;
  Geometry& g = *geos_[l.geo];
  const KvCache& kv = g.kv;
  const int32_t* table = table_of(g, r);
  MmArgs p;
  p.A = h_.p;
  p.lda = ldx_;
  p.W = l.qkv.p;
  p.M = M;
  p.N = l.n_qkv;
  p.K = cfg_.width;
  p.w_nt = w_nt_;
  MmQkv e;
  e.pos = meta<int32_t>(at_pos_);
  e.slot = meta<int32_t>(at_slot_);
  e.turn = l.rope >= 0 ? ropes_[l.rope]->turn.p : nullptr;
  e.rot = a.rope.dims;
  e.H = a.heads;
  e.G = a.kv_heads;
  e.D = a.dim;
  e.Dv = a.vdim;
  e.Dp = g.Dp;
  e.Dvp = g.Dvp;
  e.q = q_.p;
  e.table = table;
  e.slots = kv.beams;
  e.max_tiles = kv.max_tiles;
  e.num_pages = (int)kv.num_pages;
  e.k_pool = kv.k_pool;
  e.v_pool = kv.v_pool;
  e.page_stride = kv.page_stride();
  LLM_HIP_RET(mm_qkv(dt_, p, e, st));

  const Plan& plan = *plans_[l.plan];
  const int ldo = mm_pad(a.heads * a.vdim);
  GqaArgs q;
  q.q = q_.p;
  q.out = att_.p;
  q.ldo = ldo;
  q.k_pool = kv.k_pool;
  q.v_pool = kv.v_pool;
  q.page_stride = kv.page_stride();
  q.table = table;
  q.max_tiles = kv.max_tiles;
  q.num_pages = (int)kv.num_pages;
  q.H = a.heads;
  q.G = a.kv_heads;
  q.Dp = g.Dp;
  q.Dv = g.Dv;
  q.Dvp = g.Dvp;
  q.scale = a.scale;
  q.sink = a.sink ? l.sink.p : nullptr;
  q.part_o = part_o_.p;
  q.part_ml = part_ml_.p;
  for (const Launch* c : {&plan.small, &plan.big}) {
    if (c->n_items == 0) continue;
    q.items = meta<GqaItem>(c->items_at);
    q.n_items = c->n_items;
    q.merges = meta<GqaMerge>(c->merges_at);
    q.n_merges = c->n_merges;
    LLM_HIP_RET(gqa_attention(dt_, q, c->tile_rows, st));
  }

  return out_product(l, att_.p, ldo, a.heads * a.vdim, M, st);
}

int LayerStack::out_product(const Layer& l, const void* A, int lda, int K, int M, hipStream_t st) {
  MmArgs o;
  o.A = A;
  o.lda = lda;
  o.W = l.o.p;
  o.M = M;
  o.N = cfg_.width;
  o.K = K;
  o.w_nt = w_nt_;
  o.C = y_.p;
  o.ldc = ldx_;
  LLM_HIP_RET(mm(dt_, o, st));
  return LLM_OK;
}

int LayerStack::ffn(const Layer& l, int M, hipStream_t st) {
  MmArgs a;
  a.A = h_.p;
  a.lda = ldx_;
  a.W = l.ffn_in.p;
  a.M = M;
  a.N = 2 * l.s.ffn.ff;
  a.K = cfg_.width;
  a.w_nt = w_nt_;
  const int ld = mm_pad(l.s.ffn.ff);
  LLM_HIP_RET(mm_glu(dt_, a, l.s.ffn.glu, act_.p, ld, st));
  a.A = act_.p;
  a.lda = ld;
  a.W = l.ffn_out.p;
  a.N = cfg_.width;
  a.K = l.s.ffn.ff;
  a.C = y_.p;
  a.ldc = ldx_;
  LLM_HIP_RET(mm(dt_, a, st));
  return LLM_OK;
}

int LayerStack::moe(const Layer& l, int M, hipStream_t st) {
  const MoeSpec& m = l.s.moe;
  MmArgs z;
  z.A = h_.p;
  z.lda = ldx_;
  z.W = l.router.p;
  z.M = M;
  z.N = m.experts;
  z.K = cfg_.width;
  z.C = z_.p;
  z.ldc = m.experts;
  LLM_HIP_RET(mm(dt_, z, st));
  RouteArgs r;
  r.z = z_.p;
  r.ldz = m.experts;
  r.M = M;
  r.experts = m.experts;
  r.top = m.top;
  r.correction = l.correction.p;
  r.scale = m.scale;
  r.shared = m.has_shared;
  r.tile_rows = mm_group_tile_rows(M, m.top, m.experts);
  r.choice = choice_.p;
  r.weight = weight_.p;
  r.perm = perm_.p;
  r.tiles = tiles_.p;
  r.n_tiles = n_tiles_.p;
  LLM_HIP_RET(route(r, st));
  MmGrouped g;
  g.groups = l.groups.p;
  g.tiles = tiles_.p;
  g.n_tiles = n_tiles_.p;
  g.perm = perm_.p;
  g.weight = weight_.p;
  g.n_routed = m.experts;
  g.top = m.top;
  g.M = M;
  g.max_tiles = route_max_tiles(M, m.top, m.experts, m.has_shared, r.tile_rows);
  g.tile_rows = r.tile_rows;
  g.h = h_.p;
  g.ldh = ldx_;
  g.act = act_.p;
  g.lda = mm_pad(m.expert.ff);
  g.act_shared = act_shared_.p;
  g.lds = m.has_shared ? mm_pad(m.shared.ff) : 0;
  g.out = y_.p;
  g.ldo = ldx_;
  g.max_n = 2 * std::max(m.expert.ff, m.has_shared ? m.shared.ff : 0);
  g.min_ks = (cfg_.width + mm_kstep(dt_) - 1) / mm_kstep(dt_);
  LLM_HIP_RET(mm_grouped_in(dt_, g, w_nt_, st));
  g.max_n = cfg_.width;
  g.min_ks = (m.expert.ff + mm_kstep(dt_) - 1) / mm_kstep(dt_);
  LLM_HIP_RET(mm_grouped_out(dt_, g, w_nt_, st));
  return LLM_OK;
}

int LayerStack::enqueue(int M, int n_want, float* logits, hipStream_t st) {
  for (auto& r : ropes_)
    LLM_HIP_RET(rope_turns(meta<int32_t>(at_pos_), M, r->freq.p, r->spec.dims / 2, r->mul,
                           r->turn.p, st));
  NormStep n;  // what the previous sublayer left to add
  const auto fresh = [&]() {
    n = NormStep();
    n.x = x_.p;
    n.ldx = ldx_;
    n.width = cfg_.width;
    n.M = n.M_y = M;
    n.eps = cfg_.eps;
    n.emb = emb_.p;
    n.emb_scale = cfg_.embedding_scale;
    n.tok = meta<int32_t>(at_tok_);
    n.ldh = ldx_;
    n.h = h_.p;
    n.streams = cfg_.streams;
  };
  const auto leave = [&](const DevBuf<float>& post, const DevBuf<float>& scale, const Hyper& hc,
                         int parts, bool shared) {
    fresh();
    n.w_post = post.p;
    n.y_scale = scale.p;
    n.hc_mix = hc.mix.p;
    n.hc_out = hc.out.p;
    n.y = y_.p;
    n.ldy = ldx_;
    n.parts = parts;
    n.shared = shared;
  };
  const auto enter = [&](const DevBuf<float>& norm, const Hyper& hc) {
    n.w_pre = norm.p;
    n.hc_in = hc.in.p;
    return rms_norm_step(dt_, n, st);
  };
  fresh();
  n.embed = 1;
  for (size_t i = 0; i < runs_.size(); ++i) {
    const Run& r = runs_[i];
    const Layer& l = *layers_[r.layer];
    if (r.again && cfg_.loop_adds_embedding) n.embed = 2;
    LLM_HIP_RET(enter(l.norm1, l.hc1));
    switch (l.s.mixer) {
      case Mixer::kAttention: RET_IF(attention(l, r, M, st)); break;
      case Mixer::kLatent: RET_IF(latent(l, r, M, st)); break;
      case Mixer::kMamba: RET_IF(mamba(l, r, M, st)); break;
    }
    leave(l.norm1b, l.ls1, l.hc1, 1, false);
    if (l.s.has_mlp) {
      LLM_HIP_RET(enter(l.norm2, l.hc2));
      if (l.s.dense) {
        RET_IF(ffn(l, M, st));
        leave(l.norm2b, l.ls2, l.hc2, 1, false);
      } else {
        RET_IF(moe(l, M, st));
        leave(l.norm2b, l.ls2, l.hc2, l.s.moe.top, l.s.moe.has_shared);
      }
    }
    if (tap_) {
      const float* rows = x_.p;
      if (cfg_.streams > 0) {  // the sum of the streams
        if (tap_rows_.n < (size_t)M * ldx_) RET_IF(tap_rows_.alloc((size_t)M * ldx_));
        rows = n.u = tap_rows_.p;
      }
      LLM_HIP_RET(rms_norm_step(dt_, n, st));
      fresh();
      LLM_HIP_RET(hipMemcpy2DAsync(tap_ + i * (size_t)M * cfg_.width, (size_t)cfg_.width * 4, rows,
                                   (size_t)ldx_ * 4, (size_t)cfg_.width * 4, M,
                                   hipMemcpyDeviceToHost, st));
    }
  }
  if (n_want == 0) return LLM_OK;
  n.rows = meta<int32_t>(at_want_);
  n.M = n_want;
  n.w_pre = final_norm_.p;
  LLM_HIP_RET(rms_norm_step(dt_, n, st));
  MmArgs a;
  a.A = h_.p;
  a.lda = ldx_;
  a.W = head_.p;
  a.M = n_want;
  a.N = cfg_.vocab;
  a.K = cfg_.width;
  a.w_nt = w_nt_;
  a.C = logits;
  a.ldc = cfg_.vocab;
  a.softcap = cfg_.logit_softcap;
  LLM_HIP_RET(mm(dt_, a, st));
  return LLM_OK;
}

int LayerStack::forward(const std::vector<StepSeq>& batch, float* logits, hipStream_t st) {
  int M = 0, n_want = 0;
  bool decode = true;
  single_ = true;
  std::vector<char> seen(opt_.max_seqs, 0);
  for (const StepSeq& s : batch) {
    LLM_REQUIRE(s.slot >= 0 && s.slot < opt_.max_seqs && !seen[s.slot], "step: bad or repeated slot");
    seen[s.slot] = 1;
    LLM_REQUIRE(s.n >= 1 && s.tokens && s.p0 >= 0 && (long long)s.p0 + s.n <= max_len_,
                "step: a sequence grows past the longest the cache holds");
    for (int i = 0; i < s.n; ++i)
      LLM_REQUIRE(s.tokens[i] >= 0 && s.tokens[i] < cfg_.vocab, "step: token id out of range");
    for (int i = 0; i < s.n_want; ++i)
      LLM_REQUIRE(s.want && s.want[i] >= 0 && s.want[i] < s.n, "step: wanted place out of range");
    M += s.n;
    n_want += s.n_want;
    single_ = single_ && s.n == 1;
    decode = decode && s.n == 1 && s.n_want == 1;
  }
  LLM_REQUIRE(M >= 1 && M <= cap_ && n_want <= M, "step: too many tokens");
  LLM_REQUIRE(n_want == 0 || logits, "step: logits is NULL");
  RET_IF(ensure_rows(M));
  for (auto& g : geos_) {
    if (g->layers == 0) continue;
    std::lock_guard<std::mutex> lock(g->kv.mu);
    for (const StepSeq& s : batch)
      for (int t = s.p0 / kPageTokens; t <= (s.p0 + s.n - 1) / kPageTokens; ++t)
        RET_IF(g->kv.prepare_append(s.slot, t * kPageTokens));
    RET_IF(g->kv.sync(st));
  }
  RET_IF(build_meta(batch, M, n_want, st));
  if (!use_graph_ || !decode || tap_) return enqueue(M, n_want, logits, st);

  std::vector<long long> key{M, (long long)reinterpret_cast<uintptr_t>(logits)};
  for (const auto& p : plans_)
    for (const Launch* l : {&p->small, &p->big})
      key.insert(key.end(), {l->n_items, l->n_merges});
  auto it = graphs_.find(key);
  if (it == graphs_.end()) {  // first of its shape: run it, capture the next
    if (graphs_.size() >= kMaxGraphs) {  // shapes of contexts long gone
      LLM_HIP_RET(hipStreamSynchronize(st));
      clear_graphs();
    }
    graphs_[key] = nullptr;
    return enqueue(M, n_want, logits, st);
  }
  if (!it->second) {
    hipGraph_t g;
    LLM_HIP_RET(hipStreamBeginCapture(cap_stream_, hipStreamCaptureModeThreadLocal));
    const int rc = enqueue(M, n_want, logits, cap_stream_);
    const hipError_t e = hipStreamEndCapture(cap_stream_, &g);
    if (rc) return rc;
    if (e != hipSuccess) return fail(LLM_ERR_HIP, std::string("graph capture: ") + hipGetErrorString(e));
    const hipError_t ei = hipGraphInstantiate(&it->second, g, nullptr, nullptr, 0);
    (void)hipGraphDestroy(g);
    if (ei != hipSuccess) {
      it->second = nullptr;
      return fail(LLM_ERR_HIP, std::string("graph instantiate: ") + hipGetErrorString(ei));
    }
  }
  LLM_HIP_RET(hipGraphLaunch(it->second, st));
  return LLM_OK;
}

int LayerStack::release(int slot) {
  LLM_REQUIRE(slot >= 0 && slot < opt_.max_seqs, "release: bad slot");
  for (auto& g : geos_) {
    if (g->layers == 0) continue;
    std::lock_guard<std::mutex> lock(g->kv.mu);
    g->kv.release_beam(slot);
  }
  return LLM_OK;
}

int make_layer_stack(const LayerStackConfig& cfg, const std::string& dir, const ModelOptions& opt,
                     std::unique_ptr<StepModel>* out) {
  auto m = std::make_unique<LayerStack>();
  RET_IF(m->init(cfg, dir, opt));
  *out = std::move(m);
  return LLM_OK;
}

}  // namespace llm
