// The layer-stack model: weights, cache geometry and the step.
//
// One step runs every entry of a mixed batch (prompt portions beside single
// decoded tokens) as one list of token rows:
//   angles | embed + norm -> per layer run { q|k|v product, rotation, append to
//   the pages -> paged attention -> o product -> add + norm -> router product ->
//   routing -> grouped gate/up product -> grouped down product -> add + norm }
//   -> norm of the wanted rows -> head product.
// Everything a step depends on besides the weights is in one device block
// (tokens, positions, slots, attention items, wanted rows) written by one copy,
// so a decode step's launches are captured into a hipGraph per shape and
// replayed.
//
// The cache: layers of one (kv_heads, dim, vdim) share a KvCache; each run of a
// layer is a cache layer of its own, so a repeated layer keeps one cache per
// pass.
#include "layer_stack.hpp"

#include <algorithm>
#include <cmath>
#include <cstring>
#include <map>
#include <mutex>

#include "common.hpp"
#include "dev_buf.hpp"
#include "kv_cache_impl.hpp"
#include "moe.hpp"
#include "paged_gqa.hpp"
#include "rms_norm.hpp"
#include "safetensors.hpp"

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
  for (size_t i = 0; i < c.layers.size(); ++i) {
    const AttentionSpec& a = c.layers[i].attn;
    const std::string at = "config: layer " + std::to_string(i) + ": ";
    LLM_REQUIRE(a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0,
                at + "heads must be a multiple of kv_heads");
    LLM_REQUIRE(a.dim > 0 && a.vdim > 0 && a.dim <= kGqaMaxDim && a.vdim <= kGqaMaxDim &&
                    a.dim % 2 == 0,
                at + "head sizes must be in [1, 256] and dim even");
    LLM_REQUIRE(a.rope.dims >= 0 && a.rope.dims <= a.dim && a.rope.dims % 2 == 0 &&
                    (a.rope.dims == 0 || a.rope.base > 1.0),
                at + "rot.dims must be even and at most dim, rot.base > 1");
    if (!c.layers[i].has_mlp) continue;
    const MoeSpec& m = c.layers[i].moe;
    LLM_REQUIRE(m.experts >= 1 && m.experts <= kMaxExperts && m.top >= 1 && m.top <= m.experts &&
                    m.expert.ff >= 1 && (!m.has_shared || m.shared.ff >= 1),
                at + "bad expert sizes");
  }
  return LLM_OK;
}

inline int up(int v, int m) { return (v + m - 1) / m * m; }

class LayerStack final : public StepModel {
 public:
  ~LayerStack() override {
    if (meta_done_) (void)hipEventSynchronize(meta_done_);
    clear_graphs();
    if (h_meta_) (void)hipHostFree(h_meta_);
    if (meta_done_) (void)hipEventDestroy(meta_done_);
    if (cap_stream_) (void)hipStreamDestroy(cap_stream_);
  }
  int init(const LayerStackConfig& cfg, const std::string& dir, const ModelOptions& opt);

  int vocab() const override { return cfg_.vocab; }
  int max_seq_len() const override { return max_len_; }
  int max_step_tokens() const override { return cap_; }
  int page_tokens() const override { return kPageTokens; }
  long long pool_tokens() const override { return pool_pages_ * kPageTokens; }
  long long free_tokens() const override {
    long long n = pool_pages_;
    for (const auto& g : geos_) n = std::min(n, g->kv.free_count() / ((long long)g->layers * g->G));
    return n * kPageTokens;
  }
  int forward(const std::vector<StepSeq>& batch, float* logits, hipStream_t st) override;
  int release(int slot) override;
  int layer_runs() const override { return (int)runs_.size(); }
  int width() const override { return cfg_.width; }
  int set_tap(float* host) override {
    tap_ = host;
    return LLM_OK;
  }

 private:
  struct Geometry {  // cache of the layers of one head geometry
    int G = 0, D = 0, Dv = 0, Dp = 0, Dvp = 0, layers = 0;
    KvCache kv;
  };
  struct Run {
    int layer = 0, geo = 0, cache_layer = 0;
    bool add_embed = false;
  };
  struct Layer {
    LayerSpec s;
    int geo = 0, rope = -1, plan = 0;
    DevBuf<float> norm1, norm1b, norm2, norm2b, sink, correction;
    DevBuf<uint8_t> qkv, o, router, experts_in, experts_out, shared_in, shared_out;
    DevBuf<MmGroup> groups;
    int n_qkv = 0;
  };
  struct Rope {
    RopeSpec spec;
    float mul = 1.f;
    DevBuf<float> freq;
    DevBuf<float2> turn;
  };
  // one attention launch of the step: its items and merges in the meta block
  struct Launch {
    int tile_rows = 16, n_items = 0, n_merges = 0, parts = 0;
    size_t items_at = 0, merges_at = 0;
  };
  struct Plan {  // layers that cut their rows alike
    int R = 1, G = 1, big_rows = 16, max_pd = 16;
    Launch small, big;
  };

  int load(const std::string& dir);
  int pack_rows(const SafeTensors& f, const std::vector<std::pair<std::string, int>>& parts, int K,
                const std::vector<int32_t>* map, uint8_t* dst);
  int ensure_rows(int M);
  int build_meta(const std::vector<StepSeq>& batch, int M, int n_want, hipStream_t st);
  void cut(const std::vector<StepSeq>& batch, Plan& p, bool big, std::vector<GqaItem>& items,
           std::vector<GqaMerge>& merges, Launch& l);
  int enqueue(int M, int n_want, float* logits, hipStream_t st);
  int attention(const Layer& l, const Run& r, int M, hipStream_t st);
  int mlp(const Layer& l, int M, hipStream_t st);
  void clear_graphs() {
    for (auto& g : graphs_)
      if (g.second) (void)hipGraphExecDestroy(g.second);
    graphs_.clear();
  }

  LayerStackConfig cfg_;
  ModelOptions opt_;
  int dt_ = LLM_BF16, es_ = 2, ldx_ = 0, cap_ = 0, max_len_ = 0, w_nt_ = 0;
  long long pool_pages_ = 0;
  std::vector<std::unique_ptr<Geometry>> geos_;
  std::vector<std::unique_ptr<Layer>> layers_;
  std::vector<std::unique_ptr<Rope>> ropes_;
  std::vector<Run> runs_;
  std::vector<Plan> plans_;
  DevBuf<uint16_t> emb_;
  DevBuf<float> final_norm_;
  DevBuf<uint8_t> head_;
  DevBuf<uint8_t> staging_;
  DevBuf<int32_t> map_;
  size_t weight_bytes_ = 0;

  // step buffers, sized for rows_ tokens
  int rows_ = 0;
  int ld_q_ = 0, ld_att_ = 0, ld_act_ = 0, ld_shared_ = 0, max_top_ = 0, max_e_ = 0;
  DevBuf<float> x_, y_, z_, weight_, part_o_, part_ml_;
  DevBuf<uint8_t> h_, q_, att_, act_, act_shared_;
  DevBuf<int32_t> choice_, perm_, n_tiles_;
  DevBuf<MmTile> tiles_;
  // the step's meta block
  DevBuf<uint8_t> meta_;
  uint8_t* h_meta_ = nullptr;
  size_t meta_cap_ = 0;
  hipEvent_t meta_done_ = nullptr;
  size_t at_tok_ = 0, at_pos_ = 0, at_slot_ = 0, at_want_ = 0;
  float* tap_ = nullptr;

  bool use_graph_ = true;
  hipStream_t cap_stream_ = nullptr;
  std::map<std::vector<long long>, hipGraphExec_t> graphs_;  // NULL: seen once, not captured

  template <typename T>
  const T* meta(size_t at) const { return reinterpret_cast<const T*>(meta_.p + at); }
};

template <typename T>
int alloc_zero(DevBuf<T>& b, size_t n) {
  RET_IF(b.alloc(n));
  if (n) LLM_HIP_RET(hipMemset(b.p, 0, n * sizeof(T)));
  return LLM_OK;
}

template <typename T>
int upload_vec(DevBuf<T>& b, const std::vector<T>& v) {
  RET_IF(b.alloc(v.size()));
  if (!v.empty()) LLM_HIP_RET(hipMemcpy(b.p, v.data(), v.size() * sizeof(T), hipMemcpyHostToDevice));
  return LLM_OK;
}

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
    const AttentionSpec& a = s.attn;
    int g = 0;
    for (; g < (int)geos_.size(); ++g)
      if (geos_[g]->G == a.kv_heads && geos_[g]->D == a.dim && geos_[g]->Dv == a.vdim) break;
    if (g == (int)geos_.size()) {
      auto n = std::make_unique<Geometry>();
      n->G = a.kv_heads;
      n->D = a.dim;
      n->Dv = a.vdim;
      n->Dp = up(a.dim, 8);
      n->Dvp = up(a.vdim, 8);
      geos_.push_back(std::move(n));
    }
    l->geo = g;
    const Geometry& geo = *geos_[g];
    if (a.rope.dims > 0) {
      int r = 0;
      for (; r < (int)ropes_.size(); ++r)
        if (ropes_[r]->spec == a.rope) break;
      if (r == (int)ropes_.size()) {
        auto n = std::make_unique<Rope>();
        n->spec = a.rope;
        RET_IF(upload_vec(n->freq, rope_frequencies(a.rope, &n->mul)));
        ropes_.push_back(std::move(n));
      }
      l->rope = r;
    }
    Plan p;
    p.R = a.heads / a.kv_heads;
    p.G = a.kv_heads;
    p.big_rows = gqa_tile_rows(dt_, geo.Dp, geo.Dvp, 1 << 20);
    int k = 0;
    for (; k < (int)plans_.size(); ++k)
      if (plans_[k].R == p.R && plans_[k].G == p.G && plans_[k].big_rows == p.big_rows) break;
    if (k == (int)plans_.size()) plans_.push_back(p);
    plans_[k].max_pd = std::max(plans_[k].max_pd, gqa_part_dim(a.vdim));
    l->plan = k;
    ld_q_ = std::max(ld_q_, a.heads * geo.Dp);
    ld_att_ = std::max(ld_att_, mm_pad(a.heads * a.vdim));
    if (s.has_mlp) {
      max_top_ = std::max(max_top_, s.moe.top);
      max_e_ = std::max(max_e_, s.moe.experts);
      ld_act_ = std::max(ld_act_, mm_pad(s.moe.expert.ff));
      if (s.moe.has_shared) ld_shared_ = std::max(ld_shared_, mm_pad(s.moe.shared.ff));
    }
    layers_.push_back(std::move(l));
  }
  const auto add_run = [&](int i, bool again) {
    Run r;
    r.layer = i;
    r.geo = layers_[i]->geo;
    r.cache_layer = geos_[r.geo]->layers++;
    r.add_embed = again;
    runs_.push_back(r);
  };
  for (int i = 0; i < cfg.loop_start; ++i) add_run(i, false);
  for (int p = 0; p < cfg.loop_times; ++p)
    for (int i = cfg.loop_start; i < cfg.loop_stop; ++i) add_run(i, p > 0 && i == cfg.loop_start);
  for (int i = cfg.loop_stop; i < (int)layers_.size(); ++i) add_run(i, false);

  for (auto& g : geos_) {
    if (g->layers == 0) continue;
    RET_IF(g->kv.init(g->layers, opt.max_seqs, g->G, g->Dp, kPageTokens, max_len_ / kPageTokens,
                      pool_pages_ * g->layers * g->G, dt_, g->Dvp));
    RET_IF(g->kv.zero_pools(nullptr));
  }
  LLM_HIP_RET(hipEventCreateWithFlags(&meta_done_, hipEventDisableTiming));
  LLM_HIP_RET(hipStreamCreateWithFlags(&cap_stream_, hipStreamNonBlocking));
  RET_IF(load(dir));
  w_nt_ = weight_bytes_ > kKeepBytes;
  return LLM_OK;
}

// ---------------------------------------------------------------------------
// weights
// ---------------------------------------------------------------------------

// Pack the rows of one or more [rows][K] tensors, stacked and then reordered by
// `map` (packed column n takes stacked row map[n]).
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
  if (map) RET_IF(upload_vec(map_, *map));
  LLM_HIP_RET(mm_pack(dt_, reinterpret_cast<const uint16_t*>(staging_.p), map ? map_.p : nullptr, N,
                      K, dst, nullptr));
  LLM_HIP_RET(hipStreamSynchronize(nullptr));  // staging and map are used again
  weight_bytes_ += mm_packed_bytes(dt_, N, K);
  return LLM_OK;
}

int LayerStack::load(const std::string& dir) {
  SafeTensors f;
  RET_IF(f.open(dir + "/model.safetensors"));
  const int W = cfg_.width;
  const auto padded = [&](DevBuf<float>& b, const std::string& name) {
    std::vector<float> v;
    RET_IF(f.get_f32(name, {W}, &v));
    v.resize(ldx_, 0.f);
    return upload_vec(b, v);
  };
  const auto packed = [&](DevBuf<uint8_t>& b, const std::vector<std::pair<std::string, int>>& parts,
                          int K, const std::vector<int32_t>* map) {
    int N = 0;
    for (const auto& p : parts) N += p.second;
    RET_IF(b.alloc(mm_packed_bytes(dt_, N, K)));
    return pack_rows(f, parts, K, map, b.p);
  };
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
    const AttentionSpec& a = l.s.attn;
    RET_IF(padded(l.norm1, at + "norm1"));
    RET_IF(padded(l.norm1b, at + "norm1b"));
    // q | k | v with rotation partners side by side
    const int nq = a.heads * a.dim, nk = a.kv_heads * a.dim, nv = a.kv_heads * a.vdim;
    l.n_qkv = nq + nk + nv;
    std::vector<int32_t> map((size_t)l.n_qkv);
    const int half = a.rope.dims / 2;
    for (int n = 0; n < l.n_qkv; ++n) {
      const int d = n % a.dim;
      map[n] = n < nq + nk && d < a.rope.dims ? n - d + d / 2 + (d & 1) * half : n;
    }
    RET_IF(packed(l.qkv, {{mix + "q", nq}, {mix + "k", nk}, {mix + "v", nv}}, W, &map));
    RET_IF(packed(l.o, {{mix + "o", W}}, a.heads * a.vdim, nullptr));
    if (a.sink) {
      std::vector<float> s;
      RET_IF(f.get_f32(mix + "sink", {a.heads}, &s));
      RET_IF(upload_vec(l.sink, s));
    }
    if (!l.s.has_mlp) continue;
    RET_IF(padded(l.norm2, at + "norm2"));
    RET_IF(padded(l.norm2b, at + "norm2b"));
    const MoeSpec& m = l.s.moe;
    RET_IF(packed(l.router, {{ml + "router", m.experts}}, W, nullptr));
    std::vector<float> c;
    RET_IF(f.get_f32(ml + "correction", {m.experts}, &c));
    RET_IF(upload_vec(l.correction, c));
    const auto interleaved = [](int ff) {  // column 2i: gate i, 2i + 1: up i
      std::vector<int32_t> v((size_t)2 * ff);
      for (int n = 0; n < 2 * ff; ++n) v[n] = (n & 1) * ff + n / 2;
      return v;
    };
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
    const std::vector<int32_t> pairs = interleaved(ff);
    for (int e = 0; e < m.experts; ++e) {
      const std::string ex = ml + "e" + std::to_string(e) + ".";
      uint8_t *in = l.experts_in.p + b_in * e, *out = l.experts_out.p + b_out * e;
      RET_IF(pack_rows(f, {{ex + "gate", ff}, {ex + "up", ff}}, W, &pairs, in));
      RET_IF(pack_rows(f, {{ex + "down", W}}, ff, nullptr, out));
      groups.push_back(describe(m.expert, in, out));
    }
    if (m.has_shared) {
      const int sf = m.shared.ff;
      const std::vector<int32_t> sp = interleaved(sf);
      RET_IF(packed(l.shared_in, {{ml + "shared.gate", sf}, {ml + "shared.up", sf}}, W, &sp));
      RET_IF(packed(l.shared_out, {{ml + "shared.down", W}}, sf, nullptr));
      groups.push_back(describe(m.shared, l.shared_in.p, l.shared_out.p));
    }
    RET_IF(upload_vec(l.groups, groups));
  }
  RET_IF(padded(final_norm_, "final.norm"));
  RET_IF(packed(head_, {{"head", cfg_.vocab}}, W, nullptr));
  RET_IF(staging_.alloc(0));
  RET_IF(map_.alloc(0));
  return LLM_OK;
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
  RET_IF(alloc_zero(x_, (size_t)n * ldx_));
  RET_IF(alloc_zero(h_, (size_t)n * ldx_ * es_));
  RET_IF(alloc_zero(q_, (size_t)n * ld_q_ * es_));
  RET_IF(alloc_zero(att_, (size_t)n * ld_att_ * es_));
  RET_IF(alloc_zero(y_, (size_t)n * (max_top_ + 1) * ldx_));
  if (max_top_ > 0) {
    RET_IF(alloc_zero(z_, (size_t)n * max_e_));
    RET_IF(alloc_zero(act_, (size_t)n * max_top_ * ld_act_ * es_));
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

// The row tiles of one attention launch: sequences that bring few rows per
// key/value head (big false) or many, split over their pages until the launch
// holds about kTargetGroups workgroups; long tiles first.
void LayerStack::cut(const std::vector<StepSeq>& batch, Plan& p, bool big,
                     std::vector<GqaItem>& items, std::vector<GqaMerge>& merges, Launch& l) {
  l = Launch();
  l.tile_rows = big ? p.big_rows : 16;
  long long tiles = 0;
  int max_pages = 1, tok0 = 0;
  for (const StepSeq& s : batch) {
    const int rows = s.n * p.R;
    if ((rows > kGqaSmallRows) != big) continue;
    tiles += (rows + l.tile_rows - 1) / l.tile_rows;
    max_pages = std::max(max_pages, (s.p0 + s.n - 1) / kPageTokens + 1);
  }
  if (tiles == 0) return;
  const int want = (int)std::min<long long>(std::max<long long>(kTargetGroups / (tiles * p.G), 1), kMaxSplits);
  // single tokens share one split count, so a decode step keeps its launch
  // shape (and graph) while contexts grow
  const int common = std::min(want, (max_pages + kMinSplitPages - 1) / kMinSplitPages);
  for (const StepSeq& s : batch) {
    const int rows = s.n * p.R;
    const int t0 = tok0;
    tok0 += s.n;
    if ((rows > kGqaSmallRows) != big) continue;
    for (int r0 = 0; r0 < rows; r0 += l.tile_rows) {
      const int last = s.p0 + (std::min(r0 + l.tile_rows, rows) - 1) / p.R;
      const int pages = last / kPageTokens + 1;
      const int ns = big ? std::min(want, (pages + kMinSplitPages - 1) / kMinSplitPages) : common;
      for (int k = 0; k < ns; ++k)
        items.push_back(GqaItem{t0, s.slot, s.p0, r0, rows, (int)((long long)pages * k / ns),
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
  std::vector<std::vector<GqaItem>> items(plans_.size() * 2);
  std::vector<std::vector<GqaMerge>> merges(plans_.size() * 2);
  size_t at = 0, part_o = 0, part_ml = 0;
  const auto take = [&](size_t bytes) {
    const size_t a = at;
    at += (bytes + 15) / 16 * 16;
    return a;
  };
  at_tok_ = take((size_t)M * 4);
  at_pos_ = take((size_t)M * 4);
  at_slot_ = take((size_t)M * 4);
  at_want_ = take((size_t)n_want * 4);
  for (size_t i = 0; i < plans_.size(); ++i)
    for (int b = 0; b < 2; ++b) {
      Plan& p = plans_[i];
      Launch& l = b ? p.big : p.small;
      cut(batch, p, b != 0, items[2 * i + b], merges[2 * i + b], l);
      l.items_at = take(items[2 * i + b].size() * sizeof(GqaItem));
      l.merges_at = take(merges[2 * i + b].size() * sizeof(GqaMerge));
      const size_t rows = (size_t)l.parts * p.G * l.tile_rows;
      part_o = std::max(part_o, rows * p.max_pd);
      part_ml = std::max(part_ml, rows * 2);
    }
  if (part_o > part_o_.n || part_ml > part_ml_.n || at > meta_cap_) {
    LLM_HIP_RET(hipDeviceSynchronize());
    clear_graphs();
    if (part_o > part_o_.n) RET_IF(part_o_.alloc(part_o * 2));
    if (part_ml > part_ml_.n) RET_IF(part_ml_.alloc(part_ml * 2));
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
  int32_t* want = reinterpret_cast<int32_t*>(h_meta_ + at_want_);
  int m = 0, w = 0;
  for (const StepSeq& s : batch) {
    for (int i = 0; i < s.n_want; ++i) want[w++] = m + s.want[i];
    for (int i = 0; i < s.n; ++i, ++m) {
      tok[m] = s.tokens[i];
      pos[m] = s.p0 + i;
      slot[m] = s.slot;
    }
  }
  for (size_t i = 0; i < plans_.size(); ++i)
    for (int b = 0; b < 2; ++b) {
      const Launch& l = b ? plans_[i].big : plans_[i].small;
      const auto &it = items[2 * i + b];
      const auto &me = merges[2 * i + b];
      if (!it.empty()) std::memcpy(h_meta_ + l.items_at, it.data(), it.size() * sizeof(GqaItem));
      if (!me.empty()) std::memcpy(h_meta_ + l.merges_at, me.data(), me.size() * sizeof(GqaMerge));
    }
  LLM_HIP_RET(hipMemcpyAsync(meta_.p, h_meta_, at, hipMemcpyHostToDevice, st));
  LLM_HIP_RET(hipEventRecord(meta_done_, st));
  return LLM_OK;
}

int LayerStack::attention(const Layer& l, const Run& r, int M, hipStream_t st) {
  const AttentionSpec& a = l.s.attn;
  Geometry& g = *geos_[l.geo];
  const KvCache& kv = g.kv;
  const int32_t* table = kv.d_table + (size_t)r.cache_layer * kv.beams * kv.H * kv.max_tiles;
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

  const Plan& plan = plans_[l.plan];
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

  MmArgs o;
  o.A = att_.p;
  o.lda = ldo;
  o.W = l.o.p;
  o.M = M;
  o.N = cfg_.width;
  o.K = a.heads * a.vdim;
  o.w_nt = w_nt_;
  o.C = y_.p;
  o.ldc = ldx_;
  LLM_HIP_RET(mm(dt_, o, st));
  return LLM_OK;
}

int LayerStack::mlp(const Layer& l, int M, hipStream_t st) {
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
    n.tok = meta<int32_t>(at_tok_);
    n.ldh = ldx_;
    n.h = h_.p;
  };
  const auto post = [&](const float* w, int parts, bool shared) {
    fresh();
    n.w_post = w;
    n.y = y_.p;
    n.ldy = ldx_;
    n.parts = parts;
    n.shared = shared;
  };
  fresh();
  n.embed = 1;
  for (size_t i = 0; i < runs_.size(); ++i) {
    const Run& r = runs_[i];
    const Layer& l = *layers_[r.layer];
    if (r.add_embed) n.embed = 2;
    n.w_pre = l.norm1.p;
    LLM_HIP_RET(rms_norm_step(dt_, n, st));
    RET_IF(attention(l, r, M, st));
    post(l.norm1b.p, 1, false);
    if (l.s.has_mlp) {
      n.w_pre = l.norm2.p;
      LLM_HIP_RET(rms_norm_step(dt_, n, st));
      RET_IF(mlp(l, M, st));
      post(l.norm2b.p, l.s.moe.top, l.s.moe.has_shared);
    }
    if (tap_) {
      LLM_HIP_RET(rms_norm_step(dt_, n, st));
      fresh();
      LLM_HIP_RET(hipMemcpy2DAsync(tap_ + i * (size_t)M * cfg_.width, (size_t)cfg_.width * 4, x_.p,
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
  LLM_HIP_RET(mm(dt_, a, st));
  return LLM_OK;
}

int LayerStack::forward(const std::vector<StepSeq>& batch, float* logits, hipStream_t st) {
  int M = 0, n_want = 0;
  bool decode = true;
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
  for (const Plan& p : plans_)
    for (const Launch* l : {&p.small, &p.big})
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

}  // namespace

int make_layer_stack(const LayerStackConfig& cfg, const std::string& dir, const ModelOptions& opt,
                     std::unique_ptr<StepModel>* out) {
  auto m = std::make_unique<LayerStack>();
  RET_IF(m->init(cfg, dir, opt));
  *out = std::move(m);
  return LLM_OK;
}

}  // namespace llm
