// The layer-stack model's class: layer_stack.cpp has its weights, step and
// grouped-query attention, mix_latent.cpp and mix_mamba.cpp the other mixers.
#pragma once

#include <climits>
#include <map>

#include "dev_buf.hpp"
#include "kv_cache_impl.hpp"
#include "layer_stack.hpp"
#include "moe.hpp"
#include "paged_gqa.hpp"
#include "rms_norm.hpp"
#include "safetensors.hpp"
#include "selective_scan.hpp"
#include "state_cache.hpp"

namespace llm {

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
  // pages of the layers of one head geometry; latent: G = 1, D = rank, Dv = rot,
  // keys only
  struct Geometry {
    bool latent = false;
    int G = 0, D = 0, Dv = 0, Dp = 0, Dvp = 0, layers = 0;
    KvCache kv;
  };
  struct Run {
    int layer = 0, cache_layer = 0;
    bool again = false;  // first layer of a repeated pass
    std::unique_ptr<StateCache> state;
  };
  struct Hyper {  // a sublayer's stream mixing
    DevBuf<float> in, out, mix;
  };
  struct Layer {
    LayerSpec s;
    int geo = -1, rope = -1, plan = -1;
    int plan_x = -1;  // latent: the plan of portions whose keys are expanded
    int scan = -1;
    DevBuf<float> norm1, norm1b, norm2, norm2b, ls1, ls2;
    Hyper hc1, hc2;
    DevBuf<uint8_t> o;  // the mixer's output product
    // attention (qkv; latent: q and down)
    int n_qkv = 0;
    DevBuf<float> sink;
    DevBuf<uint8_t> qkv;
    // latent
    DevBuf<float> latent_norm;
    DevBuf<uint8_t> absorb, value, expand;  // per head W_uk^T, W_uv; both stacked
    size_t absorb_head = 0, value_head = 0;
    // mamba
    DevBuf<uint8_t> in, x, dt;
    DevBuf<float> conv, conv_bias, dt_bias, A, D;
    // feed-forward
    DevBuf<float> correction;
    DevBuf<uint8_t> router, experts_in, experts_out, shared_in, shared_out;
    DevBuf<MmGroup> groups;
    DevBuf<uint8_t> ffn_in, ffn_out;
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
  // Layers that cut their rows alike: R rows per token against each of G
  // key/value heads.  Portions of up to small_max rows take tiles of small_tile.
  // Only portions of min_n .. max_n tokens belong to the plan.
  struct Plan {
    int R = 1, G = 1, small_tile = 16, small_max = kGqaSmallRows, big_tile = 16;
    int min_n = 1, max_n = INT_MAX;
    int max_pd = 16;
    Launch small, big;
    // Row list of the plan's tokens (latent layers).
    bool latent = false;
    int n_rows = 0;
    size_t rows_at = 0;
    // Expanded keys: the whole context of each portion becomes keys and values
    // of G heads (key row Dp: dim, then the turned part; value size Dv) in
    // scratch pages of the plan's own.
    bool expand = false;
    int dim = 0, rot = 0, Dp = 0, Dv = 0, Dvp = 0;
    int x_rows = 0, x_tiles = 0;
    size_t x_pos = 0, x_slot = 0, x_entry = 0, x_table = 0;
    long long x_pages = 0;
    DevBuf<uint8_t> pool;
    bool same(const Plan& o) const {
      return R == o.R && G == o.G && small_tile == o.small_tile && small_max == o.small_max &&
             big_tile == o.big_tile && min_n == o.min_n && max_n == o.max_n &&
             latent == o.latent && expand == o.expand && dim == o.dim && rot == o.rot &&
             Dp == o.Dp && Dv == o.Dv && Dvp == o.Dvp;
    }
  };
  // Layers whose scans take chunks of one size.
  struct ScanPlan {
    int chunk = 0;
    int n_items = 0, n_chunks = 0, n_carry = 0, parts = 0;
    size_t items_at = 0, chunks_at = 0, carry_at = 0;
  };

  int init_latent(Layer& l);
  int init_mamba(Layer& l);
  int find_rope(const RopeSpec& spec, int* index);
  int find_geometry(bool latent, int G, int D, int Dv);
  int add_plan(std::unique_ptr<Plan> p);
  int add_run(int layer, bool again);
  int load(const std::string& dir);
  int load_attention(const SafeTensors& f, const std::string& mix, Layer& l);
  int load_latent(const SafeTensors& f, const std::string& mix, Layer& l);
  int load_mamba(const SafeTensors& f, const std::string& mix, Layer& l);
  int load_moe(const SafeTensors& f, const std::string& mlp, Layer& l);
  int load_hyper(const SafeTensors& f, const std::string& name, Hyper& h);
  // fp32 vector of n values, zero-padded to `padded`
  int load_vector(const SafeTensors& f, const std::string& name, int n, int padded, DevBuf<float>& b);
  int load_packed(const SafeTensors& f, const std::vector<std::pair<std::string, int>>& parts, int K,
                  const std::vector<int32_t>* map, DevBuf<uint8_t>& b);
  // Packed columns take row map[n] of a row-major bf16 matrix on the host.
  int pack_host(const std::vector<uint16_t>& rows, int K, const std::vector<int32_t>* map,
                uint8_t* dst);
  int pack_rows(const SafeTensors& f, const std::vector<std::pair<std::string, int>>& parts, int K,
                const std::vector<int32_t>* map, uint8_t* dst);
  int ensure_rows(int M);
  int build_meta(const std::vector<StepSeq>& batch, int M, int n_want, hipStream_t st);
  void cut(const std::vector<StepSeq>& batch, Plan& p, bool big, std::vector<GqaItem>& items,
           std::vector<GqaMerge>& merges, Launch& l);
  // rows and scratch pages of the portions whose keys are expanded
  void plan_expansion(const std::vector<StepSeq>& batch, Plan& p, std::vector<int32_t>& pos,
                      std::vector<int32_t>& slot, std::vector<int32_t>& entry,
                      std::vector<int32_t>& table);
  void plan_scan(const std::vector<StepSeq>& batch, ScanPlan& p, std::vector<ScanItem>& items,
                 std::vector<ScanItem>& chunks, std::vector<ScanCarry>& carry);
  int enqueue(int M, int n_want, float* logits, hipStream_t st);
  int attention(const Layer& l, const Run& r, int M, hipStream_t st);
  int latent(const Layer& l, const Run& r, int M, hipStream_t st);
  int mamba(const Layer& l, const Run& r, int M, hipStream_t st);
  int out_product(const Layer& l, const void* A, int lda, int K, int M, hipStream_t st);
  int moe(const Layer& l, int M, hipStream_t st);
  int ffn(const Layer& l, int M, hipStream_t st);
  const int32_t* table_of(const Geometry& g, const Run& r) const {
    return g.kv.d_table + (size_t)r.cache_layer * g.kv.beams * g.kv.H * g.kv.max_tiles;
  }
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
  std::vector<std::unique_ptr<Plan>> plans_;
  std::vector<ScanPlan> scans_;
  DevBuf<uint16_t> emb_;
  DevBuf<float> final_norm_;
  DevBuf<uint8_t> head_;
  DevBuf<uint8_t> staging_;
  DevBuf<int32_t> map_;
  size_t weight_bytes_ = 0;

  // step buffers, sized for rows_ tokens
  int rows_ = 0;
  int ld_q_ = 0, ld_att_ = 0, ld_act_ = 0, ld_shared_ = 0, max_top_ = 0, max_e_ = 0;
  DevBuf<float> x_, y_, z_, weight_, part_o_, part_ml_, tap_rows_;
  DevBuf<uint8_t> h_, q_, att_, act_, act_shared_;
  // latent: queries in the latent space, values in it, projected-down rows
  int ld_qlat_ = 0, ld_olat_ = 0, ld_down_ = 0;
  DevBuf<uint8_t> q_lat_, o_lat_;
  DevBuf<float> down_;
  // mamba: inputs (x | z), x after the convolution, low-rank step sizes, gated output
  int ld_xz_ = 0, ld_inner_ = 0, ld_low_ = 0, ld_bc_ = 0;
  DevBuf<uint8_t> xz_, xc_, low_, gated_;
  DevBuf<float> bc_, dtv_, carry_, sum_dt_;
  size_t carry_floats_ = 0;  // of a part, at most
  DevBuf<int32_t> choice_, perm_, n_tiles_;
  DevBuf<MmTile> tiles_;
  // the step's meta block
  DevBuf<uint8_t> meta_;
  uint8_t* h_meta_ = nullptr;
  size_t meta_cap_ = 0;
  hipEvent_t meta_done_ = nullptr;
  size_t at_tok_ = 0, at_pos_ = 0, at_slot_ = 0, at_seq0_ = 0, at_want_ = 0;
  bool single_ = false;  // every entry of the step is one token
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

}  // namespace llm
