// Decoder-only models given as a list of layers (csrc/layer_stack.cpp): every
// layer names its mixer and its feed-forward with sizes of their own, a run of
// layers may repeat with the same weights, norms stand before (and after) each
// sublayer, and the residual is one stream or several that are mixed around each
// sublayer.  A model family reads its config.json into LayerStackConfig.
#pragma once

#include <memory>
#include <string>
#include <vector>

#include "mm.hpp"
#include "model.hpp"

namespace llm {

// Rotary positions on the first `dims` dimensions of a head, partners half of
// `dims` apart; with yarn the frequencies are interpolated (rope_frequencies).
struct RopeSpec {
  int dims = 0;
  double base = 10000.0;
  bool yarn = false;
  double factor = 1.0, original = 1.0, fast = 32.0, slow = 1.0;
  bool operator==(const RopeSpec& o) const {
    return dims == o.dims && base == o.base && yarn == o.yarn && factor == o.factor &&
           original == o.original && fast == o.fast && slow == o.slow;
  }
};
// Frequency of each of the dims / 2 pairs; *mul: the factor on cosine and sine.
std::vector<float> rope_frequencies(const RopeSpec& r, float* mul);

struct AttentionSpec {
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
  RopeSpec rope;
  float scale = 1.f;
  bool sink = false;  // a learned term in each head's softmax denominator
};

// Keys and values are products of one normed latent per token; a rotated key part
// is shared by the heads.  The cache holds the latent and that part.
struct LatentSpec {
  int heads = 0, dim = 0, rot_dim = 0, vdim = 0, rank = 0;
  RopeSpec rope;  // dims = rot_dim, partners side by side
  float scale = 1.f;
  bool sink = false;
};

// Selective scan behind a short causal convolution.
struct MambaSpec {
  int inner = 0, state = 0, dt_rank = 0, taps = 0;
};

struct ExpertSpec {
  int ff = 0;
  GluParams glu;
};
struct MoeSpec {
  int experts = 0, top = 0;
  float scale = 1.f;
  ExpertSpec expert;
  bool has_shared = false;
  ExpertSpec shared;
};

enum class Mixer { kAttention, kLatent, kMamba };

struct LayerSpec {
  Mixer mixer = Mixer::kAttention;
  AttentionSpec attn;
  LatentSpec latent;
  MambaSpec mamba;
  bool has_mlp = false;
  bool dense = false;  // the feed-forward is `ffn`, otherwise `moe`
  ExpertSpec ffn;
  MoeSpec moe;
};

struct LayerStackConfig {
  int vocab = 0, width = 0;
  float eps = 1e-5f;
  std::vector<LayerSpec> layers;
  // layers [loop_start, loop_stop) are passed through loop_times times
  int loop_start = 0, loop_stop = 0, loop_times = 1;
  // a repeated pass starts with the tokens' embeddings added to the residual
  bool loop_adds_embedding = false;
  float embedding_scale = 1.f;
  bool post_norm = false;    // sublayer outputs are normed (norm1b, norm2b)
  bool layer_scale = false;  // and multiplied element by element (ls1, ls2)
  int streams = 0;           // residual streams mixed by hc1.*, hc2.* (0: one, plain sums)
  float logit_softcap = 0.f;  // 0: none
};

// Checks the configuration, reads the weights of dir/model.safetensors (tensor
// names: embed, l<i>.norm1 ..., final.norm, head) and builds the model.
int make_layer_stack(const LayerStackConfig& cfg, const std::string& dir, const ModelOptions& opt,
                     std::unique_ptr<StepModel>* out);

}  // namespace llm
