// The Nubosun family: config.json -> LayerStackConfig.
#include "common.hpp"
#include "config_reader.hpp"

namespace llm {
namespace {

int make_nubosun(const Json& c, const std::string& dir, const ModelOptions& opt,
                 std::unique_ptr<StepModel>* out) {
  ConfigReader r;
  LayerStackConfig cfg;
  cfg.vocab = r.size(c, "vocab", "config");
  cfg.width = r.size(c, "width", "config");
  cfg.eps = (float)r.num(c["norm"], "eps", "norm");
  cfg.embedding_scale = (float)r.num(c["embedding"], "scale", "embedding");
  cfg.streams = r.size(c, "streams", "config");
  if (r.error.empty() && cfg.streams < 1)
    return fail(LLM_ERR_INVALID, "config.json: streams must be positive");
  if (c.has("logit_softcap")) cfg.logit_softcap = (float)r.num(c, "logit_softcap", "config");
  cfg.layer_scale = true;
  for (size_t i = 0; i < c["layers"].arr.size(); ++i) {
    const Json& l = c["layers"].arr[i];
    const std::string at = "layers[" + std::to_string(i) + "]", w = at + ".mixer";
    const Json& m = l["mixer"];
    LayerSpec s;
    if (l["type"].str == "latent_attention") {
      s.mixer = Mixer::kLatent;
      s.latent.heads = r.size(m, "heads", w);
      s.latent.dim = r.size(m, "dim", w);
      s.latent.rot_dim = r.size(m, "rot_dim", w);
      s.latent.vdim = r.size(m, "vdim", w);
      s.latent.rank = r.size(m, "kv_rank", w);
      s.latent.scale = (float)r.num(m, "scale", w);
      s.latent.sink = true;
      s.latent.rope.dims = s.latent.rot_dim;
      if (s.latent.rot_dim > 0) r.rope(m["rot"], w + ".rot", &s.latent.rope);
    } else if (l["type"].str == "mamba1") {
      s.mixer = Mixer::kMamba;
      s.mamba.inner = r.size(m, "inner", w);
      s.mamba.state = r.size(m, "state", w);
      s.mamba.dt_rank = r.size(m, "dt_rank", w);
      s.mamba.taps = r.size(m, "conv", w);
    } else {
      return fail(LLM_ERR_UNSUPPORTED, "config.json: " + at + ".type '" + l["type"].str + "'");
    }
    if (l.has("mlp")) {
      const Json& f = l["mlp"];
      if (f.has("kind") && f["kind"].str != "dense")
        return fail(LLM_ERR_UNSUPPORTED, "config.json: " + at + ".mlp.kind '" + f["kind"].str + "'");
      s.has_mlp = s.dense = true;
      r.glu(f, at + ".mlp", &s.ffn);
    }
    cfg.layers.push_back(s);
  }
  r.loop(c, &cfg);
  if (!r.error.empty()) return fail(LLM_ERR_INVALID, r.error);
  return make_layer_stack(cfg, dir, opt, out);
}

const ModelRegistrar reg("Nubosun", &make_nubosun);

}  // namespace
}  // namespace llm
