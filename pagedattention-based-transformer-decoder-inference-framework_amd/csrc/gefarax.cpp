// The Gefarax family: config.json -> LayerStackConfig.
#include "common.hpp"
#include "config_reader.hpp"

namespace llm {
namespace {

int make_gefarax(const Json& c, const std::string& dir, const ModelOptions& opt,
                 std::unique_ptr<StepModel>* out) {
  ConfigReader r;
  LayerStackConfig cfg;
  cfg.vocab = r.size(c, "vocab", "config");
  cfg.width = r.size(c, "width", "config");
  cfg.eps = (float)r.num(c["norm"], "eps", "norm");
  for (size_t i = 0; i < c["layers"].arr.size(); ++i) {
    const Json& l = c["layers"].arr[i];
    const std::string at = "layers[" + std::to_string(i) + "]";
    if (l["type"].str != "attention")
      return fail(LLM_ERR_UNSUPPORTED, "config.json: " + at + ".type '" + l["type"].str + "'");
    LayerSpec s;
    const Json& m = l["mixer"];
    s.attn.heads = r.size(m, "heads", at + ".mixer");
    s.attn.kv_heads = r.size(m, "kv_heads", at + ".mixer");
    s.attn.dim = r.size(m, "dim", at + ".mixer");
    s.attn.vdim = r.size(m, "vdim", at + ".mixer");
    s.attn.scale = (float)r.num(m, "scale", at + ".mixer");
    s.attn.sink = true;
    if (m.has("rot")) {
      const Json& rot = m["rot"];
      s.attn.rope.dims = r.size(rot, "dims", at + ".mixer.rot");
      r.rope(rot, at + ".mixer.rot", &s.attn.rope);
    }
    if (l.has("mlp")) {
      const Json& f = l["mlp"];
      const std::string w = at + ".mlp";
      if (f.has("kind") && f["kind"].str != "moe")
        return fail(LLM_ERR_UNSUPPORTED, "config.json: " + w + ".kind '" + f["kind"].str + "'");
      s.has_mlp = true;
      s.moe.experts = r.size(f["router"], "experts", w + ".router");
      s.moe.top = r.size(f["router"], "top", w + ".router");
      s.moe.scale = (float)r.num(f["router"], "scale", w + ".router");
      r.glu(f["expert"], w + ".expert", &s.moe.expert);
      if (f.has("shared")) {
        s.moe.has_shared = true;
        r.glu(f["shared"], w + ".shared", &s.moe.shared);
      }
    }
    cfg.layers.push_back(s);
  }
  r.loop(c, &cfg);
  cfg.loop_adds_embedding = true;
  cfg.post_norm = true;
  if (!r.error.empty()) return fail(LLM_ERR_INVALID, r.error);
  return make_layer_stack(cfg, dir, opt, out);
}

const ModelRegistrar reg("Gefarax", &make_gefarax);

}  // namespace
}  // namespace llm
