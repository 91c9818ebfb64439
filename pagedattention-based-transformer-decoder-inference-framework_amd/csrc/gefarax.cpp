// The Gefarax family: config.json -> LayerStackConfig.
#include <cmath>

#include "common.hpp"
#include "layer_stack.hpp"

namespace llm {
namespace {

constexpr float kGluAlpha = 1.702f;
constexpr float kGluUpBias = 1.f;

struct Reader {
  std::string error;
  double num(const Json& o, const char* key, const std::string& where) {
    const Json& v = o[key];
    if (v.kind != Json::Number && error.empty())
      error = "config.json: " + where + "." + key + " is missing or not a number";
    return v.num;
  }
  int size(const Json& o, const char* key, const std::string& where) {
    const double d = num(o, key, where);
    if (error.empty() && (d < 0 || d > 1e9 || d != std::floor(d)))
      error = "config.json: " + where + "." + key + " is not a size";
    return (int)d;
  }
};

void read_expert(Reader& r, const Json& j, const std::string& where, ExpertSpec* e) {
  e->ff = r.size(j, "ff", where);
  e->glu.limit = (float)r.num(j, "limit", where);
  e->glu.alpha = kGluAlpha;
  e->glu.up_bias = kGluUpBias;
}

int make_gefarax(const Json& c, const std::string& dir, const ModelOptions& opt,
                 std::unique_ptr<StepModel>* out) {
  Reader r;
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
      s.attn.rope.base = r.num(rot, "base", at + ".mixer.rot");
      if (rot.has("scaling")) {
        const Json& sc = rot["scaling"];
        const std::string w = at + ".mixer.rot.scaling";
        s.attn.rope.yarn = true;
        s.attn.rope.factor = r.num(sc, "factor", w);
        s.attn.rope.original = r.num(sc, "original", w);
        s.attn.rope.fast = r.num(sc, "fast", w);
        s.attn.rope.slow = r.num(sc, "slow", w);
      }
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
      read_expert(r, f["expert"], w + ".expert", &s.moe.expert);
      if (f.has("shared")) {
        s.moe.has_shared = true;
        read_expert(r, f["shared"], w + ".shared", &s.moe.shared);
      }
    }
    cfg.layers.push_back(s);
  }
  if (c.has("loop")) {
    cfg.loop_start = r.size(c["loop"], "start", "loop");
    cfg.loop_stop = r.size(c["loop"], "stop", "loop");
    cfg.loop_times = r.size(c["loop"], "times", "loop");
  }
  if (!r.error.empty()) return fail(LLM_ERR_INVALID, r.error);
  return make_layer_stack(cfg, dir, opt, out);
}

const ModelRegistrar reg("Gefarax", &make_gefarax);

}  // namespace
}  // namespace llm
