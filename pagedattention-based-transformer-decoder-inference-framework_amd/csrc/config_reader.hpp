// Reads the parts of config.json that the layer-stack families share.  The first
// fault is kept in `error`.
#pragma once

#include <cmath>
#include <string>

#include "json.hpp"
#include "layer_stack.hpp"

namespace llm {

// the clamped GLU of the layer-stack families: g sigmoid(1.702 g) (u + 1)
constexpr float kGluAlpha = 1.702f;
constexpr float kGluUpBias = 1.f;

struct ConfigReader {
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
  void rope(const Json& rot, const std::string& where, RopeSpec* r) {
    r->base = num(rot, "base", where);
    if (!rot.has("scaling")) return;
    const Json& sc = rot["scaling"];
    const std::string w = where + ".scaling";
    r->yarn = true;
    r->factor = num(sc, "factor", w);
    r->original = num(sc, "original", w);
    r->fast = num(sc, "fast", w);
    r->slow = num(sc, "slow", w);
  }
  void glu(const Json& j, const std::string& where, ExpertSpec* e) {
    e->ff = size(j, "ff", where);
    e->glu.limit = (float)num(j, "limit", where);
    e->glu.alpha = kGluAlpha;
    e->glu.up_bias = kGluUpBias;
  }
  void loop(const Json& c, LayerStackConfig* cfg) {
    if (!c.has("loop")) return;
    cfg->loop_start = size(c["loop"], "start", "loop");
    cfg->loop_stop = size(c["loop"], "stop", "loop");
    cfg->loop_times = size(c["loop"], "times", "loop");
  }
};

}  // namespace llm
