// What the serving engine (csrc/engine.cpp) needs of a model, and the registry
// that finds a model by its config.json.
#pragma once

#include <hip/hip_runtime.h>

#include <cstdint>
#include <memory>
#include <string>
#include <vector>

#include "json.hpp"
#include "llm_decoder.h"

namespace llm {

// The new tokens of one sequence in a step: n tokens at positions p0 .. of
// cache slot `slot`; logits are wanted after tokens want[0 .. n_want).
struct StepSeq {
  int slot = 0, p0 = 0, n = 0;
  const int32_t* tokens = nullptr;
  const int32_t* want = nullptr;
  int n_want = 0;
};

class StepModel {
 public:
  virtual ~StepModel() = default;
  virtual int vocab() const = 0;
  virtual int max_seq_len() const = 0;
  virtual int max_step_tokens() const = 0;
  virtual int page_tokens() const = 0;
  // cache pages: tokens the pool holds in whole pages, and still has free
  virtual long long pool_tokens() const = 0;
  virtual long long free_tokens() const = 0;
  // Run the batch (all entries together, from what earlier steps left in the
  // slots) and write the wanted rows' logits, in order, to logits[rows][vocab]
  // on the device.  At most max_step_tokens() tokens.  Enqueued on `st`.
  virtual int forward(const std::vector<StepSeq>& batch, float* logits, hipStream_t st) = 0;
  // Give back what the slot holds.
  virtual int release(int slot) = 0;
  // The residual stream after every layer of the next forwards, copied to the
  // host: tap[layer run][tokens of the batch][width] (NULL: off).
  virtual int layer_runs() const { return 0; }
  virtual int width() const { return 0; }
  virtual int set_tap(float* host) { return host ? LLM_ERR_UNSUPPORTED : LLM_OK; }
};

struct ModelOptions {
  int dtype = LLM_BF16;
  int max_seqs = 1;
  long long max_tokens = 0;  // most tokens live sequences hold, each in whole pages
  int max_seq_len = 0;       // longest sequence (0: max_tokens)
  int max_step_tokens = 0;   // 0: the model's default
};

// Builds the model of a folder whose config.json names it; an llm_status.
using ModelFactory = int (*)(const Json& config, const std::string& dir, const ModelOptions& opt,
                             std::unique_ptr<StepModel>* out);
// A model family enters the registry from its own source file:
//   static const ModelRegistrar reg("Name", &make_name);
struct ModelRegistrar {
  ModelRegistrar(const char* architecture, ModelFactory make);
};
// The model named by config.json's "architecture".
int make_model(const std::string& dir, const ModelOptions& opt, std::unique_ptr<StepModel>* out);
// Registered architectures, comma-separated.
std::string model_names();

}  // namespace llm
