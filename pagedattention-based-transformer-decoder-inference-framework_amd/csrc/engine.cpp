// The serving engine: the model registry, sequences and their cache slots, the
// mixed-batch step and the scheduler over it.
#include <algorithm>
#include <cstring>
#include <deque>
#include <fstream>
#include <map>
#include <memory>
#include <mutex>
#include <sstream>
#include <vector>

#include "common.hpp"
#include "dev_buf.hpp"
#include "model.hpp"
#include "row_ops.hpp"

namespace llm {

static std::map<std::string, ModelFactory>& registry() {
  static std::map<std::string, ModelFactory> r;  // filled while the library loads
  return r;
}

ModelRegistrar::ModelRegistrar(const char* architecture, ModelFactory make) {
  registry()[architecture] = make;
}

std::string model_names() {
  std::string s;
  for (const auto& m : registry()) s += (s.empty() ? "" : ",") + m.first;
  return s;
}

int make_model(const std::string& dir, const ModelOptions& opt, std::unique_ptr<StepModel>* out) {
  std::ifstream f(dir + "/config.json", std::ios::binary);
  if (!f) return fail(LLM_ERR_IO, "cannot open " + dir + "/config.json");
  std::stringstream ss;
  ss << f.rdbuf();
  const std::string text = ss.str();
  Json c;
  if (!JsonReader(text.data(), text.size()).parse(c) || !c.is_object())
    return fail(LLM_ERR_IO, dir + "/config.json is not a JSON object");
  const auto it = registry().find(c["architecture"].str);
  if (it == registry().end())
    return fail(LLM_ERR_UNSUPPORTED, "config.json: architecture '" + c["architecture"].str +
                                         "' is not one of " + model_names());
  return it->second(c, dir, opt, out);
}

namespace {

struct Sequence {
  bool open = false;
  int len = 0;
};

struct Request {
  int id = 0, slot = -1;
  std::vector<int32_t> tokens;  // prompt, then what was generated
  int prompt = 0, done = 0;     // done: tokens in the cache
  llm_request_params p{};
  long long pages = 0;
  bool finished = false;
  int generated() const { return (int)tokens.size() - prompt; }
};

}  // namespace
}  // namespace llm

using namespace llm;

struct llm_engine {
  std::unique_ptr<StepModel> model;
  hipStream_t stream = nullptr;
  std::mutex mu;
  int max_seqs = 1;
  std::vector<Sequence> seqs;
  DevBuf<float> logits;   // [rows][vocab]
  DevBuf<int32_t> next;   // [rows] chosen ids
  DevBuf<int32_t> draw;   // [rows] draw counters
  size_t rows_cap = 0;

  std::deque<std::unique_ptr<Request>> waiting;
  std::vector<std::unique_ptr<Request>> running;
  std::map<int, std::unique_ptr<Request>> finished;
  int next_id = 1;
  long long promised = 0;  // pages the running requests may come to hold

  ~llm_engine() {
    if (stream) (void)hipStreamSynchronize(stream);
    model.reset();
    if (stream) (void)hipStreamDestroy(stream);
  }
  int ensure_logits(size_t rows) {
    if (rows <= rows_cap) return LLM_OK;
    LLM_HIP_RET(hipStreamSynchronize(stream));
    const size_t n = std::max<size_t>(rows, 16);
    rows_cap = 0;
    RET_IF(logits.alloc(n * model->vocab()));
    RET_IF(next.alloc(n));
    RET_IF(draw.alloc(n));
    rows_cap = n;
    return LLM_OK;
  }
  int open_slot(int* seq) {
    for (int i = 0; i < max_seqs; ++i)
      if (!seqs[i].open) {
        seqs[i].open = true;
        seqs[i].len = 0;
        *seq = i;
        return LLM_OK;
      }
    return fail(LLM_ERR_OOM, "engine: every sequence slot is in use");
  }
  int close_slot(int seq) {
    seqs[seq].open = false;
    seqs[seq].len = 0;
    return model->release(seq);
  }
  long long pages_for(long long tokens) const {
    return (tokens + model->page_tokens() - 1) / model->page_tokens();
  }
  int step(const llm_engine_entry* entries, int n, float* host);
  int run(int* active);
  int choose(const std::vector<Request*>& rows);
};

// Batches past the model's step size run as several passes, cut anywhere.
int llm_engine::step(const llm_engine_entry* entries, int n, float* host) {
  std::vector<char> seen(max_seqs, 0);
  size_t wanted = 0;
  for (int i = 0; i < n; ++i) {
    const llm_engine_entry& t = entries[i];
    LLM_REQUIRE(t.seq >= 0 && t.seq < max_seqs && seqs[t.seq].open, "engine step: sequence not open");
    LLM_REQUIRE(!seen[t.seq], "engine step: a sequence appears twice");
    seen[t.seq] = 1;
    LLM_REQUIRE(t.n >= 1 && t.tokens && t.n_want >= 0 && (t.n_want == 0 || t.want),
                "engine step: an entry needs tokens");
    LLM_REQUIRE((long long)seqs[t.seq].len + t.n <= model->max_seq_len(),
                "engine step: sequence past max_seq_len");
    for (int k = 0; k < t.n_want; ++k)
      LLM_REQUIRE(t.want[k] >= 0 && t.want[k] < t.n, "engine step: wanted place out of range");
    for (int k = 0; k < t.n; ++k)
      LLM_REQUIRE(t.tokens[k] >= 0 && t.tokens[k] < model->vocab(),
                  "engine step: token id out of range");
    wanted += (size_t)t.n_want;
  }
  LLM_REQUIRE(wanted == 0 || host, "engine step: logits is NULL");
  const int cap = model->max_step_tokens();
  const int V = model->vocab();
  std::vector<StepSeq> batch;
  std::vector<std::vector<int32_t>> wants;
  std::vector<size_t> rows;
  std::vector<int> len0(n);
  for (int i = 0; i < n; ++i) len0[i] = seqs[entries[i].seq].len;
  int used = 0;
  const auto flush = [&]() -> int {
    if (batch.empty()) return LLM_OK;
    for (size_t i = 0; i < batch.size(); ++i) {
      batch[i].want = wants[i].data();
      batch[i].n_want = (int)wants[i].size();
    }
    RET_IF(ensure_logits(rows.size()));
    RET_IF(model->forward(batch, logits.p, stream));
    bool in_order = true;
    for (size_t r = 1; r < rows.size(); ++r) in_order = in_order && rows[r] == rows[r - 1] + 1;
    if (!rows.empty() && in_order)
      LLM_HIP_RET(hipMemcpyAsync(host + rows[0] * V, logits.p, rows.size() * V * sizeof(float),
                                 hipMemcpyDeviceToHost, stream));
    else
      for (size_t r = 0; r < rows.size(); ++r)
        LLM_HIP_RET(hipMemcpyAsync(host + rows[r] * V, logits.p + r * V, V * sizeof(float),
                                   hipMemcpyDeviceToHost, stream));
    LLM_HIP_RET(hipStreamSynchronize(stream));
    for (const StepSeq& s : batch) seqs[s.slot].len = s.p0 + s.n;
    batch.clear();
    wants.clear();
    rows.clear();
    used = 0;
    return LLM_OK;
  };
  int rc = LLM_OK;
  size_t row0 = 0;
  for (int i = 0; i < n && !rc; ++i) {
    const llm_engine_entry& t = entries[i];
    for (int at = 0; at < t.n && !rc;) {
      const int m = std::min(t.n - at, cap - used);
      StepSeq s;
      s.slot = t.seq;
      s.p0 = len0[i] + at;
      s.n = m;
      s.tokens = t.tokens + at;
      std::vector<int32_t> w;
      for (int k = 0; k < t.n_want; ++k)
        if (t.want[k] >= at && t.want[k] < at + m) {
          w.push_back(t.want[k] - at);
          rows.push_back(row0 + k);
        }
      batch.push_back(s);
      wants.push_back(std::move(w));
      used += m;
      at += m;
      if (used == cap) rc = flush();
    }
    row0 += (size_t)t.n_want;
  }
  if (!rc) rc = flush();
  if (rc)
    for (int i = 0; i < n; ++i) seqs[entries[i].seq].len = len0[i];
  return rc;
}

// Ids of the step's logits rows into `next` on the device: greedy rows in one
// launch, every drawn row with its request's own settings.
int llm_engine::choose(const std::vector<Request*>& rows) {
  const int V = model->vocab(), n = (int)rows.size();
  std::vector<int32_t> ctr(n);
  bool greedy = false;
  for (int i = 0; i < n; ++i) {
    ctr[i] = rows[i]->done - 1;  // the position whose logits these are
    greedy = greedy || rows[i]->p.temperature <= 0.f || rows[i]->p.top_k == 1;
  }
  LLM_HIP_RET(hipMemcpyAsync(draw.p, ctr.data(), n * sizeof(int32_t), hipMemcpyHostToDevice, stream));
  if (greedy) LLM_HIP_RET(launch_argmax(logits.p, n, V, next.p, nullptr, 0, stream));
  for (int i = 0; i < n; ++i) {
    const llm_request_params& p = rows[i]->p;
    if (p.temperature <= 0.f || p.top_k == 1) continue;
    LLM_HIP_RET(launch_sample(logits.p + (size_t)i * V, 1, 0, V, p.temperature, p.top_k,
                              p.top_p > 0.f ? p.top_p : 1.f, p.seed, draw.p + i, next.p + i, stream));
  }
  std::vector<int32_t> ids(n);
  LLM_HIP_RET(hipMemcpyAsync(ids.data(), next.p, n * sizeof(int32_t), hipMemcpyDeviceToHost, stream));
  LLM_HIP_RET(hipStreamSynchronize(stream));
  for (int i = 0; i < n; ++i) {
    Request& r = *rows[i];
    r.tokens.push_back(ids[i]);
    r.finished = r.generated() >= r.p.max_new_tokens || ids[i] == r.p.eos_token;
  }
  return LLM_OK;
}

int llm_engine::run(int* active) {
  while (!waiting.empty()) {
    Request& r = *waiting.front();
    if (promised + r.pages > pages_for(model->pool_tokens())) break;
    int free = 0;
    for (const Sequence& s : seqs) free += !s.open;
    if (free == 0) break;
    RET_IF(open_slot(&r.slot));
    promised += r.pages;
    running.push_back(std::move(waiting.front()));
    waiting.pop_front();
  }
  // one token of every generating request first, then prompt portions
  const int cap = model->max_step_tokens();
  int used = 0;
  std::vector<StepSeq> batch;
  std::vector<Request*> in_batch, rows;
  static const int32_t kFirst = 0;
  std::vector<int32_t> last(running.size());
  for (int pass = 0; pass < 2; ++pass)
    for (size_t i = 0; i < running.size() && used < cap; ++i) {
      Request& r = *running[i];
      const int left = (int)r.tokens.size() - r.done;
      if ((left == 1 && r.done > 0) != (pass == 0)) continue;
      StepSeq s;
      s.slot = r.slot;
      s.p0 = r.done;
      s.n = std::min(left, cap - used);
      s.tokens = r.tokens.data() + r.done;
      if (s.n == left) {
        last[i] = s.n - 1;
        s.want = s.n == 1 ? &kFirst : &last[i];
        s.n_want = 1;
        rows.push_back(&r);
      }
      used += s.n;
      batch.push_back(s);
      in_batch.push_back(&r);
    }
  if (!batch.empty()) {
    RET_IF(ensure_logits(std::max<size_t>(rows.size(), 1)));
    RET_IF(model->forward(batch, logits.p, stream));
    for (size_t i = 0; i < batch.size(); ++i) {
      in_batch[i]->done += batch[i].n;
      seqs[batch[i].slot].len = in_batch[i]->done;
    }
    if (!rows.empty()) RET_IF(choose(rows));
    else LLM_HIP_RET(hipStreamSynchronize(stream));
    for (size_t i = 0; i < running.size();) {
      if (!running[i]->finished) { ++i; continue; }
      promised -= running[i]->pages;
      RET_IF(close_slot(running[i]->slot));
      const int id = running[i]->id;
      finished[id] = std::move(running[i]);
      running.erase(running.begin() + i);
    }
  }
  *active = (int)(waiting.size() + running.size());
  return LLM_OK;
}

extern "C" const char* llm_model_architectures(void) {
  static const std::string names = model_names();
  return names.c_str();
}

extern "C" int llm_engine_create(const char* model_dir, const llm_engine_config* cfg,
                                 llm_engine** out) {
  LLM_REQUIRE(model_dir && cfg && out, "llm_engine_create: NULL");
  LLM_REQUIRE(cfg->max_seqs >= 1 && cfg->max_tokens >= 1 && cfg->max_seq_len >= 0 &&
                  cfg->max_step_tokens >= 0,
              "llm_engine_create: max_seqs and max_tokens must be positive");
  std::unique_ptr<llm_engine> e(new llm_engine());
  e->max_seqs = cfg->max_seqs;
  e->seqs.resize(cfg->max_seqs);
  ModelOptions o;
  o.dtype = cfg->dtype;
  o.max_seqs = cfg->max_seqs;
  o.max_tokens = cfg->max_tokens;
  o.max_seq_len = cfg->max_seq_len;
  o.max_step_tokens = cfg->max_step_tokens;
  RET_IF(make_model(model_dir, o, &e->model));
  LLM_HIP_RET(hipStreamCreateWithFlags(&e->stream, hipStreamNonBlocking));
  RET_IF(e->ensure_logits((size_t)std::max(16, cfg->max_seqs)));
  *out = e.release();
  return LLM_OK;
}

extern "C" void llm_engine_destroy(llm_engine* e) { delete e; }

extern "C" int llm_engine_vocab(const llm_engine* e) { return e ? e->model->vocab() : -1; }
extern "C" int llm_engine_max_seq_len(const llm_engine* e) { return e ? e->model->max_seq_len() : -1; }
extern "C" int llm_engine_page_tokens(const llm_engine* e) { return e ? e->model->page_tokens() : -1; }
extern "C" int llm_engine_layer_runs(const llm_engine* e) { return e ? e->model->layer_runs() : -1; }
extern "C" int llm_engine_width(const llm_engine* e) { return e ? e->model->width() : -1; }

extern "C" long long llm_engine_free_tokens(llm_engine* e) {
  if (!e) return -1;
  std::lock_guard<std::mutex> g(e->mu);
  return e->model->free_tokens();
}

extern "C" int llm_engine_open(llm_engine* e, int* seq) {
  LLM_REQUIRE(e && seq, "llm_engine_open: NULL");
  std::lock_guard<std::mutex> g(e->mu);
  return e->open_slot(seq);
}

extern "C" int llm_engine_close(llm_engine* e, int seq) {
  LLM_REQUIRE(e, "llm_engine_close: NULL");
  std::lock_guard<std::mutex> g(e->mu);
  LLM_REQUIRE(seq >= 0 && seq < e->max_seqs && e->seqs[seq].open, "llm_engine_close: not open");
  for (const auto& r : e->running)
    LLM_REQUIRE(r->slot != seq, "llm_engine_close: the sequence belongs to a request");
  return e->close_slot(seq);
}

extern "C" int llm_engine_seq_len(llm_engine* e, int seq) {
  if (!e || seq < 0 || seq >= e->max_seqs) return -1;
  std::lock_guard<std::mutex> g(e->mu);
  return e->seqs[seq].open ? e->seqs[seq].len : -1;
}

extern "C" int llm_engine_step(llm_engine* e, const llm_engine_entry* entries, int n, float* logits) {
  LLM_REQUIRE(e && (entries || n == 0) && n >= 0, "llm_engine_step: NULL");
  std::lock_guard<std::mutex> g(e->mu);
  return e->step(entries, n, logits);
}

extern "C" int llm_engine_set_tap(llm_engine* e, float* tap) {
  LLM_REQUIRE(e, "llm_engine_set_tap: NULL");
  std::lock_guard<std::mutex> g(e->mu);
  return e->model->set_tap(tap);
}

extern "C" int llm_engine_submit(llm_engine* e, const int32_t* prompt, int n,
                                 const llm_request_params* p, int* request) {
  LLM_REQUIRE(e && prompt && p && request, "llm_engine_submit: NULL");
  std::lock_guard<std::mutex> g(e->mu);
  LLM_REQUIRE(n >= 1 && p->max_new_tokens >= 1, "llm_engine_submit: needs a prompt and a length");
  LLM_REQUIRE(p->top_k >= 0 && p->top_p >= 0.f && p->top_p <= 1.f &&
                  (p->temperature <= 0.f || p->top_k == 1 || e->model->vocab() <= 65536),
              "llm_engine_submit: top_k >= 0, 0 <= top_p <= 1, sampling needs a vocabulary <= 65536");
  for (int i = 0; i < n; ++i)
    LLM_REQUIRE(prompt[i] >= 0 && prompt[i] < e->model->vocab(),
                "llm_engine_submit: token id out of range");
  // the last generated token never enters the cache
  const long long len = (long long)n + p->max_new_tokens - 1;
  LLM_REQUIRE(len <= e->model->max_seq_len() &&
                  e->pages_for(len) <= e->pages_for(e->model->pool_tokens()),
              "llm_engine_submit: prompt and generation exceed what the cache holds");
  auto r = std::make_unique<Request>();
  r->id = e->next_id++;
  r->tokens.assign(prompt, prompt + n);
  r->prompt = n;
  r->p = *p;
  r->pages = e->pages_for(len);
  *request = r->id;
  e->waiting.push_back(std::move(r));
  return LLM_OK;
}

extern "C" int llm_engine_run(llm_engine* e, int* active) {
  LLM_REQUIRE(e && active, "llm_engine_run: NULL");
  std::lock_guard<std::mutex> g(e->mu);
  return e->run(active);
}

extern "C" int llm_engine_result(llm_engine* e, int request, int32_t* out, int cap, int* n,
                                 int* finished) {
  LLM_REQUIRE(e && n && finished && (out || cap == 0), "llm_engine_result: NULL");
  std::lock_guard<std::mutex> g(e->mu);
  const Request* r = nullptr;
  const auto it = e->finished.find(request);
  if (it != e->finished.end()) r = it->second.get();
  for (const auto& q : e->running)
    if (q->id == request) r = q.get();
  for (const auto& q : e->waiting)
    if (q->id == request) r = q.get();
  LLM_REQUIRE(r, "llm_engine_result: no such request");
  *n = r->generated();
  *finished = r->finished;
  for (int i = 0; i < std::min(*n, cap); ++i) out[i] = r->tokens[r->prompt + i];
  if (*finished && cap >= *n) e->finished.erase(it);
  return LLM_OK;
}
