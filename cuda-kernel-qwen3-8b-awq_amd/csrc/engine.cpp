// The step driver: sequence state, step state on the device, captured steps, the prompt and generation loops, and
// the registry of model classes.  What runs inside a step is the model's (engine.hpp).
//
// Replaces the loops of class QWen3AWQInfer of the reference: generateResponse (Inference.cu:1297-1408) and the
// call order around runOneLayer and sampleNextToken.
#include "engine.hpp"
#include "checkpoint.hpp"

#include <stdio.h>
#include <string.h>
#include <fcntl.h>
#include <sys/stat.h>
#include <unistd.h>

#include <algorithm>
#include <chrono>
#include <thread>

static thread_local std::string g_last_error;
void awq_set_error(const std::string& msg) { g_last_error = msg; }
extern "C" const char* awq_last_error(void) { return g_last_error.c_str(); }


// ---------------------------------------------------------------------------
// the registry
// ---------------------------------------------------------------------------
ModelClass* ModelClass::first = nullptr;
ModelClass::ModelClass(const char* arch, int (*fn)(const char*, const awq_open_options&, awq_engine**))
    : architecture(arch), open(fn), next(first) {
  first = this;
}

extern "C" int awq_open(const char* dir, const awq_open_options* opt_in, awq_engine** out) {
  AWQ_REQUIRE(dir != nullptr && out != nullptr, "NULL argument");
  *out = nullptr;
  awq_open_options opt{};
  if (opt_in) opt = *opt_in;
  AWQ_REQUIRE(opt.dtype >= AWQ_DTYPE_DEFAULT && opt.dtype <= AWQ_DTYPE_FLOAT32, "unknown dtype");
  AWQ_REQUIRE(opt.max_positions >= 0, "max_positions must not be negative");
  std::string arch = AWQ_RAW_DIRECTORY;
  struct stat st;
  if (stat((std::string(dir) + "/config.json").c_str(), &st) == 0)
    if (int rc = awq_config_architecture(dir, &arch)) return rc;
  for (ModelClass* c = ModelClass::first; c; c = c->next)
    if (arch == c->architecture) return c->open(dir, opt, out);
  awq_set_error("no model class for architecture \"" + arch + "\"");
  return AWQ_ERR_ARG;
}

extern "C" const char* awq_architecture(const awq_engine* e) { return e ? e->architecture() : ""; }
extern "C" int64_t awq_vocab_size(const awq_engine* e) { return e ? e->vocab_size() : 0; }
extern "C" int64_t awq_hidden_size(const awq_engine* e) { return e ? e->hidden_size() : 0; }
extern "C" int64_t awq_max_positions(const awq_engine* e) { return e ? e->max_positions() : 0; }

// ---------------------------------------------------------------------------
// what every engine owns
// ---------------------------------------------------------------------------
int awq_engine::dev_alloc(void** p, int64_t bytes) {
  AWQ_HIP_TRY(hipMalloc(p, (size_t)(bytes > 0 ? bytes : 4)));
  allocations.push_back(*p);
  return AWQ_OK;
}

int awq_engine::dev_free(void* p) {
  for (auto& a : allocations)
    if (a == p) {
      a = nullptr;
      AWQ_HIP_TRY(hipFree(p));
      return AWQ_OK;
    }
  return AWQ_OK;
}

int awq_engine::init_driver(int64_t positions) {
  int ndev = 0;
  AWQ_HIP_TRY(hipGetDeviceCount(&ndev));
  if (ndev < 1) {
    awq_set_error("no HIP device found");
    return AWQ_ERR_HIP;
  }
  AWQ_HIP_TRY(hipGetDevice(&device));
  AWQ_HIP_TRY(hipStreamCreateWithFlags(&stream, hipStreamNonBlocking));
  if (int rc = dev_alloc((void**)&d_state, sizeof(StepState))) return rc;
  if (int rc = dev_alloc((void**)&d_token, 4)) return rc;
  return dev_alloc((void**)&d_out, positions * 4);
}

void awq_engine::drop_graphs() {
  for (auto& row : graphs)
    for (hipGraphExec_t& g : row)
      if (g) {
        (void)hipGraphExecDestroy(g);
        g = nullptr;
      }
}

awq_engine::~awq_engine() {
  if (stream) (void)hipStreamSynchronize(stream);
  drop_graphs();
  for (void* p : allocations)
    if (p) (void)hipFree(p);
  if (stream) (void)hipStreamDestroy(stream);
}

extern "C" void awq_destroy(awq_engine* e) { delete e; }

// ---------------------------------------------------------------------------
// steps
// ---------------------------------------------------------------------------
namespace {
constexpr int kStepsPerGraph = 4;

int length_bucket(const awq_engine* e, int64_t len) {
  const std::vector<int64_t>& bounds = e->length_bounds();
  int bucket = 0;
  while (len > bounds[bucket]) ++bucket;
  return bucket;
}

int build_graph(awq_engine* e, StepKind kind, int64_t len_bound, hipGraphExec_t* out, int n_steps = 1) {
  hipGraph_t graph = nullptr;
  AWQ_HIP_TRY(hipStreamBeginCapture(e->stream, hipStreamCaptureModeThreadLocal));
  int rc = 0;
  for (int i = 0; i < n_steps && !rc; ++i) rc = e->enqueue_step(kind, len_bound);
  hipError_t err = hipStreamEndCapture(e->stream, &graph);
  if (rc) {
    if (graph) hipGraphDestroy(graph);
    return rc;
  }
  AWQ_HIP_TRY(err);
  AWQ_HIP_TRY(hipGraphInstantiate(out, graph, nullptr, nullptr, 0));
  AWQ_HIP_TRY(hipGraphDestroy(graph));
  return AWQ_OK;
}

// `write_state` false: the device already holds `s` (the previous generation step advanced it)
int run_step(awq_engine* e, StepKind kind, StepState s, bool write_state = true, int n_steps = 1) {
  s.epoch = e->epoch_next;
  for (int i = 0; i < n_steps && kind != STEP_SAMPLE; ++i)
    e->epoch_next = (e->epoch_next + e->epoch_step()) & 0x3fffffff;  // what the step's last launch adds on the device
  if (write_state)
    if (int rc = launch_set_state(e->d_state, s, e->stream)) return rc;
  const int bucket = length_bucket(e, s.len_hi);
  const int64_t len_bound = std::min(e->length_bounds()[bucket], e->max_positions());
  if (e->graph_mode && kind != STEP_SAMPLE) {
    hipGraphExec_t* g = &e->graphs[n_steps > 1 ? 2 : (kind == STEP_GENERATE ? 1 : 0)][bucket];
    if (!*g)
      if (int rc = build_graph(e, kind, len_bound, g, n_steps)) return rc;
    AWQ_HIP_TRY(hipGraphLaunch(*g, e->stream));
    return AWQ_OK;
  }
  return e->enqueue_step(kind, len_bound);
}

int prompt_step(awq_engine* e, int32_t token) {
  const int t = e->n_positions;
  StepState s{};
  s.pos = t;
  s.len_lo = e->current_seq_len + 1;  // layer 0 still sees the previous value (Inference.cu:1118 before :1331)
  s.len_hi = t + 1;                   // later layers see current_seq_len_ = t
  s.token = token;
  if (int rc = run_step(e, STEP_PROMPT, s)) return rc;
  e->current_seq_len = t;
  e->n_positions = t + 1;
  return AWQ_OK;
}

// a prompt portion may start
int check_prompt(awq_engine* e, const int32_t* ids, int32_t n, const char* who) {
  if (!e->finalized) {
    awq_set_error(std::string(who) + " before awq_finalize");
    return AWQ_ERR_STATE;
  }
  AWQ_REQUIRE(e->n_generated == 0, "prompt tokens cannot follow generated ones; call awq_reset");
  AWQ_REQUIRE((int64_t)e->n_positions + n <= e->max_positions(), "prompt does not fit max_pos");
  const int64_t vocab = e->vocab_size();
  for (int32_t i = 0; i < n; ++i) AWQ_REQUIRE(ids[i] >= 0 && ids[i] < vocab, "token id out of range");
  return AWQ_OK;
}

// A prompt portion in passes of several positions (token by token where the model asks for it).  `want`: ascending
// places of the portion whose logits go to `logits`, one row of vocab values each.
int prompt_passes(awq_engine* e, const int32_t* ids, int32_t n, const int32_t* want, int32_t n_want, float* logits) {
  int32_t w = 0;
  std::vector<int32_t> rows;
  for (int64_t off = 0, M = 0; off < n; off += M) {
    const int64_t pos0 = e->n_positions;
    M = e->prompt_pass_tokens(pos0, n - off);
    const bool batched = M > 0;
    if (batched) {
      if (int rc = e->enqueue_prompt_pass(ids + off, pos0, M)) return rc;
      AWQ_HIP_TRY(hipStreamSynchronize(e->stream));  // the token ids were read from the caller's buffer
      if (int rc = e->check_prompt_pass()) return rc;
      e->current_seq_len = (int)(pos0 + M - 1);
      e->n_positions = (int)(pos0 + M);
    } else {
      M = 1;
      if (int rc = prompt_step(e, ids[off])) return rc;
    }
    rows.clear();
    for (; w < n_want && want[w] < off + M; ++w) rows.push_back((int32_t)(want[w] - off));
    if (!rows.empty()) {
      if (int rc = e->read_rows_logits(batched, rows.data(), (int32_t)rows.size(), logits)) return rc;
      logits += (int64_t)rows.size() * e->vocab_size();
    }
  }
  AWQ_HIP_TRY(hipStreamSynchronize(e->stream));
  return e->check_steps();
}

thread_local double g_last_load_seconds = 0.0;
}  // namespace

// readBinaryFileToDevice's host half (Inference.cu:297-308): exactly `bytes` bytes of the file from `offset` on (more are
// ignored, fewer are an error).  A large file is read by four threads, a quarter each: one thread copies
// out of the page cache at 8-10 GB/s, well below what the copy to the device takes.
int awq_read_file(const std::string& path, int64_t offset, int64_t bytes, void* dst, std::string* err) {
  const int fd = open(path.c_str(), O_RDONLY);
  if (fd < 0) {
    *err = "could not open " + path;  // Inference.cu:299-302
    return AWQ_ERR_IO;
  }
  auto read_range = [fd, dst, offset](int64_t from, int64_t to) {
    while (from < to) {
      const ssize_t got = pread(fd, (char*)dst + from, (size_t)(to - from), (off_t)(offset + from));
      if (got <= 0) return false;  // end of file or an error: the file is short
      from += got;
    }
    return true;
  };
  // from a cold disk: have the whole range scheduled as one sequential read before four threads ask for
  // quarters of it (no effect on cached files)
  (void)posix_fadvise(fd, (off_t)offset, (off_t)bytes, POSIX_FADV_WILLNEED);
  bool ok = true;
  constexpr int64_t kParallelFrom = 8ll << 20;
  constexpr int kReaders = 4;
  if (bytes >= kParallelFrom) {
    bool part_ok[kReaders];
    std::thread helper[kReaders - 1];
    const int64_t piece = ((bytes / kReaders) + 4095) & ~4095ll;
    for (int i = 1; i < kReaders; ++i)
      helper[i - 1] = std::thread([&, i] { part_ok[i] = read_range(std::min(bytes, i * piece), std::min(bytes, (i + 1) * piece)); });
    part_ok[0] = read_range(0, std::min(bytes, piece));
    for (auto& h : helper) h.join();
    for (bool p_ok : part_ok) ok = ok && p_ok;
  } else {
    ok = read_range(0, bytes);
  }
  close(fd);
  if (!ok) {
    *err = "read failed for " + path;  // :305-308
    return AWQ_ERR_IO;
  }
  return AWQ_OK;
}


extern "C" double awq_last_load_seconds(void) { return g_last_load_seconds; }

void awq_note_load_seconds(double s) { g_last_load_seconds = s; }

extern "C" int awq_set_graph_mode(awq_engine* e, int enabled) {
  AWQ_REQUIRE(e != nullptr, "engine is NULL");
  e->graph_mode = enabled != 0;
  return AWQ_OK;
}

extern "C" int awq_reset(awq_engine* e) {
  AWQ_REQUIRE(e != nullptr, "engine is NULL");
  if (!e->finalized) {
    awq_set_error("awq_reset before awq_finalize");
    return AWQ_ERR_STATE;
  }
  // The reference initialises current_seq_len_ in the constructor only
  // (Inference.cu:430); a second generateResponse would attend stale positions.
  // Each sequence starts clean here, with a zero hidden state.
  e->current_seq_len = 0;
  e->n_positions = 0;
  e->n_generated = 0;
  return e->begin_sequence();
}

// prompt loop, Inference.cu:1304-1343
extern "C" int awq_prefill(awq_engine* e, const int32_t* prompt_ids, int32_t n_prompt) {
  AWQ_REQUIRE(e != nullptr && n_prompt >= 0 && (n_prompt == 0 || prompt_ids), "bad arguments");
  if (int rc = check_prompt(e, prompt_ids, n_prompt, "awq_prefill")) return rc;
  for (int32_t i = 0; i < n_prompt; ++i)
    if (int rc = prompt_step(e, prompt_ids[i])) return rc;
  AWQ_HIP_TRY(hipStreamSynchronize(e->stream));
  return e->check_steps();
}

// The prompt loop (Inference.cu:1304-1343) with all prompt positions of a chunk
// going through each layer together: the weights are read once per chunk and
// the products run on the matrix cores.  Every token still sees exactly the
// positions the sequential loop shows it.  The products are summed in another
// order than the one-token kernel's, so the cache it leaves agrees with
// awq_prefill's to rounding noise, not bit for bit.
extern "C" int awq_prefill_batched(awq_engine* e, const int32_t* prompt_ids, int32_t n_prompt) {
  AWQ_REQUIRE(e != nullptr && n_prompt >= 0 && (n_prompt == 0 || prompt_ids), "bad arguments");
  if (int rc = check_prompt(e, prompt_ids, n_prompt, "awq_prefill_batched")) return rc;
  return prompt_passes(e, prompt_ids, n_prompt, nullptr, 0, nullptr);
}

extern "C" int awq_forward(awq_engine* e, const int32_t* ids, int32_t n, const int32_t* want, int32_t n_want,
                           float* logits) {
  AWQ_REQUIRE(e != nullptr && n >= 0 && (n == 0 || ids), "bad arguments");
  AWQ_REQUIRE(n_want >= 0 && (n_want == 0 || (want && logits)), "bad arguments");
  for (int32_t i = 0; i < n_want; ++i)
    AWQ_REQUIRE(want[i] >= (i ? want[i - 1] : 0) && want[i] < n, "wanted places must ascend within the portion");
  if (int rc = check_prompt(e, ids, n, "awq_forward")) return rc;
  return prompt_passes(e, ids, n, want, n_want, logits);
}

extern "C" int awq_set_prefill_mode(awq_engine* e, int batched) {
  AWQ_REQUIRE(e != nullptr, "engine is NULL");
  e->batched_prefill = batched != 0;
  return AWQ_OK;
}

// generation loop, Inference.cu:1352-1405
extern "C" int awq_decode(awq_engine* e, int32_t n_steps, int32_t* out_ids) {
  AWQ_REQUIRE(e != nullptr && n_steps >= 0 && (n_steps == 0 || out_ids), "bad arguments");
  if (!e->finalized) {
    awq_set_error("awq_decode before awq_finalize");
    return AWQ_ERR_STATE;
  }
  AWQ_REQUIRE((int64_t)e->n_positions + n_steps <= e->max_positions(), "sequence does not fit max_pos");
  AWQ_REQUIRE(e->refeeds_hidden() || e->n_positions > 0 || n_steps == 0, "nothing to continue: the sequence is empty");
  const int first = e->n_generated;
  for (int32_t i = 0; i < n_steps; ++i) {
    const int pos = e->n_positions;
    StepState s{};
    s.pos = pos;
    s.len_lo = e->current_seq_len + 1;  // layers below split_idx run before Inference.cu:1364
    s.len_hi = pos + 1;                 // the others after it
    s.token = -1;
    s.out_index = e->n_generated;
    s.sample = 1;
    if (e->n_generated == 0 && !e->refeeds_hidden()) {
      // the prompt's last position has not been sampled from yet; the step that follows starts behind it
      s.pos = pos - 1;
      if (int rc = run_step(e, STEP_SAMPLE, s)) return rc;
      e->n_generated += 1;
      continue;
    }
    // kStepsPerGraph steps as one graph launch where the call has that many left and they share a length bound
    // (the steps advance their own state on the device, so the nodes of one step are those of the next): a
    // graph launch costs about 8 us beyond its kernels, 1031 -> 1037 tok/s with four steps per launch, the
    // same with 8, 16 or 32
    const bool several = e->graph_mode && i > 0 && i + kStepsPerGraph <= n_steps &&
                         length_bucket(e, pos + 1) == length_bucket(e, pos + kStepsPerGraph);
    const int k = several ? kStepsPerGraph : 1;
    // the state is written for the first step of the call; every step leaves the next one's on the device
    if (int rc = run_step(e, STEP_GENERATE, s, i == 0, k)) return rc;
    e->current_seq_len = pos + k - 1;
    e->n_positions = pos + k;
    e->n_generated += k;
    i += k - 1;
  }
  AWQ_HIP_TRY(hipStreamSynchronize(e->stream));
  if (int rc = e->check_steps()) return rc;
  if (n_steps > 0)
    AWQ_HIP_TRY(hipMemcpy(out_ids, e->d_out + first, (size_t)n_steps * 4, hipMemcpyDeviceToHost));
  return AWQ_OK;
}

extern "C" int awq_generate(awq_engine* e, const int32_t* prompt_ids, int32_t n_prompt, int32_t max_new_tokens,
                            int32_t* out_ids) {
  AWQ_REQUIRE(e != nullptr, "engine is NULL");
  AWQ_REQUIRE(n_prompt >= 0 && max_new_tokens >= 0, "negative count");
  AWQ_REQUIRE((int64_t)n_prompt + max_new_tokens <= e->max_positions(), "prompt + new tokens exceed max_pos");
  auto once = [&]() -> int {
    if (int rc = awq_reset(e)) return rc;
    if (int rc = e->batched_prefill ? awq_prefill_batched(e, prompt_ids, n_prompt) : awq_prefill(e, prompt_ids, n_prompt))
      return rc;
    return awq_decode(e, max_new_tokens, out_ids);
  };
  int rc = once();
  if (rc == AWQ_ERR_HIP && e->retry_unfused()) rc = once();
  return rc;
}

namespace {
template <typename F>
int read_f32(awq_engine* e, float* host_dst, F f) {
  AWQ_REQUIRE(e && host_dst, "NULL argument");
  AWQ_REQUIRE(e->finalized, "the engine has no weights yet");
  return f();
}
}  // namespace
extern "C" int awq_read_hidden_f32(awq_engine* e, float* host_dst) {
  return read_f32(e, host_dst, [&] { return e->read_hidden_f32(host_dst); });
}
extern "C" int awq_read_logits_f32(awq_engine* e, float* host_dst) {
  return read_f32(e, host_dst, [&] { return e->read_logits_f32(host_dst); });
}
extern "C" int awq_set_layer_tap(awq_engine* e, int on) {
  AWQ_REQUIRE(e != nullptr, "engine is NULL");
  return e->set_layer_tap(on);
}
extern "C" int64_t awq_read_layer_tap(awq_engine* e, float* host_dst, int64_t capacity) {
  return e ? e->read_layer_tap(host_dst, capacity) : -1;
}
