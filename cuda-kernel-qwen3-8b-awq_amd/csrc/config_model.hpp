// What the models that a config.json describes share: reading the configuration and the tensors, the embedding and output
// head, passes over a prompt and single steps, logits of any rows, the layer tap.  A model adds its layers.
#pragma once
#include <memory>

#include "checkpoint.hpp"
#include "engine.hpp"
#include "layers.hpp"

// --- config.json: a value that is missing or out of range is refused with its place (`at`) ---------------------------
int bad_config(const std::string& why);
int get_number(const Json& j, const std::string& at, const char* key, double* out);
int get_int(const Json& j, const std::string& at, const char* key, double lo, double hi, int32_t* out);
int get_float(const Json& j, const std::string& at, const char* key, float* out);
const Json* section(const Json& j, const char* key);  // an object, or nullptr

// --- tensors ------------------------------------------------------------------------------------------------------
typedef std::vector<std::pair<std::string, std::vector<int64_t>>> TensorTable;
// every tensor is there, of that shape, bfloat16 or float
int check_tensors(const TensorTable& expected, const Safetensors& file);

struct ConfigModel;
struct Loader {
  ConfigModel* e;
  const Safetensors& file;
  void* staging = nullptr;

  int stage(const Tensor* t);
  static bool wide(const Tensor* t) { return t->dtype == "F32"; }
  int vector(const std::string& name, const float** out, float plus = 0.0f);  // float, `plus` added to every entry
  int table(const std::string& name, void** out);                             // in the activations' type
  // into rows row0.., inputs col0.. of a block of padded inputs k
  int matrix(const std::string& name, void* w, int64_t k, int64_t row0, int64_t col0, int form = PACK_PLAIN);
  int block(void** w, int64_t rows, int64_t k);  // zeroed
  int constants(const std::vector<float>& v, const float** out);
  int constants(const std::vector<double>& v, const double** out);
  void numbers(const std::string& name, std::vector<double>* out);
};

// --- the engine ---------------------------------------------------------------------------------------------------
constexpr int64_t kPassTokens = 2048;   // prompt positions per pass
constexpr int64_t kLogitRows = 128;     // rows whose logits are formed at once

struct ConfigModel : awq_engine {
  int32_t vocab = 0, width = 0, norm_groups = 1;
  float eps = 0.0f, softcap = 0.0f;  // softcap 0: none
  float norm_shift = 0.0f;           // added to the stored weights of the model's norm
  bool f32 = false;
  int64_t max_pos = 0, pass_tokens = 0;
  int64_t ld = 0;  // a normalised token vector, padded
  void *embed = nullptr, *head = nullptr;
  const float* final_norm = nullptr;
  int32_t* tokens = nullptr;
  int32_t* rows = nullptr;  // which rows' logits are asked for
  void* head_in = nullptr;  // [kLogitRows][ld]
  float* logits = nullptr;  // [kLogitRows][vocab]
  unsigned long long* best = nullptr;
  float* dense_ws = nullptr;
  int64_t dense_ws_floats = 0;
  std::vector<int64_t> bounds;
  bool tap_on = false, tap_saved_graphs = true;
  float* tap = nullptr;
  int64_t tap_tokens = 0;

  // --- the model's part
  virtual int load_layers(Loader& ld) = 0;
  virtual int make_buffers() = 0;  // activations, caches, recurrent state
  virtual int64_t layer_runs() const = 0;
  // the residual stream of the one-token step or of a prompt pass
  virtual float* stream_of(bool one) = 0;
  // the embedding and all layers for M tokens: the ids on the device, or the step state's token (one)
  virtual int run_pass(bool one, const int32_t* ids, int64_t M, PassPos pos) = 0;

  int64_t vocab_size() const override { return vocab; }
  int64_t hidden_size() const override { return width; }
  int64_t max_positions() const override { return max_pos; }
  // nothing to clear: a run at position 0 reads no state of an earlier sequence, and attention sees only rows of the
  // running one
  int begin_sequence() override { return AWQ_OK; }
  const std::vector<int64_t>& length_bounds() const override { return bounds; }
  int32_t epoch_step() const override { return 1; }
  bool refeeds_hidden() const override { return false; }
  int enqueue_step(StepKind kind, int64_t len_bound) override;
  int64_t prompt_pass_tokens(int64_t done, int64_t rest) const override;
  int enqueue_prompt_pass(const int32_t* ids, int64_t pos0, int64_t M) override;
  int read_rows_logits(bool batched, const int32_t* which, int32_t n, float* host_dst) override;
  int read_logits_f32(float* host_dst) override;
  int read_hidden_f32(float* host_dst) override;
  int set_layer_tap(int on) override;
  int64_t read_layer_tap(float* host_dst, int64_t capacity) override;

  int64_t unit() const { return f32 ? 4 : 2; }
  int zeroed(void** p, int64_t bytes);
  // a pass calls it behind layer run `run`; the pass's last call ends it
  int tap_layer(int64_t run, const float* x, int64_t M);
  int logits_of(const float* x, const int32_t* which, int64_t n, bool sample);
  // weights, buffers and driver behind a checked folder; `e` stays the caller's when it fails
  static int open(std::unique_ptr<ConfigModel> e, const Safetensors& file, const awq_open_options& opt, awq_engine** out);
};
