// Host-side engine declarations: the state and the step driver every model shares (engine.cpp), what a model
// supplies to it, and the registry by which a model folder finds its class.
#pragma once
#include <string>
#include <vector>

#include "common.hpp"

// What one recorded or eager pass over the layers does (awq_engine::enqueue_step).
enum StepKind {
  STEP_PROMPT = 0,    // the state's token goes through the layers
  STEP_GENERATE = 1,  // ... and the next token is sampled; the step leaves the next one's state on the device
  STEP_SAMPLE = 2,    // no position: the next token is sampled from the hidden state as it stands
};

// One engine: the sequence, its step state on the device and the captured steps are the driver's (engine.cpp);
// weights, caches, recurrent state and launches are the model's, behind the virtual functions.
struct awq_engine {
  int device = 0;
  hipStream_t stream = nullptr;
  StepState* d_state = nullptr;
  int32_t* d_token = nullptr;  // the token sampled last
  int32_t* d_out = nullptr;    // [max_positions] generated tokens
  // sequence state
  int current_seq_len = 0;  // current_seq_len_ of Inference.cu:408
  int n_positions = 0;      // forward passes since reset
  int n_generated = 0;
  bool finalized = false;
  bool graph_mode = true;
  bool batched_prefill = false;
  int32_t epoch_next = 0;  // the epoch of the next step (mirrors what the device adds per step)
  static constexpr int kMaxBuckets = 8;
  hipGraphExec_t graphs[3][kMaxBuckets] = {};  // [prompt | generation step | kStepsPerGraph generation steps][length bound]
  std::vector<void*> allocations;

  virtual ~awq_engine();
  virtual const char* architecture() const = 0;
  virtual int64_t vocab_size() const = 0;
  virtual int64_t hidden_size() const = 0;
  virtual int64_t max_positions() const = 0;
  // everything the model holds beyond the driver's counters at the start of a sequence
  virtual int begin_sequence() = 0;
  // the launches of one step, position and lengths from d_state; `len_bound` >= every attended length
  virtual int enqueue_step(StepKind kind, int64_t len_bound) = 0;
  // The launches may be specialised by an upper bound of the attended length: ascending bounds, the last one
  // unreachable; one captured graph per bound.
  virtual const std::vector<int64_t>& length_bounds() const = 0;
  // what a step adds to the state's epoch on the device
  virtual int32_t epoch_step() const = 0;
  // true: the first generated position feeds the last hidden state again (Inference.cu:1357); false: the first
  // token is sampled from it without another position
  virtual bool refeeds_hidden() const = 0;
  // after the stream has drained: did a launch of the steps report a fault?
  virtual int check_steps() { return AWQ_OK; }
  // after a failed request: switch to a slower form of the launches and say so, or false
  virtual bool retry_unfused() { return false; }

  // Several prompt positions at once.  How many of `rest` tokens the next pass takes after `done` positions
  // (0: token by token), its launches (the host's token ids are read before the stream has drained), and the
  // check after the stream has drained.
  virtual int64_t prompt_pass_tokens(int64_t done, int64_t rest) const = 0;
  virtual int enqueue_prompt_pass(const int32_t* tokens, int64_t pos0, int64_t M) = 0;
  virtual int check_prompt_pass() { return AWQ_OK; }

  // 32-bit logits of `n` rows of the latest pass (`batched`: a prompt pass, row = token of the pass; otherwise the
  // latest step's only row) to host memory, synchronously
  virtual int read_rows_logits(bool batched, const int32_t* rows, int32_t n, float* host_dst) = 0;
  // the last sampled position's logits [vocab] and the hidden state [hidden], binary32
  virtual int read_logits_f32(float* host_dst) = 0;
  virtual int read_hidden_f32(float* host_dst) = 0;
  // the residual stream after every layer of the next passes goes to the host (tests); not every model has it
  virtual int set_layer_tap(int) {
    awq_set_error("this model has no layer tap");
    return AWQ_ERR_ARG;
  }
  virtual int64_t read_layer_tap(float*, int64_t) { return -1; }

  // device memory that lives as long as the engine
  int dev_alloc(void** p, int64_t bytes);
  int dev_free(void* p);
  // stream, step state, sampled token, output array
  int init_driver(int64_t max_positions);
  void drop_graphs();
};

// A model class of the registry: `architecture` is config.json's entry of that name.  A source file that defines a
// model holds one of these as a static object, so a program serves the models whose object files it is linked from.
struct ModelClass {
  const char* architecture;
  int (*open)(const char* dir, const awq_open_options& opt, awq_engine** out);
  ModelClass* next;
  ModelClass(const char* arch, int (*fn)(const char*, const awq_open_options&, awq_engine**));
  static ModelClass* first;
};
// the name under which the class of config.json-less weight directories is registered
#define AWQ_RAW_DIRECTORY "raw weight directory"

// exactly `bytes` bytes of a file from `offset` on (Inference.cu:297-308); a large range is read by four threads
int awq_read_file(const std::string& path, int64_t offset, int64_t bytes, void* dst, std::string* err);
// on the calling thread, set by the loaders (awq_last_load_seconds)
void awq_note_load_seconds(double s);

// one file of the weight directory (Inference.cu:780-899)
struct WeightFile {
  std::string name;
  int layer, kind, part;
  int64_t bytes;
};

int awq_check_config(const awq_config* cfg);
std::vector<WeightFile> awq_weight_files(const awq_config& cfg);
// rows (outputs) and columns (inputs) of a quantised tensor kind
void awq_tensor_dims(const awq_config& cfg, int kind, int64_t* out_dim, int64_t* in_dim);
bool awq_zp_all_integral(const uint16_t* zp, int64_t n);
