// What the models that a config.json describes share (config_model.hpp).
#include "config_model.hpp"

#include <math.h>
#include <string.h>

#include <chrono>

// --- config.json -------------------------------------------------------------------------------------------
int bad_config(const std::string& why) {
  awq_set_error("config.json: " + why);
  return AWQ_ERR_ARG;
}

int get_number(const Json& j, const std::string& at, const char* key, double* out) {
  const Json* v = j.find(key);
  if (!v || !v->is(Json::Number)) return bad_config(at + key + " is missing or no number");
  *out = v->number;
  return AWQ_OK;
}
int get_int(const Json& j, const std::string& at, const char* key, double lo, double hi, int32_t* out) {
  double d;
  if (int rc = get_number(j, at, key, &d)) return rc;
  if (!(d >= lo && d <= hi) || d != floor(d)) return bad_config(at + key + " is out of range");
  *out = (int32_t)d;
  return AWQ_OK;
}
int get_float(const Json& j, const std::string& at, const char* key, float* out) {
  double d;
  if (int rc = get_number(j, at, key, &d)) return rc;
  *out = (float)d;
  return AWQ_OK;
}
const Json* section(const Json& j, const char* key) {
  const Json* v = j.find(key);
  return v && v->is(Json::Object) ? v : nullptr;
}

// --- tensors -----------------------------------------------------------------------------------------------
int check_tensors(const TensorTable& expected, const Safetensors& file) {
  for (const auto& want : expected) {
    const Tensor* t = file.find(want.first);
    if (!t) {
      awq_set_error("model.safetensors has no tensor " + want.first);
      return AWQ_ERR_IO;
    }
    if (t->shape != want.second || (t->dtype != "BF16" && t->dtype != "F32")) {
      awq_set_error("tensor " + want.first + " has another shape or type than config.json says");
      return AWQ_ERR_IO;
    }
  }
  return AWQ_OK;
}

namespace {
__global__ __launch_bounds__(256) void add_constant_kernel(float* x, float v, int64_t n) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n) x[i] += v;
}
int64_t count_of(const Tensor* t) {
  int64_t n = 1;
  for (int64_t d : t->shape) n *= d;
  return n;
}
}  // namespace

int Loader::stage(const Tensor* t) {
  AWQ_HIP_TRY(hipMemcpyAsync(staging, t->data, (size_t)t->bytes, hipMemcpyHostToDevice, e->stream));
  return AWQ_OK;
}
int Loader::vector(const std::string& name, const float** out, float plus) {
  const Tensor* t = file.find(name);
  const int64_t n = count_of(t);
  float* dst = nullptr;
  if (int rc = e->dev_alloc((void**)&dst, n * 4)) return rc;
  if (int rc = stage(t)) return rc;
  *out = dst;
  if (int rc = launch_convert(staging, wide(t), dst, true, n, e->stream)) return rc;
  if (plus != 0.0f) {
    hipLaunchKernelGGL(add_constant_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, e->stream, dst, plus, n);
    AWQ_HIP_TRY(hipGetLastError());
  }
  return AWQ_OK;
}
int Loader::table(const std::string& name, void** out) {
  const Tensor* t = file.find(name);
  const int64_t n = count_of(t);
  if (int rc = e->dev_alloc(out, n * e->unit())) return rc;
  if (int rc = stage(t)) return rc;
  return launch_convert(staging, wide(t), *out, e->f32, n, e->stream);
}
int Loader::matrix(const std::string& name, void* w, int64_t k, int64_t row0, int64_t col0, int form) {
  const Tensor* t = file.find(name);
  if (int rc = stage(t)) return rc;
  return launch_dense_pack(staging, wide(t), t->shape[0], t->shape[1], w, k, row0, col0, e->f32, e->stream, form);
}
int Loader::block(void** w, int64_t n, int64_t k) { return e->zeroed(w, dense_weight_bytes(n, k, e->f32)); }
int Loader::constants(const std::vector<float>& v, const float** out) {
  float* dst = nullptr;
  if (int rc = e->dev_alloc((void**)&dst, (int64_t)v.size() * 4)) return rc;
  AWQ_HIP_TRY(hipMemcpy(dst, v.data(), v.size() * 4, hipMemcpyHostToDevice));
  *out = dst;
  return AWQ_OK;
}
int Loader::constants(const std::vector<double>& v, const double** out) {
  double* dst = nullptr;
  if (int rc = e->dev_alloc((void**)&dst, (int64_t)v.size() * 8)) return rc;
  AWQ_HIP_TRY(hipMemcpy(dst, v.data(), v.size() * 8, hipMemcpyHostToDevice));
  *out = dst;
  return AWQ_OK;
}
void Loader::numbers(const std::string& name, std::vector<double>* out) {
  const Tensor* t = file.find(name);
  out->clear();
  for (int64_t i = 0; i < t->shape[0]; ++i) {
    uint32_t bits;
    if (wide(t)) {
      memcpy(&bits, (const char*)t->data + 4 * i, 4);
    } else {
      uint16_t h;
      memcpy(&h, (const char*)t->data + 2 * i, 2);
      bits = (uint32_t)h << 16;
    }
    float f;
    memcpy(&f, &bits, 4);
    out->push_back(f);
  }
}

// --- the engine --------------------------------------------------------------------------------------------
int ConfigModel::zeroed(void** p, int64_t bytes) {
  bytes = round_up(std::max<int64_t>(bytes, 4), 4);
  if (int rc = dev_alloc(p, bytes)) return rc;
  return launch_fill_zero(*p, bytes, stream);
}

int ConfigModel::open(std::unique_ptr<ConfigModel> e, const Safetensors& file, const awq_open_options& opt, awq_engine** out) {
  e->f32 = opt.dtype == AWQ_DTYPE_FLOAT32;
  constexpr int64_t kDefaultPositions = 8192;
  e->max_pos = opt.max_positions ? opt.max_positions : kDefaultPositions;
  AWQ_REQUIRE(e->max_pos <= (1 << 24), "max_positions is too large");
  e->pass_tokens = std::min<int64_t>(kPassTokens, e->max_pos);
  e->ld = round_up(e->width, kDenseKAlign);
  e->bounds = {1ll << 40};
  e->batched_prefill = true;
  if (int rc = e->init_driver(e->max_pos)) return rc;

  const auto t0 = std::chrono::steady_clock::now();
  Loader ldr{e.get(), file};
  int64_t largest = 4;
  for (const auto& t : file.tensors()) largest = std::max(largest, t.second.bytes);
  AWQ_HIP_TRY(hipMalloc(&ldr.staging, (size_t)largest));
  const auto all = [&]() -> int {
    if (int rc = ldr.table("embed", &e->embed)) return rc;
    if (int rc = ldr.vector("final.norm", &e->final_norm, e->norm_shift)) return rc;
    if (int rc = ldr.block(&e->head, round_up(e->vocab, kDenseRowAlign), e->ld)) return rc;
    if (int rc = ldr.matrix("head", e->head, e->ld, 0, 0)) return rc;
    return e->load_layers(ldr);
  };
  const int rc = all();
  (void)hipStreamSynchronize(e->stream);  // nothing may still read the staging buffer or the mapped file
  (void)hipFree(ldr.staging);
  if (rc) return rc;
  awq_note_load_seconds(std::chrono::duration<double>(std::chrono::steady_clock::now() - t0).count());

  if (!e->f32) {  // for products that are cut along k
    constexpr int64_t kDenseWorkspace = 32ll << 20;
    e->dense_ws_floats = std::min<int64_t>(kDenseWorkspace, 4 * e->pass_tokens * round_up(e->width, kDenseRowAlign));
    if (int rc2 = e->dev_alloc((void**)&e->dense_ws, e->dense_ws_floats * 4)) return rc2;
  }
  if (int rc2 = e->make_buffers()) return rc2;
  if (int rc2 = e->zeroed((void**)&e->tokens, e->pass_tokens * 4)) return rc2;
  if (int rc2 = e->zeroed((void**)&e->rows, kLogitRows * 4)) return rc2;
  if (int rc2 = e->zeroed(&e->head_in, kLogitRows * e->ld * e->unit())) return rc2;
  if (int rc2 = e->zeroed((void**)&e->logits, kLogitRows * e->vocab * 4)) return rc2;
  if (int rc2 = e->zeroed((void**)&e->best, 8)) return rc2;
  if (int rc2 = launch_fill_zero(e->d_token, 4, e->stream)) return rc2;
  AWQ_HIP_TRY(hipStreamSynchronize(e->stream));
  e->finalized = true;
  if (int rc2 = awq_reset(e.get())) return rc2;
  *out = e.release();
  return AWQ_OK;
}

int ConfigModel::logits_of(const float* x, const int32_t* which, int64_t n, bool sample) {
  NormConvArgs a;
  a.x = x;
  a.rows = which;
  a.M = n;
  a.width = width;
  a.groups = norm_groups;
  a.eps = eps;
  a.w1 = final_norm;
  a.out1 = head_in;
  a.ld = ld;
  if (int rc = launch_norm_conv(a, f32, stream)) return rc;
  DenseArgs d;
  d.w = head;
  d.k = ld;
  d.M = n;
  d.out = sample ? DENSE_ARGMAX : DENSE_F32;
  d.best = best;
  d.workspace = dense_ws;
  d.workspace_floats = dense_ws_floats;
  d.seg[0].x = head_in;
  d.seg[0].ldx = ld;
  d.seg[0].y = logits;
  d.seg[0].ldy = vocab;
  d.seg[0].rows = vocab;
  if (softcap != 0.0f) {
    d.seg[0].act = DENSE_SOFTCAP;
    d.seg[0].act_pos = softcap;
  }
  return launch_dense(d, f32, stream);
}

int ConfigModel::enqueue_step(StepKind kind, int64_t) {
  PassPos pos;
  pos.dyn = d_state;
  if (kind != STEP_SAMPLE)
    if (int rc = run_pass(true, nullptr, 1, pos)) return rc;
  if (kind == STEP_PROMPT) return AWQ_OK;
  if (int rc = logits_of(stream_of(true), nullptr, 1, true)) return rc;
  return launch_take_best(best, d_token, d_out, d_state, kind == STEP_GENERATE ? 1 : 0, stream);
}

int64_t ConfigModel::prompt_pass_tokens(int64_t, int64_t rest) const {
  if (rest == 1 || pass_tokens < 2) return 0;
  // equal passes of whole tiles rather than full ones and a small rest
  const int64_t passes = (rest + pass_tokens - 1) / pass_tokens;
  return std::min<int64_t>(rest, std::min<int64_t>(pass_tokens, round_up((rest + passes - 1) / passes, 128)));
}

int ConfigModel::enqueue_prompt_pass(const int32_t* ids, int64_t pos0, int64_t M) {
  PassPos pos;
  pos.pos0 = (int32_t)pos0;
  pos.epoch = epoch_next;
  epoch_next = (epoch_next + 1) & 0x3fffffff;
  AWQ_HIP_TRY(hipMemcpyAsync(tokens, ids, (size_t)M * 4, hipMemcpyHostToDevice, stream));
  if (int rc = run_pass(false, tokens, M, pos)) return rc;
  // the row the first generated token is sampled from
  AWQ_HIP_TRY(hipMemcpyAsync(stream_of(true), stream_of(false) + (M - 1) * width, (size_t)width * 4, hipMemcpyDeviceToDevice, stream));
  return AWQ_OK;
}

int ConfigModel::read_rows_logits(bool batched, const int32_t* which, int32_t n, float* host_dst) {
  for (int64_t at = 0; at < n; at += kLogitRows) {
    const int64_t k = std::min<int64_t>(kLogitRows, n - at);
    if (batched) AWQ_HIP_TRY(hipMemcpyAsync(rows, which + at, (size_t)k * 4, hipMemcpyHostToDevice, stream));
    if (int rc = logits_of(stream_of(!batched), batched ? rows : nullptr, k, false)) return rc;
    AWQ_HIP_TRY(hipMemcpyAsync(host_dst + at * vocab, logits, (size_t)(k * vocab) * 4, hipMemcpyDeviceToHost, stream));
    AWQ_HIP_TRY(hipStreamSynchronize(stream));
  }
  return AWQ_OK;
}

int ConfigModel::read_logits_f32(float* host_dst) {
  AWQ_HIP_TRY(hipStreamSynchronize(stream));
  AWQ_HIP_TRY(hipMemcpy(host_dst, logits, (size_t)vocab * 4, hipMemcpyDeviceToHost));
  return AWQ_OK;
}

int ConfigModel::read_hidden_f32(float* host_dst) {
  AWQ_HIP_TRY(hipStreamSynchronize(stream));
  AWQ_HIP_TRY(hipMemcpy(host_dst, stream_of(true), (size_t)width * 4, hipMemcpyDeviceToHost));
  return AWQ_OK;
}

int ConfigModel::tap_layer(int64_t run, const float* x, int64_t M) {
  AWQ_HIP_TRY(hipMemcpyAsync(tap + run * M * width, x, (size_t)(M * width) * 4, hipMemcpyDeviceToDevice, stream));
  if (run + 1 == layer_runs()) tap_tokens = M;
  return AWQ_OK;
}

int ConfigModel::set_layer_tap(int on) {
  AWQ_HIP_TRY(hipStreamSynchronize(stream));
  if (on && !tap)
    if (int rc = dev_alloc((void**)&tap, layer_runs() * pass_tokens * width * 4)) return rc;
  if ((on != 0) != tap_on) {
    if (on) {
      tap_saved_graphs = graph_mode;
      graph_mode = false;
    } else {
      graph_mode = tap_saved_graphs;
    }
  }
  tap_on = on != 0;
  tap_tokens = 0;
  return AWQ_OK;
}

int64_t ConfigModel::read_layer_tap(float* host_dst, int64_t capacity) {
  if (!tap_on || tap_tokens == 0) {
    awq_set_error("no pass was tapped");
    return -1;
  }
  const int64_t n = layer_runs() * tap_tokens * width;
  if (host_dst) {
    if (hipStreamSynchronize(stream) != hipSuccess ||
        hipMemcpy(host_dst, tap, (size_t)std::min(n, capacity) * 4, hipMemcpyDeviceToHost) != hipSuccess) {
      awq_set_error("reading the tapped layers failed");
      return -1;
    }
  }
  return n;
}
