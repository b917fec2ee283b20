// Kugilix: a decoder-only model of attention layers over a sliding window and linear-attention layers, parallel
// mixer and feed-forward behind two grouped norms, a causal convolution in front of every mixer, a run of layers
// that is repeated with the embedding added again, sinusoidal positions at the input.  config.json gives every size
// and constant; the order of the layers is data.  Runs in bfloat16 (residual, norms, scores and recurrent state in
// binary32) or wholly in binary32, behind the step driver of engine.cpp.
//
// A layer is four launches (five in a pass with linear attention, and with attention over more than 64 keys):
//   norms + convolution     x -> h = conv(norm1(x)) and n = norm2(x)
//   one product             q, k, v (and the gate) of h, and act(W_up n): two segments of one weight block
//   the mixer               -> ctx
//   one product             x += [W_o | W_down] [ctx, mid], both halves in one block along k
#include "config_model.hpp"

#include <math.h>

namespace {

enum MixerType { MIX_ATTENTION, MIX_LIGHTNING };

struct LayerSpec {
  MixerType type = MIX_ATTENTION;
  int32_t heads = 0, kv_heads = 0, dim = 0, vdim = 0;
  int32_t window = 0;
  float scale = 1.0f, temp_coef = 0.0f;
  double temp_every = 1.0;
  std::vector<double> decay;
  int32_t ff = 0;  // 0: no feed-forward
  int32_t mixed() const { return heads * vdim; }
};

struct Spec {
  int32_t vocab = 0, width = 0, taps = 1, groups = 1;
  float eps = 0.0f, embed_scale = 1.0f;
  std::vector<LayerSpec> layers;
  int32_t loop_start = 0, loop_stop = 0, loop_times = 1;
};

// --- config.json -------------------------------------------------------------------------------------------
int read_layer(const Json& j, const std::string& at, LayerSpec* s) {
  const Json *type = j.find("type"), *m = section(j, "mixer");
  if (!type || !type->is(Json::String) || !m) return bad_config(at + "type or mixer is missing");
  const std::string mx = at + "mixer.";
  constexpr double kMany = 1 << 20;
  if (int rc = get_int(*m, mx, "heads", 1, 65535, &s->heads)) return rc;
  if (int rc = get_int(*m, mx, "dim", 1, kMany, &s->dim)) return rc;
  if (int rc = get_int(*m, mx, "vdim", 1, kMany, &s->vdim)) return rc;
  if (type->str == "attention") {
    s->type = MIX_ATTENTION;
    if (int rc = get_int(*m, mx, "kv_heads", 1, 65535, &s->kv_heads)) return rc;
    if (s->heads % s->kv_heads) return bad_config(mx + "heads is no multiple of kv_heads");
    if (int rc = get_float(*m, mx, "scale", &s->scale)) return rc;
    if (const Json* mask = section(*m, "mask"))
      if (int rc = get_int(*mask, mx + "mask.", "size", 1, 1 << 30, &s->window)) return rc;
    if (const Json* t = section(*m, "q_temp")) {
      if (int rc = get_float(*t, mx + "q_temp.", "coef", &s->temp_coef)) return rc;
      if (int rc = get_number(*t, mx + "q_temp.", "every", &s->temp_every)) return rc;
      if (!(s->temp_every > 0.0)) return bad_config(mx + "q_temp.every must be positive");
    }
  } else if (type->str == "lightning") {
    s->type = MIX_LIGHTNING;
    const Json* d = m->find("decay");
    if (!d || !d->is(Json::Array) || (int32_t)d->items.size() != s->heads) return bad_config(mx + "decay needs one number per head");
    for (const Json& v : d->items) {
      if (!v.is(Json::Number)) return bad_config(mx + "decay needs one number per head");
      s->decay.push_back(v.number);
    }
  } else {
    return bad_config(at + "type \"" + type->str + "\" is unknown");
  }
  const Json* f = j.find("mlp");
  if (f && f->is(Json::Object)) {
    const Json* kind = f->find("kind");
    if (!kind || kind->str != "dense") return bad_config(at + "mlp.kind is unknown");
    if (int rc = get_int(*f, at + "mlp.", "ff", 1, 1 << 28, &s->ff)) return rc;
  }
  return AWQ_OK;
}

int read_spec(const std::string& dir, Spec* s) {
  Json j;
  if (int rc = awq_read_json(dir + "/config.json", &j)) return rc;
  if (int rc = get_int(j, "", "vocab", 1, 1 << 28, &s->vocab)) return rc;
  if (int rc = get_int(j, "", "width", 1, 1 << 24, &s->width)) return rc;
  const Json *norm = section(j, "norm"), *canon = section(j, "canon"), *emb = section(j, "embedding"), *layers = j.find("layers");
  if (!norm || !canon || !emb) return bad_config("norm, canon or embedding is missing");
  if (int rc = get_float(*norm, "norm.", "eps", &s->eps)) return rc;
  if (int rc = get_int(*norm, "norm.", "groups", 1, 65535, &s->groups)) return rc;
  if (s->width % s->groups) return bad_config("width is no multiple of norm.groups");
  if (int rc = get_int(*canon, "canon.", "taps", 1, 1024, &s->taps)) return rc;
  if (int rc = get_float(*emb, "embedding.", "scale", &s->embed_scale)) return rc;
  if (!layers || !layers->is(Json::Array) || layers->items.empty() || layers->items.size() > 65535)
    return bad_config("layers is missing or empty");
  for (size_t i = 0; i < layers->items.size(); ++i) {
    s->layers.emplace_back();
    if (int rc = read_layer(layers->items[i], "layers[" + std::to_string(i) + "].", &s->layers.back())) return rc;
  }
  if (const Json* loop = section(j, "loop")) {
    const double n = (double)s->layers.size();
    if (int rc = get_int(*loop, "loop.", "start", 0, n, &s->loop_start)) return rc;
    if (int rc = get_int(*loop, "loop.", "stop", s->loop_start, n, &s->loop_stop)) return rc;
    if (int rc = get_int(*loop, "loop.", "times", 1, 4096, &s->loop_times)) return rc;
  }
  return AWQ_OK;
}

// every tensor of the model and its shape
TensorTable expected_tensors(const Spec& c) {
  const int64_t W = c.width;
  TensorTable v = {{"embed", {c.vocab, W}}, {"final.norm", {W}}, {"head", {c.vocab, W}}};
  for (size_t i = 0; i < c.layers.size(); ++i) {
    const LayerSpec& s = c.layers[i];
    const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.";
    const int64_t mixed = s.mixed(), kv = s.type == MIX_ATTENTION ? s.kv_heads : s.heads;
    v.push_back({p + "norm1", {W}});
    v.push_back({p + "canon1", {W, c.taps}});
    v.push_back({m + "q", {(int64_t)s.heads * s.dim, W}});
    v.push_back({m + "k", {kv * s.dim, W}});
    v.push_back({m + "v", {kv * s.vdim, W}});
    v.push_back({m + "o", {W, mixed}});
    if (s.type == MIX_LIGHTNING) {
      v.push_back({m + "g", {mixed, W}});
      v.push_back({m + "norm", {mixed}});
    }
    if (s.ff) {
      v.push_back({p + "norm2", {W}});
      v.push_back({p + "mlp.up", {s.ff, W}});
      v.push_back({p + "mlp.down", {W, s.ff}});
      v.push_back({p + "mlp.act", {2}});
    }
  }
  return v;
}

// --- the model ---------------------------------------------------------------------------------------------
struct LayerDev {
  const float *norm1 = nullptr, *norm2 = nullptr, *conv = nullptr;
  void *w_in = nullptr, *w_out = nullptr;
  int32_t rows_in = 0;           // of the first segment: q, k, v and the gate
  int32_t up_row = 0;            // where the second segment, W_up, starts
  int64_t ldp = 0;               // projections of a token
  int64_t mixed_k = 0, k_out = 0;  // inputs of W_o and of both, padded
  float act_pos = 0.0f, act_neg = 0.0f;
  const float *mix_norm = nullptr, *decay = nullptr, *log2_decay = nullptr, *slope = nullptr;
};

// one run of a layer: a looped layer has one per pass
struct LayerRun {
  int32_t layer = 0;
  bool add_embedding = false;  // the embedding output is added to x behind this run: another pass of the loop starts
  float* conv_state[2] = {nullptr, nullptr};
  float* state = nullptr;
  void *k_cache = nullptr, *v_cache = nullptr;
  RingLayout kl, vl;
};

// activations of a pass of up to `tokens` tokens
struct Buffers {
  int64_t tokens = 0;
  float *x = nullptr, *keep = nullptr, *o = nullptr;
  void *h = nullptr, *n = nullptr, *proj = nullptr;
  std::vector<void*> cat;  // [ctx, mid] per layer (layers of one shape share)
};

struct KugilixEngine final : ConfigModel {
  Spec spec;
  const double* freq = nullptr;
  std::vector<LayerDev> layers;
  std::vector<LayerRun> runs;
  Buffers step, pass;
  float* attn_parts = nullptr;

  const char* architecture() const override { return "Kugilix"; }
  int load_layers(Loader& ldr) override;
  int make_buffers() override;
  int64_t layer_runs() const override { return (int64_t)runs.size(); }
  float* stream_of(bool one) override { return one ? step.x : pass.x; }
  int run_pass(bool one, const int32_t* ids, int64_t M, PassPos pos) override;

  int make_activations(Buffers* b, int64_t n_tokens);
  int make_runs();
};

double softplus(double z) { return log1p(exp(-fabs(z))) + fmax(z, 0.0); }

int load_layer(Loader& ld, KugilixEngine* e, int i) {
  const LayerSpec& s = e->spec.layers[i];
  const int64_t W = e->spec.width;
  LayerDev L;
  const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.";
  if (int rc = ld.vector(p + "norm1", &L.norm1)) return rc;
  if (int rc = ld.vector(p + "canon1", &L.conv)) return rc;
  struct Part {
    const char* name;
    int64_t rows;
  };
  std::vector<Part> parts;
  if (s.type == MIX_ATTENTION)
    parts = {{"q", (int64_t)s.heads * s.dim}, {"k", (int64_t)s.kv_heads * s.dim}, {"v", (int64_t)s.kv_heads * s.vdim}};
  else
    parts = {{"q", (int64_t)s.heads * s.dim}, {"k", (int64_t)s.heads * s.dim}, {"v", s.mixed()}, {"g", s.mixed()}};
  int64_t rows = 0;
  for (const Part& q : parts) rows += q.rows;
  AWQ_REQUIRE(rows + s.ff < (1 << 28), "layer too large");
  L.rows_in = (int32_t)rows;
  L.ldp = round_up(rows, 8);
  L.up_row = (int32_t)round_up(rows, kDenseRowAlign);
  if (int rc = ld.block(&L.w_in, L.up_row + round_up(s.ff, kDenseRowAlign), e->ld)) return rc;
  int64_t at = 0;
  for (const Part& q : parts) {
    if (int rc = ld.matrix(m + q.name, L.w_in, e->ld, at, 0)) return rc;
    at += q.rows;
  }
  L.mixed_k = round_up(s.mixed(), kDenseKAlign);
  L.k_out = L.mixed_k + round_up(s.ff, kDenseKAlign);
  if (int rc = ld.block(&L.w_out, round_up(W, kDenseRowAlign), L.k_out)) return rc;
  if (int rc = ld.matrix(m + "o", L.w_out, L.k_out, 0, 0)) return rc;
  if (s.ff) {
    if (int rc = ld.vector(p + "norm2", &L.norm2)) return rc;
    if (int rc = ld.matrix(p + "mlp.up", L.w_in, e->ld, L.up_row, 0)) return rc;
    if (int rc = ld.matrix(p + "mlp.down", L.w_out, L.k_out, 0, L.mixed_k)) return rc;
    std::vector<double> act;
    ld.numbers(p + "mlp.act", &act);
    L.act_pos = (float)softplus(act[0]);
    L.act_neg = (float)(0.5 + softplus(act[1]));
  }
  if (s.type == MIX_LIGHTNING) {
    if (int rc = ld.vector(m + "norm", &L.mix_norm)) return rc;
    if (int rc = ld.constants(std::vector<float>(s.decay.begin(), s.decay.end()), &L.decay)) return rc;
    std::vector<float> lg;
    for (double d : s.decay)
      if (d > 0.0) lg.push_back((float)log2(d));
    if (lg.size() == s.decay.size())
      if (int rc = ld.constants(lg, &L.log2_decay)) return rc;
  } else {
    std::vector<float> slope;
    for (int h = 0; h < s.heads; ++h) slope.push_back((float)exp2(-8.0 * (h + 1) / s.heads));
    if (int rc = ld.constants(slope, &L.slope)) return rc;
  }
  e->layers.push_back(L);
  return AWQ_OK;
}

int KugilixEngine::load_layers(Loader& ldr) {
  std::vector<double> f;
  for (int64_t i = 0; 2 * i < width; ++i) f.push_back(pow(10000.0, -2.0 * (double)i / (double)width));
  if (int rc = ldr.constants(f, &freq)) return rc;
  for (size_t i = 0; i < spec.layers.size(); ++i)
    if (int rc = load_layer(ldr, this, (int)i)) return rc;
  return AWQ_OK;
}

// --- activations, caches and recurrent state ---------------------------------------------------------------
int KugilixEngine::make_activations(Buffers* b, int64_t n) {
  const int64_t W = spec.width;
  int64_t proj = 0, o = 0;
  b->cat.resize(layers.size());
  for (size_t i = 0; i < layers.size(); ++i) {
    proj = std::max(proj, layers[i].ldp);
    if (spec.layers[i].type == MIX_LIGHTNING) o = std::max<int64_t>(o, spec.layers[i].mixed());
    for (size_t j = 0; j < i && !b->cat[i]; ++j)
      if (spec.layers[j].mixed() == spec.layers[i].mixed() && spec.layers[j].ff == spec.layers[i].ff) b->cat[i] = b->cat[j];
    // the padding between and behind the two halves stays zero
    if (!b->cat[i])
      if (int rc = zeroed(&b->cat[i], n * layers[i].k_out * unit())) return rc;
  }
  if (int rc = zeroed((void**)&b->x, n * W * 4)) return rc;
  if (int rc = zeroed((void**)&b->keep, n * W * 4)) return rc;
  if (int rc = zeroed((void**)&b->o, n * o * 4)) return rc;
  if (int rc = zeroed(&b->h, n * ld * unit())) return rc;
  if (int rc = zeroed(&b->n, n * ld * unit())) return rc;
  if (int rc = zeroed(&b->proj, n * proj * unit())) return rc;
  b->tokens = n;
  return AWQ_OK;
}

int KugilixEngine::make_buffers() {
  if (int rc = make_activations(&step, 1)) return rc;
  if (int rc = make_activations(&pass, pass_tokens)) return rc;
  return make_runs();
}

int KugilixEngine::make_runs() {
  const int n = (int)spec.layers.size();
  for (int i = 0; i < n;) {
    if (i == spec.loop_start && spec.loop_stop > i) {
      for (int t = 0; t < spec.loop_times; ++t)
        for (int l = spec.loop_start; l < spec.loop_stop; ++l) {
          LayerRun r;
          r.layer = l;
          r.add_embedding = l == spec.loop_stop - 1 && t + 1 < spec.loop_times;
          runs.push_back(r);
        }
      i = spec.loop_stop;
    } else {
      LayerRun r;
      r.layer = i++;
      runs.push_back(r);
    }
  }
  int64_t parts = 4;
  for (LayerRun& r : runs) {
    const LayerSpec& s = spec.layers[r.layer];
    if (spec.taps > 1)
      for (float*& p : r.conv_state)
        if (int rc = zeroed((void**)&p, (int64_t)(spec.taps - 1) * spec.width * 4)) return rc;
    if (s.type == MIX_LIGHTNING) {
      if (int rc = zeroed((void**)&r.state, linear_state_floats(s.heads, s.dim, s.vdim) * 4)) return rc;
      continue;
    }
    // a pass appends its rows before it attends: the ring holds a window behind the pass's first position
    const int64_t need = s.window ? std::min<int64_t>(max_pos, (int64_t)s.window - 1 + pass_tokens) : max_pos;
    r.kl = RingLayout{(int32_t)round_up(need, 64), s.kv_heads, window_row_padded(s.dim)};
    r.vl = RingLayout{r.kl.slots, s.kv_heads, window_row_padded(s.vdim)};
    if (int rc = zeroed(&r.k_cache, r.kl.elements() * unit())) return rc;
    if (int rc = zeroed(&r.v_cache, r.vl.elements() * unit())) return rc;
    parts = std::max(parts, window_parts_floats(s.heads, s.vdim, s.window, max_pos));
  }
  return zeroed((void**)&attn_parts, parts * 4);
}

// --- passes ------------------------------------------------------------------------------------------------
int KugilixEngine::run_pass(bool one, const int32_t* ids, int64_t M, PassPos pos) {
  const int64_t W = spec.width;
  Buffers& b = one ? step : pass;
  if (int rc = launch_embed_sinusoid(embed, f32, ids, d_token, pos, M, W, spec.embed_scale, freq, b.x, b.keep, stream)) return rc;
  for (size_t ri = 0; ri < runs.size(); ++ri) {
    const LayerRun& r = runs[ri];
    const LayerSpec& s = spec.layers[r.layer];
    const LayerDev& L = layers[r.layer];
    void* const cat = b.cat[r.layer];
    char* const mid = (char*)cat + L.mixed_k * unit();
    {
      NormConvArgs a;
      a.x = b.x;
      a.M = M;
      a.width = W;
      a.groups = spec.groups;
      a.eps = spec.eps;
      a.w1 = L.norm1;
      a.conv = L.conv;
      a.taps = spec.taps;
      a.state[0] = r.conv_state[0];
      a.state[1] = r.conv_state[1];
      a.out1 = b.h;
      a.w2 = L.norm2;
      a.out2 = b.n;
      a.ld = ld;
      a.pos = pos;
      if (int rc = launch_norm_conv(a, f32, stream)) return rc;
    }
    {
      DenseArgs a;
      a.w = L.w_in;
      a.k = ld;
      a.M = M;
      a.workspace = dense_ws;
      a.workspace_floats = dense_ws_floats;
      DenseSegment& in = a.seg[0];
      in.x = b.h;
      in.ldx = ld;
      in.y = b.proj;
      in.ldy = L.ldp;
      in.rows = L.rows_in;
      if (s.type == MIX_LIGHTNING) {
        in.act = DENSE_SILU;
        in.act_rows = s.heads * (2 * s.dim + s.vdim);
      }
      if (s.ff) {
        a.n_seg = 2;
        DenseSegment& up = a.seg[1];
        up.x = b.n;
        up.ldx = ld;
        up.y = mid;
        up.ldy = L.k_out;
        up.row0 = L.up_row;
        up.rows = s.ff;
        up.act = DENSE_XIELU;
        up.act_pos = L.act_pos;
        up.act_neg = L.act_neg;
      }
      if (int rc = launch_dense(a, f32, stream)) return rc;
    }
    const char* gate = nullptr;
    bool gate_fused = false;
    if (s.type == MIX_ATTENTION) {
      WindowAttnArgs a;
      a.proj = b.proj;
      a.ldp = L.ldp;
      a.heads = s.heads;
      a.kv_heads = s.kv_heads;
      a.dim = s.dim;
      a.vdim = s.vdim;
      a.window = s.window;
      a.scale = s.scale;
      a.eps = spec.eps;
      a.temp_coef = s.temp_coef;
      a.temp_every = s.temp_every;
      a.slope = L.slope;
      a.k_cache = r.k_cache;
      a.v_cache = r.v_cache;
      a.kl = r.kl;
      a.vl = r.vl;
      a.ctx = cat;
      a.ldc = L.k_out;
      a.M = M;
      a.pos = pos;
      a.parts = attn_parts;
      a.len_bound = (int32_t)max_pos;
      if (int rc = launch_window_attention(a, f32, stream)) return rc;
    } else {
      LinearAttnArgs a;
      a.proj = b.proj;
      a.ldp = L.ldp;
      a.heads = s.heads;
      a.dim = s.dim;
      a.vdim = s.vdim;
      a.decay = L.decay;
      a.log2_decay = L.log2_decay;
      a.state = r.state;
      a.o = b.o;
      a.M = M;
      a.pos = pos;
      if (int rc = launch_linear_attention(a, f32, stream)) return rc;
      gate = (const char*)b.proj + (int64_t)s.heads * (2 * s.dim + s.vdim) * unit();
      // a single token's gated norm is part of the product below
      gate_fused = dense_gate_fused(s.mixed(), L.mixed_k, M, f32) && ((uintptr_t)gate & 7) == 0;
      if (!gate_fused)
        if (int rc = launch_gated_norm(b.o, s.mixed(), gate, L.ldp, L.mix_norm, cat, L.k_out, s.mixed(), M, spec.eps, f32, stream))
          return rc;
    }
    {
      DenseArgs a;
      a.w = L.w_out;
      a.k = L.k_out;
      a.M = M;
      a.out = DENSE_RESIDUAL;
      a.workspace = dense_ws;
      a.workspace_floats = dense_ws_floats;
      a.seg[0].x = cat;
      a.seg[0].ldx = L.k_out;
      a.seg[0].y = b.x;
      a.seg[0].ldy = W;
      a.seg[0].rows = (int32_t)W;
      if (gate_fused) {
        a.gate_o = b.o;
        a.gate_g = gate;
        a.gate_w = L.mix_norm;
        a.gate_n = s.mixed();
        a.gate_k = (int32_t)L.mixed_k;
        a.gate_eps = spec.eps;
      }
      // the tap sees the stream as the layer leaves it
      if (r.add_embedding && !tap_on) a.addend = b.keep;
      if (int rc = launch_dense(a, f32, stream)) return rc;
    }
    if (tap_on) {
      if (int rc = tap_layer((int64_t)ri, b.x, M)) return rc;
      if (r.add_embedding)
        if (int rc = launch_add_rows(b.x, b.keep, M * W, stream)) return rc;
    }
  }
  return AWQ_OK;
}

int open_kugilix(const char* dir, const awq_open_options& opt, awq_engine** out) {
  std::unique_ptr<KugilixEngine> e(new KugilixEngine());
  // look at the folder before touching the GPU
  Safetensors file;
  if (int rc = read_spec(dir, &e->spec)) return rc;
  if (int rc = file.open(std::string(dir) + "/model.safetensors")) return rc;
  if (int rc = check_tensors(expected_tensors(e->spec), file)) return rc;
  e->vocab = e->spec.vocab;
  e->width = e->spec.width;
  e->norm_groups = e->spec.groups;
  e->eps = e->spec.eps;
  return ConfigModel::open(std::move(e), file, opt, out);
}

ModelClass g_class("Kugilix", open_kugilix);

}  // namespace
