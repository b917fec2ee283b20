// Tudasun: a decoder-only model whose layers mix tokens by linear attention with a decay per channel (two kinds) or by
// attention over a shared latent, with norms on both sides of every sublayer, gated sublayer results, a dense or routed
// feed-forward and an input per token and layer behind it.  config.json gives every size and constant; the order of the
// layers is data.  Runs in bfloat16 (residual, norms, scores, routers, decays and recurrent state in binary32) or wholly in
// binary32, behind the step driver of engine.cpp.
//
// A layer, with h = norm1(x) left by the launch that ended the layer ahead:
//   one product             what the mixer takes from h, and the gate of its result
//   the mixer               -> ctx
//   one product             y = W_o ctx
//   join                    x += norm(y * gate), h = norm2(x)
//   one product             the feed-forward's first half (or router and shared expert) of h, and its gate
//   feed-forward            -> y (experts: pairs of token and expert)
//   join                    x += norm(y * gate), x in the activations' type
//   two products, join      the token input: x += norm(W_p (gelu(W_g x) * e)), h = norm1(x) of the next layer
#include "config_model.hpp"

#include <math.h>

namespace {

enum MixerType { MIX_GLA, MIX_HGRN2, MIX_LATENT };
enum MlpType { MLP_NONE, MLP_DENSE, MLP_EXPERTS };

struct LayerSpec {
  MixerType type = MIX_GLA;
  int32_t heads = 0, dim = 0, vdim = 0;
  double tau = 1.0;                  // gated linear attention: the root of the decay
  int32_t decay_rank = 0;            // ... rows of its first decay matrix
  int32_t rank = 0, rot = 0;         // latent attention
  double base = 1.0;
  float scale = 1.0f;
  int32_t kv_from = -1;              // the layer whose latents are used; -1: this layer's own
  MlpType mlp = MLP_NONE;
  int32_t ff = 0;                    // of the dense feed-forward or of an expert
  int32_t experts = 0, identity = 0, top = 0, groups = 0, keep = 0;
  int32_t shared_ff = 0;             // 0: no shared expert
  int32_t mixed() const { return heads * vdim; }
  int32_t outputs() const { return experts + identity; }
};

struct Spec {
  int32_t vocab = 0, width = 0, side = 0;  // side 0: no input per layer
  float eps = 0.0f, softcap = 0.0f;
  std::vector<LayerSpec> layers;
};

// --- config.json -------------------------------------------------------------------------------------------
int read_mlp(const Json& f, const std::string& at, LayerSpec* s) {
  const Json* kind = f.find("kind");
  if (kind && kind->str == "dense") {
    s->mlp = MLP_DENSE;
    return get_int(f, at, "ff", 1, 1 << 28, &s->ff);
  }
  if (!kind || kind->str != "moe") return bad_config(at + "kind is unknown");
  s->mlp = MLP_EXPERTS;
  const Json *expert = section(f, "expert"), *router = section(f, "router");
  if (!expert || !router) return bad_config(at + "expert or router is missing");
  if (int rc = get_int(*expert, at + "expert.", "ff", 1, 1 << 24, &s->ff)) return rc;
  const std::string r = at + "router.";
  if (int rc = get_int(*router, r, "experts", 0, 4096, &s->experts)) return rc;
  const Json* identity = router->find("identity");
  if (identity && !identity->is(Json::Null))
    if (int rc = get_int(*router, r, "identity", 0, 4096, &s->identity)) return rc;
  if (s->outputs() < 1 || s->outputs() > 4096) return bad_config(r + "experts and identity are out of range");
  if (int rc = get_int(*router, r, "top", 1, s->outputs(), &s->top)) return rc;
  if (const Json* g = section(*router, "groups")) {
    if (int rc = get_int(*g, r + "groups.", "count", 1, s->outputs(), &s->groups)) return rc;
    if (s->outputs() % s->groups) return bad_config(r + "groups.count does not divide the outputs");
    if (int rc = get_int(*g, r + "groups.", "keep", 1, s->groups, &s->keep)) return rc;
    if (s->keep * (s->outputs() / s->groups) < s->top) return bad_config(r + "groups.keep leaves fewer outputs than top");
  }
  if (const Json* shared = section(f, "shared"))
    if (int rc = get_int(*shared, at + "shared.", "ff", 1, 1 << 24, &s->shared_ff)) return rc;
  return AWQ_OK;
}

int read_layer(const Json& j, const std::string& at, const std::vector<LayerSpec>& before, LayerSpec* s) {
  const Json *type = j.find("type"), *m = section(j, "mixer");
  if (!type || !type->is(Json::String) || !m) return bad_config(at + "type or mixer is missing");
  const std::string mx = at + "mixer.";
  const bool latent = type->str == "latent_attention";
  if (!latent && type->str != "gla" && type->str != "hgrn2") return bad_config(at + "type \"" + type->str + "\" is unknown");
  if (int rc = get_int(*m, mx, "heads", 1, 65535, &s->heads)) return rc;
  if (int rc = get_int(*m, mx, "dim", 1, latent ? 1 << 16 : 512, &s->dim)) return rc;
  if (int rc = get_int(*m, mx, "vdim", 1, 8192, &s->vdim)) return rc;
  if ((int64_t)s->heads * std::max(s->dim, s->vdim) > (1 << 24)) return bad_config(mx + "heads is out of range");
  if (latent) {
    s->type = MIX_LATENT;
    if (int rc = get_int(*m, mx, "kv_rank", 1, 1024, &s->rank)) return rc;
    if (int rc = get_int(*m, mx, "rot_dim", 2, 1024, &s->rot)) return rc;
    if (int rc = get_float(*m, mx, "scale", &s->scale)) return rc;
    const Json* rot = section(*m, "rot");
    if (!rot) return bad_config(mx + "rot is missing");
    int32_t dims;
    if (int rc = get_int(*rot, mx + "rot.", "dims", 2, 1024, &dims)) return rc;
    if (dims != s->rot || dims % 2) return bad_config(mx + "rot.dims must be rot_dim, and even");
    if (int rc = get_number(*rot, mx + "rot.", "base", &s->base)) return rc;
    if (!(s->base > 0.0)) return bad_config(mx + "rot.base must be positive");
    const Json* from = m->find("kv_from");
    if (from && !from->is(Json::Null)) {
      if (int rc = get_int(*m, mx, "kv_from", 0, (double)before.size() - 1, &s->kv_from)) return rc;
      const LayerSpec& o = before[s->kv_from];
      if (o.type != MIX_LATENT || o.kv_from >= 0 || o.rank != s->rank || o.rot != s->rot || o.base != s->base)
        return bad_config(mx + "kv_from names a layer without latents of this shape and rotation");
    }
  } else if (type->str == "gla") {
    s->type = MIX_GLA;
    if (int rc = get_number(*m, mx, "tau", &s->tau)) return rc;
    if (!(s->tau > 0.0)) return bad_config(mx + "tau must be positive");
  } else {
    s->type = MIX_HGRN2;
  }
  const Json* f = j.find("mlp");
  if (f && f->is(Json::Object)) return read_mlp(*f, at + "mlp.", s);
  if (f && !f->is(Json::Null)) return bad_config(at + "mlp is no object");
  return AWQ_OK;
}

int read_spec(const std::string& dir, Spec* s) {
  Json j;
  if (int rc = awq_read_json(dir + "/config.json", &j)) return rc;
  if (int rc = get_int(j, "", "vocab", 1, 1 << 28, &s->vocab)) return rc;
  if (int rc = get_int(j, "", "width", 1, 16000, &s->width)) return rc;
  const Json *norm = section(j, "norm"), *layers = j.find("layers"), *cap = j.find("logit_softcap");
  if (!norm) return bad_config("norm is missing");
  if (int rc = get_float(*norm, "norm.", "eps", &s->eps)) return rc;
  if (cap && !cap->is(Json::Null)) {
    if (int rc = get_float(j, "", "logit_softcap", &s->softcap)) return rc;
    if (!(s->softcap > 0.0f)) return bad_config("logit_softcap must be positive");
  }
  if (const Json* side = section(j, "token_side"))
    if (int rc = get_int(*side, "token_side.", "dim", 1, 1 << 16, &s->side)) return rc;
  if (!layers || !layers->is(Json::Array) || layers->items.empty() || layers->items.size() > 4096)
    return bad_config("layers is missing or empty");
  for (size_t i = 0; i < layers->items.size(); ++i) {
    LayerSpec l;
    if (int rc = read_layer(layers->items[i], "layers[" + std::to_string(i) + "].", s->layers, &l)) return rc;
    s->layers.push_back(l);
  }
  return AWQ_OK;
}

// a size that only a tensor's shape gives
int read_shapes(const Safetensors& file, Spec* c) {
  for (size_t i = 0; i < c->layers.size(); ++i) {
    if (c->layers[i].type != MIX_GLA) continue;
    const std::string name = "l" + std::to_string(i) + ".mix.a1";
    const Tensor* t = file.find(name);
    if (!t || t->shape.size() != 2 || t->shape[0] < 1 || t->shape[0] > (1 << 16)) {
      awq_set_error("model.safetensors has no matrix " + name);
      return AWQ_ERR_IO;
    }
    c->layers[i].decay_rank = (int32_t)t->shape[0];
  }
  return AWQ_OK;
}

// every tensor of the model and its shape
TensorTable expected_tensors(const Spec& c) {
  const int64_t W = c.width;
  TensorTable v = {{"embed", {c.vocab, W}}, {"final.norm", {W}}, {"head", {c.vocab, W}}};
  if (c.side) v.push_back({"side.embed", {c.vocab, (int64_t)c.layers.size() * c.side}});
  for (size_t i = 0; i < c.layers.size(); ++i) {
    const LayerSpec& s = c.layers[i];
    const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.", f = p + "mlp.";
    const int64_t keys = (int64_t)s.heads * s.dim, mixed = s.mixed();
    v.push_back({p + "norm1", {W}});
    v.push_back({p + "norm1b", {W}});
    v.push_back({p + "rg1", {W, W}});
    v.push_back({p + "rg1.b", {W}});
    v.push_back({m + "o", {W, mixed}});
    if (s.type == MIX_LATENT) {
      v.push_back({m + "q", {(int64_t)s.heads * (s.dim + s.rot), W}});
      v.push_back({m + "uk", {keys, s.rank}});
      v.push_back({m + "uv", {mixed, s.rank}});
      v.push_back({m + "sink", {s.heads}});
      if (s.kv_from < 0) {
        v.push_back({m + "dkv", {s.rank + s.rot, W}});
        v.push_back({m + "dkv.norm", {s.rank}});
      }
    } else {
      v.push_back({m + "q", {keys, W}});
      v.push_back({m + "v", {mixed, W}});
      v.push_back({m + "norm", {s.vdim}});
      if (s.type == MIX_GLA) {
        v.push_back({m + "k", {keys, W}});
        v.push_back({m + "g", {mixed, W}});
        v.push_back({m + "a1", {s.decay_rank, W}});
        v.push_back({m + "a2", {keys, s.decay_rank}});
        v.push_back({m + "a2.b", {keys}});
      } else {
        v.push_back({m + "f", {keys, W}});
        v.push_back({m + "f.b", {keys}});
        v.push_back({m + "lower", {keys}});
      }
    }
    if (s.mlp != MLP_NONE) {
      v.push_back({p + "norm2", {W}});
      v.push_back({p + "norm2b", {W}});
      v.push_back({p + "rg2", {W, W}});
      v.push_back({p + "rg2.b", {W}});
    }
    if (s.mlp == MLP_DENSE) {
      v.push_back({f + "up", {s.ff, W}});
      v.push_back({f + "down", {W, s.ff}});
      v.push_back({f + "act", {4}});
    }
    const auto expert = [&](const std::string& e, int64_t ff) {
      v.push_back({e + "gate", {ff, W}});
      v.push_back({e + "up", {ff, W}});
      v.push_back({e + "down", {W, ff}});
    };
    if (s.mlp == MLP_EXPERTS) {
      v.push_back({f + "router", {s.outputs(), W}});
      v.push_back({f + "correction", {s.outputs()}});
      for (int e = 0; e < s.experts; ++e) expert(f + "e" + std::to_string(e) + ".", s.ff);
      if (s.shared_ff) {
        expert(f + "shared.", s.shared_ff);
        v.push_back({f + "shared.sg", {1, W}});
      }
    }
    if (c.side) {
      v.push_back({p + "side.gate", {c.side, W}});
      v.push_back({p + "side.proj", {W, c.side}});
      v.push_back({p + "side.norm", {W}});
    }
  }
  return v;
}

// --- the model ---------------------------------------------------------------------------------------------
// a block of matrices that are applied to the same vectors, each at a multiple of kDenseSharedAlign rows
struct InBlock {
  void* w = nullptr;
  std::vector<int32_t> at;  // first rows, in the order they were asked for
};

struct LayerDev {
  const float *norm1 = nullptr, *norm1b = nullptr, *norm2 = nullptr, *norm2b = nullptr, *rg1_b = nullptr, *rg2_b = nullptr;
  InBlock in, mid;                   // products of norm1(x) and norm2(x)
  void* w_o = nullptr;
  int64_t ldp = 0, mixed_k = 0;      // projections of a token, inputs of W_o padded
  // linear attention
  void* w_a2 = nullptr;
  int64_t decay_k = 0;
  const float *decay_b = nullptr, *lower = nullptr, *mix_norm = nullptr;
  // latent attention
  const float *latent_norm = nullptr, *sink = nullptr;
  const double* freq = nullptr;
  void *w_uk = nullptr, *w_uv = nullptr, *w_kv = nullptr;
  void* cache = nullptr;             // the owner's
  // feed-forward
  void *w_down = nullptr, *w_shared_down = nullptr, *w_gate_up = nullptr, *w_expert_down = nullptr;
  const float *act = nullptr, *correction = nullptr;
  int64_t ff_k = 0, shared_k = 0, gate_up_block = 0, expert_down_block = 0;
  // token input
  void *w_side_gate = nullptr, *w_side_proj = nullptr;
  const float* side_norm = nullptr;
};

// activations of a pass of up to `tokens` tokens
struct Buffers {
  float *x = nullptr, *y = nullptr, *o = nullptr, *decay = nullptr, *down = nullptr, *router = nullptr, *shared_gate = nullptr,
        *pairs = nullptr, *weights = nullptr;
  void *h = nullptr, *xt = nullptr, *proj = nullptr, *gate = nullptr, *low = nullptr, *ctx = nullptr, *mid = nullptr,
       *shared_mid = nullptr, *side = nullptr, *side_mid = nullptr;
  int32_t *ids = nullptr, *list = nullptr;
  DenseTile* tiles = nullptr;
};

struct TudasunEngine final : ConfigModel {
  Spec spec;
  void* side_embed = nullptr;
  int64_t side_k = 0, ldg = 0;
  std::vector<LayerDev> layers;
  Buffers step, pass;
  LatentScratch scratch_bytes;
  void *s_qa = nullptr, *s_ql = nullptr, *s_ol = nullptr, *s_kv = nullptr, *s_parts = nullptr;
  std::vector<float*> states;

  const char* architecture() const override { return "Tudasun"; }
  int load_layers(Loader& ldr) override;
  int make_buffers() override;
  int64_t layer_runs() const override { return (int64_t)layers.size(); }
  float* stream_of(bool one) override { return one ? step.x : pass.x; }
  int run_pass(bool one, const int32_t* ids, int64_t M, PassPos pos) override;

  int load_layer(Loader& ldr, int i);
  int make_activations(Buffers* b, int64_t n_tokens);
  LatentAttnArgs latent_args(int i) const;
  int64_t side_width() const { return (int64_t)layers.size() * spec.side; }

  // the parts of a layer
  DenseArgs product(const void* w, int64_t k, int64_t M) const;
  int mix(int i, Buffers& b, int64_t M, PassPos pos);
  int dense_feed_forward(int i, Buffers& b, int64_t M);
  int routed_feed_forward(int i, Buffers& b, int64_t M, JoinArgs* end);
  int token_input(int i, Buffers& b, int64_t M, JoinArgs* end);
};

// --- weights -----------------------------------------------------------------------------------------------
// what goes into an InBlock
struct Part {
  std::string name;
  int64_t rows;       // of the block
  int form = PACK_PLAIN;
  bool joins = false;  // continues the part ahead: no alignment, the same segment
};

int load_in(Loader& ldr, ConfigModel* e, const std::vector<Part>& parts, InBlock* b) {
  int64_t rows = 0;
  std::vector<int64_t> first;
  for (const Part& p : parts) {
    if (!p.joins) {
      rows = round_up(rows, kDenseSharedAlign);
      b->at.push_back((int32_t)rows);
    }
    if (p.form == PACK_UP) {  // interleaved with the gate rows ahead of it
      first.push_back(first.back());
      continue;
    }
    first.push_back(rows);
    rows += p.rows;
  }
  AWQ_REQUIRE(rows < (1 << 28), "layer too large");
  if (int rc = ldr.block(&b->w, round_up(rows, kDenseRowAlign), e->ld)) return rc;
  for (size_t i = 0; i < parts.size(); ++i)
    if (int rc = ldr.matrix(parts[i].name, b->w, e->ld, first[i], 0, parts[i].form)) return rc;
  return AWQ_OK;
}

int load_out(Loader& ldr, const std::string& name, int64_t width, int64_t k, void** w) {
  if (int rc = ldr.block(w, round_up(width, kDenseRowAlign), k)) return rc;
  return ldr.matrix(name, *w, k, 0, 0);
}

LatentAttnArgs TudasunEngine::latent_args(int i) const {
  const LayerSpec& s = spec.layers[i];
  LatentAttnArgs a;
  a.heads = s.heads;
  a.dim = s.dim;
  a.vdim = s.vdim;
  a.l.rank = s.rank;
  a.l.rot = s.rot;
  a.scale = s.scale;
  a.eps = eps;
  a.max_pos = max_pos;
  return a;
}

int TudasunEngine::load_layer(Loader& ldr, int i) {
  const LayerSpec& s = spec.layers[i];
  const int64_t W = width, keys = (int64_t)s.heads * s.dim, mixed = s.mixed();
  const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.", f = p + "mlp.";
  layers.emplace_back();
  LayerDev& L = layers.back();
  if (int rc = ldr.vector(p + "norm1", &L.norm1, norm_shift)) return rc;
  if (int rc = ldr.vector(p + "norm1b", &L.norm1b, norm_shift)) return rc;
  if (int rc = ldr.vector(p + "rg1.b", &L.rg1_b)) return rc;
  std::vector<Part> in;
  if (s.type == MIX_GLA) {
    in = {{m + "q", keys}, {m + "k", keys, PACK_PLAIN, true}, {m + "v", mixed, PACK_PLAIN, true}, {m + "g", mixed, PACK_PLAIN, true},
          {m + "a1", s.decay_rank}};
    L.ldp = round_up(2 * keys + 2 * mixed, 8);
  } else if (s.type == MIX_HGRN2) {
    in = {{m + "q", keys}, {m + "v", mixed, PACK_PLAIN, true}, {m + "f", keys}};
    L.ldp = round_up(keys + mixed, 8);
  } else {
    in = {{m + "q", (int64_t)s.heads * (s.dim + s.rot)}};
    if (s.kv_from < 0) in.push_back({m + "dkv", s.rank + s.rot});
    L.ldp = round_up((int64_t)s.heads * (s.dim + s.rot), 8);
  }
  in.push_back({p + "rg1", W});
  if (int rc = load_in(ldr, this, in, &L.in)) return rc;
  L.mixed_k = round_up(mixed, kDenseKAlign);
  if (int rc = load_out(ldr, m + "o", W, L.mixed_k, &L.w_o)) return rc;

  if (s.type == MIX_LATENT) {
    LatentAttnArgs a = latent_args(i);
    const int64_t qk = round_up(s.dim, kDenseKAlign), vk = round_up(s.rank, kDenseKAlign);
    if (int rc = ldr.block(&L.w_uk, s.heads * latent_uk_block(a) / qk, qk)) return rc;
    if (int rc = ldr.block(&L.w_uv, s.heads * latent_uv_block(a) / vk, vk)) return rc;
    if (latent_forms_keys(a, pass_tokens, f32))
      if (int rc = ldr.block(&L.w_kv, latent_kv_rows(a), vk)) return rc;
    for (const char* name : {"uk", "uv"}) {
      const Tensor* t = ldr.file.find(m + name);
      if (int rc = ldr.stage(t)) return rc;
      const bool k = name[1] == 'k';
      if (int rc = launch_latent_pack(a, k ? ldr.staging : nullptr, k ? nullptr : ldr.staging, Loader::wide(t), L.w_uk, L.w_uv, L.w_kv,
                                      f32, stream))
        return rc;
    }
    if (int rc = ldr.vector(m + "sink", &L.sink)) return rc;
    std::vector<double> freq;
    for (int d = 0; 2 * d < s.rot; ++d) freq.push_back(pow(s.base, -2.0 * d / s.rot));
    if (int rc = ldr.constants(freq, &L.freq)) return rc;
    if (s.kv_from < 0) {
      if (int rc = ldr.vector(m + "dkv.norm", &L.latent_norm)) return rc;
      if (int rc = zeroed(&L.cache, round_up(max_pos, 64) * a.l.row() * unit())) return rc;
    } else {
      L.cache = layers[s.kv_from].cache;
    }
  } else {
    if (int rc = ldr.vector(m + "norm", &L.mix_norm)) return rc;
    if (s.type == MIX_GLA) {
      L.decay_k = round_up(s.decay_rank, kDenseKAlign);
      if (int rc = load_out(ldr, m + "a2", keys, L.decay_k, &L.w_a2)) return rc;
      if (int rc = ldr.vector(m + "a2.b", &L.decay_b)) return rc;
    } else {
      if (int rc = ldr.vector(m + "f.b", &L.decay_b)) return rc;
      if (int rc = ldr.vector(m + "lower", &L.lower)) return rc;
    }
  }

  if (s.mlp != MLP_NONE) {
    if (int rc = ldr.vector(p + "norm2", &L.norm2, norm_shift)) return rc;
    if (int rc = ldr.vector(p + "norm2b", &L.norm2b, norm_shift)) return rc;
    if (int rc = ldr.vector(p + "rg2.b", &L.rg2_b)) return rc;
    std::vector<Part> mid = {{p + "rg2", W}};
    L.ff_k = round_up(s.ff, kDenseKAlign);
    if (s.mlp == MLP_DENSE) {
      mid.push_back({f + "up", s.ff});
      if (int rc = load_out(ldr, f + "down", W, L.ff_k, &L.w_down)) return rc;
      if (int rc = ldr.vector(f + "act", &L.act)) return rc;
    } else {
      mid.push_back({f + "router", s.outputs()});
      if (s.shared_ff) {
        mid.push_back({f + "shared.gate", dense_glu_rows(s.shared_ff), PACK_GATE});
        mid.push_back({f + "shared.up", 0, PACK_UP, true});
        mid.push_back({f + "shared.sg", 1});
        L.shared_k = round_up(s.shared_ff, kDenseKAlign);
        if (int rc = load_out(ldr, f + "shared.down", W, L.shared_k, &L.w_shared_down)) return rc;
      }
      if (int rc = ldr.vector(f + "correction", &L.correction)) return rc;
      const int64_t gu_rows = round_up(dense_glu_rows(s.ff), kDenseRowAlign), down_rows = round_up(W, kDenseRowAlign);
      L.gate_up_block = gu_rows * ld;
      L.expert_down_block = down_rows * L.ff_k;
      if (int rc = ldr.block(&L.w_gate_up, s.experts * gu_rows, ld)) return rc;
      if (int rc = ldr.block(&L.w_expert_down, s.experts * down_rows, L.ff_k)) return rc;
      for (int e = 0; e < s.experts; ++e) {
        const std::string x = f + "e" + std::to_string(e) + ".";
        if (int rc = ldr.matrix(x + "gate", L.w_gate_up, ld, e * gu_rows, 0, PACK_GATE)) return rc;
        if (int rc = ldr.matrix(x + "up", L.w_gate_up, ld, e * gu_rows, 0, PACK_UP)) return rc;
        if (int rc = ldr.matrix(x + "down", L.w_expert_down, L.ff_k, e * down_rows, 0)) return rc;
      }
    }
    if (int rc = load_in(ldr, this, mid, &L.mid)) return rc;
  }
  if (spec.side) {
    if (int rc = load_out(ldr, p + "side.gate", spec.side, ld, &L.w_side_gate)) return rc;
    if (int rc = load_out(ldr, p + "side.proj", W, side_k, &L.w_side_proj)) return rc;
    if (int rc = ldr.vector(p + "side.norm", &L.side_norm)) return rc;
  }
  return AWQ_OK;
}

int TudasunEngine::load_layers(Loader& ldr) {
  side_k = round_up(spec.side, kDenseKAlign);
  ldg = round_up(width, 8);
  if (spec.side)
    if (int rc = ldr.table("side.embed", &side_embed)) return rc;
  layers.reserve(spec.layers.size());
  for (size_t i = 0; i < spec.layers.size(); ++i)
    if (int rc = load_layer(ldr, (int)i)) return rc;
  return AWQ_OK;
}

// --- activations, caches and recurrent state ---------------------------------------------------------------
int TudasunEngine::make_activations(Buffers* b, int64_t n) {
  int64_t proj = 8, o = 1, decay = 1, down = 1, low = 8, ctx = 8, mid = 8, shared_mid = 8, router = 1, pairs = 1, top = 1, tiles = 1;
  for (size_t i = 0; i < layers.size(); ++i) {
    const LayerSpec& s = spec.layers[i];
    const LayerDev& L = layers[i];
    proj = std::max(proj, L.ldp);
    ctx = std::max(ctx, L.mixed_k);
    if (s.type == MIX_LATENT) {
      down = std::max<int64_t>(down, s.rank + s.rot);
    } else {
      o = std::max<int64_t>(o, s.mixed());
      decay = std::max<int64_t>(decay, (int64_t)s.heads * s.dim);
      low = std::max(low, L.decay_k);
    }
    if (s.mlp == MLP_DENSE) mid = std::max(mid, L.ff_k);
    if (s.mlp == MLP_EXPERTS) {
      mid = std::max(mid, s.top * L.ff_k);
      shared_mid = std::max(shared_mid, L.shared_k);
      router = std::max<int64_t>(router, s.outputs());
      pairs = std::max<int64_t>(pairs, (int64_t)s.top * width);
      top = std::max<int64_t>(top, s.top);
      tiles = std::max<int64_t>(tiles, route_max_tiles(n, s.top, s.experts, 64));
    }
  }
  // every buffer starts as zeros: what pads a product's inputs meets zero weights, and has to be finite
  struct Need {
    void** p;
    int64_t bytes;
  };
  const int64_t u = unit();
  const Need all[] = {{(void**)&b->x, n * width * 4}, {(void**)&b->y, n * width * 4}, {(void**)&b->o, n * o * 4},
                      {(void**)&b->decay, n * decay * 4}, {(void**)&b->down, n * down * 4}, {(void**)&b->router, n * router * 4},
                      {(void**)&b->shared_gate, n * 4}, {(void**)&b->pairs, n * pairs * 4}, {(void**)&b->weights, n * top * 4},
                      {(void**)&b->ids, n * top * 4}, {(void**)&b->list, n * top * 4},
                      {(void**)&b->tiles, tiles * (int64_t)sizeof(DenseTile)}, {&b->h, n * ld * u}, {&b->xt, n * ld * u},
                      {&b->proj, n * proj * u}, {&b->gate, n * ldg * u}, {&b->low, n * low * u}, {&b->ctx, n * ctx * u},
                      {&b->mid, n * mid * u}, {&b->shared_mid, n * shared_mid * u}, {&b->side, n * std::max<int64_t>(1, side_width()) * u},
                      {&b->side_mid, n * std::max<int64_t>(8, side_k) * u}};
  for (const Need& need : all)
    if (int rc = zeroed(need.p, need.bytes)) return rc;
  return AWQ_OK;
}

int TudasunEngine::make_buffers() {
  if (int rc = make_activations(&step, 1)) return rc;
  if (int rc = make_activations(&pass, pass_tokens)) return rc;
  states.assign(layers.size(), nullptr);
  for (size_t i = 0; i < layers.size(); ++i) {
    const LayerSpec& s = spec.layers[i];
    if (s.type == MIX_LATENT) {
      const LatentScratch need = latent_scratch(latent_args((int)i), pass_tokens, f32);
      scratch_bytes.qa = std::max(scratch_bytes.qa, need.qa);
      scratch_bytes.ql = std::max(scratch_bytes.ql, need.ql);
      scratch_bytes.ol = std::max(scratch_bytes.ol, need.ol);
      scratch_bytes.kv = std::max(scratch_bytes.kv, need.kv);
      scratch_bytes.parts = std::max(scratch_bytes.parts, need.parts);
    } else if (int rc = zeroed((void**)&states[i], linear_state_floats(s.heads, s.dim, s.vdim) * 4)) {
      return rc;
    }
  }
  if (int rc = zeroed(&s_qa, scratch_bytes.qa)) return rc;
  if (int rc = zeroed(&s_ql, scratch_bytes.ql)) return rc;
  if (int rc = zeroed(&s_ol, scratch_bytes.ol)) return rc;
  if (int rc = zeroed(&s_kv, scratch_bytes.kv)) return rc;
  return zeroed(&s_parts, scratch_bytes.parts);
}

// --- passes ------------------------------------------------------------------------------------------------
DenseArgs TudasunEngine::product(const void* w, int64_t k, int64_t M) const {
  DenseArgs a;
  a.w = w;
  a.k = k;
  a.M = M;
  a.n_seg = 0;
  a.workspace = dense_ws;
  a.workspace_floats = dense_ws_floats;
  return a;
}

DenseSegment& segment(DenseArgs* a, const void* x, int64_t ldx, void* y, int64_t ldy, int32_t row0, int64_t rows) {
  DenseSegment& s = a->seg[a->n_seg++];
  s.x = x;
  s.ldx = ldx;
  s.y = y;
  s.ldy = ldy;
  s.row0 = row0;
  s.rows = (int32_t)rows;
  return s;
}

int TudasunEngine::mix(int i, Buffers& b, int64_t M, PassPos pos) {
  const LayerSpec& s = spec.layers[i];
  const LayerDev& L = layers[i];
  const int64_t keys = (int64_t)s.heads * s.dim, mixed = s.mixed();
  const auto proj = [&](int64_t at) -> char* { return (char*)b.proj + at * unit(); };
  {
    DenseArgs a = product(L.in.w, ld, M);
    size_t part = 0;
    const auto rows = [&](void* y, int64_t ldy, int64_t n) -> DenseSegment& {
      return segment(&a, b.h, ld, y, ldy, L.in.at[part++], n);
    };
    if (s.type == MIX_GLA) {
      rows(b.proj, L.ldp, 2 * keys + 2 * mixed);
      rows(b.low, L.decay_k, s.decay_rank);
    } else if (s.type == MIX_HGRN2) {
      DenseSegment& q = rows(b.proj, L.ldp, keys + mixed);
      q.act = DENSE_SILU;
      q.act_rows = (int32_t)keys;
      DenseSegment& f = rows(b.decay, keys, keys);
      f.act = DENSE_FORGET;
      f.y_f32 = 1;
      f.bias = L.decay_b;
      f.lower = L.lower;
    } else {
      rows(b.proj, L.ldp, (int64_t)s.heads * (s.dim + s.rot));
      if (s.kv_from < 0) rows(b.down, s.rank + s.rot, s.rank + s.rot).y_f32 = 1;
    }
    DenseSegment& g = rows(b.gate, ldg, width);
    g.act = DENSE_SIGMOID;
    g.bias = L.rg1_b;
    if (int rc = launch_dense(a, f32, stream)) return rc;
  }
  if (s.type == MIX_LATENT) {
    LatentAttnArgs a = latent_args(i);
    a.q = b.proj;
    a.ldq = L.ldp;
    if (s.kv_from < 0) a.down = b.down;
    a.ldd = s.rank + s.rot;
    a.norm = L.latent_norm;
    a.freq = L.freq;
    a.sink = L.sink;
    a.cache = L.cache;
    a.w_uk = L.w_uk;
    a.w_uv = L.w_uv;
    a.w_kv = L.w_kv;
    a.ctx = b.ctx;
    a.ldc = L.mixed_k;
    a.M = M;
    a.pos = pos;
    a.qa = s_qa;
    a.ql = s_ql;
    a.ol = s_ol;
    a.kv = s_kv;
    a.parts = (float*)s_parts;
    a.dense_ws = dense_ws;
    a.dense_ws_floats = dense_ws_floats;
    return launch_latent_attention(a, f32, stream);
  }
  if (s.type == MIX_GLA) {
    DenseArgs a = product(L.w_a2, L.decay_k, M);
    DenseSegment& z = segment(&a, b.low, L.decay_k, b.decay, keys, 0, keys);
    z.act = DENSE_LOG_DECAY;
    z.act_pos = (float)(1.4426950408889634074 / s.tau);  // binary logarithms
    z.y_f32 = 1;
    z.bias = L.decay_b;
    if (int rc = launch_dense(a, f32, stream)) return rc;
  }
  GatedStateArgs a;
  a.q = proj(0);
  if (s.type == MIX_GLA) a.k = proj(keys);
  a.v = proj(s.type == MIX_GLA ? 2 * keys : keys);
  a.ldp = L.ldp;
  a.g = b.decay;
  a.ldg = keys;
  a.heads = s.heads;
  a.dim = s.dim;
  a.vdim = s.vdim;
  if (s.type == MIX_GLA) a.q_scale = (float)(1.0 / sqrt((double)s.dim));
  a.state = states[i];
  a.o = b.o;
  a.M = M;
  a.pos = pos;
  const void* gate = s.type == MIX_GLA ? proj(2 * keys + mixed) : nullptr;
  if (M == 1) {
    a.norm = L.mix_norm;
    a.gate = gate;
    a.ctx = b.ctx;
    a.eps = eps;
    return launch_gated_state(a, f32, stream);
  }
  if (int rc = launch_gated_state(a, f32, stream)) return rc;
  return launch_head_norm(b.o, gate, L.ldp, L.mix_norm, b.ctx, L.mixed_k, s.heads, s.vdim, M, eps, f32, stream);
}

int TudasunEngine::dense_feed_forward(int i, Buffers& b, int64_t M) {
  const LayerSpec& s = spec.layers[i];
  const LayerDev& L = layers[i];
  {
    DenseArgs a = product(L.mid.w, ld, M);
    DenseSegment& g = segment(&a, b.h, ld, b.gate, ldg, L.mid.at[0], width);
    g.act = DENSE_SIGMOID;
    g.bias = L.rg2_b;
    segment(&a, b.h, ld, b.mid, L.ff_k, L.mid.at[1], s.ff);
    if (int rc = launch_dense(a, f32, stream)) return rc;
  }
  if (int rc = launch_polynorm(b.mid, L.ff_k, s.ff, M, L.act, eps, f32, stream)) return rc;
  DenseArgs a = product(L.w_down, L.ff_k, M);
  a.out = DENSE_F32;
  segment(&a, b.mid, L.ff_k, b.y, width, 0, width);
  return launch_dense(a, f32, stream);
}

int TudasunEngine::routed_feed_forward(int i, Buffers& b, int64_t M, JoinArgs* end) {
  const LayerSpec& s = spec.layers[i];
  const LayerDev& L = layers[i];
  {
    DenseArgs a = product(L.mid.w, ld, M);
    DenseSegment& g = segment(&a, b.h, ld, b.gate, ldg, L.mid.at[0], width);
    g.act = DENSE_SIGMOID;
    g.bias = L.rg2_b;
    segment(&a, b.h, ld, b.router, s.outputs(), L.mid.at[1], s.outputs()).y_f32 = 1;
    if (s.shared_ff) {
      DenseSegment& m = segment(&a, b.h, ld, b.shared_mid, L.shared_k, L.mid.at[2], dense_glu_rows(s.shared_ff));
      m.act = DENSE_GLU;
      m.glu_rows = s.shared_ff;
      segment(&a, b.h, ld, b.shared_gate, 1, L.mid.at[3], 1).y_f32 = 1;
    }
    if (int rc = launch_dense(a, f32, stream)) return rc;
  }
  const int32_t tile_tokens = route_tile_tokens(M, s.top, s.outputs(), f32);
  {
    RouteArgs r;
    r.logits = b.router;
    r.ld = s.outputs();
    r.correction = L.correction;
    r.outputs = s.outputs();
    r.experts = s.experts;
    r.top = s.top;
    r.groups = s.groups;
    r.keep = s.keep;
    r.ids = b.ids;
    r.weights = b.weights;
    r.M = M;
    r.tile_tokens = tile_tokens;
    r.tiles = b.tiles;
    r.list = b.list;
    if (int rc = launch_route(r, stream)) return rc;
  }
  if (s.experts) {
    // entry t * top + j is token t's j-th choice; one token finds its weights by number, several by the plan
    const auto choose = [&](DenseArgs* a, int64_t w_block, int64_t x_step, int64_t y_step, int32_t reads_token) {
      a->w_batch = w_block;
      if (M == 1) {
        a->batch = s.top;
        a->ids = b.ids;
        a->n_groups = s.experts;
        a->x_batch = x_step;
        a->y_batch = y_step;
      } else {
        a->tiles = b.tiles;
        a->list = b.list;
        a->max_tiles = route_max_tiles(M, s.top, s.experts, tile_tokens);
        a->tile_tokens = tile_tokens;
        a->list_div = reads_token ? s.top : 1;
      }
    };
    DenseArgs up = product(L.w_gate_up, ld, M);
    DenseSegment& m = segment(&up, b.h, ld, b.mid, L.ff_k, 0, dense_glu_rows(s.ff));
    m.act = DENSE_GLU;
    m.glu_rows = s.ff;
    choose(&up, L.gate_up_block, 0, L.ff_k, 1);
    if (int rc = launch_dense(up, f32, stream)) return rc;
    DenseArgs down = product(L.w_expert_down, L.ff_k, M);
    segment(&down, b.mid, L.ff_k, b.pairs, width, 0, width).y_f32 = 1;
    choose(&down, L.expert_down_block, L.ff_k, width, 0);
    if (int rc = launch_dense(down, f32, stream)) return rc;
  }
  if (s.shared_ff) {
    DenseArgs a = product(L.w_shared_down, L.shared_k, M);
    a.out = DENSE_F32;
    segment(&a, b.shared_mid, L.shared_k, b.y, width, 0, width);
    if (int rc = launch_dense(a, f32, stream)) return rc;
  }
  end->y = s.shared_ff ? b.y : nullptr;
  end->y_gate = s.shared_ff ? b.shared_gate : nullptr;
  end->pairs = b.pairs;
  end->ids = b.ids;
  end->weights = b.weights;
  end->top = s.top;
  end->experts = s.experts;
  end->h = b.h;
  end->ldh = ld;
  return AWQ_OK;
}

int TudasunEngine::token_input(int i, Buffers& b, int64_t M, JoinArgs* end) {
  const LayerDev& L = layers[i];
  DenseArgs a = product(L.w_side_gate, ld, M);
  DenseSegment& g = segment(&a, b.xt, ld, b.side_mid, side_k, 0, spec.side);
  g.act = DENSE_GELU;
  g.mul = (const char*)b.side + (int64_t)i * spec.side * unit();
  g.ldmul = side_width();
  if (int rc = launch_dense(a, f32, stream)) return rc;
  DenseArgs p = product(L.w_side_proj, side_k, M);
  p.out = DENSE_F32;
  segment(&p, b.side_mid, side_k, b.y, width, 0, width);
  end->y = b.y;
  end->w_post = L.side_norm;
  return launch_dense(p, f32, stream);
}

int TudasunEngine::run_pass(bool one, const int32_t* ids, int64_t M, PassPos pos) {
  Buffers& b = one ? step : pass;
  const int n = (int)layers.size();
  if (int rc = launch_embed_tokens(embed, side_embed, f32, ids, d_token, pos, M, width, side_width(), b.x, b.side, stream)) return rc;
  {
    NormConvArgs a;
    a.x = b.x;
    a.M = M;
    a.width = width;
    a.eps = eps;
    a.w1 = layers[0].norm1;
    a.out1 = b.h;
    a.ld = ld;
    if (int rc = launch_norm_conv(a, f32, stream)) return rc;
  }
  for (int i = 0; i < n; ++i) {
    const LayerSpec& s = spec.layers[i];
    const LayerDev& L = layers[i];
    const auto ending = [&]() {
      JoinArgs e;
      e.x = b.x;
      e.M = M;
      e.width = width;
      e.eps = eps;
      e.ldo = ld;
      return e;
    };
    // what the next sublayer reads: x itself for the token input, the next layer's first norm, nothing behind the last
    const auto leaves = [&](JoinArgs* e, bool token_input_next) {
      if (token_input_next) {
        e->out = b.xt;
      } else if (i + 1 < n) {
        e->w_next = layers[i + 1].norm1;
        e->out = b.h;
      }
    };
    if (int rc = mix(i, b, M, pos)) return rc;
    {
      DenseArgs a = product(L.w_o, L.mixed_k, M);
      a.out = DENSE_F32;
      segment(&a, b.ctx, L.mixed_k, b.y, width, 0, width);
      if (int rc = launch_dense(a, f32, stream)) return rc;
      JoinArgs e = ending();
      e.y = b.y;
      e.gate = b.gate;
      e.ldg = ldg;
      e.w_post = L.norm1b;
      if (s.mlp != MLP_NONE) {
        e.w_next = L.norm2;
        e.out = b.h;
      } else {
        leaves(&e, spec.side > 0);
      }
      if (int rc = launch_join(e, f32, stream)) return rc;
    }
    if (s.mlp != MLP_NONE) {
      JoinArgs e = ending();
      e.y = b.y;
      if (int rc = s.mlp == MLP_DENSE ? dense_feed_forward(i, b, M) : routed_feed_forward(i, b, M, &e)) return rc;
      e.gate = b.gate;
      e.ldg = ldg;
      e.w_post = L.norm2b;
      leaves(&e, spec.side > 0);
      if (int rc = launch_join(e, f32, stream)) return rc;
    }
    if (spec.side) {
      JoinArgs e = ending();
      if (int rc = token_input(i, b, M, &e)) return rc;
      leaves(&e, false);
      if (int rc = launch_join(e, f32, stream)) return rc;
    }
    if (tap_on)
      if (int rc = tap_layer(i, b.x, M)) return rc;
  }
  return AWQ_OK;
}

int open_tudasun(const char* dir, const awq_open_options& opt, awq_engine** out) {
  std::unique_ptr<TudasunEngine> e(new TudasunEngine());
  // look at the folder before touching the GPU
  Safetensors file;
  if (int rc = read_spec(dir, &e->spec)) return rc;
  if (int rc = file.open(std::string(dir) + "/model.safetensors")) return rc;
  if (int rc = read_shapes(file, &e->spec)) return rc;
  if (int rc = check_tensors(expected_tensors(e->spec), file)) return rc;
  e->vocab = e->spec.vocab;
  e->width = e->spec.width;
  e->eps = e->spec.eps;
  e->softcap = e->spec.softcap;
  e->norm_shift = 1.0f;
  return ConfigModel::open(std::move(e), file, opt, out);
}

ModelClass g_class("Tudasun", open_tudasun);

}  // namespace
