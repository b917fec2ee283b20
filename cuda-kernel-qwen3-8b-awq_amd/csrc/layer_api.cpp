// The entry points of include/awq_infer.h for single layer building blocks: argument checks around the launchers of
// layers.hpp.
#include "layers.hpp"

extern "C" int64_t awq_dense_weight_bytes(int64_t rows_padded, int64_t k_padded, int32_t f32) {
  return dense_weight_bytes(rows_padded, k_padded, f32 != 0);
}

extern "C" int awq_dense_pack(const void* src, int32_t src_f32, int64_t rows, int64_t cols, void* w, int64_t k_padded,
                              int64_t row0, int64_t col0, int32_t f32, void* stream) {
  AWQ_REQUIRE(src && w, "NULL pointer");
  return launch_dense_pack(src, src_f32 != 0, rows, cols, w, k_padded, row0, col0, f32 != 0, (hipStream_t)stream);
}

extern "C" int awq_dense_pack_form(const void* src, int32_t src_f32, int64_t rows, int64_t cols, void* w, int64_t k_padded,
                                   int64_t row0, int64_t col0, int32_t form, int32_t f32, void* stream) {
  AWQ_REQUIRE(src && w, "NULL pointer");
  AWQ_REQUIRE(form >= AWQ_PACK_PLAIN && form <= AWQ_PACK_TRANSPOSED, "bad form");
  return launch_dense_pack(src, src_f32 != 0, rows, cols, w, k_padded, row0, col0, f32 != 0, (hipStream_t)stream, form);
}

static_assert(sizeof(awq_dense_tile) == sizeof(DenseTile) && AWQ_DENSE_SEGMENTS == kDenseSegments, "awq_infer.h and layers.hpp differ");

extern "C" int awq_dense(const awq_dense_args* u, int32_t f32, void* stream) {
  AWQ_REQUIRE(u != nullptr, "args is NULL");
  AWQ_REQUIRE(u->n_segments >= 1 && u->n_segments <= AWQ_DENSE_SEGMENTS, "too few or too many segments");
  AWQ_REQUIRE(u->out >= AWQ_DENSE_STORE && u->out <= AWQ_DENSE_F32, "bad output");
  DenseArgs a;
  a.w = u->w;
  a.k = u->k;
  a.M = u->tokens;
  a.n_seg = u->n_segments;
  a.out = u->out;
  a.addend = u->addend;
  a.workspace = u->workspace;
  a.workspace_floats = u->workspace ? u->workspace_floats : 0;
  a.batch = u->batch > 0 ? u->batch : 1;
  a.w_batch = u->w_batch;
  a.x_batch = u->x_batch;
  a.y_batch = u->y_batch;
  a.ids = u->ids;
  a.n_groups = u->n_groups;
  a.tiles = reinterpret_cast<const DenseTile*>(u->tiles);
  a.list = u->list;
  a.max_tiles = u->max_tiles;
  a.tile_tokens = u->tile_tokens;
  a.list_div = u->list_div;
  for (int i = 0; i < u->n_segments; ++i) {
    const awq_dense_segment& s = u->segment[i];
    AWQ_REQUIRE(s.act >= AWQ_ACT_NONE && s.act <= AWQ_ACT_FORGET, "bad activation");
    DenseSegment& d = a.seg[i];
    d.x = s.x;
    d.y = s.y;
    d.ldx = s.ldx;
    d.ldy = s.ldy;
    d.row0 = s.row0;
    d.rows = s.rows;
    d.act = s.act;
    d.act_rows = s.act_rows;
    d.act_pos = s.act_pos;
    d.act_neg = s.act_neg;
    d.y_f32 = s.y_f32;
    d.glu_rows = s.glu_rows;
    d.bias = s.bias;
    d.lower = s.lower;
    d.mul = s.mul;
    d.ldmul = s.ldmul;
  }
  return launch_dense(a, f32 != 0, (hipStream_t)stream);
}

static PassPos at_position(int64_t pos0) {
  PassPos p;
  p.pos0 = (int32_t)pos0;
  return p;
}

extern "C" int awq_embed_sinusoid(const void* table, int32_t f32, const int32_t* tokens, int64_t pos0, int64_t n_tokens,
                                  int64_t width, float scale, const double* freq, float* x, void* stream) {
  return launch_embed_sinusoid(table, f32 != 0, tokens, nullptr, at_position(pos0), n_tokens, width, scale, freq, x, nullptr,
                               (hipStream_t)stream);
}

extern "C" int awq_norm_conv(const float* x, int64_t n_tokens, int64_t width, int32_t groups, float eps, const float* w1,
                             const float* conv, int32_t taps, const float* state_in, float* state_out, void* out1,
                             const float* w2, void* out2, int64_t ld, int64_t pos0, int32_t f32, void* stream) {
  AWQ_REQUIRE(state_in == nullptr || state_in != state_out, "the convolution's states must differ");
  NormConvArgs a;
  a.x = x;
  a.M = n_tokens;
  a.width = width;
  a.groups = groups;
  a.eps = eps;
  a.w1 = w1;
  a.conv = conv;
  a.taps = taps;
  a.state[0] = const_cast<float*>(state_in);
  a.state[1] = state_out;
  a.out1 = out1;
  a.w2 = w2;
  a.out2 = out2;
  a.ld = ld;
  a.pos = at_position(pos0);
  return launch_norm_conv(a, f32 != 0, (hipStream_t)stream);
}

extern "C" int awq_gated_norm(const float* o, int64_t ldo, const void* g, int64_t ldg, const float* w, void* y, int64_t ldy,
                              int64_t n, int64_t n_tokens, float eps, int32_t f32, void* stream) {
  return launch_gated_norm(o, ldo, g, ldg, w, y, ldy, n, n_tokens, eps, f32 != 0, (hipStream_t)stream);
}

extern "C" int32_t awq_window_row(int32_t dim) { return window_row_padded(dim); }

extern "C" int64_t awq_window_workspace_floats(int32_t heads, int32_t vdim, int64_t window, int64_t max_pos) {
  return window_parts_floats(heads, vdim, window, max_pos);
}

extern "C" int awq_window_attention(const awq_window_args* u, int32_t f32, void* stream) {
  AWQ_REQUIRE(u != nullptr, "args is NULL");
  AWQ_REQUIRE(u->n_tokens >= 1 && u->pos0 >= 0 && u->pos0 + u->n_tokens <= u->max_pos && u->max_pos < (1ll << 31) && u->window >= 0,
              "positions out of range");
  AWQ_REQUIRE(u->slots >= std::min<int64_t>(u->max_pos, u->window ? u->window - 1 + u->n_tokens : u->max_pos),
              "the cache does not hold the window and the new positions");
  WindowAttnArgs a;
  a.proj = u->proj;
  a.ldp = u->ldp;
  a.heads = u->heads;
  a.kv_heads = u->kv_heads;
  a.dim = u->dim;
  a.vdim = u->vdim;
  a.window = u->window;
  a.scale = u->scale;
  a.eps = u->eps;
  a.temp_coef = u->temp_coef;
  a.temp_every = u->temp_every;
  a.slope = u->slope;
  a.k_cache = u->k_cache;
  a.v_cache = u->v_cache;
  a.kl = RingLayout{u->slots, u->kv_heads, window_row_padded(u->dim)};
  a.vl = RingLayout{u->slots, u->kv_heads, window_row_padded(u->vdim)};
  a.ctx = u->ctx;
  a.ldc = u->ldc;
  a.M = u->n_tokens;
  a.pos = at_position(u->pos0);
  a.parts = u->workspace;
  a.len_bound = (int32_t)u->max_pos;
  return launch_window_attention(a, f32 != 0, (hipStream_t)stream);
}

extern "C" int awq_linear_attention(const void* proj, int64_t ldp, int32_t heads, int32_t dim, int32_t vdim,
                                    const float* decay, const float* log2_decay, float* state, float* o, int64_t n_tokens,
                                    int64_t pos0, int32_t f32, void* stream) {
  LinearAttnArgs a;
  a.proj = proj;
  a.ldp = ldp;
  a.heads = heads;
  a.dim = dim;
  a.vdim = vdim;
  a.decay = decay;
  a.log2_decay = log2_decay;
  a.state = state;
  a.o = o;
  a.M = n_tokens;
  a.pos = at_position(pos0);
  return launch_linear_attention(a, f32 != 0, (hipStream_t)stream);
}

extern "C" int awq_gated_state(const awq_gated_state_args* u, int32_t f32, void* stream) {
  AWQ_REQUIRE(u != nullptr, "args is NULL");
  GatedStateArgs a;
  a.q = u->q;
  a.k = u->k;
  a.v = u->v;
  a.ldp = u->ldp;
  a.g = u->g;
  a.ldg = u->ldg;
  a.heads = u->heads;
  a.dim = u->dim;
  a.vdim = u->vdim;
  a.q_scale = u->q_scale;
  a.state = u->state;
  a.o = u->o;
  a.M = u->n_tokens;
  a.pos = at_position(u->pos0);
  a.norm = u->norm;
  a.gate = u->gate;
  a.ctx = u->ctx;
  a.eps = u->eps;
  return launch_gated_state(a, f32 != 0, (hipStream_t)stream);
}

extern "C" int awq_head_norm(const float* o, const void* gate, int64_t ldg, const float* w, void* ctx, int64_t ldc, int32_t heads,
                             int32_t vdim, int64_t n_tokens, float eps, int32_t f32, void* stream) {
  return launch_head_norm(o, gate, ldg, w, ctx, ldc, heads, vdim, n_tokens, eps, f32 != 0, (hipStream_t)stream);
}

static LatentAttnArgs latent_of(const awq_latent_args& u) {
  LatentAttnArgs a;
  a.q = u.q;
  a.ldq = u.ldq;
  a.down = u.down;
  a.ldd = u.ldd;
  a.norm = u.norm;
  a.freq = u.freq;
  a.sink = u.sink;
  a.heads = u.heads;
  a.dim = u.dim;
  a.vdim = u.vdim;
  a.scale = u.scale;
  a.eps = u.eps;
  a.l.rank = u.rank;
  a.l.rot = u.rot;
  a.cache = u.cache;
  a.w_uk = u.w_uk;
  a.w_uv = u.w_uv;
  a.w_kv = u.w_kv;
  a.ctx = u.ctx;
  a.ldc = u.ldc;
  a.M = u.n_tokens;
  a.pos = at_position(u.pos0);
  a.max_pos = u.max_pos;
  a.qa = u.qa;
  a.ql = u.ql;
  a.ol = u.ol;
  a.kv = u.kv;
  a.parts = u.parts;
  return a;
}

extern "C" int32_t awq_latent_row(int32_t rank, int32_t rot) {
  LatentLayout l;
  l.rank = rank;
  l.rot = rot;
  return l.row();
}

extern "C" int awq_latent_sizes(const awq_latent_args* u, int64_t max_tokens, int32_t f32, awq_latent_bytes* out) {
  AWQ_REQUIRE(u && out && u->heads >= 1 && u->dim >= 1 && u->vdim >= 1 && u->rank >= 1 && u->rot >= 2 && max_tokens >= 1, "bad arguments");
  const LatentAttnArgs a = latent_of(*u);
  const LatentScratch s = latent_scratch(a, max_tokens, f32 != 0);
  const int64_t unit = f32 ? 4 : 2;
  out->w_uk = latent_uk_block(a) * a.heads * unit;
  out->w_uv = latent_uv_block(a) * a.heads * unit;
  out->w_kv = latent_forms_keys(a, max_tokens, f32 != 0) ? latent_kv_rows(a) * round_up(a.l.rank, kDenseKAlign) * unit : 0;
  out->qa = s.qa;
  out->ql = s.ql;
  out->ol = s.ol;
  out->kv = s.kv;
  out->parts = s.parts;
  return AWQ_OK;
}

extern "C" int awq_latent_pack(const awq_latent_args* u, const void* uk, const void* uv, int32_t f32, void* stream) {
  AWQ_REQUIRE(u && uk && uv && u->w_uk && u->w_uv, "NULL pointer");
  return launch_latent_pack(latent_of(*u), uk, uv, false, const_cast<void*>(u->w_uk), const_cast<void*>(u->w_uv),
                            const_cast<void*>(u->w_kv), f32 != 0, (hipStream_t)stream);
}

extern "C" int awq_latent_attention(const awq_latent_args* u, int32_t f32, void* stream) {
  AWQ_REQUIRE(u != nullptr, "args is NULL");
  AWQ_REQUIRE(u->pos0 >= 0 && u->n_tokens >= 1 && u->pos0 + u->n_tokens <= u->max_pos && u->max_pos < (1ll << 31), "positions out of range");
  return launch_latent_attention(latent_of(*u), f32 != 0, (hipStream_t)stream);
}

extern "C" int32_t awq_route_max_tiles(int64_t n_tokens, int32_t top, int32_t experts, int32_t tile_tokens) {
  return tile_tokens > 0 ? route_max_tiles(n_tokens, top, experts, tile_tokens) : 0;
}

extern "C" int awq_route(const float* logits, int64_t ld, const float* correction, int32_t outputs, int32_t experts, int32_t top,
                         int32_t groups, int32_t keep, int64_t n_tokens, int32_t* ids, float* weights, int32_t tile_tokens,
                         awq_dense_tile* tiles, int32_t* list, void* stream) {
  RouteArgs a;
  a.logits = logits;
  a.ld = ld;
  a.correction = correction;
  a.outputs = outputs;
  a.experts = experts;
  a.top = top;
  a.groups = groups;
  a.keep = keep;
  a.ids = ids;
  a.weights = weights;
  a.M = n_tokens;
  a.tile_tokens = tile_tokens;
  a.tiles = reinterpret_cast<DenseTile*>(tiles);
  a.list = list;
  return launch_route(a, (hipStream_t)stream);
}

extern "C" int awq_join(const awq_join_args* u, int32_t f32, void* stream) {
  AWQ_REQUIRE(u != nullptr, "args is NULL");
  JoinArgs a;
  a.x = u->x;
  a.M = u->n_tokens;
  a.width = u->width;
  a.eps = u->eps;
  a.y = u->y;
  a.y_gate = u->y_gate;
  a.pairs = u->pairs;
  a.ids = u->ids;
  a.weights = u->weights;
  a.top = u->pairs ? u->top : 0;
  a.experts = u->experts;
  a.h = u->h;
  a.ldh = u->ldh;
  a.gate = u->gate;
  a.ldg = u->ldg;
  a.w_post = u->w_post;
  a.w_next = u->w_next;
  a.out = u->out;
  a.ldo = u->ldo;
  return launch_join(a, f32 != 0, (hipStream_t)stream);
}

extern "C" int awq_polynorm(void* z, int64_t ld, int64_t n, int64_t n_tokens, const float* abce, float eps, int32_t f32, void* stream) {
  return launch_polynorm(z, ld, n, n_tokens, abce, eps, f32 != 0, (hipStream_t)stream);
}
