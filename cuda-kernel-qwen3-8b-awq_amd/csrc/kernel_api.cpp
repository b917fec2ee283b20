// The kernel-level entry points of include/awq_infer.h: argument checks around the launchers.
#include "engine.hpp"

#include <string.h>

bool awq_zp_all_integral(const uint16_t* zp, int64_t n) {
  for (int64_t i = 0; i < n; ++i) {
    half_t h;
    memcpy(&h, &zp[i], 2);
    float f = (float)h;
    if (!(f >= 0.0f && f <= 1024.0f) || f != (float)(int)f) return false;
  }
  return true;
}

extern "C" int awq_dequant(const void* packed, const void* scale, const void* zp, void* out, int64_t rows, int64_t cols,
                           int64_t n_groups, void* stream) {
  AWQ_REQUIRE(packed && scale && zp && out, "NULL pointer");
  return launch_dequant((const uint8_t*)packed, (const half_t*)scale, (const half_t*)zp, (half_t*)out, rows, cols,
                        n_groups, (hipStream_t)stream);
}

extern "C" int awq_linear_repack(const void* packed_in, void* repacked_out, int64_t m, int64_t k, void* stream) {
  AWQ_REQUIRE(packed_in && repacked_out && packed_in != repacked_out, "NULL or aliased pointers");
  return launch_repack((const uint8_t*)packed_in, repacked_out, m, k, (hipStream_t)stream);
}

extern "C" int64_t awq_gemv_workspace_bytes(int64_t m, int64_t k) { return gemv_workspace_bytes(m, k); }

extern "C" int awq_gemv_fused(const awq_linear_args* u, void* stream) {
  AWQ_REQUIRE(u != nullptr, "args is NULL");
  AWQ_REQUIRE(u->repacked && u->scale && u->zp && u->x && u->y && u->workspace, "NULL pointer");
  AWQ_REQUIRE(u->m > 0 && u->m % 128 == 0, "m must be a positive multiple of 128");
  AWQ_REQUIRE(u->prologue == AWQ_PRO_NONE || u->prologue == AWQ_PRO_RMSNORM, "bad prologue");
  AWQ_REQUIRE(u->epilogue >= AWQ_EPI_STORE && u->epilogue <= AWQ_EPI_ARGMAX, "bad epilogue");
  LinearArgs a;
  a.wq = u->repacked;
  a.scale = (const half_t*)u->scale;
  a.zp = (const half_t*)u->zp;
  a.x = (const half_t*)u->x;
  a.y = (half_t*)u->y;
  a.res = (const half_t*)u->residual;
  a.best = (unsigned long long*)u->workspace;  // the sampler's best candidate
  a.m = u->m;
  a.k = u->k;
  a.prologue = u->prologue;
  a.epilogue = u->epilogue;
  a.gamma = (const half_t*)u->gamma;
  a.eps = u->eps;
  a.cos_t = (const half_t*)u->cos_t;
  a.sin_t = (const half_t*)u->sin_t;
  a.k_cache = (half_t*)u->k_cache;
  a.v_cache = (half_t*)u->v_cache;
  a.hidden = u->hidden;
  a.pos = (int32_t)u->pos;
  a.max_pos = u->max_pos;
  a.kv = kv_head_major(u->max_pos);
  a.out_token = (int32_t*)u->out_token;
  return launch_gemv(a, (hipStream_t)stream);
}

// workspace of awq_qkv_attention: the step state the launch reads, the status word, then the exchange buffers
namespace {
constexpr int64_t kQkvWsHeader = 256;  // StepState at 0, status word at 128
}
extern "C" int64_t awq_qkv_attention_workspace_bytes(int32_t n_heads) {
  if (n_heads <= 0) return -1;
  return kQkvWsHeader + fused_qkv_attn_exchange_bytes(n_heads);
}

extern "C" int awq_qkv_attention_supported(int64_t hidden, int32_t n_heads, void* stream) {
  return fused_qkv_attn_supported(hidden, n_heads, (hipStream_t)stream);
}

extern "C" int64_t awq_kv_parts_bytes(int32_t n_heads, int64_t parts_pos) {
  if (n_heads <= 0 || parts_pos <= 0) return -1;
  return fused_qkv_attn_parts_bytes(n_heads, parts_pos);
}

extern "C" int awq_kv_cache_to_parts(const void* k_cache, const void* v_cache, int64_t max_pos, int32_t n_heads,
                                     void* k_parts, void* v_parts, int64_t parts_pos, int64_t pos0, int64_t n,
                                     void* stream) {
  AWQ_REQUIRE(max_pos > 0 && pos0 >= 0 && n >= 0 && pos0 + n <= max_pos && parts_pos > 0 && parts_pos < (1ll << 30),
              "positions out of range");
  return launch_kv_to_parts((const half_t*)k_cache, (const half_t*)v_cache, kv_head_major(max_pos), (half_t*)k_parts,
                            (half_t*)v_parts, n_heads, (int)parts_pos, pos0, n, (hipStream_t)stream);
}

extern "C" int awq_qkv_attention(const void* wqkv_repacked, const void* scale, const void* zp, const void* x,
                                 const void* gamma, float eps, const void* cos_t, const void* sin_t, void* k_cache,
                                 void* v_cache, int64_t max_pos, void* k_parts, void* v_parts, int64_t parts_pos,
                                 int32_t n_heads, int64_t pos, int64_t L, void* q_out, void* ctx, void* workspace,
                                 int32_t call_tag, void* stream) {
  AWQ_REQUIRE(workspace != nullptr, "workspace is NULL");
  AWQ_REQUIRE(n_heads == 32, "the fused launch is built for 32 heads of 128");
  AWQ_REQUIRE(max_pos > 0 && pos >= 0 && pos < max_pos, "pos out of range");
  AWQ_REQUIRE(L >= 0 && L <= pos + 1 && L <= kFusedQkvAttnMax, "attended length out of range for the fused launch");
  AWQ_REQUIRE(parts_pos > 0 && parts_pos < (1ll << 30) && L <= parts_pos, "the parts arrays do not hold the attended positions");
  AWQ_REQUIRE(call_tag >= 1 && call_tag < (1 << 30), "call_tag must be in [1, 2^30)");
  hipStream_t st = (hipStream_t)stream;
  char* ws = (char*)workspace;
  StepState s{};
  s.pos = (int32_t)pos;
  s.len_lo = s.len_hi = (int32_t)L;
  s.token = -1;
  s.epoch = call_tag;
  if (int rc = launch_set_state((StepState*)ws, s, st)) return rc;
  const int64_t hidden = (int64_t)n_heads * AWQ_HEAD_DIM;
  uint32_t* score_tag = (uint32_t*)(ws + kQkvWsHeader);
  // the words of an earlier call must not meet their tag again
  if (int rc = launch_fill_zero(score_tag, fused_qkv_attn_exchange_bytes(n_heads), st)) return rc;
  return launch_fused_qkv_attn(wqkv_repacked, (const half_t*)scale, (const half_t*)zp, 3 * hidden, (const half_t*)x,
                               (const half_t*)gamma, eps, (const half_t*)cos_t, (const half_t*)sin_t, (half_t*)k_cache,
                               (half_t*)v_cache, kv_head_major(max_pos), (half_t*)k_parts, (half_t*)v_parts, (int)parts_pos,
                               (half_t*)q_out, (half_t*)ctx, score_tag,
                               (int32_t*)(ws + 128), (const StepState*)ws, 0, 0, L > 0 ? L : 1, n_heads, nullptr, st);
}

// after the stream has drained: 0, or AWQ_ERR_HIP when a wait of the last launches gave up (the word is cleared)
extern "C" int awq_qkv_attention_status(void* workspace, void* stream) {
  AWQ_REQUIRE(workspace != nullptr, "workspace is NULL");
  AWQ_HIP_TRY(hipStreamSynchronize((hipStream_t)stream));
  int32_t word = 0;
  AWQ_HIP_TRY(hipMemcpy(&word, (char*)workspace + 128, 4, hipMemcpyDeviceToHost));
  if (word == 0) return AWQ_OK;
  AWQ_HIP_TRY(hipMemset((char*)workspace + 128, 0, 4));
  awq_set_error("a fused launch gave up waiting for what other workgroups hand over");
  return AWQ_ERR_HIP;
}

extern "C" int awq_gemv(const void* repacked, const void* scale, const void* zp, int64_t m, int64_t k, const void* x,
                        void* y, void* workspace, void* stream) {
  awq_linear_args u;
  memset(&u, 0, sizeof(u));
  u.repacked = repacked;
  u.scale = scale;
  u.zp = zp;
  u.m = m;
  u.k = k;
  u.x = x;
  u.y = y;
  u.workspace = workspace;
  return awq_gemv_fused(&u, stream);
}

extern "C" int64_t awq_gemm_workspace_bytes(int64_t m, int64_t k, int64_t M) { return gemm_workspace_bytes(m, k, M); }
extern "C" int awq_gemm_plan(int64_t m, int64_t k, int64_t M, int has_workspace) {
  return gemm_plan(m, k, M, has_workspace);
}

extern "C" int awq_gemm(const void* repacked, const void* scale, const void* zp, int64_t m, int64_t k, const void* x,
                        void* y, int64_t M, int32_t zp_integral, void* workspace, void* stream) {
  AWQ_REQUIRE(repacked && scale && zp && x && y, "NULL pointer");
  AWQ_REQUIRE(m > 0 && m % 128 == 0, "m must be a positive multiple of 128");
  if (zp_integral < 0) {
    std::vector<uint16_t> zph((size_t)(m / 128));
    AWQ_HIP_TRY(hipMemcpyAsync(zph.data(), zp, zph.size() * 2, hipMemcpyDeviceToHost, (hipStream_t)stream));
    AWQ_HIP_TRY(hipStreamSynchronize((hipStream_t)stream));
    zp_integral = awq_zp_all_integral(zph.data(), (int64_t)zph.size());
  }
  return launch_gemm(repacked, (const half_t*)scale, (const half_t*)zp, m, k, (const half_t*)x, (half_t*)y, M,
                     zp_integral != 0, EPI_STORE, nullptr, workspace, workspace ? gemm_workspace_bytes(m, k, M) : 0,
                     (hipStream_t)stream);
}

extern "C" int awq_rmsnorm(const void* x, const void* gamma, void* out, int64_t n, float eps, void* stream) {
  AWQ_REQUIRE(x && gamma && out, "NULL pointer");
  return launch_rmsnorm((const half_t*)x, (const half_t*)gamma, (half_t*)out, n, eps, (hipStream_t)stream);
}

extern "C" int awq_rope_kv_append(const void* qkv, const void* cos_t, const void* sin_t, void* q_out, void* k_cache,
                                  void* v_cache, int32_t n_heads, int64_t max_pos, int64_t pos, void* stream) {
  AWQ_REQUIRE(qkv && cos_t && sin_t && q_out && k_cache && v_cache, "NULL pointer");
  return launch_rope_kv_append((const half_t*)qkv, (const half_t*)cos_t, (const half_t*)sin_t, (half_t*)q_out,
                               (half_t*)k_cache, (half_t*)v_cache, n_heads, max_pos, kv_head_major(max_pos), pos, nullptr,
                               (hipStream_t)stream);
}

extern "C" int64_t awq_attention_workspace_bytes(int32_t n_heads, int64_t max_pos) {
  return attention_workspace_bytes(n_heads, max_pos);
}

extern "C" int awq_decode_attention(const void* q, const void* k_cache, const void* v_cache, void* ctx, int32_t n_heads,
                                    int64_t max_pos, int64_t L, void* workspace, void* stream) {
  AWQ_REQUIRE(q && k_cache && v_cache && ctx, "NULL pointer");
  return launch_attention((const half_t*)q, (const half_t*)k_cache, (const half_t*)v_cache, (half_t*)ctx, n_heads,
                          max_pos, kv_head_major(max_pos), L, nullptr, 0, 0, workspace, (hipStream_t)stream);
}

extern "C" int awq_decode_attention_static(const void* q, const void* k_cache, const void* v_cache, void* ctx,
                                           int32_t n_heads, int64_t max_pos, int64_t L, void* stream) {
  AWQ_REQUIRE(q && k_cache && v_cache && ctx, "NULL pointer");
  return launch_attention_static((const half_t*)q, (const half_t*)k_cache, (const half_t*)v_cache, (half_t*)ctx, n_heads,
                                 max_pos, L, (hipStream_t)stream);
}

extern "C" int awq_prefill_attention(const void* q, const void* k_cache, const void* v_cache, void* ctx,
                                     int32_t n_heads, int64_t max_pos, int64_t pos0, int64_t n_tokens,
                                     int32_t first_layer, void* stream) {
  AWQ_REQUIRE(q && k_cache && v_cache && ctx, "NULL pointer");
  return launch_prefill_attention((const half_t*)q, (const half_t*)k_cache, (const half_t*)v_cache, (half_t*)ctx,
                                  n_heads, max_pos, kv_head_major(max_pos), pos0, n_tokens, first_layer ? 0 : 1,
                                  (hipStream_t)stream);
}

extern "C" int awq_residual_add(const void* a, const void* b, void* out, int64_t n, void* stream) {
  AWQ_REQUIRE(a && b && out, "NULL pointer");
  return launch_residual((const half_t*)a, (const half_t*)b, (half_t*)out, n, (hipStream_t)stream);
}

extern "C" int awq_gelu(void* x, int64_t n, void* stream) {
  AWQ_REQUIRE(x != nullptr, "NULL pointer");
  return launch_gelu((half_t*)x, n, (hipStream_t)stream);
}

extern "C" int64_t awq_argmax_workspace_bytes(int64_t n) { return argmax_workspace_bytes(n); }

extern "C" int awq_logits_argmax(const void* logits, int64_t n, void* out_token, void* workspace, void* stream) {
  AWQ_REQUIRE(logits && out_token, "NULL pointer");
  return launch_argmax((const half_t*)logits, n, (int32_t*)out_token, workspace, nullptr, nullptr, (hipStream_t)stream);
}

extern "C" int awq_embed_gather(const void* packed, const void* scale, const void* zp, int64_t hidden, int64_t vocab,
                                int32_t tok, void* out, void* stream) {
  AWQ_REQUIRE(packed && scale && zp && out, "NULL pointer");
  return launch_embed((const uint8_t*)packed, (const half_t*)scale, (const half_t*)zp, hidden, vocab, tok, nullptr,
                      (half_t*)out, (hipStream_t)stream);
}
