// Building blocks of decoder layers in bfloat16 or binary32, shared by the models that are described by a
// config.json: dense products, grouped RMS norms with a causal convolution over time, attention over a sliding
// window with a distance bias, attention over a shared latent, linear attention with a decaying state (a decay per head or
// per channel), routed experts, gated and normalised sums into the residual stream, greedy sampling from binary32 logits.
// Every size and constant is an argument.  `f32` selects the binary32 form of a launch: weights and activations
// are then float, and no product runs at less than binary32; otherwise they are bfloat16 with binary32 sums.
// What is stated as float here is float in both forms.
#pragma once
#include <algorithm>

#include "common.hpp"

typedef __bf16 bf16_t;
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));

inline int64_t round_up(int64_t v, int64_t to) { return (v + to - 1) / to * to; }

// Where a pass stands in its sequence: from the step state on the device if `dyn` is set (so that a captured step
// can be replayed), by value otherwise.  The epoch counts the passes; its parity selects between two copies of
// state that a launch reads and writes in different workgroups.
struct PassPos {
  int32_t pos0 = 0;
  int32_t epoch = 0;
  const StepState* dyn = nullptr;
  __device__ __forceinline__ int position() const { return dyn ? dyn->pos : pos0; }
  __device__ __forceinline__ int parity() const { return (dyn ? dyn->epoch : epoch) & 1; }
};

// --- dense products (dense.hip) ----------------------------------------------------------------------------
// y[t][r] = act(sum_k w[r][k] x[t][k]).  The rows of several matrices that are applied to the same tokens form one
// weight block; a segment is a run of rows with an output of its own.  bfloat16 blocks are stored in the matrix
// instruction's operand order, [row / 32][k / 16][64 lanes][8]: lane l of a 1 KB piece holds row l % 32, inputs
// 8 (l / 32) .. + 7; binary32 blocks are row major.  k is padded with zeros to a multiple of 64.  A segment with an
// input of its own starts at a multiple of 256 rows, one that shares the input of the segment ahead of it at a
// multiple of 32; a block has a multiple of 256 rows.
constexpr int kDenseRowAlign = 256;
constexpr int kDenseSharedAlign = 32;
constexpr int kDenseKAlign = 64;
constexpr int kDenseSegments = 8;

enum DenseAct {
  DENSE_NONE = 0,
  DENSE_SILU = 1,     // z * sigmoid(z) on the segment's first act_rows rows
  DENSE_XIELU = 2,    // z > 0: softplus(p) z^2 + z/2; z <= 0: (1/2 + softplus(q)) (exp(z) - 1 - z) + z/2
  DENSE_SIGMOID = 3,  // sigmoid(z + bias)
  DENSE_GELU = 4,     // z/2 (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3)))
  DENSE_GLU = 5,      // silu(gate) * up: rows 16 i .. + 7 are gate rows 8 i .., rows 16 i + 8 .. + 15 their up rows
  DENSE_SOFTCAP = 6,  // act_pos * tanh(z / act_pos)
  DENSE_LOG_DECAY = 7,  // act_pos * ln(sigmoid(z + bias))
  DENSE_FORGET = 8,     // (1 - lower) * (1 - sigmoid(z + bias))
};
struct DenseSegment {
  const void* x = nullptr;  // [tokens][ldx]
  void* y = nullptr;        // [tokens][ldy]
  int64_t ldx = 0, ldy = 0;
  int32_t row0 = 0, rows = 0;
  int32_t act = DENSE_NONE, act_rows = 0;
  float act_pos = 0.0f, act_neg = 0.0f;  // softplus(p), 1/2 + softplus(q); the cap
  int32_t y_f32 = 0;                     // DENSE_STORE: y is float
  int32_t glu_rows = 0;                  // DENSE_GLU: outputs; rows is dense_glu_rows of it
  const float* bias = nullptr;           // DENSE_SIGMOID, DENSE_LOG_DECAY, DENSE_FORGET: [rows]
  const float* lower = nullptr;          // DENSE_FORGET: [rows]
  const void* mul = nullptr;             // DENSE_GELU: the result times mul[token][row], in the activations' type; may be null
  int64_t ldmul = 0;
};
enum DenseOut {
  DENSE_STORE = 0,     // y in the activations' type, or float where the segment says so
  DENSE_RESIDUAL = 1,  // y is float: y = (y + sum) + addend (addend: same shape, may be null)
  DENSE_F32 = 2,       // y is float
  DENSE_ARGMAX = 3,    // one token: y is float, and *best becomes the largest (value, -row) candidate
};
// A run of tokens that one weight block of several is applied to: rows first .. first + count - 1 of the list.
struct DenseTile {
  int32_t group, first, count;
};
struct DenseArgs {
  const void* w = nullptr;
  int64_t k = 0;  // padded
  int64_t M = 0;
  int32_t n_seg = 1;
  int32_t out = DENSE_STORE;
  int32_t start[kDenseSegments] = {};  // the segments' first rows (launch_dense)
  DenseSegment seg[kDenseSegments];
  const float* addend = nullptr;
  unsigned long long* best = nullptr;  // DENSE_ARGMAX: zero between launches
  // one token, DENSE_RESIDUAL: the first gate_k inputs of segment 0 are not read from x but formed in the launch, the RMS
  // norm of o over gate_n values times w times sigmoid(g), zeros behind them (dense_gate_fused says where it can be)
  const float* gate_o = nullptr;
  const void* gate_g = nullptr;
  const float* gate_w = nullptr;
  int32_t gate_n = 0, gate_k = 0;
  float gate_eps = 0.0f;
  float* workspace = nullptr;          // sums of products that are cut along k; may be null
  int64_t workspace_floats = 0;
  // Several products in one launch (DENSE_STORE): product b has its weight block w_batch elements (rows padded times k)
  // behind the one ahead, its input x_batch and its output y_batch elements.  ids (device, one token only): product b
  // takes weight block ids[b], and is left out where that is not below n_groups.
  int32_t batch = 1;
  int64_t w_batch = 0, x_batch = 0, y_batch = 0;
  const int32_t* ids = nullptr;
  int32_t n_groups = 0;
  // Many tokens, each with weight blocks of its own (DENSE_STORE): `tiles` (device, max_tiles of them, count 0 behind the
  // last) name runs of `list`; entry p of the list reads input row p / list_div and writes output row p.
  const DenseTile* tiles = nullptr;
  const int32_t* list = nullptr;
  int32_t max_tiles = 0, tile_tokens = 64, list_div = 1;
};
inline int64_t dense_glu_rows(int64_t n) { return round_up(n, 8) * 2; }
int64_t dense_weight_bytes(int64_t rows_padded, int64_t k_padded, bool f32);
// src [rows][cols] bfloat16 or float, row major on the device, into rows row0.., inputs col0.. of a block (col0 a
// multiple of 8); the rest of the block is left as it is (zero it first)
enum DensePack {
  PACK_PLAIN = 0,
  PACK_GATE = 1,       // as the gate rows of a DENSE_GLU segment
  PACK_UP = 2,         // as its up rows
  PACK_TRANSPOSED = 3  // rows and columns of src exchanged
};
int launch_dense_pack(const void* src, bool src_f32, int64_t rows, int64_t cols, void* w, int64_t k_padded, int64_t row0,
                      int64_t col0, bool f32, hipStream_t st, int form = PACK_PLAIN);
int launch_dense(const DenseArgs& a, bool f32, hipStream_t st);
bool dense_gate_fused(int64_t n, int64_t k_padded, int64_t M, bool f32);

// --- per-token operators (token_ops.hip) -------------------------------------------------------------------
// src [n] -> dst [n], each bfloat16 or float
int launch_convert(const void* src, bool src_f32, void* dst, bool dst_f32, int64_t n, hipStream_t st);
// x[t][i] = table[token][i] * scale + (i even: sin, odd: cos of position * freq[i / 2]), also kept in `keep` (may be
// null).  With pos.dyn the one token is the step state's, or *last where that is negative.
int launch_embed_sinusoid(const void* table, bool f32, const int32_t* tokens, const int32_t* last, PassPos pos, int64_t M,
                          int64_t width, float scale, const double* freq, float* x, float* keep, hipStream_t st);
struct NormConvArgs {
  const float* x = nullptr;         // [M][width]
  const int32_t* rows = nullptr;    // take row rows[t] of x instead of t (without convolution)
  int64_t M = 0, width = 0;
  int32_t groups = 1;
  float eps = 0.0f;
  const float* w1 = nullptr;        // first norm, [width]
  const float* conv = nullptr;      // [width][taps] or null: out1 = h + conv(h), h the first norm's output
  int32_t taps = 0;
  float* state[2] = {nullptr, nullptr};  // [taps - 1][width]: the last inputs h of the convolution, by parity
  void* out1 = nullptr;             // [M][ld]
  const float* w2 = nullptr;        // second norm or null
  void* out2 = nullptr;
  int64_t ld = 0;
  PassPos pos;
};
int launch_norm_conv(const NormConvArgs& a, bool f32, hipStream_t st);
// y[t][i] = RMS norm over all n of o[t] * w * sigmoid(g[t][i]); o is float
int launch_gated_norm(const float* o, int64_t ldo, const void* g, int64_t ldg, const float* w, void* y, int64_t ldy,
                      int64_t n, int64_t M, float eps, bool f32, hipStream_t st);
int launch_add_rows(float* x, const float* y, int64_t n, hipStream_t st);  // x += y
// the best candidate becomes the token; `state` moves on to the next position (epoch + epoch_step)
int launch_take_best(unsigned long long* best, int32_t* out_token, int32_t* out_array, StepState* state,
                     int32_t epoch_step, hipStream_t st);

// --- attention over a sliding window (window_attention.hip) --------------------------------------------------
// Row (kv head, position) of a key or value cache: blocks of 64 positions, [block][head][64][row], and a position's
// slot is position % slots, so a layer whose window is shorter than the sequence keeps a ring.
struct RingLayout {
  int32_t slots = 0;  // a multiple of 64
  int32_t heads = 0;
  int32_t row = 0;    // elements, padded
  __host__ __device__ int64_t elements() const { return (int64_t)slots * heads * row; }
};
__device__ __forceinline__ int64_t ring_row(const RingLayout& l, int head, int slot) {
  return (((int64_t)(slot >> 6) * l.heads + head) * 64 + (slot & 63)) * l.row;
}
struct WindowAttnArgs {
  // projections of the pass, [M][ldp]: heads * dim of q, kv_heads * dim of k, kv_heads * vdim of v; the prompt form
  // normalises q in place
  void* proj = nullptr;
  int64_t ldp = 0;
  int32_t heads = 0, kv_heads = 0, dim = 0, vdim = 0;
  int32_t window = 0;       // keys a position sees, itself included; 0: all before it
  float scale = 1.0f, eps = 0.0f;
  float temp_coef = 0.0f;   // scores times 1 + coef * ln(floor((p + 1) / every) + 1); 0: none
  double temp_every = 1.0;
  const float* slope = nullptr;  // [heads], taken off per position of distance
  void* k_cache = nullptr;
  void* v_cache = nullptr;
  RingLayout kl, vl;
  void* ctx = nullptr;      // [M][ldc]
  int64_t ldc = 0;
  int64_t M = 0;
  PassPos pos;
  // one-token form: partial results of the parts a window is cut into
  float* parts = nullptr;
  int32_t len_bound = 0;  // >= positions the sequence will hold
};
int32_t window_row_padded(int32_t dim);
int64_t window_parts_floats(int32_t heads, int32_t vdim, int64_t window, int64_t max_pos);
// normalise q and k, append k and v, attend
int launch_window_attention(const WindowAttnArgs& a, bool f32, hipStream_t st);

// --- linear attention with a decaying state (linear_attention.hip) -------------------------------------------
// per head S <- decay S + k v^T, o = S^T q; state [heads][vdim][round_up(dim, 64)] float (S transposed), zero ahead of
// position 0
struct LinearAttnArgs {
  const void* proj = nullptr;  // [M][ldp]: heads * dim of q, heads * dim of k, heads * vdim of v
  int64_t ldp = 0;
  int32_t heads = 0, dim = 0, vdim = 0;
  const float* decay = nullptr;       // [heads]
  const float* log2_decay = nullptr;  // [heads], null unless every decay is positive: many tokens then go in chunks
  float* state = nullptr;
  float* o = nullptr;  // [M][heads * vdim]
  int64_t M = 0;
  PassPos pos;
};
int64_t linear_state_floats(int32_t heads, int32_t dim, int32_t vdim);
int launch_linear_attention(const LinearAttnArgs& a, bool f32, hipStream_t st);

// --- linear attention whose state decays per channel (gated_state.hip) -----------------------------------------
// Per head S <- diag(decay_t) S + k_t v_t^T, o_t = S^T (q_scale q_t); the decay of a token is one number per row of S.
// State as above, [heads][vdim][round_up(dim, 64)] float (S transposed), zero ahead of position 0.
struct GatedStateArgs {
  const void *q = nullptr, *k = nullptr, *v = nullptr;  // [M][ldp]: heads * dim, heads * dim, heads * vdim
  int64_t ldp = 0;
  // [M][ldg], heads * dim: with k the binary logarithms of the decays (at most 0); without k the numbers 1 - decay,
  // which then are the keys as well
  const float* g = nullptr;
  int64_t ldg = 0;
  int32_t heads = 0, dim = 0, vdim = 0;
  float q_scale = 1.0f;
  float* state = nullptr;
  float* o = nullptr;  // [M][heads * vdim]
  int64_t M = 0;
  PassPos pos;
  // one token: ctx = the heads' norm below instead of o, in the same launch; null: none
  const float* norm = nullptr;
  const void* gate = nullptr;
  void* ctx = nullptr;
  float eps = 0.0f;
};
int launch_gated_state(const GatedStateArgs& a, bool f32, hipStream_t st);
// ctx[t][h][c] = RMS norm over a head's vdim values of o, times w [vdim], times silu(gate) (gate may be null)
int launch_head_norm(const float* o, const void* gate, int64_t ldg, const float* w, void* ctx, int64_t ldc, int32_t heads,
                     int32_t vdim, int64_t M, float eps, bool f32, hipStream_t st);

// --- attention over a shared latent (latent_attention.hip) -----------------------------------------------------
// A position's cache row is [latent, zeros to a multiple of 32, rotated key part, zeros to a multiple of 32].  Queries meet
// it in two forms: taken into the latent space (q W_uk, one key for all heads, values are the latents themselves), or
// with every head's keys and values formed from the latents first, where a pass has enough queries to pay for it.
struct LatentLayout {
  int32_t rank = 0, rot = 0;
  __host__ __device__ int32_t rank_padded() const { return (rank + 31) / 32 * 32; }
  __host__ __device__ int32_t row() const { return rank_padded() + (rot + 31) / 32 * 32; }
};
struct LatentAttnArgs {
  void* q = nullptr;  // [M][ldq]: per head dim unrotated and rot rotated values; the second form rotates them in place
  int64_t ldq = 0;
  const float* down = nullptr;  // [M][ldd]: latent and key part as projected; null: another layer's rows are used
  int64_t ldd = 0;
  const float* norm = nullptr;  // [rank]
  const double* freq = nullptr; // [rot / 2]
  const float* sink = nullptr;  // [heads] or null
  int32_t heads = 0, dim = 0, vdim = 0;
  float scale = 1.0f, eps = 0.0f;
  LatentLayout l;
  void* cache = nullptr;        // [max_pos rounded up to 64][l.row()]
  const void* w_uk = nullptr;   // batch of heads: rank rows of dim inputs (W_uk transposed)
  const void* w_uv = nullptr;   // batch of heads: vdim rows of rank inputs
  const void* w_kv = nullptr;   // one block: heads * dim rows of W_uk, then heads * vdim of W_uv, of rank inputs
  void* ctx = nullptr;          // [M][ldc], heads * vdim
  int64_t ldc = 0;
  int64_t M = 0;
  PassPos pos;
  int64_t max_pos = 0;
  // scratch, latent_scratch_bytes of each
  void *qa = nullptr, *ql = nullptr, *ol = nullptr, *kv = nullptr;
  float* parts = nullptr;
  float* dense_ws = nullptr;
  int64_t dense_ws_floats = 0;
};
struct LatentScratch {
  int64_t qa = 0, ql = 0, ol = 0, kv = 0, parts = 0;  // bytes
};
// will passes of up to max_tokens tokens form keys and values?  Only then w_kv (and kv) are needed
bool latent_forms_keys(const LatentAttnArgs& a, int64_t max_tokens, bool f32);
LatentScratch latent_scratch(const LatentAttnArgs& a, int64_t max_tokens, bool f32);
int64_t latent_uk_block(const LatentAttnArgs& a);  // elements between heads of w_uk
int64_t latent_uv_block(const LatentAttnArgs& a);  // ... of w_uv
int64_t latent_kv_rows(const LatentAttnArgs& a);   // padded rows of w_kv
// W_uk [heads * dim][rank] and W_uv [heads * vdim][rank] on the device into the zeroed blocks (either source may be null: it
// is left out; w_kv may be null)
int launch_latent_pack(const LatentAttnArgs& a, const void* uk, const void* uv, bool src_f32, void* w_uk, void* w_uv, void* w_kv,
                       bool f32, hipStream_t st);
int launch_latent_attention(const LatentAttnArgs& a, bool f32, hipStream_t st);

// --- routed feed-forward (experts.hip) ---------------------------------------------------------------------------
struct RouteArgs {
  const float* logits = nullptr;  // [M][ld], one per output: experts, then identity experts
  int64_t ld = 0;
  const float* correction = nullptr;  // [outputs], added to the softmax scores for the choice only; may be null
  int32_t outputs = 0, experts = 0, top = 0;
  int32_t groups = 0, keep = 0;   // only outputs of the `keep` groups with the largest choice score; 0: no groups
  int32_t* ids = nullptr;         // [M][top]
  float* weights = nullptr;       // [M][top], the chosen scores over their sum
  int64_t M = 0;
  // more than one token: the plan of the experts' products, token t's j-th choice is entry t * top + j
  int32_t tile_tokens = 64;
  DenseTile* tiles = nullptr;     // [route_max_tiles]
  int32_t* list = nullptr;        // [M * top]
};
// tokens of a tile: 64, or 128 where an expert has as many on average and the products have tiles of that size
int32_t route_tile_tokens(int64_t M, int32_t top, int32_t outputs, bool f32);
int32_t route_max_tiles(int64_t M, int32_t top, int32_t experts, int32_t tile_tokens);
int launch_route(const RouteArgs& a, hipStream_t st);

// --- around a sublayer (sublayer_ops.hip) --------------------------------------------------------------------------
// x[t] = table[token] (float), side[t] = side_table[token] (both tables in the activations' type); the one token of
// pos.dyn as in launch_embed_sinusoid
int launch_embed_tokens(const void* table, const void* side_table, bool f32, const int32_t* tokens, const int32_t* last,
                        PassPos pos, int64_t M, int64_t width, int64_t side_width, float* x, void* side, hipStream_t st);
// What ends a sublayer: x += RMS norm(y * gate) * w_post, then out = RMS norm(x) * w_next.
struct JoinArgs {
  float* x = nullptr;         // [M][width]
  int64_t M = 0, width = 0;
  float eps = 0.0f;
  const float* y = nullptr;   // [M][width], or null
  // y is to be multiplied by sigmoid(y_gate[t]) (null: by 1), and the experts' outputs are added to it: sum over j < top
  // of weights[t][j] * (ids[t][j] < experts ? pairs[t * top + j] : h[t])
  const float* y_gate = nullptr;
  const float* pairs = nullptr;
  const int32_t* ids = nullptr;
  const float* weights = nullptr;
  int32_t top = 0, experts = 0;
  const void* h = nullptr;    // [M][ldh]
  int64_t ldh = 0;
  const void* gate = nullptr; // [M][ldg], in the activations' type; may be null
  int64_t ldg = 0;
  const float* w_post = nullptr;
  const float* w_next = nullptr;  // null: out = x
  void* out = nullptr;            // [M][ldo] in the activations' type; may be null
  int64_t ldo = 0;
};
int launch_join(const JoinArgs& a, bool f32, hipStream_t st);
// z <- a N(z) + b N(z^2) + c N(z^3) + e with N the division of a token's n values by their root mean square; [M][ld]
int launch_polynorm(void* z, int64_t ld, int64_t n, int64_t M, const float* abce, float eps, bool f32, hipStream_t st);
