// Building blocks of decoder layers in bfloat16 or binary32, shared by the models that are described by a
// config.json: dense products, grouped RMS norms with a causal convolution over time, attention over a sliding
// window with a distance bias, linear attention with a decaying state, greedy sampling from binary32 logits.
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
// weight block; a segment is a run of rows with an input and an output of its own.  bfloat16 blocks are stored in
// the matrix instruction's operand order, [row / 32][k / 16][64 lanes][8]: lane l of a 1 KB piece holds row l % 32,
// inputs 8 (l / 32) .. + 7; binary32 blocks are row major.  k is padded with zeros to a multiple of 64 and a
// segment starts at a multiple of 256 rows.
constexpr int kDenseRowAlign = 256;
constexpr int kDenseKAlign = 64;

enum DenseAct {
  DENSE_NONE = 0,
  DENSE_SILU = 1,   // z * sigmoid(z) on the segment's first act_rows rows
  DENSE_XIELU = 2,  // z > 0: softplus(p) z^2 + z/2; z <= 0: (1/2 + softplus(q)) (exp(z) - 1 - z) + z/2
};
struct DenseSegment {
  const void* x = nullptr;  // [tokens][ldx]
  void* y = nullptr;        // [tokens][ldy]
  int64_t ldx = 0, ldy = 0;
  int32_t row0 = 0, rows = 0;
  int32_t act = DENSE_NONE, act_rows = 0;
  float act_pos = 0.0f, act_neg = 0.0f;  // softplus(p), 1/2 + softplus(q)
};
enum DenseOut {
  DENSE_STORE = 0,     // y in the activations' type
  DENSE_RESIDUAL = 1,  // y is float: y = (y + sum) + addend (addend: same shape, may be null)
  DENSE_F32 = 2,       // y is float
  DENSE_ARGMAX = 3,    // one token: y is float, and *best becomes the largest (value, -row) candidate
};
struct DenseArgs {
  const void* w = nullptr;
  int64_t k = 0;  // padded
  int64_t M = 0;
  int32_t n_seg = 1;
  int32_t out = DENSE_STORE;
  DenseSegment seg[2];
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
};
int64_t dense_weight_bytes(int64_t rows_padded, int64_t k_padded, bool f32);
// src [rows][cols] bfloat16 or float, row major on the device, into rows row0.., inputs col0.. of a block (col0 a
// multiple of 8); the rest of the block is left as it is (zero it first)
int launch_dense_pack(const void* src, bool src_f32, int64_t rows, int64_t cols, void* w, int64_t k_padded, int64_t row0,
                      int64_t col0, bool f32, hipStream_t st);
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
