// Dense products of bfloat16 (matrix cores) or binary32 weights with one token or many (layers.hpp).
#include "layers.hpp"

namespace {

typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef float f32x16_t __attribute__((ext_vector_type(16)));
typedef const __attribute__((address_space(1))) void* gptr_t;
typedef __attribute__((address_space(3))) void* lptr_t;

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + __expf(-z)); }
__device__ __forceinline__ float sigmoid_exact(float z) { return 1.0f / (1.0f + expf(-z)); }

// exp(z) - 1 - z for z <= 0.  Near zero the difference cancels: there the series z^2/2 + z^3/6 + ...
__device__ __forceinline__ float exp_minus_1_minus(float z) {
  if (z > -0.25f) {
    const float t = z * (1.0f / 7.0f) + 1.0f;
    float s = __builtin_fmaf(z * (1.0f / 6.0f), t, 1.0f);
    s = __builtin_fmaf(z * (1.0f / 5.0f), s, 1.0f);
    s = __builtin_fmaf(z * (1.0f / 4.0f), s, 1.0f);
    s = __builtin_fmaf(z * (1.0f / 3.0f), s, 1.0f);
    return 0.5f * z * z * s;
  }
  return (expf(z) - 1.0f) - z;
}

// `bias` and `lower`: the row's entries, where the activation has them
template <bool F32>
__device__ __forceinline__ float activate_with(const DenseSegment& s, int row, float z, float bias, float lower) {
  if (s.act == DENSE_SILU) return row < s.act_rows ? z * (F32 ? sigmoid_exact(z) : sigmoid_f32(z)) : z;
  if (s.act == DENSE_XIELU) {
    const float h = 0.5f * z;
    return z > 0.0f ? __builtin_fmaf(s.act_pos * z, z, h) : __builtin_fmaf(s.act_neg, exp_minus_1_minus(z), h);
  }
  if (s.act == DENSE_SIGMOID) return F32 ? sigmoid_exact(z + bias) : sigmoid_f32(z + bias);
  if (s.act == DENSE_GELU) {  // (1 + tanh u) / 2 = sigmoid(2 u)
    const float u2 = 1.5957691216057307117f * __builtin_fmaf(0.044715f * z * z, z, z);
    return z * (F32 ? sigmoid_exact(u2) : sigmoid_f32(u2));
  }
  if (s.act == DENSE_LOG_DECAY) {
    z += bias;
    if (F32) return -s.act_pos * (log1pf(expf(-fabsf(z))) + fmaxf(-z, 0.0f));
    // (off by what one rounding of the decay itself is off)
    const float e = __builtin_amdgcn_exp2f(-1.44269504088896340736f * fabsf(z));
    return -s.act_pos * __builtin_fmaf(0.693147180559945309417f, __builtin_amdgcn_logf(1.0f + e), fmaxf(-z, 0.0f));
  }
  if (s.act == DENSE_FORGET) return (1.0f - lower) * sigmoid_exact(-(z + bias));
  return z;
}

// the same for four rows, with one look at which it is
__device__ __forceinline__ void activate_four(const DenseSegment& s, int row, f32x4_t& v, const float (&bias)[4], const float (&lower)[4]) {
  switch (s.act) {
#define AWQ_ACTIVATE(ACT)                                                                      \
  case ACT:                                                                                    \
    _Pragma("unroll") for (int j = 0; j < 4; ++j) {                                            \
      __builtin_assume(s.act == ACT);                                                          \
      v[j] = activate_with<false>(s, row + j, v[j], bias[j], lower[j]);                        \
    }                                                                                          \
    break;
    AWQ_ACTIVATE(DENSE_SILU)
    AWQ_ACTIVATE(DENSE_XIELU)
    AWQ_ACTIVATE(DENSE_SIGMOID)
    AWQ_ACTIVATE(DENSE_GELU)
    AWQ_ACTIVATE(DENSE_LOG_DECAY)
    AWQ_ACTIVATE(DENSE_FORGET)
#undef AWQ_ACTIVATE
  }
}

template <bool F32>
__device__ __forceinline__ float activate(const DenseSegment& s, int row, float z) {
  return activate_with<F32>(s, row, z, s.bias ? s.bias[row] : 0.0f, s.lower ? s.lower[row] : 0.0f);
}

__device__ __forceinline__ float softcap(const DenseSegment& s, float z) { return s.act_pos * tanhf(z / s.act_pos); }

template <bool F32>
__device__ __forceinline__ float glu(float gate, float up) {
  return gate * (F32 ? sigmoid_exact(gate) : sigmoid_f32(gate)) * up;
}

__device__ __forceinline__ int32_t f32_key(float v) {
  if (v != v) return INT32_MIN;  // NaN never wins
  const uint32_t b = __float_as_uint(v);
  if ((b & 0x7fffffffu) == 0) return 0;
  return (b & 0x80000000u) ? -(int32_t)(b & 0x7fffffffu) : (int32_t)b;
}

// the lanes' LDS writes ahead of this are seen by all lanes' reads behind it
__device__ __forceinline__ void wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

__device__ __forceinline__ const DenseSegment& segment_of(const DenseArgs& a, int row) {
  int i = 0;
#pragma unroll
  for (int j = 1; j < kDenseSegments; ++j) i += j < a.n_seg && row >= a.start[j] ? 1 : 0;
  return a.seg[i];
}

// one output of one token (DENSE_STORE), `y0` elements into the segment's output
template <typename T>
__device__ __forceinline__ void store_one(const DenseSegment& s, int64_t y0, int64_t t, int row, float v) {
  if (s.act == DENSE_GELU && s.mul) v *= (float)reinterpret_cast<const T*>(s.mul)[t * s.ldmul + row];
  const int64_t at = y0 + t * s.ldy + row;
  if (s.y_f32) reinterpret_cast<float*>(s.y)[at] = v;
  else reinterpret_cast<T*>(s.y)[at] = (T)v;
}

// one finished sum of one token
template <typename T, int OUT>
__device__ __forceinline__ void finish_one(const DenseArgs& a, const DenseSegment& s, int64_t t, int row, float sum, int64_t y0 = 0) {
  if constexpr (OUT == DENSE_STORE) {
    store_one<T>(s, y0, t, row, activate<sizeof(T) == 4>(s, row, sum));
  } else if constexpr (OUT == DENSE_RESIDUAL) {
    const int64_t at = t * s.ldy + row;
    float* y = reinterpret_cast<float*>(s.y);
    float v = y[at] + sum;
    if (a.addend) v += a.addend[at];
    y[at] = v;
  } else {
    reinterpret_cast<float*>(s.y)[t * s.ldy + row] = s.act == DENSE_SOFTCAP ? softcap(s, sum) : sum;
  }
}

// --- one token, bfloat16 -----------------------------------------------------------------------------------
// A workgroup owns 16 rows and all of k, its wavefronts a run of k each; a load of a wavefront is four pieces of 256
// contiguous bytes of the block.  v_mfma_f32_16x16x32_bf16 with the token in every column: the matrix unit does the
// additions, and nothing but loads stands between the wavefront and memory.
// GATED: the first gate_k inputs are formed here, RMS norm of o times w times sigmoid(g) (token_ops.hip has it as a
// launch of its own for many tokens): every workgroup normalises for itself while its first weights are on their way.
template <int NW, int OUT, bool GATED>
__global__ __launch_bounds__(NW * 64) void dense_one_kernel(DenseArgs a) {
  extern __shared__ __attribute__((aligned(16))) bf16_t gated[];  // [gate_k]
  __shared__ float part[NW][16];
  __shared__ float squares[NW];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int row0 = blockIdx.x * 16;
  const DenseSegment& s = segment_of(a, row0);
  const int local = row0 - s.row0;
  if (local >= s.rows) return;  // padding
  int group = blockIdx.y;
  if (a.ids) {
    group = a.ids[blockIdx.y];
    if (group >= a.n_groups) return;
  }
  const int steps = (int)(a.k >> 5);  // even: k is a multiple of 64
  const int per = (steps + NW - 1) / NW;
  const int s0 = min(wave * per, steps), s1 = min(s0 + per, steps);
  const int r = lane & 15, c = lane >> 4;
  // piece of (row, 8-wide chunk c of step i): block (row / 32, 2 i + c / 2), lane 32 (c % 2) + row % 32
  const bf16x8_t* w = reinterpret_cast<const bf16x8_t*>(reinterpret_cast<const bf16_t*>(a.w) + group * a.w_batch) +
                      ((int64_t)(row0 >> 5) * (a.k >> 4) + (c >> 1)) * 64 + 32 * (c & 1) + (row0 & 16) + r;
  const bf16x8_t* x = reinterpret_cast<const bf16x8_t*>(reinterpret_cast<const bf16_t*>(s.x) + blockIdx.y * a.x_batch) + c;
  f32x4_t acc = {0.0f, 0.0f, 0.0f, 0.0f};
  constexpr int U = 8;
  bf16x8_t wv[U], xv[U];
  auto weights = [&](int i) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < U; ++u) wv[u] = __builtin_nontemporal_load(w + (int64_t)(i + u) * 128);
  };
  auto input = [&](int i) __attribute__((always_inline)) {
    if (GATED && i * 32 < a.gate_k) return reinterpret_cast<const bf16x8_t*>(gated)[i * 4 + c];
    return x[i * 4];
  };
  int i = s0;
  if (i + U <= s1) weights(i);
  if constexpr (GATED) {
    constexpr int NT = NW * 64;
    const bf16_t* gate = reinterpret_cast<const bf16_t*>(a.gate_g);
    float sq = 0.0f;
    for (int j = tid * 4; j < a.gate_n; j += NT * 4) {
      const f32x4_t o = *reinterpret_cast<const f32x4_t*>(a.gate_o + j);
#pragma unroll
      for (int e = 0; e < 4; ++e) sq = __builtin_fmaf(o[e], o[e], sq);
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) sq += __shfl_xor(sq, off, 64);
    if (lane == 0) squares[wave] = sq;
    __syncthreads();
    float all = 0.0f;
#pragma unroll
    for (int v = 0; v < NW; ++v) all += squares[v];
    const float inv = 1.0f / sqrtf(all / (float)a.gate_n + a.gate_eps);
    for (int j = tid * 4; j < a.gate_k; j += NT * 4) {
      bf16x4_t y = {(bf16_t)0.0f, (bf16_t)0.0f, (bf16_t)0.0f, (bf16_t)0.0f};
      if (j < a.gate_n) {
        const f32x4_t o = *reinterpret_cast<const f32x4_t*>(a.gate_o + j), gw = *reinterpret_cast<const f32x4_t*>(a.gate_w + j);
        const bf16x4_t g = *reinterpret_cast<const bf16x4_t*>(gate + j);
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = (bf16_t)(o[e] * inv * gw[e] * sigmoid_exact((float)g[e]));
      }
      *reinterpret_cast<bf16x4_t*>(gated + j) = y;
    }
    __syncthreads();
  }
  for (; i + U <= s1; i += U) {
    if (i != s0) weights(i);
#pragma unroll
    for (int u = 0; u < U; ++u) xv[u] = input(i + u);
#pragma unroll
    for (int u = 0; u < U; ++u) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[u], xv[u], acc, 0, 0, 0);
  }
  for (; i < s1; ++i)
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_nontemporal_load(w + (int64_t)i * 128), input(i), acc, 0, 0, 0);
  if (r == 0) {
#pragma unroll
    for (int j = 0; j < 4; ++j) part[wave][4 * c + j] = acc[j];
  }
  __syncthreads();
  if (tid >= 16) return;
  float sum = 0.0f;
#pragma unroll
  for (int v = 0; v < NW; ++v) sum += part[v][tid];
  const int row = local + tid;
  const int64_t y0 = blockIdx.y * a.y_batch;
  if constexpr (OUT == DENSE_STORE) {
    if (s.act == DENSE_GLU) {
      const float up = __shfl_down(sum, 8, 16);
      if (tid < 8 && local / 2 + tid < s.glu_rows) store_one<bf16_t>(s, y0, 0, local / 2 + tid, glu<false>(sum, up));
      return;
    }
  }
  if (row < s.rows) finish_one<bf16_t, OUT>(a, s, 0, row, sum, y0);
  if constexpr (OUT == DENSE_ARGMAX) {
    if (s.act == DENSE_SOFTCAP) sum = softcap(s, sum);
    unsigned long long b = row < s.rows ? awq_pack_candidate(f32_key(sum), (uint32_t)row) : 0ull;
#pragma unroll
    for (int off = 8; off > 0; off >>= 1) {
      const unsigned long long o = __shfl_xor(b, off, 16);
      b = o > b ? o : b;
    }
    if (tid == 0 && b > __hip_atomic_load(a.best, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT)) atomicMax(a.best, b);
  }
}

// --- many tokens, bfloat16 ---------------------------------------------------------------------------------
// A workgroup of four wavefronts takes 256 rows and 32 TT tokens: 64 rows per wavefront as 2 x TT accumulators of
// v_mfma_f32_32x32x16_bf16.  The weights go from memory into registers in operand order, every byte once per
// workgroup; the tokens go through LDS (global_load_lds_dwordx4, 128 bytes per token and step of 64 inputs, the
// eight 16-byte pieces of row r at positions c ^ (r & 7)).  Both are requested a step ahead.  Where the tiles do not
// fill the device, k is cut over `cuts` workgroups whose sums go to the workspace, [cut][token][row]; a second launch
// adds them in order.
constexpr int DENSE_PART = 100;
// LISTED: the tokens come from runs of a list, each with a weight block of its own.
template <int TT, int OUT, bool LISTED = false>
__global__ __launch_bounds__(256, 2) void dense_many_kernel(DenseArgs a, int row_tiles, int tok_tiles, int cuts) {
  __shared__ __attribute__((aligned(16))) bf16_t tile0[2 * 32 * TT * 64];
  bf16_t* const tile1 = tile0 + 32 * TT * 64;
  const int total = row_tiles * tok_tiles * cuts;
  // workgroups whose indices agree modulo 8 share a die: each die walks its own run of row tiles
  const int per = (total + 7) >> 3;
  const int work = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  if (work >= total) return;
  const int rc = work / tok_tiles, tile = work - rc * tok_tiles, tt0 = LISTED ? 0 : tile * 32 * TT;
  const int rt = rc / cuts, cut = rc - rt * cuts;
  int64_t group = blockIdx.y;
  int n_tok = (int)min((int64_t)1 << 30, a.M);
  const int32_t* list = nullptr;
  if constexpr (LISTED) {
    const DenseTile run = a.tiles[tile];
    if (run.count == 0) return;
    group = run.group;
    n_tok = run.count;
    list = a.list + run.first;
  }
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n = lane & 31, kh = lane >> 5;
  const DenseSegment& s = segment_of(a, rt * 256);
  const int all_steps = (int)(a.k >> 6);
  const int first_step = (int)((int64_t)all_steps * cut / cuts);
  const int steps = (int)((int64_t)all_steps * (cut + 1) / cuts) - first_step;
  const int64_t k16 = a.k >> 4;

  // this lane's pieces of the token tile
  const bf16_t* src[TT];
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    const int row = (wave * TT + i) * 8 + (lane >> 3);
    int64_t tok = min(tt0 + row, n_tok - 1);
    if constexpr (LISTED) tok = list[tok] / a.list_div;
    src[i] = reinterpret_cast<const bf16_t*>(s.x) + blockIdx.y * a.x_batch + tok * s.ldx + first_step * 64 +
             (((lane & 7) ^ (row & 7)) << 3);
  }
  auto request = [&](bf16_t* tile, int step) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < TT; ++i)
      __builtin_amdgcn_global_load_lds((gptr_t)(src[i] + step * 64), (lptr_t)(tile + (wave * TT + i) * 8 * 64), 16, 0, 0);
  };
  const bf16x8_t* wp = reinterpret_cast<const bf16x8_t*>(reinterpret_cast<const bf16_t*>(a.w) + group * a.w_batch) +
                       ((int64_t)(rt * 8 + wave * 2) * k16 + first_step * 4) * 64 + lane;
  auto weights = [&](bf16x8_t (&wv)[2][4], int step) __attribute__((always_inline)) {
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int j = 0; j < 4; ++j) wv[b][j] = wp[(b * k16 + step * 4 + j) * 64];
  };
  f32x16_t acc[2][TT];
#pragma unroll
  for (int b = 0; b < 2; ++b)
#pragma unroll
    for (int t = 0; t < TT; ++t)
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[b][t][i] = 0.0f;
  auto multiply = [&](const bf16_t* tile, const bf16x8_t (&wv)[2][4]) __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      bf16x8_t xv[TT];
#pragma unroll
      for (int t = 0; t < TT; ++t)
        xv[t] = *reinterpret_cast<const bf16x8_t*>(tile + (32 * t + n) * 64 + (((2 * j + kh) ^ (n & 7)) << 3));
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int t = 0; t < TT; ++t) acc[b][t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wv[b][j], xv[t], acc[b][t], 0, 0, 0);
    }
  };
  bf16x8_t w0[2][4], w1[2][4];
  request(tile0, 0);
  weights(w0, 0);
  for (int st = 0; st < steps; st += 2) {
    __syncthreads();  // tile0 has arrived, tile1's readers are done
    if (st + 1 < steps) {
      request(tile1, st + 1);
      weights(w1, st + 1);
    }
    multiply(tile0, w0);
    if (st + 1 < steps) {
      __syncthreads();
      if (st + 2 < steps) {
        request(tile0, st + 2);
        weights(w0, st + 2);
      }
      multiply(tile1, w1);
    }
  }
  // acc[b][t][i]: row 32 b + 8 (i / 4) + 4 kh + i % 4 of the wavefront's 64, token 32 t + n
  // A block of 32 tokens and 32 rows is turned in LDS, 4 KB of its own per wavefront, so that eight lanes hold and store the
  // rows of a token side by side; four rows (a piece) of token n are at place piece ^ (n % 8).
  const int row_w = rt * 256 + wave * 64;
  const int64_t y0 = blockIdx.y * a.y_batch;
  float* const turn = reinterpret_cast<float*>(tile0) + wave * 1024;
  __syncthreads();  // the last step's readers are done
#pragma unroll
  for (int b = 0; b < 2; ++b) {
    const DenseSegment out = segment_of(a, row_w + 32 * b);
    const int local_b = row_w + 32 * b - out.row0;
    const bool gated = OUT == DENSE_STORE && out.act == DENSE_GLU;
    const int n_rows = gated ? out.glu_rows : out.rows;
    if (OUT != DENSE_PART && local_b >= out.rows) continue;  // padding
    const bool by_four = ((out.ldy | a.y_batch) & 3) == 0 && !(OUT == DENSE_STORE && out.mul);
    // pieces of a token: 8, or 4 of a gated segment
    const int shift = gated ? 2 : 3, piece = lane & ((1 << shift) - 1);
    const int row = (gated ? local_b / 2 : local_b) + 4 * piece;
    float bias[4] = {}, lower[4] = {};  // of this lane's rows
    if (OUT == DENSE_STORE && out.bias) {
#pragma unroll
      for (int j = 0; j < 4; ++j) bias[j] = out.bias[min(row + j, n_rows - 1)];
    }
    if (OUT == DENSE_STORE && out.lower) {
#pragma unroll
      for (int j = 0; j < 4; ++j) lower[j] = out.lower[min(row + j, n_rows - 1)];
    }
#pragma unroll
    for (int t = 0; t < TT; ++t) {
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        if (gated && (g & 1)) continue;
        f32x4_t v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = gated ? glu<false>(acc[b][t][4 * g + j], acc[b][t][(4 * g + 4 + j) & 15]) : acc[b][t][4 * g + j];
        const int p = gated ? g + kh : 2 * g + kh;
        *reinterpret_cast<f32x4_t*>(turn + n * 32 + ((p ^ (n & 7)) << 2)) = v;
      }
      wave_sync();
#pragma unroll 1
      for (int token = lane >> shift; token < 32; token += 64 >> shift) {
        f32x4_t v = *reinterpret_cast<const f32x4_t*>(turn + token * 32 + ((piece ^ (token & 7)) << 2));
        int64_t tok = tt0 + 32 * t + token;
        if (tok >= n_tok) continue;
        if constexpr (LISTED) tok = list[tok];
        if constexpr (OUT == DENSE_PART) {
          *reinterpret_cast<f32x4_t*>(a.workspace + ((int64_t)cut * a.M + tok) * row_tiles * 256 + row_w + 32 * b + 4 * piece) = v;
        } else {
          if (OUT == DENSE_STORE && !gated) activate_four(out, row, v, bias, lower);
          const int64_t at = y0 + tok * out.ldy + row;
          if (row + 3 < n_rows && by_four) {
            if (OUT == DENSE_STORE && !out.y_f32) {
              *reinterpret_cast<bf16x4_t*>(reinterpret_cast<bf16_t*>(out.y) + at) =
                  bf16x4_t{(bf16_t)v[0], (bf16_t)v[1], (bf16_t)v[2], (bf16_t)v[3]};
              continue;
            }
            if (OUT == DENSE_F32 && out.act == DENSE_SOFTCAP) {
#pragma unroll
              for (int j = 0; j < 4; ++j) v[j] = softcap(out, v[j]);
            }
            f32x4_t* y = reinterpret_cast<f32x4_t*>(reinterpret_cast<float*>(out.y) + at);
            if constexpr (OUT == DENSE_RESIDUAL) {
              v = *y + v;
              if (a.addend) v = v + *reinterpret_cast<const f32x4_t*>(a.addend + at);
            }
            *y = v;
          } else {
#pragma unroll
            for (int j = 0; j < 4; ++j) {
              if (row + j >= n_rows) continue;
              if constexpr (OUT == DENSE_STORE) store_one<bf16_t>(out, y0, tok, row + j, v[j]);
              else finish_one<bf16_t, OUT>(a, out, tok, row + j, v[j]);
            }
          }
        }
      }
      wave_sync();
    }
  }
}

// adds the sums of the workgroups that shared k: a thread takes four rows of a token
template <int OUT>
__global__ __launch_bounds__(256) void dense_parts_kernel(DenseArgs a, int rows, int cuts) {
  const int row = (blockIdx.x * 256 + threadIdx.x) * 4;
  const int64_t tok = blockIdx.y;
  if (row >= rows) return;
  const DenseSegment& s = segment_of(a, row);
  const int local = row - s.row0;
  if (local >= s.rows) return;
  const f32x4_t* p = reinterpret_cast<const f32x4_t*>(a.workspace + tok * rows + row);
  const int64_t stride = a.M * rows / 4;
  f32x4_t sum = p[0];
  for (int c = 1; c < cuts; ++c) sum = sum + p[c * stride];
  if constexpr (OUT == DENSE_STORE) {
    if (s.act == DENSE_GLU) {
      if (local & 8) return;
      f32x4_t up = p[2];
      for (int c = 1; c < cuts; ++c) up = up + p[c * stride + 2];
      const int r0 = (local >> 4) * 8 + (local & 7);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (r0 + j < s.glu_rows) store_one<bf16_t>(s, 0, tok, r0 + j, glu<false>(sum[j], up[j]));
      return;
    }
  }
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (local + j < s.rows) finish_one<bf16_t, OUT>(a, s, tok, local + j, sum[j]);
}

// --- binary32 ----------------------------------------------------------------------------------------------
// one wavefront per row
template <int OUT>
__global__ __launch_bounds__(256) void dense_one_f32_kernel(DenseArgs a) {
  const int lane = threadIdx.x & 63;
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
  const DenseSegment& s = segment_of(a, row);
  const int local = row - s.row0;
  if (local >= s.rows) return;
  int group = blockIdx.y;
  if (a.ids) {
    group = a.ids[blockIdx.y];
    if (group >= a.n_groups) return;
  }
  const float* x = reinterpret_cast<const float*>(s.x) + blockIdx.y * a.x_batch;
  auto product = [&](int r) {
    const f32x4_t* w = reinterpret_cast<const f32x4_t*>(reinterpret_cast<const float*>(a.w) + group * a.w_batch + (int64_t)r * a.k);
    float acc = 0.0f;
    for (int i = lane; i < (int)(a.k >> 2); i += 64) {
      const f32x4_t wv = w[i];
#pragma unroll
      for (int j = 0; j < 4; ++j) acc = __builtin_fmaf(wv[j], x[4 * i + j], acc);
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) acc += __shfl_xor(acc, off, 64);
    return acc;
  };
  const int64_t y0 = blockIdx.y * a.y_batch;
  if constexpr (OUT == DENSE_STORE) {
    if (s.act == DENSE_GLU) {
      const int r = (local >> 4) * 8 + (local & 7);
      if ((local & 8) || r >= s.glu_rows) return;
      const float gate = product(row), up = product(row + 8);
      if (lane == 0) store_one<float>(s, y0, 0, r, glu<true>(gate, up));
      return;
    }
  }
  float acc = product(row);
  if (lane != 0) return;
  finish_one<float, OUT>(a, s, 0, local, acc, y0);
  if constexpr (OUT == DENSE_ARGMAX) {
    if (s.act == DENSE_SOFTCAP) acc = softcap(s, acc);
    atomicMax(a.best, awq_pack_candidate(f32_key(acc), (uint32_t)local));
  }
}

// 64 rows x 64 tokens per workgroup, 4 x 4 per thread, through LDS.  A thread's rows are two of an eight and the same two of
// the eight behind it: a gate and its up row meet.
template <int OUT, bool LISTED = false>
__global__ __launch_bounds__(256) void dense_many_f32_kernel(DenseArgs a) {
  __shared__ float ws[16][68], xs[16][68];
  const int tid = threadIdx.x;
  const int row0 = blockIdx.x * 64;
  const int64_t tok0 = LISTED ? 0 : (int64_t)blockIdx.y * 64;
  const DenseSegment& s = segment_of(a, row0);
  if (row0 >= a.seg[a.n_seg - 1].row0 + a.seg[a.n_seg - 1].rows) return;
  int64_t group = blockIdx.z, n_tok = a.M;
  const int32_t* list = nullptr;
  if constexpr (LISTED) {
    const DenseTile run = a.tiles[blockIdx.y];
    if (run.count == 0) return;
    group = run.group;
    n_tok = run.count;
    list = a.list + run.first;
  }
  const int lr = tid >> 2, lk = (tid & 3) * 4;
  const float* w = reinterpret_cast<const float*>(a.w) + group * a.w_batch + (int64_t)(row0 + lr) * a.k + lk;
  int64_t tok = min(tok0 + lr, n_tok - 1);
  if constexpr (LISTED) tok = list[tok] / a.list_div;
  const float* x = reinterpret_cast<const float*>(s.x) + blockIdx.z * a.x_batch + tok * s.ldx + lk;
  const int tc = (tid >> 4) * 4;
  int tr[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) tr[i] = 16 * ((tid & 15) >> 2) + 2 * (tid & 3) + (i & 1) + 8 * (i >> 1);
  float acc[4][4] = {};
  for (int k0 = 0; k0 < (int)a.k; k0 += 16) {
    const f32x4_t wv = *reinterpret_cast<const f32x4_t*>(w + k0);
    f32x4_t xv;
#pragma unroll
    for (int j = 0; j < 4; ++j) xv[j] = x[k0 + j];
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 4; ++j) ws[lk + j][lr] = wv[j], xs[lk + j][lr] = xv[j];
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = __builtin_fmaf(ws[k][tr[i]], xs[k][tc + j], acc[i][j]);
  }
  const int64_t y0 = blockIdx.z * a.y_batch;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    if (tok0 + tc + j >= n_tok) continue;
    int64_t t = tok0 + tc + j;
    if constexpr (LISTED) t = list[t];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const DenseSegment& out = segment_of(a, row0 + tr[i]);
      const int row = row0 + tr[i] - out.row0;
      if (row >= out.rows) continue;
      if constexpr (OUT == DENSE_STORE) {
        if (out.act == DENSE_GLU) {
          const int r = (row >> 4) * 8 + (row & 7);
          if (i < 2 && r < out.glu_rows) store_one<float>(out, y0, t, r, glu<true>(acc[i][j], acc[i | 2][j]));
          continue;
        }
      }
      finish_one<float, OUT>(a, out, t, row, acc[i][j], y0);
    }
  }
}

template <typename S>
__global__ __launch_bounds__(256) void dense_pack_kernel(const S* __restrict__ src, int64_t rows, int64_t cols, void* w,
                                                         int64_t k, int64_t row0, int64_t col0, int f32, int form) {
  const int64_t n = rows * cols;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
    int64_t r = i / cols, c = i % cols;
    if (form == PACK_TRANSPOSED) {
      const int64_t was = r;
      r = c;
      c = was;
    } else if (form != PACK_PLAIN) {
      r = (r >> 3) * 16 + (r & 7) + (form == PACK_UP ? 8 : 0);
    }
    r += row0;
    c += col0;
    if (f32)
      reinterpret_cast<float*>(w)[r * k + c] = (float)src[i];
    else
      reinterpret_cast<bf16_t*>(w)[(((r >> 5) * (k >> 4) + (c >> 4)) * 64 + ((c >> 3) & 1) * 32 + (r & 31)) * 8 + (c & 7)] =
          (bf16_t)(float)src[i];
  }
}

template <int OUT>
int launch_one(const DenseArgs& a, bool f32, int64_t rows, hipStream_t st) {
  if (f32) {
    hipLaunchKernelGGL(dense_one_f32_kernel<OUT>, dim3((unsigned)(rows / 4), (unsigned)a.batch), dim3(256), 0, st, a);
  } else {
    const dim3 g((unsigned)(rows / 16), (unsigned)a.batch);
    if constexpr (OUT == DENSE_RESIDUAL) {
      if (a.gate_o) {
        const size_t lds = (size_t)a.gate_k * 2;
        if (a.k > 8192) hipLaunchKernelGGL((dense_one_kernel<16, OUT, true>), g, dim3(1024), lds, st, a);
        else if (a.k > 1024) hipLaunchKernelGGL((dense_one_kernel<8, OUT, true>), g, dim3(512), lds, st, a);
        else hipLaunchKernelGGL((dense_one_kernel<4, OUT, true>), g, dim3(256), lds, st, a);
        AWQ_HIP_TRY(hipGetLastError());
        return AWQ_OK;
      }
    }
    if (a.k > 8192) hipLaunchKernelGGL((dense_one_kernel<16, OUT, false>), g, dim3(1024), 0, st, a);
    else if (a.k > 1024) hipLaunchKernelGGL((dense_one_kernel<8, OUT, false>), g, dim3(512), 0, st, a);
    else hipLaunchKernelGGL((dense_one_kernel<4, OUT, false>), g, dim3(256), 0, st, a);
  }
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

template <int OUT>
int launch_many(const DenseArgs& a, bool f32, int64_t rows, hipStream_t st) {
  if (f32) {
    hipLaunchKernelGGL(dense_many_f32_kernel<OUT>, dim3((unsigned)(rows / 64), (unsigned)((a.M + 63) / 64), (unsigned)a.batch),
                       dim3(256), 0, st, a);
  } else {
    const int row_tiles = (int)(rows / 256);
    // few weights (few rows or a short k) are read again for less: tiles of 64 tokens where those of 128 are few
    const bool small = (row_tiles <= 4 || a.k <= 512) && row_tiles * ((a.M + 127) / 128) <= 256;
    const bool wide = a.M > 64 && !small;
    const int64_t tok_tiles = wide ? (a.M + 127) / 128 : (a.M + 63) / 64;
    const int64_t tiles = row_tiles * tok_tiles;
    // two workgroups per compute unit, at least eight steps each (four in a small product)
    int64_t cuts = 1;
    if (a.workspace && a.batch == 1 && a.M <= 65535 && tiles < 384) {
      cuts = std::min<int64_t>((512 + tiles / 2) / tiles, (a.k >> 6) / (small ? 4 : 8));
      cuts = std::max<int64_t>(1, std::min<int64_t>(cuts, a.workspace_floats / (a.M * rows)));
    }
    const dim3 grid((unsigned)((tiles * cuts + 7) / 8 * 8), (unsigned)a.batch);
    if (cuts > 1) {
      if (wide)
        hipLaunchKernelGGL((dense_many_kernel<4, DENSE_PART>), grid, dim3(256), 0, st, a, row_tiles, (int)tok_tiles, (int)cuts);
      else
        hipLaunchKernelGGL((dense_many_kernel<2, DENSE_PART>), grid, dim3(256), 0, st, a, row_tiles, (int)tok_tiles, (int)cuts);
      AWQ_HIP_TRY(hipGetLastError());
      hipLaunchKernelGGL(dense_parts_kernel<OUT>, dim3((unsigned)((rows / 4 + 255) / 256), (unsigned)a.M), dim3(256), 0, st, a,
                         (int)rows, (int)cuts);
    } else if (wide) {
      hipLaunchKernelGGL((dense_many_kernel<4, OUT>), grid, dim3(256), 0, st, a, row_tiles, (int)tok_tiles, 1);
    } else {
      hipLaunchKernelGGL((dense_many_kernel<2, OUT>), grid, dim3(256), 0, st, a, row_tiles, (int)tok_tiles, 1);
    }
  }
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

// tokens with weight blocks of their own
int launch_listed(const DenseArgs& a, bool f32, int64_t rows, hipStream_t st) {
  if (f32) {
    hipLaunchKernelGGL((dense_many_f32_kernel<DENSE_STORE, true>), dim3((unsigned)(rows / 64), (unsigned)a.max_tiles), dim3(256), 0,
                       st, a);
  } else {
    const int row_tiles = (int)(rows / 256);
    const unsigned grid = (unsigned)(((int64_t)row_tiles * a.max_tiles + 7) / 8 * 8);
    if (a.tile_tokens <= 64)
      hipLaunchKernelGGL((dense_many_kernel<2, DENSE_STORE, true>), dim3(grid), dim3(256), 0, st, a, row_tiles, a.max_tiles, 1);
    else
      hipLaunchKernelGGL((dense_many_kernel<4, DENSE_STORE, true>), dim3(grid), dim3(256), 0, st, a, row_tiles, a.max_tiles, 1);
  }
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

}  // namespace

bool dense_gate_fused(int64_t n, int64_t k_padded, int64_t M, bool f32) {
  return !f32 && M == 1 && n % 4 == 0 && n > 0 && n <= k_padded && k_padded % kDenseKAlign == 0 && k_padded <= 16384;
}

int64_t dense_weight_bytes(int64_t rows_padded, int64_t k_padded, bool f32) { return rows_padded * k_padded * (f32 ? 4 : 2); }

int launch_dense_pack(const void* src, bool src_f32, int64_t rows, int64_t cols, void* w, int64_t k_padded, int64_t row0,
                      int64_t col0, bool f32, hipStream_t st, int form) {
  AWQ_REQUIRE(rows > 0 && cols > 0 && k_padded % kDenseKAlign == 0 && col0 % 8 == 0 &&
                  col0 + (form == PACK_TRANSPOSED ? rows : cols) <= k_padded,
              "bad block");
  const unsigned grid = (unsigned)std::min<int64_t>((rows * cols + 255) / 256, 65536);
  if (src_f32)
    hipLaunchKernelGGL(dense_pack_kernel<float>, dim3(grid), dim3(256), 0, st, (const float*)src, rows, cols, w, k_padded,
                       row0, col0, f32 ? 1 : 0, form);
  else
    hipLaunchKernelGGL(dense_pack_kernel<bf16_t>, dim3(grid), dim3(256), 0, st, (const bf16_t*)src, rows, cols, w, k_padded,
                       row0, col0, f32 ? 1 : 0, form);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

int launch_dense(const DenseArgs& args, bool f32, hipStream_t st) {
  DenseArgs a = args;
  AWQ_REQUIRE(a.w && a.M >= 1 && a.k > 0 && a.k % kDenseKAlign == 0, "bad product");
  AWQ_REQUIRE(a.n_seg >= 1 && a.n_seg <= kDenseSegments, "too few or too many segments");
  for (int i = 0; i < a.n_seg; ++i) {
    const DenseSegment& s = a.seg[i];
    const bool shares = i > 0 && s.x == a.seg[i - 1].x;
    AWQ_REQUIRE(s.x && s.y && s.rows > 0 && s.row0 % (shares ? kDenseSharedAlign : kDenseRowAlign) == 0 && s.ldx % 8 == 0,
                "bad segment");
    AWQ_REQUIRE(i == 0 || s.row0 >= a.seg[i - 1].row0 + a.seg[i - 1].rows, "segments overlap");
    AWQ_REQUIRE(s.act != DENSE_GLU || (a.out == DENSE_STORE && s.glu_rows > 0 && s.rows == dense_glu_rows(s.glu_rows)), "bad gated segment");
    AWQ_REQUIRE((s.act != DENSE_SIGMOID && s.act != DENSE_LOG_DECAY && s.act != DENSE_FORGET) || s.bias, "a segment lacks its bias");
    AWQ_REQUIRE(s.act != DENSE_FORGET || s.lower, "a segment lacks its lower bound");
    a.start[i] = s.row0;
  }
  AWQ_REQUIRE(!a.gate_o || (a.out == DENSE_RESIDUAL && a.n_seg == 1 && dense_gate_fused(a.gate_n, a.gate_k, a.M, f32) && a.gate_g &&
                            a.gate_w && a.gate_k <= a.k),
              "the gated norm cannot be part of this product");
  const DenseSegment& last = a.seg[a.n_seg - 1];
  const int64_t rows = round_up(last.row0 + last.rows, kDenseRowAlign);
  AWQ_REQUIRE(rows < (1ll << 30) && a.M < (1ll << 30), "too large");
  AWQ_REQUIRE(a.batch >= 1 && a.batch <= 65535 && (a.batch == 1 || (a.out == DENSE_STORE && a.w_batch % 8 == 0 && a.x_batch % 8 == 0)),
              "bad batch");
  AWQ_REQUIRE(!a.ids || (a.M == 1 && a.n_groups >= 0), "weight blocks by number take one token");
  if (a.tiles) {
    AWQ_REQUIRE(a.out == DENSE_STORE && a.list && a.list_div >= 1 && a.batch == 1 && a.max_tiles >= 1 && a.max_tiles <= 65535 &&
                    a.tile_tokens >= 1 && a.tile_tokens <= (f32 ? 64 : 128),
                "bad list of tokens");
    return launch_listed(a, f32, rows, st);
  }
  switch (a.out) {
    case DENSE_STORE: return a.M == 1 ? launch_one<DENSE_STORE>(a, f32, rows, st) : launch_many<DENSE_STORE>(a, f32, rows, st);
    case DENSE_RESIDUAL:
      return a.M == 1 ? launch_one<DENSE_RESIDUAL>(a, f32, rows, st) : launch_many<DENSE_RESIDUAL>(a, f32, rows, st);
    case DENSE_F32: return a.M == 1 ? launch_one<DENSE_F32>(a, f32, rows, st) : launch_many<DENSE_F32>(a, f32, rows, st);
    case DENSE_ARGMAX:
      AWQ_REQUIRE(a.M == 1 && a.best, "sampling takes one token");
      return launch_one<DENSE_ARGMAX>(a, f32, rows, st);
  }
  awq_set_error("launch_dense: unknown output");
  return AWQ_ERR_ARG;
}
