// Linear attention whose state decays per channel (layers.hpp): per head S <- diag(decay_t) S + k_t v_t^T, o_t = S^T q_t.
#include "layers.hpp"

#include <type_traits>

namespace {

typedef float f32x4_t __attribute__((ext_vector_type(4)));

// decay and key of one channel and token; without keys of its own the layer writes 1 - decay
__device__ __forceinline__ void decay_and_key(float g, bool keys, float k, float& decay, float& key) {
  decay = keys ? exp2f(g) : 1.0f - g;
  key = keys ? k : g;
}

// The recurrence token by token: a wavefront holds kCols columns of the state, lane l the rows l, l + 64, ... of each.
// HEAD: one token, a workgroup per head; the head's norm and gate are formed behind the recurrence in the same launch.
// Otherwise a workgroup takes 4 kCols columns.
template <typename T, int DPL, bool HEAD, int kCols>
__global__ __launch_bounds__(HEAD ? 1024 : 256) void gated_step_kernel(GatedStateArgs a) {
  extern __shared__ float row[];  // HEAD: [vdim]
  __shared__ float sums[16];
  const int head = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = blockDim.x >> 6;
  const int dimp = DPL * 64;
  const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)head * a.dim;
  const T* k = reinterpret_cast<const T*>(a.k) + (int64_t)head * a.dim;
  const T* v = reinterpret_cast<const T*>(a.v) + (int64_t)head * a.vdim;
  const float* g = a.g + (int64_t)head * a.dim;
  float* o = a.o + (int64_t)head * a.vdim;
  const int64_t ldo = (int64_t)a.heads * a.vdim;
  const bool keys = a.k != nullptr, fresh = a.pos.position() == 0;
  const int first = HEAD ? wave * kCols : (blockIdx.y * 4 + wave) * kCols, step = HEAD ? waves * kCols : a.vdim;
  for (int col0 = first; col0 < a.vdim; col0 += step) {
    float* state = a.state + ((int64_t)head * a.vdim + col0) * dimp;
    const int nc = min(kCols, a.vdim - col0);
    float s[kCols][DPL];
#pragma unroll
    for (int c = 0; c < kCols; ++c)
#pragma unroll
      for (int i = 0; i < DPL; ++i) s[c][i] = fresh || c >= nc ? 0.0f : state[c * dimp + i * 64 + lane];
    for (int64_t t = 0; t < a.M; ++t) {
      float qv[DPL], kv[DPL], dv[DPL], out[kCols];
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        const int d = i * 64 + lane;
        qv[i] = kv[i] = dv[i] = 0.0f;
        if (d < a.dim) {
          qv[i] = (float)q[t * a.ldp + d] * a.q_scale;
          decay_and_key(g[t * a.ldg + d], keys, keys ? (float)k[t * a.ldp + d] : 0.0f, dv[i], kv[i]);
        }
      }
#pragma unroll
      for (int c = 0; c < kCols; ++c) {
        const float vv = c < nc ? (float)v[t * a.ldp + col0 + c] : 0.0f;
        out[c] = 0.0f;
#pragma unroll
        for (int i = 0; i < DPL; ++i) {
          s[c][i] = __builtin_fmaf(kv[i], vv, dv[i] * s[c][i]);
          out[c] = __builtin_fmaf(s[c][i], qv[i], out[c]);
        }
      }
#pragma unroll
      for (int c = 0; c < kCols; ++c) {
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) out[c] += __shfl_xor(out[c], off, 64);
        if (lane == c && c < nc) {
          if constexpr (HEAD) row[col0 + c] = out[c];
          else o[t * ldo + col0 + c] = out[c];
        }
      }
    }
#pragma unroll
    for (int c = 0; c < kCols; ++c)
      if (c < nc)
#pragma unroll
        for (int i = 0; i < DPL; ++i) state[c * dimp + i * 64 + lane] = s[c][i];
  }
  if constexpr (HEAD) {
    __syncthreads();
    float sq = 0.0f;
    for (int c = threadIdx.x; c < a.vdim; c += blockDim.x) sq = __builtin_fmaf(row[c], row[c], sq);
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) sq += __shfl_xor(sq, off, 64);
    if (lane == 0) sums[wave] = sq;
    __syncthreads();
    float all = 0.0f;
    for (int i = 0; i < waves; ++i) all += sums[i];
    const float inv = 1.0f / sqrtf(all / (float)a.vdim + a.eps);
    const T* gate = reinterpret_cast<const T*>(a.gate);
    T* ctx = reinterpret_cast<T*>(a.ctx) + (int64_t)head * a.vdim;
    for (int c = threadIdx.x; c < a.vdim; c += blockDim.x) {
      float y = row[c] * inv * a.norm[c];
      if (gate) {
        const float z = (float)gate[(int64_t)head * a.vdim + c];
        y *= z / (1.0f + expf(-z));
      }
      ctx[c] = (T)y;
    }
  }
}

// Many tokens on the binary32 matrix instruction (v_mfma_f32_16x16x4_f32), C tokens (a chunk) after the other in blocks
// of 16.  Inside a block, with L_t the sum of the logarithms of the decays up to and with token t (a number per
// channel), T that of all 16, S the state ahead of the block and
//     Q_t = q_t 2^(L_t - T/2),   K_s = k_s 2^(T/2 - L_s),   R = 2^(T/2) S,
// the outputs and the state behind the block are
//     o_t = R^T Q_t + sum over s <= t of (Q_t . K_s) v_s,   S <- 2^(T/2) (R + sum over s of K_s v_s^T).
// A workgroup takes 16 columns of one head's state.  Wavefronts 4 .. 7 form a chunk's Q, K and 2^(T/2) in LDS (two channels
// and eight tokens a thread) and add up and store the outputs of the chunk before the running one, while wavefronts 0 .. 3
// go through the running one: wavefront w holds the D / 4 rows from w D / 4 on of the state in its accumulators and takes
// them for both sums over channels as well, so that nothing passes between wavefronts inside a chunk.
// Operands, lane (n, j) = (lane % 16, lane / 16), step i: an accumulator holds rows 4 j + i of column n, and used as an
// operand it is just that for an order of the summed index of 4 j + i.
//     A^T[s][t] = K Q^T,  O^T[c][t] = R^T Q^T + V^T (A^T, s <= t),  R[d][c] += K^T V
// Where a channel of a block decays by more than 2^-kSafe the factors could leave the range of binary32: such a block goes
// token by token, in the same accumulators.
constexpr int kBlock = 16;
constexpr float kSafe = 200.0f;
constexpr int kValueStride = 20;

template <typename T>
struct Pair {
  typedef T type __attribute__((ext_vector_type(2)));
};
typedef float f32x2_t __attribute__((ext_vector_type(2)));

template <int D>
constexpr int chunk_blocks() { return 256 / D; }
template <int D>
constexpr int chunk_lds() {
  constexpr int B = chunk_blocks<D>(), C = B * kBlock;
  return 2 * (2 * C * (D + 4) + C * kValueStride + B * D + 4 * B * 256) * 4;
}

// EVEN: dim is even, two channels make one load; keys: there are keys beside the decays
template <typename T, int D, bool EVEN, bool keys>
__global__ __launch_bounds__(512) void gated_chunk_kernel(GatedStateArgs a) {
  constexpr int B = chunk_blocks<D>(), C = B * kBlock, S4 = D + 4, VS = kValueStride;
  constexpr int NT = D / 64;                  // tiles of 16 state rows per wavefront
  constexpr int kHalf = kBlock / 2;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* const qs2 = lds;                     // [2][C][S4]
  float* const ks2 = qs2 + 2 * C * S4;        // [2][C][S4]
  float* const vs2 = ks2 + 2 * C * S4;        // [2][C][VS]
  float* const ts2 = vs2 + 2 * C * VS;        // [2][B][D]: 2^(T/2)
  float* const red2 = ts2 + 2 * B * D;        // [2][4][B][256]
  __shared__ int unsafe[3][B];                // of the running chunk, the one being formed, and one to be cleared
  const int head = blockIdx.x, c0 = blockIdx.y * 16;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int M = (int)a.M, nv = min(16, a.vdim - c0), chunks = (M + C - 1) / C;
  const T* const q = reinterpret_cast<const T*>(a.q) + (int64_t)head * a.dim;
  const T* const k = keys ? reinterpret_cast<const T*>(a.k) + (int64_t)head * a.dim : q;
  const T* const v = reinterpret_cast<const T*>(a.v) + (int64_t)head * a.vdim + c0;
  const float* const g = a.g + (int64_t)head * a.dim;
  if (tid < 3 * B) unsafe[tid / B][tid % B] = 0;
  __syncthreads();

  if (wave >= 4) {
    const int p = tid - 256;
    const int pair = (p >> 6) * 32 + (lane & 31), half = lane >> 5;
    const int d = (pair % (D / 2)) * 2, blk = pair / (D / 2);
    const bool has[2] = {d < a.dim, d + 1 < a.dim};
    const int dc = has[0] ? d : 0, t0 = blk * kBlock + half * kHalf;  // this thread's tokens of a chunk
    T vr[B];
    f32x2_t gr[kHalf];
    typename Pair<T>::type qr[kHalf], kr[kHalf];
    auto two = [&](const auto* x) __attribute__((always_inline)) {
      typedef typename Pair<std::remove_cv_t<std::remove_reference_t<decltype(*x)>>>::type P;
      if constexpr (EVEN) return *reinterpret_cast<const P*>(x);
      else return P{x[0], x[has[1] ? 1 : 0]};
    };
    auto load = [&](int chunk) __attribute__((always_inline)) {
      const int at = chunk * C;
#pragma unroll
      for (int t = 0; t < kHalf; ++t) {
        const int64_t tok = min(at + t0 + t, M - 1);
        gr[t] = two(g + tok * a.ldg + dc);
        qr[t] = two(q + tok * a.ldp + dc);
        if constexpr (keys) kr[t] = two(k + tok * a.ldp + dc);
      }
#pragma unroll
      for (int i = 0; i < B; ++i) vr[i] = v[(int64_t)min(at + i * 16 + (p >> 4), M - 1) * a.ldp + min(p & 15, nv - 1)];
    };
    auto form = [&](int chunk) __attribute__((always_inline)) {
      const int at = chunk * C + t0, par = chunk & 1;
      f32x2_t L[kHalf];
      float sum[2] = {0.0f, 0.0f};
#pragma unroll
      for (int t = 0; t < kHalf; ++t)
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const float x = has[e] && at + t < M ? gr[t][e] : 0.0f;
          gr[t][e] = x;
          // (a decay of zero: nothing of binary32 is left behind 2^-150)
          sum[e] += fmaxf(keys ? x : __builtin_amdgcn_logf(1.0f - x), -150.0f);
          L[t][e] = sum[e];
        }
      f32x2_t mid, ahead;  // T / 2, and what the block's first half adds to the second
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const float other = __shfl_xor(sum[e], 32, 64);
        mid[e] = 0.5f * (sum[e] + other);
        ahead[e] = half ? other : 0.0f;
      }
      if (half == 0 && fminf(mid[0], mid[1]) < -0.5f * kSafe) unsafe[chunk % 3][blk] = 1;
      float* const qs = qs2 + (par * C + t0) * S4 + d;
      float* const ks = ks2 + (par * C + t0) * S4 + d;
#pragma unroll
      for (int t = 0; t < kHalf; ++t) {
        f32x2_t qv, kv;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const bool there = has[e] && at + t < M;
          const float x = L[t][e] + ahead[e] - mid[e];
          qv[e] = (there ? (float)qr[t][e] * a.q_scale : 0.0f) * __builtin_amdgcn_exp2f(x);
          kv[e] = (keys ? (there ? (float)kr[t][e] : 0.0f) : gr[t][e]) * __builtin_amdgcn_exp2f(-x);
        }
        *reinterpret_cast<f32x2_t*>(qs + t * S4) = qv;
        *reinterpret_cast<f32x2_t*>(ks + t * S4) = kv;
      }
      if (half == 0)
        *reinterpret_cast<f32x2_t*>(ts2 + (par * B + blk) * D + d) =
            f32x2_t{__builtin_amdgcn_exp2f(mid[0]), __builtin_amdgcn_exp2f(mid[1])};
#pragma unroll
      for (int i = 0; i < B; ++i)  // (behind the last token and column: values that meet keys of zero, or are not stored)
        vs2[(par * C + i * 16 + (p >> 4)) * VS + (p & 15)] = (float)vr[i];
    };
    auto store = [&](int chunk) __attribute__((always_inline)) {
      if (p >= C * 4) return;
      const int t = p >> 2, c = (p & 3) * 4;  // four columns of a token
      const float* const red = red2 + (chunk & 1) * 4 * B * 256 + t * 16 + c;
      f32x4_t sum = *reinterpret_cast<const f32x4_t*>(red);
#pragma unroll
      for (int w = 1; w < 4; ++w) sum = sum + *reinterpret_cast<const f32x4_t*>(red + w * B * 256);
      if (chunk * C + t >= M) return;
      float* const out = a.o + ((int64_t)(chunk * C + t) * a.heads + head) * a.vdim + c0 + c;
      if (c + 3 < nv && (a.vdim & 3) == 0) {
        *reinterpret_cast<f32x4_t*>(out) = sum;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (c + e < nv) out[e] = sum[e];
      }
    };
    load(0);
    form(0);
    if (chunks > 1) load(1);
    __syncthreads();
    for (int i = 0; i < chunks; ++i) {
      if (p < B) unsafe[(i + 2) % 3][p] = 0;
      if (i + 1 < chunks) form(i + 1);
      if (i + 2 < chunks) load(i + 2);
      if (i > 0) store(i - 1);
      __syncthreads();
    }
    store(chunks - 1);
    return;
  }

  const int n = lane & 15, j4 = (lane >> 4) * 4;
  const int dimp = (a.dim + 63) & ~63;
  const int row0 = wave * (D / 4);        // this wavefront's rows of the state
  float* const state = a.state + ((int64_t)head * a.vdim + c0 + n) * dimp;
  f32x4_t s[NT];                          // s[i]: rows row0 + 16 i + j4 .. + 3 of column n
  const bool fresh = a.pos.position() == 0;
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int d = row0 + 16 * i + j4;
    s[i] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    if (!fresh && d < dimp && n < nv) s[i] = *reinterpret_cast<const f32x4_t*>(state + d);
  }
  __syncthreads();
  for (int chunk = 0; chunk < chunks; ++chunk) {
    const int par = chunk & 1;
    const float* const qs = qs2 + par * C * S4;
    const float* const ks = ks2 + par * C * S4;
    const float* const vs = vs2 + par * C * VS;
    const float* const ts = ts2 + par * B * D;
    float* const red = red2 + par * 4 * B * 256;
#pragma unroll
    for (int b = 0; b < B; ++b) {
      f32x4_t o = {0.0f, 0.0f, 0.0f, 0.0f};
      float vv[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) vv[i] = vs[(b * kBlock + j4 + i) * VS + n];
      if (unsafe[chunk % 3][b] == 0) {
        f32x4_t w = {0.0f, 0.0f, 0.0f, 0.0f}, f[NT];
#pragma unroll
        for (int i = 0; i < NT; ++i) {
          f[i] = *reinterpret_cast<const f32x4_t*>(ts + b * D + row0 + 16 * i + j4);
#pragma unroll
          for (int e = 0; e < 4; ++e) s[i][e] *= f[i][e];
          const f32x4_t qv = *reinterpret_cast<const f32x4_t*>(qs + (b * kBlock + n) * S4 + row0 + 16 * i + j4);
          const f32x4_t kv = *reinterpret_cast<const f32x4_t*>(ks + (b * kBlock + n) * S4 + row0 + 16 * i + j4);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            w = __builtin_amdgcn_mfma_f32_16x16x4f32(kv[e], qv[e], w, 0, 0, 0);
            o = __builtin_amdgcn_mfma_f32_16x16x4f32(s[i][e], qv[e], o, 0, 0, 0);
          }
        }
#pragma unroll
        for (int i = 0; i < NT; ++i) {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            s[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(b * kBlock + j4 + e) * S4 + row0 + 16 * i + n], vv[e], s[i], 0, 0, 0);
#pragma unroll
          for (int e = 0; e < 4; ++e) s[i][e] *= f[i][e];
        }
        // w[i]: key token j4 + i, query token n
#pragma unroll
        for (int i = 0; i < 4; ++i) o = __builtin_amdgcn_mfma_f32_16x16x4f32(vv[i], j4 + i <= n ? w[i] : 0.0f, o, 0, 0, 0);
      } else {
        for (int t = 0; t < kBlock && chunk * C + b * kBlock + t < M; ++t) {
          const int64_t tok = chunk * C + b * kBlock + t;
          const float value = vs[(b * kBlock + t) * VS + n];
          float out = 0.0f;
#pragma unroll
          for (int i = 0; i < NT; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              const int r = row0 + 16 * i + j4 + e;
              if (r >= a.dim) continue;
              float decay, key;
              decay_and_key(g[tok * a.ldg + r], keys, keys ? (float)k[tok * a.ldp + r] : 0.0f, decay, key);
              s[i][e] = __builtin_fmaf(key, value, decay * s[i][e]);
              out = __builtin_fmaf(s[i][e], (float)q[tok * a.ldp + r] * a.q_scale, out);
            }
          out += __shfl_xor(out, 16, 64);
          out += __shfl_xor(out, 32, 64);
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float x = __shfl(out, j4 + i, 64);
            if (n == t) o[i] = x;
          }
        }
      }
      *reinterpret_cast<f32x4_t*>(red + (wave * B + b) * 256 + n * 16 + j4) = o;
    }
    __syncthreads();
  }
  if (n < nv)
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int d = row0 + 16 * i + j4;
      if (d < dimp) *reinterpret_cast<f32x4_t*>(state + d) = s[i];
    }
}

template <typename T, int D, bool EVEN, bool KEYS>
int launch_chunk_form(const GatedStateArgs& a, hipStream_t st) {
  static bool raised = false;  // more LDS than the default limit of a launch
  if (!raised) {
    AWQ_HIP_TRY(hipFuncSetAttribute((const void*)gated_chunk_kernel<T, D, EVEN, KEYS>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                    chunk_lds<D>()));
    raised = true;
  }
  hipLaunchKernelGGL((gated_chunk_kernel<T, D, EVEN, KEYS>), dim3((unsigned)a.heads, (unsigned)((a.vdim + 15) / 16)), dim3(512),
                     chunk_lds<D>(), st, a);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}
template <typename T, int D>
int launch_chunks(const GatedStateArgs& a, hipStream_t st) {
  const uintptr_t parts = (uintptr_t)a.q | (uintptr_t)a.k;  // two values of T, two floats
  const bool even = a.dim % 2 == 0 && a.ldp % 2 == 0 && a.ldg % 2 == 0 && parts % (2 * sizeof(T)) == 0 && (uintptr_t)a.g % 8 == 0;
  if (a.k) return even ? launch_chunk_form<T, D, true, true>(a, st) : launch_chunk_form<T, D, false, true>(a, st);
  return even ? launch_chunk_form<T, D, true, false>(a, st) : launch_chunk_form<T, D, false, false>(a, st);
}

template <typename T, int DPL>
void launch_steps(const GatedStateArgs& a, hipStream_t st) {
  constexpr int kHeadCols = DPL <= 4 ? 8 : 4, kCols = 4;
  if (a.ctx)
    hipLaunchKernelGGL((gated_step_kernel<T, DPL, true, kHeadCols>), dim3((unsigned)a.heads),
                       dim3((unsigned)std::min<int64_t>(1024, (a.vdim + kHeadCols - 1) / kHeadCols * 64)), (size_t)a.vdim * 4, st, a);
  else
    hipLaunchKernelGGL((gated_step_kernel<T, DPL, false, kCols>),
                       dim3((unsigned)a.heads, (unsigned)((a.vdim + 4 * kCols - 1) / (4 * kCols))), dim3(256), 0, st, a);
}

// below this many tokens the token-by-token form is as fast
constexpr int kChunkFrom = 16;

template <typename T>
int launch(const GatedStateArgs& a, hipStream_t st) {
  if (a.M >= kChunkFrom && a.dim <= 256) {
    if (a.dim <= 64) return launch_chunks<T, 64>(a, st);
    return a.dim <= 128 ? launch_chunks<T, 128>(a, st) : launch_chunks<T, 256>(a, st);
  }
  switch ((a.dim + 63) / 64) {
    case 1: launch_steps<T, 1>(a, st); break;
    case 2: launch_steps<T, 2>(a, st); break;
    case 3: launch_steps<T, 3>(a, st); break;
    case 4: launch_steps<T, 4>(a, st); break;
    case 5: launch_steps<T, 5>(a, st); break;
    case 6: launch_steps<T, 6>(a, st); break;
    case 7: launch_steps<T, 7>(a, st); break;
    default: launch_steps<T, 8>(a, st); break;
  }
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

}  // namespace

int launch_gated_state(const GatedStateArgs& a, bool f32, hipStream_t st) {
  AWQ_REQUIRE(a.q && a.v && a.g && a.state && (a.o || a.ctx) && a.M >= 1 && a.M < (1 << 30), "bad arguments");
  AWQ_REQUIRE(a.heads >= 1 && a.heads <= 65535 && a.dim >= 1 && a.dim <= 512 && a.vdim >= 1 && a.vdim <= 8192, "bad shape");
  AWQ_REQUIRE(!a.ctx || (a.M == 1 && a.norm), "the heads' norm in the launch is for one token");
  return f32 ? launch<float>(a, st) : launch<bf16_t>(a, st);
}
