// Linear attention whose state decays per channel (layers.hpp): per head S <- diag(decay_t) S + k_t v_t^T, o_t = S^T q_t.
#include "layers.hpp"

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
constexpr int kCols = 4;

template <typename T, int DPL, bool HEAD>
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

// Many tokens on the binary32 matrix instruction (v_mfma_f32_16x16x4_f32), C tokens (a chunk, read ahead of time) after the
// other in blocks of 16.  Inside a block, with L_t the sum of the logarithms of the decays up to and with token t (a
// number per channel), T that of all 16 and S the state ahead of the block,
//     o_t = S^T (q_t 2^L_t) + sum over s <= t of ((q_t 2^L_t) . (k_s 2^-L_s)) v_s
//     S  <- 2^T (S + sum over s of (k_s 2^-L_s) v_s^T)
// A workgroup takes 16 columns of one head's state; wavefront w the D / 4 rows from w D / 4 on, in its accumulators, for
// the state and for both sums over channels, so that nothing passes between wavefronts inside a chunk; their
// shares of the outputs are added at its end.  Operands, lane (n, j) = (lane % 16, lane / 16), step i: an accumulator holds
// rows 4 j + i of column n, and used as an operand it is just that for an order of the summed index of 4 j + i.
//     A^T[s][t] = K Q^T,  O^T[c][t] = S^T Q^T + V^T (A^T, s <= t),  S[d][c] += K^T V
// Where a channel of a block decays by more than 2^-kSafe the factors 2^-L_s could leave the range of binary32: such a
// block goes token by token, in the same accumulators.
constexpr int kBlock = 16;
constexpr float kSafe = 60.0f;

template <int D>
constexpr int chunk_tokens() { return D <= 128 ? 64 : 32; }
template <int D>
constexpr int chunk_lds() {
  constexpr int C = chunk_tokens<D>(), B = C / kBlock;
  return (2 * C * (D + 4) + C * 20 + B * D + 4 * B * 256) * 4;
}

template <typename T, int D>
__global__ __launch_bounds__(256) void gated_chunk_kernel(GatedStateArgs a) {
  constexpr int C = chunk_tokens<D>(), B = C / kBlock, S4 = D + 4;
  constexpr int NT = D / 64;              // tiles of 16 state rows per wavefront
  constexpr int TASKS = D * B / 256;      // (channel, block) pairs per thread
  constexpr int VS = 20;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* const qs = lds;                  // [C][S4]
  float* const ks = qs + C * S4;          // [C][S4]
  float* const vs = ks + C * S4;          // [C][VS]
  float* const ts = vs + C * VS;          // [B][D]: 2^T
  float* const red = ts + B * D;          // [4][B][256]
  __shared__ int unsafe[2][B];
  const int head = blockIdx.x, c0 = blockIdx.y * 16;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n = lane & 15, j4 = (lane >> 4) * 4;
  const int M = (int)a.M, nv = min(16, a.vdim - c0);
  const T* const q = reinterpret_cast<const T*>(a.q) + (int64_t)head * a.dim;
  const bool keys = a.k != nullptr;
  const T* const k = keys ? reinterpret_cast<const T*>(a.k) + (int64_t)head * a.dim : q;
  const T* const v = reinterpret_cast<const T*>(a.v) + (int64_t)head * a.vdim + c0;
  const float* const g = a.g + (int64_t)head * a.dim;
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
  if (tid < 2 * B) unsafe[tid / B][tid % B] = 0;

  // what a chunk needs, a chunk ahead
  float gr[TASKS][kBlock], vr[C / 16];
  T qr[TASKS][kBlock], kr[TASKS][kBlock];
  auto load = [&](int at) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < TASKS; ++i) {
      const int task = tid + 256 * i, d = task % D, t0 = at + task / D * kBlock;
#pragma unroll
      for (int t = 0; t < kBlock; ++t) {
        const bool there = d < a.dim && t0 + t < M;
        const int64_t tok = there ? t0 + t : 0;
        const int dd = there ? d : 0;
        gr[i][t] = g[tok * a.ldg + dd];
        qr[i][t] = q[tok * a.ldp + dd];
        kr[i][t] = k[tok * a.ldp + dd];
      }
    }
#pragma unroll
    for (int i = 0; i < C / 16; ++i) {
      const int t = at + i * 16 + (tid >> 4), c = tid & 15;
      vr[i] = t < M && c < nv ? (float)v[(int64_t)t * a.ldp + c] : 0.0f;
    }
  };
  load(0);
  __syncthreads();
  for (int at = 0, par = 0; at < M; at += C, par ^= 1) {
    float L[TASKS][kBlock];
#pragma unroll
    for (int i = 0; i < TASKS; ++i) {
      const int task = tid + 256 * i, d = task % D, t0 = at + task / D * kBlock;
      float sum = 0.0f;
#pragma unroll
      for (int t = 0; t < kBlock; ++t) {
        const bool there = d < a.dim && t0 + t < M;
        const float x = there ? gr[i][t] : 0.0f;
        gr[i][t] = x;
        // (a decay of zero: nothing of binary32 is left behind 2^-150)
        sum += keys ? fmaxf(x, -150.0f) : fmaxf(__log2f(1.0f - x), -150.0f);
        L[i][t] = sum;
      }
      if (sum < -kSafe) unsafe[par][task / D] = 1;
    }
    __syncthreads();  // the flags are whole, the previous chunk's readers are done
    if (tid < B) unsafe[par ^ 1][tid] = 0;
#pragma unroll
    for (int i = 0; i < TASKS; ++i) {
      const int task = tid + 256 * i, d = task % D, b = task / D, t0 = at + b * kBlock;
      const bool plain = unsafe[par][b] != 0;
#pragma unroll
      for (int t = 0; t < kBlock; ++t) {
        const bool there = d < a.dim && t0 + t < M;
        const float qv = there ? (float)qr[i][t] * a.q_scale : 0.0f;
        const float kv = there ? (keys ? (float)kr[i][t] : gr[i][t]) : 0.0f;
        qs[(b * kBlock + t) * S4 + d] = plain ? qv : qv * exp2f(L[i][t]);
        ks[(b * kBlock + t) * S4 + d] = plain ? kv : kv * exp2f(-L[i][t]);
      }
      ts[b * D + d] = exp2f(L[i][kBlock - 1]);
    }
#pragma unroll
    for (int i = 0; i < C / 16; ++i) vs[(i * 16 + (tid >> 4)) * VS + (tid & 15)] = vr[i];
    __syncthreads();
    if (at + C < M) load(at + C);

#pragma unroll
    for (int b = 0; b < B; ++b) {
      f32x4_t o = {0.0f, 0.0f, 0.0f, 0.0f};
      float vv[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) vv[i] = vs[(b * kBlock + j4 + i) * VS + n];
      if (unsafe[par][b] == 0) {
        f32x4_t w = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int i = 0; i < NT; ++i) {
          const f32x4_t qv = *reinterpret_cast<const f32x4_t*>(qs + (b * kBlock + n) * S4 + row0 + 16 * i + j4);
          const f32x4_t kv = *reinterpret_cast<const f32x4_t*>(ks + (b * kBlock + n) * S4 + row0 + 16 * i + j4);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            w = __builtin_amdgcn_mfma_f32_16x16x4f32(kv[e], qv[e], w, 0, 0, 0);
            o = __builtin_amdgcn_mfma_f32_16x16x4f32(s[i][e], qv[e], o, 0, 0, 0);
          }
        }
        // w[i]: key token j4 + i, query token n
#pragma unroll
        for (int i = 0; i < 4; ++i) o = __builtin_amdgcn_mfma_f32_16x16x4f32(vv[i], j4 + i <= n ? w[i] : 0.0f, o, 0, 0, 0);
#pragma unroll
        for (int i = 0; i < NT; ++i) {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            s[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(b * kBlock + j4 + e) * S4 + row0 + 16 * i + n], vv[e], s[i], 0, 0, 0);
          const f32x4_t f = *reinterpret_cast<const f32x4_t*>(ts + b * D + row0 + 16 * i + j4);
#pragma unroll
          for (int e = 0; e < 4; ++e) s[i][e] *= f[e];
        }
      } else {
        for (int t = 0; t < kBlock && at + b * kBlock + t < M; ++t) {
          const int tt = b * kBlock + t;
          const float value = vs[tt * VS + n];
          float out = 0.0f;
#pragma unroll
          for (int i = 0; i < NT; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              const int d = row0 + 16 * i + j4 + e;
              const float x = d < a.dim ? g[(int64_t)(at + tt) * a.ldg + d] : 0.0f;
              const float decay = keys ? exp2f(x) : 1.0f - x;
              s[i][e] = __builtin_fmaf(ks[tt * S4 + d], value, decay * s[i][e]);
              out = __builtin_fmaf(s[i][e], qs[tt * S4 + d], out);
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
#pragma unroll
    for (int i = 0; i < C / 64; ++i) {
      const int p = tid + 256 * i, t = p >> 2, c = (p & 3) * 4;  // four columns of a token
      f32x4_t sum = *reinterpret_cast<const f32x4_t*>(red + t * 16 + c);
#pragma unroll
      for (int w = 1; w < 4; ++w) sum = sum + *reinterpret_cast<const f32x4_t*>(red + w * B * 256 + t * 16 + c);
      if (at + t < M) {
        float* const out = a.o + ((int64_t)(at + t) * a.heads + head) * a.vdim + c0 + c;
        if (c + 3 < nv && (a.vdim & 3) == 0) {
          *reinterpret_cast<f32x4_t*>(out) = sum;
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (c + e < nv) out[e] = sum[e];
        }
      }
    }
    if (C < 64 && tid < C * 4) {
      const int t = tid >> 2, c = (tid & 3) * 4;
      f32x4_t sum = *reinterpret_cast<const f32x4_t*>(red + t * 16 + c);
#pragma unroll
      for (int w = 1; w < 4; ++w) sum = sum + *reinterpret_cast<const f32x4_t*>(red + w * B * 256 + t * 16 + c);
      if (at + t < M)
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (c + e < nv) a.o[((int64_t)(at + t) * a.heads + head) * a.vdim + c0 + c + e] = sum[e];
    }
  }
  if (n < nv)
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int d = row0 + 16 * i + j4;
      if (d < dimp) *reinterpret_cast<f32x4_t*>(state + d) = s[i];
    }
}

template <typename T, int D>
int launch_chunks(const GatedStateArgs& a, hipStream_t st) {
  static bool raised = false;  // more LDS than the default limit of a launch
  if (!raised) {
    AWQ_HIP_TRY(hipFuncSetAttribute((const void*)gated_chunk_kernel<T, D>, hipFuncAttributeMaxDynamicSharedMemorySize, chunk_lds<D>()));
    raised = true;
  }
  hipLaunchKernelGGL((gated_chunk_kernel<T, D>), dim3((unsigned)a.heads, (unsigned)((a.vdim + 15) / 16)), dim3(256), chunk_lds<D>(),
                     st, a);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

template <typename T, int DPL>
void launch_steps(const GatedStateArgs& a, hipStream_t st) {
  if (a.ctx)
    hipLaunchKernelGGL((gated_step_kernel<T, DPL, true>), dim3((unsigned)a.heads),
                       dim3((unsigned)std::min<int64_t>(1024, round_up((a.vdim + kCols - 1) / kCols * 64, 64))), (size_t)a.vdim * 4, st, a);
  else
    hipLaunchKernelGGL((gated_step_kernel<T, DPL, false>), dim3((unsigned)a.heads, (unsigned)((a.vdim + 4 * kCols - 1) / (4 * kCols))),
                       dim3(256), 0, st, a);
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
