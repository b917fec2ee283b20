// Linear attention with a decaying state (layers.hpp): per head S <- decay S + k v^T, o = S^T q.
#include "layers.hpp"

namespace {

// The recurrence token by token: a wavefront holds kCols columns of the state, lane l the rows l, l + 64, ...
// of each.  Used for single tokens and for the binary32 form; the state never leaves the registers inside a pass.
constexpr int kCols = 4;

template <typename T, int DPL>
__global__ __launch_bounds__(256) void linear_step_kernel(LinearAttnArgs a) {
  const int head = blockIdx.x, lane = threadIdx.x & 63;
  const int col0 = (blockIdx.y * 4 + (threadIdx.x >> 6)) * kCols;
  if (col0 >= a.vdim) return;
  const int dimp = DPL * 64;
  float* state = a.state + ((int64_t)head * a.vdim + col0) * dimp;
  const T* p = reinterpret_cast<const T*>(a.proj);
  const T* q = p + (int64_t)head * a.dim;
  const T* k = p + (int64_t)(a.heads + head) * a.dim;
  const T* v = p + (int64_t)2 * a.heads * a.dim + (int64_t)head * a.vdim + col0;
  float* o = a.o + (int64_t)head * a.vdim + col0;
  const int64_t ldo = (int64_t)a.heads * a.vdim;
  const int nc = min(kCols, a.vdim - col0);
  const float decay = a.decay[head];
  float s[kCols][DPL];
  const bool fresh = a.pos.position() == 0;
#pragma unroll
  for (int c = 0; c < kCols; ++c)
#pragma unroll
    for (int i = 0; i < DPL; ++i) s[c][i] = fresh || c >= nc ? 0.0f : state[c * dimp + i * 64 + lane];
  for (int64_t t = 0; t < a.M; ++t) {
    float qv[DPL], kv[DPL], out[kCols];
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int d = i * 64 + lane;
      qv[i] = d < a.dim ? (float)q[t * a.ldp + d] : 0.0f;
      kv[i] = d < a.dim ? (float)k[t * a.ldp + d] : 0.0f;
    }
#pragma unroll
    for (int c = 0; c < kCols; ++c) {
      const float vv = c < nc ? (float)v[t * a.ldp + c] : 0.0f;
      out[c] = 0.0f;
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        s[c][i] = __builtin_fmaf(kv[i], vv, decay * s[c][i]);
        out[c] = __builtin_fmaf(s[c][i], qv[i], out[c]);
      }
    }
#pragma unroll
    for (int c = 0; c < kCols; ++c) {
#pragma unroll
      for (int off = 32; off > 0; off >>= 1) out[c] += __shfl_xor(out[c], off, 64);
      if (lane == c && c < nc) o[t * ldo + c] = out[c];
    }
  }
#pragma unroll
  for (int c = 0; c < kCols; ++c)
    if (c < nc)
#pragma unroll
      for (int i = 0; i < DPL; ++i) state[c * dimp + i * 64 + lane] = s[c][i];
}

template <typename T>
int launch_step(const LinearAttnArgs& a, hipStream_t st) {
  const dim3 g((unsigned)a.heads, (unsigned)((a.vdim + 4 * kCols - 1) / (4 * kCols)));
  switch ((a.dim + 63) / 64) {
    case 1: hipLaunchKernelGGL((linear_step_kernel<T, 1>), g, dim3(256), 0, st, a); break;
    case 2: hipLaunchKernelGGL((linear_step_kernel<T, 2>), g, dim3(256), 0, st, a); break;
    case 3: hipLaunchKernelGGL((linear_step_kernel<T, 3>), g, dim3(256), 0, st, a); break;
    case 4: hipLaunchKernelGGL((linear_step_kernel<T, 4>), g, dim3(256), 0, st, a); break;
    case 5: hipLaunchKernelGGL((linear_step_kernel<T, 5>), g, dim3(256), 0, st, a); break;
    case 6: hipLaunchKernelGGL((linear_step_kernel<T, 6>), g, dim3(256), 0, st, a); break;
    case 7: hipLaunchKernelGGL((linear_step_kernel<T, 7>), g, dim3(256), 0, st, a); break;
    case 8: hipLaunchKernelGGL((linear_step_kernel<T, 8>), g, dim3(256), 0, st, a); break;
    default: awq_set_error("launch_linear_attention: dim must be at most 512"); return AWQ_ERR_ARG;
  }
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

}  // namespace

int64_t linear_state_floats(int32_t heads, int32_t dim, int32_t vdim) { return (int64_t)heads * vdim * round_up(dim, 64); }

int launch_linear_attention(const LinearAttnArgs& a, bool f32, hipStream_t st) {
  AWQ_REQUIRE(a.proj && a.decay && a.state && a.o && a.M >= 1, "bad arguments");
  AWQ_REQUIRE(a.heads >= 1 && a.dim >= 1 && a.vdim >= 1 && a.vdim <= 65536 && a.ldp >= (int64_t)a.heads * (2 * a.dim + a.vdim), "bad shape");
  return f32 ? launch_step<float>(a, st) : launch_step<bf16_t>(a, st);
}
