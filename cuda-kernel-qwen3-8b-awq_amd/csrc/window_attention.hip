// Attention over a sliding window with a distance bias (layers.hpp).
#include "layers.hpp"

namespace {

__device__ __forceinline__ float temperature(const WindowAttnArgs& a, int p) {
  if (a.temp_coef == 0.0f) return 1.0f;
  return 1.0f + a.temp_coef * logf((float)floor((double)(p + 1) / a.temp_every) + 1.0f);
}

// One wavefront per (token, head of q, k or v): q normalised in place, k normalised into its cache row, v copied
// into its cache row.
template <typename T>
__global__ __launch_bounds__(256) void window_append_kernel(WindowAttnArgs a) {
  const int lane = threadIdx.x & 63, item = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int t = blockIdx.y;
  if (item >= a.heads + 2 * a.kv_heads) return;
  T* row = reinterpret_cast<T*>(a.proj) + (int64_t)t * a.ldp;
  const int pos = a.pos.position() + t;
  if (item >= a.heads + a.kv_heads) {
    const int g = item - a.heads - a.kv_heads;
    const T* v = row + (int64_t)(a.heads + a.kv_heads) * a.dim + (int64_t)g * a.vdim;
    T* dst = reinterpret_cast<T*>(a.v_cache) + ring_row(a.vl, g, pos % a.vl.slots);
    for (int d = lane; d < a.vl.row; d += 64) dst[d] = d < a.vdim ? v[d] : (T)0.0f;
    return;
  }
  T* x = row + (int64_t)item * a.dim;
  float acc = 0.0f;
  for (int d = lane; d < a.dim; d += 64) acc = __builtin_fmaf((float)x[d], (float)x[d], acc);
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) acc += __shfl_xor(acc, off, 64);
  const float inv = 1.0f / sqrtf(acc / (float)a.dim + a.eps);
  if (item < a.heads) {
    for (int d = lane; d < a.dim; d += 64) x[d] = (T)((float)x[d] * inv);
  } else {
    T* dst = reinterpret_cast<T*>(a.k_cache) + ring_row(a.kl, item - a.heads, pos % a.kl.slots);
    for (int d = lane; d < a.kl.row; d += 64) dst[d] = d < a.dim ? (T)((float)x[d] * inv) : (T)0.0f;
  }
}

// A query at a time: a workgroup per (token, head), a thread per key, blocks of 256 keys with a running maximum.
// Any sizes; the binary32 form and what the tiled kernel has no instance for.
constexpr int kMaxColsPerThread = 4;
template <typename T>
__global__ __launch_bounds__(256) void window_query_kernel(WindowAttnArgs a) {
  extern __shared__ float lds[];
  float* q = lds;              // [dim]
  float* p = lds + a.dim;      // [256]
  float* red = p + 256;        // [4]
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x;
  const int g = h / (a.heads / a.kv_heads);
  const int pos = a.pos.position() + t;
  const T* qrow = reinterpret_cast<const T*>(a.proj) + (int64_t)t * a.ldp + (int64_t)h * a.dim;
  for (int d = tid; d < a.dim; d += 256) q[d] = (float)qrow[d];
  const float mul = a.scale * temperature(a, pos), slope = a.slope[h];
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  float m = -INFINITY, l = 0.0f, acc[kMaxColsPerThread] = {};
  __syncthreads();
  for (int k0 = lo; k0 <= pos; k0 += 256) {
    const int key = k0 + tid;
    float s = -INFINITY;
    if (key <= pos) {
      const T* kr = reinterpret_cast<const T*>(a.k_cache) + ring_row(a.kl, g, key % a.kl.slots);
      float dot = 0.0f;
      for (int d = 0; d < a.dim; ++d) dot = __builtin_fmaf(q[d], (float)kr[d], dot);
      s = dot * mul - slope * (float)(pos - key);
    }
    float mx = s;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float m_new = fmaxf(m, mx), alpha = expf(m - m_new), e = expf(s - m_new);
    p[tid] = e;
    float sum = e;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) sum += __shfl_xor(sum, off, 64);
    __syncthreads();
    if ((tid & 63) == 0) red[tid >> 6] = sum;
    __syncthreads();
    l = l * alpha + ((red[0] + red[1]) + (red[2] + red[3]));
    m = m_new;
    const int n = min(256, pos + 1 - k0);
#pragma unroll
    for (int c = 0; c < kMaxColsPerThread; ++c) {
      const int col = c * 256 + tid;
      if (col < a.vdim) {
        float v = acc[c] * alpha;
        for (int j = 0; j < n; ++j)
          v = __builtin_fmaf(p[j], (float)reinterpret_cast<const T*>(a.v_cache)[ring_row(a.vl, g, (k0 + j) % a.vl.slots) + col], v);
        acc[c] = v;
      }
    }
    __syncthreads();
  }
  T* out = reinterpret_cast<T*>(a.ctx) + (int64_t)t * a.ldc + (int64_t)h * a.vdim;
#pragma unroll
  for (int c = 0; c < kMaxColsPerThread; ++c)
    if (c * 256 + tid < a.vdim) out[c * 256 + tid] = (T)(acc[c] / l);
}

template <typename T>
int launch_simple(const WindowAttnArgs& a, hipStream_t st) {
  const dim3 ga((unsigned)((a.heads + 2 * a.kv_heads + 3) / 4), (unsigned)a.M);
  hipLaunchKernelGGL(window_append_kernel<T>, ga, dim3(256), 0, st, a);
  AWQ_HIP_TRY(hipGetLastError());
  hipLaunchKernelGGL(window_query_kernel<T>, dim3((unsigned)a.heads, (unsigned)a.M), dim3(256),
                     (size_t)(a.dim + 256 + 4) * sizeof(float), st, a);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

}  // namespace

// rows are padded so that a row is whole 16-byte pieces of the matrix instructions' operands
int32_t window_row_padded(int32_t dim) { return (int32_t)round_up(dim, 32); }

int64_t window_parts_floats(int32_t heads, int32_t vdim, int64_t window, int64_t max_pos) { return 4; }
int64_t window_counter_count(int32_t heads, int32_t kv_heads) { return 4; }

int launch_window_attention(const WindowAttnArgs& a, bool f32, hipStream_t st) {
  AWQ_REQUIRE(a.proj && a.k_cache && a.v_cache && a.ctx && a.slope && a.M >= 1 && a.M <= 65535, "bad arguments");
  AWQ_REQUIRE(a.heads >= 1 && a.kv_heads >= 1 && a.heads % a.kv_heads == 0, "heads must be a multiple of kv_heads");
  AWQ_REQUIRE(a.dim >= 1 && a.dim <= 1024 && a.vdim >= 1 && a.vdim <= 256 * kMaxColsPerThread, "head sizes must be at most 1024");
  AWQ_REQUIRE(a.kl.slots > 0 && a.kl.slots % 64 == 0 && a.vl.slots == a.kl.slots && a.kl.row >= a.dim && a.vl.row >= a.vdim,
              "bad cache layout");
  return f32 ? launch_simple<float>(a, st) : launch_simple<bf16_t>(a, st);
}
