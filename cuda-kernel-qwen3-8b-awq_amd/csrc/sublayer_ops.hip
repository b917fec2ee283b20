// What stands around the products of a sublayer (layers.hpp): token rows, the gated and normalised sum into the residual
// stream with the next norm behind it, PolyNorm.
#include "layers.hpp"

namespace {

template <typename T, int V>
struct Vec {
  typedef T type __attribute__((ext_vector_type(V)));
};
template <typename T, int V>
__device__ __forceinline__ void read(const T* p, float (&v)[V]) {
  if constexpr (V == 1) {
    v[0] = (float)*p;
  } else {
    const typename Vec<T, V>::type r = *reinterpret_cast<const typename Vec<T, V>::type*>(p);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = (float)r[i];
  }
}
template <typename T, int V>
__device__ __forceinline__ void write(T* p, const float (&v)[V]) {
  if constexpr (V == 1) {
    *p = (T)v[0];
  } else {
    typename Vec<T, V>::type r;
#pragma unroll
    for (int i = 0; i < V; ++i) r[i] = (T)v[i];
    *reinterpret_cast<typename Vec<T, V>::type*>(p) = r;
  }
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
  return v;
}
// sum over the workgroup; `sums` has a place per wavefront and is free again behind the next barrier
__device__ __forceinline__ float group_sum(float v, float* sums) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) sums[threadIdx.x >> 6] = v;
  __syncthreads();
  float all = 0.0f;
  for (int i = 0; i < (int)(blockDim.x >> 6); ++i) all += sums[i];
  return all;
}

template <typename T, int V>
__global__ __launch_bounds__(256) void embed_tokens_kernel(const T* __restrict__ table, const T* __restrict__ side_table,
                                                           const int32_t* __restrict__ tokens, const int32_t* __restrict__ last,
                                                           PassPos pos, int64_t width, int64_t side_width, float* __restrict__ x,
                                                           T* __restrict__ side) {
  const int t = blockIdx.y;
  int64_t tok;
  if (pos.dyn) {
    tok = pos.dyn->token;
    if (tok < 0) tok = *last;
  } else {
    tok = tokens[t];
  }
  for (int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * V; i < width + side_width; i += (int64_t)gridDim.x * 256 * V) {
    float v[V];
    if (i < width) {
      read<T, V>(table + tok * width + i, v);
      write<float, V>(x + t * width + i, v);
    } else {
      read<T, V>(side_table + tok * side_width + i - width, v);
      write<T, V>(side + t * side_width + i - width, v);
    }
  }
}

// A workgroup per token; the sum, then the new residual, wait in LDS.
template <typename T, int V>
__global__ __launch_bounds__(1024) void join_kernel(JoinArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // [width]
  __shared__ float sums[2][16];
  const int tid = threadIdx.x, step = blockDim.x * V, W = (int)a.width;
  const int64_t t = blockIdx.x;
  float* const x = a.x + t * W;
  const float y_mul = a.y_gate ? 1.0f / (1.0f + expf(-a.y_gate[t])) : 1.0f;
  float sq = 0.0f;
  for (int c = tid * V; c < W; c += step) {
    float v[V] = {};
    if (a.y) {
      read<float, V>(a.y + t * W + c, v);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] *= y_mul;
    }
    for (int j = 0; j < a.top; ++j) {
      const int64_t p = t * a.top + j;
      const float w = a.weights[p];
      float u[V];
      if (a.ids[p] < a.experts) read<float, V>(a.pairs + p * W + c, u);
      else read<T, V>(reinterpret_cast<const T*>(a.h) + t * a.ldh + c, u);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] = __builtin_fmaf(w, u[i], v[i]);
    }
    if (a.gate) {
      float g[V];
      read<T, V>(reinterpret_cast<const T*>(a.gate) + t * a.ldg + c, g);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] *= g[i];
    }
#pragma unroll
    for (int i = 0; i < V; ++i) sq = __builtin_fmaf(v[i], v[i], sq);
    write<float, V>(row + c, v);
  }
  const float inv = 1.0f / sqrtf(group_sum(sq, sums[0]) / (float)W + a.eps);
  sq = 0.0f;
  for (int c = tid * V; c < W; c += step) {
    float v[V], w[V], r[V];
    read<float, V>(row + c, v);
    read<float, V>(a.w_post + c, w);
    read<float, V>(x + c, r);
#pragma unroll
    for (int i = 0; i < V; ++i) {
      r[i] = r[i] + v[i] * inv * w[i];
      sq = __builtin_fmaf(r[i], r[i], sq);
    }
    write<float, V>(x + c, r);
    if (a.out) write<float, V>(row + c, r);
  }
  if (!a.out) return;
  const float next = a.w_next ? 1.0f / sqrtf(group_sum(sq, sums[1]) / (float)W + a.eps) : 1.0f;
  T* const out = reinterpret_cast<T*>(a.out) + t * a.ldo;
  for (int c = tid * V; c < W; c += step) {
    float v[V], w[V];
    read<float, V>(row + c, v);
    if (a.w_next) {
      read<float, V>(a.w_next + c, w);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] = v[i] * next * w[i];
    }
    write<T, V>(out + c, v);
  }
}

template <typename T, int V>
__global__ __launch_bounds__(1024) void polynorm_kernel(T* z, int64_t ld, int n, const float* __restrict__ abce, float eps) {
  __shared__ float sums[3][16];
  const int tid = threadIdx.x, step = blockDim.x * V;
  z += blockIdx.x * ld;
  float s1 = 0.0f, s2 = 0.0f, s3 = 0.0f;
  for (int c = tid * V; c < n; c += step) {
    float v[V];
    read<T, V>(z + c, v);
#pragma unroll
    for (int i = 0; i < V; ++i) {
      const float q = v[i] * v[i], q2 = q * q;
      s1 += q;
      s2 += q2;
      s3 = __builtin_fmaf(q2, q, s3);
    }
  }
  s1 = wave_sum(s1);
  s2 = wave_sum(s2);
  s3 = wave_sum(s3);
  if ((tid & 63) == 0) sums[0][tid >> 6] = s1, sums[1][tid >> 6] = s2, sums[2][tid >> 6] = s3;
  __syncthreads();
  s1 = s2 = s3 = 0.0f;
  for (int i = 0; i < (int)(blockDim.x >> 6); ++i) s1 += sums[0][i], s2 += sums[1][i], s3 += sums[2][i];
  const float m = 1.0f / (float)n;
  const float a = abce[0] / sqrtf(s1 * m + eps), b = abce[1] / sqrtf(s2 * m + eps), c3 = abce[2] / sqrtf(s3 * m + eps), e = abce[3];
  for (int c = tid * V; c < n; c += step) {
    float v[V];
    read<T, V>(z + c, v);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = __builtin_fmaf(__builtin_fmaf(__builtin_fmaf(c3, v[i], b), v[i], a), v[i], e);
    write<T, V>(z + c, v);
  }
}

// a wavefront per token and head
template <typename T>
__global__ __launch_bounds__(256) void head_norm_kernel(const float* __restrict__ o, const T* __restrict__ gate, int64_t ldg,
                                                        const float* __restrict__ w, T* __restrict__ ctx, int64_t ldc, int heads,
                                                        int vdim, int64_t rows, float eps) {
  const int lane = threadIdx.x & 63;
  const int64_t at = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (at >= rows) return;
  const int64_t t = at / heads;
  const int c0 = (int)(at - t * heads) * vdim;
  o += t * heads * vdim + c0;
  float sq = 0.0f;
  for (int c = lane; c < vdim; c += 64) sq = __builtin_fmaf(o[c], o[c], sq);
  const float inv = 1.0f / sqrtf(wave_sum(sq) / (float)vdim + eps);
  for (int c = lane; c < vdim; c += 64) {
    float y = o[c] * inv * w[c];
    if (gate) {
      const float g = (float)gate[t * ldg + c0 + c];
      y *= g / (1.0f + expf(-g));
    }
    ctx[t * ldc + c0 + c] = (T)y;
  }
}

template <typename T>
void embed_tokens(const void* table, const void* side_table, const int32_t* tokens, const int32_t* last, PassPos pos, int64_t M,
                  int64_t width, int64_t side_width, float* x, void* side, hipStream_t st) {
  const bool quads = ((width | side_width) & 3) == 0;
  const dim3 g((unsigned)std::min<int64_t>((width + side_width + 1023) / (quads ? 1024 : 256), 64), (unsigned)M);
  if (quads)
    hipLaunchKernelGGL((embed_tokens_kernel<T, 4>), g, dim3(256), 0, st, (const T*)table, (const T*)side_table, tokens, last, pos, width,
                       side_width, x, (T*)side);
  else
    hipLaunchKernelGGL((embed_tokens_kernel<T, 1>), g, dim3(256), 0, st, (const T*)table, (const T*)side_table, tokens, last, pos, width,
                       side_width, x, (T*)side);
}

template <typename T>
int join(const JoinArgs& a, hipStream_t st) {
  const size_t lds = (size_t)a.width * 4;
  const bool quads = ((a.width | a.ldo | a.ldg | a.ldh) & 3) == 0;
  const dim3 g((unsigned)a.M);
  const int64_t items = a.width / (quads ? 4 : 1);
  const dim3 b((unsigned)std::min<int64_t>(a.M < 512 ? 1024 : 256, round_up(items, 64)));
  if (quads) hipLaunchKernelGGL((join_kernel<T, 4>), g, b, lds, st, a);
  else hipLaunchKernelGGL((join_kernel<T, 1>), g, b, lds, st, a);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

template <typename T>
int polynorm(void* z, int64_t ld, int64_t n, int64_t M, const float* abce, float eps, hipStream_t st) {
  const bool quads = ((n | ld) & 3) == 0;
  const dim3 b((unsigned)std::min<int64_t>(M < 512 ? 1024 : 256, round_up(n / (quads ? 4 : 1), 64)));
  if (quads) hipLaunchKernelGGL((polynorm_kernel<T, 4>), dim3((unsigned)M), b, 0, st, (T*)z, ld, (int)n, abce, eps);
  else hipLaunchKernelGGL((polynorm_kernel<T, 1>), dim3((unsigned)M), b, 0, st, (T*)z, ld, (int)n, abce, eps);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

}  // namespace

int launch_embed_tokens(const void* table, const void* side_table, bool f32, const int32_t* tokens, const int32_t* last,
                        PassPos pos, int64_t M, int64_t width, int64_t side_width, float* x, void* side, hipStream_t st) {
  AWQ_REQUIRE(table && x && (pos.dyn ? last != nullptr && M == 1 : tokens != nullptr), "bad arguments");
  AWQ_REQUIRE(M >= 1 && M <= 65535 && width >= 1 && side_width >= 0 && (side_width == 0 || (side_table && side)), "bad shape");
  if (f32) embed_tokens<float>(table, side_table, tokens, last, pos, M, width, side_width, x, side, st);
  else embed_tokens<bf16_t>(table, side_table, tokens, last, pos, M, width, side_width, x, side, st);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

int launch_join(const JoinArgs& a, bool f32, hipStream_t st) {
  AWQ_REQUIRE(a.x && a.w_post && (a.y || a.top > 0) && a.M >= 1 && a.M < (1ll << 31), "bad arguments");
  AWQ_REQUIRE(a.width >= 1 && a.width <= 16000, "width must be at most 16000");  // a row in 64 KB of LDS, sums beside it
  AWQ_REQUIRE(a.top == 0 || (a.pairs && a.ids && a.weights && a.h && a.ldh >= a.width), "bad experts");
  AWQ_REQUIRE((!a.out || a.ldo >= a.width) && (!a.gate || a.ldg >= a.width), "bad shape");
  return f32 ? join<float>(a, st) : join<bf16_t>(a, st);
}

int launch_polynorm(void* z, int64_t ld, int64_t n, int64_t M, const float* abce, float eps, bool f32, hipStream_t st) {
  AWQ_REQUIRE(z && abce && n >= 1 && n < (1 << 30) && ld >= n && M >= 1 && M < (1ll << 31), "bad arguments");
  return f32 ? polynorm<float>(z, ld, n, M, abce, eps, st) : polynorm<bf16_t>(z, ld, n, M, abce, eps, st);
}

int launch_head_norm(const float* o, const void* gate, int64_t ldg, const float* w, void* ctx, int64_t ldc, int32_t heads,
                     int32_t vdim, int64_t M, float eps, bool f32, hipStream_t st) {
  AWQ_REQUIRE(o && w && ctx && heads >= 1 && vdim >= 1 && M >= 1 && ldc >= (int64_t)heads * vdim, "bad arguments");
  const int64_t rows = M * heads;
  AWQ_REQUIRE(rows < (1ll << 32), "too large");
  const dim3 g((unsigned)((rows + 3) / 4));
  if (f32)
    hipLaunchKernelGGL(head_norm_kernel<float>, g, dim3(256), 0, st, o, (const float*)gate, ldg, w, (float*)ctx, ldc, heads, vdim,
                       rows, eps);
  else
    hipLaunchKernelGGL(head_norm_kernel<bf16_t>, g, dim3(256), 0, st, o, (const bf16_t*)gate, ldg, w, (bf16_t*)ctx, ldc, heads, vdim,
                       rows, eps);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}
