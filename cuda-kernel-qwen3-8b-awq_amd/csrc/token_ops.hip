// Per-token operators of the layers in layers.hpp: embedding with a sinusoidal position vector, grouped RMS norms
// with a causal convolution over time, a gated norm, and the end of a sampling step.
#include "layers.hpp"

namespace {

template <typename S, typename D>
__global__ __launch_bounds__(256) void convert_kernel(const S* __restrict__ src, D* __restrict__ dst, int64_t n) {
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) dst[i] = (D)(float)src[i];
}

__global__ __launch_bounds__(256) void add_rows_kernel(float* __restrict__ x, const float* __restrict__ y, int64_t n) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n) x[i] += y[i];
}

// One thread per pair of entries.  The angle is formed and brought into [-pi, pi] in binary64: at a few thousand
// positions a binary32 product would already be off by 1e-4.
template <typename T>
__global__ __launch_bounds__(256) void embed_sinusoid_kernel(const T* __restrict__ table, const int32_t* __restrict__ tokens,
                                                             const int32_t* __restrict__ last, PassPos pos, int width,
                                                             float scale, const double* __restrict__ freq,
                                                             float* __restrict__ x, float* __restrict__ keep) {
  const int t = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x;
  if (2 * i >= width) return;
  int tok;
  if (pos.dyn) {
    tok = pos.dyn->token;
    if (tok < 0) tok = *last;
  } else {
    tok = tokens[t];
  }
  const double angle = (double)(pos.position() + t) * freq[i];
  const double turns = angle * 0.15915494309189533577;  // 1 / 2 pi
  const float a = (float)((turns - rint(turns)) * 6.28318530717958647693);
  float v[2] = {sinf(a), cosf(a)};
#pragma unroll
  for (int e = 0; e < 2; ++e)
    if (2 * i + e < width) {
      const int64_t at = (int64_t)t * width + 2 * i + e;
      const float y = (float)table[(int64_t)tok * width + 2 * i + e] * scale + v[e];
      x[at] = y;
      if (keep) keep[at] = y;
    }
}

// Tokens per workgroup.  The convolution needs the norms of the taps - 1 tokens ahead of a token: the workgroup
// forms their statistics again rather than waiting for another workgroup's.
constexpr int kNormTokens = 4;

// blockIdx.x: token block, blockIdx.y: part of the vector
template <typename T>
__global__ __launch_bounds__(256) void norm_conv_kernel(NormConvArgs a) {
  extern __shared__ float inv[];  // [kNormTokens + taps - 1]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int width = (int)a.width, part = width / a.groups, c0 = blockIdx.y * part;
  const int t0 = blockIdx.x * kNormTokens, t1 = min(t0 + kNormTokens, (int)a.M);
  const int back = a.conv ? a.taps - 1 : 0;
  for (int t = t0 - back + wave; t < t1; t += 4) {
    if (t < 0) continue;
    const float* x = a.x + (int64_t)(a.rows ? a.rows[t] : t) * width + c0;
    float acc = 0.0f;
    for (int c = lane; c < part; c += 64) acc = __builtin_fmaf(x[c], x[c], acc);
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) acc += __shfl_xor(acc, off, 64);
    if (lane == 0) inv[t - t0 + back] = 1.0f / sqrtf(acc / (float)part + a.eps);
  }
  __syncthreads();
  const int pos0 = a.conv ? a.pos.position() : 0, par = a.conv ? a.pos.parity() : 0;
  const float* before = a.state[par];
  float* after = a.state[par ^ 1];
  const int keep0 = (int)a.M - back;  // tokens from here on go into the state
  for (int c = c0 + tid; c < c0 + part; c += 256) {
    const float w1 = a.w1[c], w2 = a.w2 ? a.w2[c] : 0.0f;
    auto h_at = [&](int t) -> float {  // the first norm's output at token t of the pass, or ahead of it
      if (t >= 0) return a.x[(int64_t)t * width + c] * inv[t - t0 + back] * w1;
      return pos0 + t >= 0 ? before[(int64_t)(back + t) * width + c] : 0.0f;
    };
    if (blockIdx.x == 0)
      for (int t = keep0; t < 0; ++t) after[(int64_t)(t - keep0) * width + c] = h_at(t);
    for (int t = t0; t < t1; ++t) {
      const float n = a.x[(int64_t)(a.rows ? a.rows[t] : t) * width + c] * inv[t - t0 + back];
      const float h = n * w1;
      float y = h;
      if (a.conv) {
        const float* k = a.conv + (int64_t)c * a.taps;
        for (int j = 0; j < back; ++j) y = __builtin_fmaf(k[j], h_at(t - back + j), y);
        y = __builtin_fmaf(k[back], h, y);
        if (t >= keep0) after[(int64_t)(t - keep0) * width + c] = h;
      }
      reinterpret_cast<T*>(a.out1)[(int64_t)t * a.ld + c] = (T)y;
      if (a.w2) reinterpret_cast<T*>(a.out2)[(int64_t)t * a.ld + c] = (T)(n * w2);
    }
  }
}

typedef float f32x4_t __attribute__((ext_vector_type(4)));
template <typename T>
struct Vec4;
template <>
struct Vec4<float> {
  typedef f32x4_t type;
};
template <>
struct Vec4<bf16_t> {
  typedef bf16x4_t type;
};
template <typename T>
__device__ __forceinline__ void store4(T* p, f32x4_t v) {
  typename Vec4<T>::type o;
#pragma unroll
  for (int i = 0; i < 4; ++i) o[i] = (T)v[i];
  *reinterpret_cast<typename Vec4<T>::type*>(p) = o;
}

// The same with four channels per thread and the convolution's inputs passed on in registers, for parts that are
// whole float4 and a known number of taps (0: no convolution).  `tokens` per workgroup; one token alone is reduced by
// the whole workgroup, and what does not depend on the statistic is requested ahead of it.
constexpr int kNormMaxTokens = 8;
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void norm_conv4_kernel(NormConvArgs a, int tokens) {
  constexpr int BACK = TAPS > 0 ? TAPS - 1 : 0, KN = TAPS > 0 ? TAPS : 1, HN = BACK > 0 ? BACK : 1;
  __shared__ float inv[kNormMaxTokens + BACK];
  __shared__ float sums[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nt = blockDim.x, nw = nt >> 6;
  const int width = (int)a.width, part = width / a.groups, c0 = blockIdx.y * part, quads = part >> 2;
  const int t0 = blockIdx.x * tokens, t1 = min(t0 + tokens, (int)a.M);
  auto x_row = [&](int t) { return a.x + (int64_t)(a.rows ? a.rows[t] : t) * width; };
  const int pos0 = TAPS > 0 ? a.pos.position() : 0, par = TAPS > 0 ? a.pos.parity() : 0;
  const float* before = a.state[par];
  float* after = a.state[par ^ 1];
  const int keep0 = (int)a.M - BACK;  // tokens from here on go into the state
  f32x4_t w1, w2 = {0.0f, 0.0f, 0.0f, 0.0f}, k[KN], past[HN];
  // norms' weights, taps, and the inputs ahead of the pass for channels c ..
  auto constants = [&](int c) __attribute__((always_inline)) {
    w1 = *reinterpret_cast<const f32x4_t*>(a.w1 + c);
    if (a.w2) w2 = *reinterpret_cast<const f32x4_t*>(a.w2 + c);
    if constexpr (TAPS > 0) {
      f32x4_t raw[KN];  // four channels of TAPS taps each, contiguous
#pragma unroll
      for (int i = 0; i < TAPS; ++i) raw[i] = *reinterpret_cast<const f32x4_t*>(a.conv + (int64_t)c * TAPS + 4 * i);
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) k[j][i] = raw[(i * TAPS + j) >> 2][(i * TAPS + j) & 3];
#pragma unroll
      for (int j = 0; j < BACK; ++j) {
        const int t = t0 - BACK + j;
        past[j] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
        if (t < 0 && pos0 + t >= 0) past[j] = *reinterpret_cast<const f32x4_t*>(before + (int64_t)(BACK + t) * width + c);
      }
    }
  };
  const bool once = quads <= nt;
  if (once && tid < quads) constants(c0 + 4 * tid);
  auto sum_row = [&](const float* x, int from, int by) {
    float acc = 0.0f;
    for (int q = from; q < quads; q += by) {
      const f32x4_t v = *reinterpret_cast<const f32x4_t*>(x + c0 + 4 * q);
#pragma unroll
      for (int i = 0; i < 4; ++i) acc = __builtin_fmaf(v[i], v[i], acc);
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) acc += __shfl_xor(acc, off, 64);
    return acc;
  };
  if (a.M == 1) {
    const float acc = sum_row(x_row(0), tid, nt);
    if (lane == 0) sums[wave] = acc;
    __syncthreads();
    float all = 0.0f;
    for (int w = 0; w < nw; ++w) all += sums[w];
    if (tid == 0) inv[BACK] = 1.0f / sqrtf(all / (float)part + a.eps);
  } else {
    for (int t = max(0, t0 - BACK) + wave; t < t1; t += nw) {
      const float acc = sum_row(x_row(t), lane, 64);
      if (lane == 0) inv[t - t0 + BACK] = 1.0f / sqrtf(acc / (float)part + a.eps);
    }
  }
  __syncthreads();
  for (int q = tid; q < quads; q += nt) {
    const int c = c0 + 4 * q;
    if (!once) constants(c);
    if constexpr (TAPS > 1) {
#pragma unroll
      for (int j = 0; j < BACK; ++j) {
        const int t = t0 - BACK + j;
        if (t >= 0) past[j] = *reinterpret_cast<const f32x4_t*>(x_row(t) + c) * inv[t - t0 + BACK] * w1;
      }
      if (blockIdx.x == 0)
#pragma unroll
        for (int j = 0; j < BACK; ++j)
          if (j - BACK >= keep0) *reinterpret_cast<f32x4_t*>(after + (int64_t)(j - BACK - keep0) * width + c) = past[j];
    }
    for (int t = t0; t < t1; ++t) {
      const f32x4_t n = *reinterpret_cast<const f32x4_t*>(x_row(t) + c) * inv[t - t0 + BACK];
      const f32x4_t h = n * w1;
      f32x4_t y = h;
      if constexpr (TAPS > 0) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
#pragma unroll
          for (int j = 0; j < BACK; ++j) y[i] = __builtin_fmaf(k[j][i], past[j][i], y[i]);
          y[i] = __builtin_fmaf(k[BACK][i], h[i], y[i]);
        }
        if constexpr (TAPS > 1) {
          if (t >= keep0) *reinterpret_cast<f32x4_t*>(after + (int64_t)(t - keep0) * width + c) = h;
#pragma unroll
          for (int j = 0; j + 1 < BACK; ++j) past[j] = past[j + 1];
          past[BACK - 1] = h;
        }
      }
      store4(reinterpret_cast<T*>(a.out1) + (int64_t)t * a.ld + c, y);
      if (a.w2) store4(reinterpret_cast<T*>(a.out2) + (int64_t)t * a.ld + c, n * w2);
    }
  }
}

template <typename T>
bool launch_norm4(const NormConvArgs& a, hipStream_t st) {
  const int64_t part = a.width / a.groups;
  const int taps = a.conv ? a.taps : 0;
  if (part % 4 || a.ld % 4 || taps > 8) return false;
  // (without a convolution nothing is shared between the tokens of a workgroup but the weights)
  const int tokens = a.M == 1 ? 1 : a.M >= 512 && taps > 0 ? 8 : a.M >= 64 ? 4 : 2;
  const dim3 g((unsigned)((a.M + tokens - 1) / tokens), (unsigned)a.groups);
  const dim3 b((unsigned)std::min<int64_t>(256, round_up(part / 4, 64)));
  switch (taps) {
    case 0: hipLaunchKernelGGL((norm_conv4_kernel<T, 0>), g, b, 0, st, a, tokens); break;
    case 1: hipLaunchKernelGGL((norm_conv4_kernel<T, 1>), g, b, 0, st, a, tokens); break;
    case 2: hipLaunchKernelGGL((norm_conv4_kernel<T, 2>), g, b, 0, st, a, tokens); break;
    case 3: hipLaunchKernelGGL((norm_conv4_kernel<T, 3>), g, b, 0, st, a, tokens); break;
    case 4: hipLaunchKernelGGL((norm_conv4_kernel<T, 4>), g, b, 0, st, a, tokens); break;
    case 5: hipLaunchKernelGGL((norm_conv4_kernel<T, 5>), g, b, 0, st, a, tokens); break;
    case 6: hipLaunchKernelGGL((norm_conv4_kernel<T, 6>), g, b, 0, st, a, tokens); break;
    case 7: hipLaunchKernelGGL((norm_conv4_kernel<T, 7>), g, b, 0, st, a, tokens); break;
    case 8: hipLaunchKernelGGL((norm_conv4_kernel<T, 8>), g, b, 0, st, a, tokens); break;
  }
  return true;
}

// Four elements per thread and turn; what the first kKeep turns need is requested ahead of the statistic.
template <typename T>
__global__ __launch_bounds__(1024) void gated_norm4_kernel(const float* __restrict__ o, int64_t ldo, const T* __restrict__ g,
                                                           int64_t ldg, const float* __restrict__ w, T* __restrict__ y,
                                                           int64_t ldy, int n, float eps) {
  __shared__ float sums[16];
  constexpr int kKeep = 4;
  const int tid = threadIdx.x, nt = blockDim.x, quads = n >> 2;
  o += (int64_t)blockIdx.x * ldo;
  g += (int64_t)blockIdx.x * ldg;
  y += (int64_t)blockIdx.x * ldy;
  f32x4_t ov[kKeep], wv[kKeep];
  typename Vec4<T>::type gv[kKeep];
  float acc = 0.0f;
#pragma unroll
  for (int i = 0; i < kKeep; ++i) {
    const int q = tid + i * nt;
    if (q < quads) {
      ov[i] = *reinterpret_cast<const f32x4_t*>(o + 4 * q);
      wv[i] = *reinterpret_cast<const f32x4_t*>(w + 4 * q);
      gv[i] = *reinterpret_cast<const typename Vec4<T>::type*>(g + 4 * q);
    }
  }
#pragma unroll
  for (int i = 0; i < kKeep; ++i)
    if (tid + i * nt < quads)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc = __builtin_fmaf(ov[i][j], ov[i][j], acc);
  for (int q = tid + kKeep * nt; q < quads; q += nt) {
    const f32x4_t v = *reinterpret_cast<const f32x4_t*>(o + 4 * q);
#pragma unroll
    for (int j = 0; j < 4; ++j) acc = __builtin_fmaf(v[j], v[j], acc);
  }
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) acc += __shfl_xor(acc, off, 64);
  if ((tid & 63) == 0) sums[tid >> 6] = acc;
  __syncthreads();
  float all = 0.0f;
  for (int i = 0; i < nt >> 6; ++i) all += sums[i];
  const float inv = 1.0f / sqrtf(all / (float)n + eps);
  auto finish = [&](int q, f32x4_t a, f32x4_t b, typename Vec4<T>::type c) __attribute__((always_inline)) {
    f32x4_t r;
#pragma unroll
    for (int j = 0; j < 4; ++j) r[j] = a[j] * inv * b[j] * (1.0f / (1.0f + expf(-(float)c[j])));
    store4(y + 4 * q, r);
  };
#pragma unroll
  for (int i = 0; i < kKeep; ++i)
    if (tid + i * nt < quads) finish(tid + i * nt, ov[i], wv[i], gv[i]);
  for (int q = tid + kKeep * nt; q < quads; q += nt)
    finish(q, *reinterpret_cast<const f32x4_t*>(o + 4 * q), *reinterpret_cast<const f32x4_t*>(w + 4 * q),
           *reinterpret_cast<const typename Vec4<T>::type*>(g + 4 * q));
}

template <typename T>
__global__ __launch_bounds__(256) void gated_norm_kernel(const float* __restrict__ o, int64_t ldo, const T* __restrict__ g,
                                                         int64_t ldg, const float* __restrict__ w, T* __restrict__ y,
                                                         int64_t ldy, int n, float eps) {
  __shared__ float sums[4];
  const int tid = threadIdx.x;
  o += (int64_t)blockIdx.x * ldo;
  g += (int64_t)blockIdx.x * ldg;
  y += (int64_t)blockIdx.x * ldy;
  float acc = 0.0f;
  for (int i = tid; i < n; i += 256) acc = __builtin_fmaf(o[i], o[i], acc);
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) acc += __shfl_xor(acc, off, 64);
  if ((tid & 63) == 0) sums[tid >> 6] = acc;
  __syncthreads();
  const float inv = 1.0f / sqrtf(((sums[0] + sums[1]) + (sums[2] + sums[3])) / (float)n + eps);
  for (int i = tid; i < n; i += 256) y[i] = (T)(o[i] * inv * w[i] * (1.0f / (1.0f + expf(-(float)g[i]))));
}

__global__ void take_best_kernel(unsigned long long* best, int32_t* out_token, int32_t* out_array, StepState* state,
                                 int32_t epoch_step) {
  if (threadIdx.x != 0) return;
  const int32_t tok = (int32_t)(0xffffffffu - (uint32_t)(*best & 0xffffffffull));
  *out_token = tok;
  StepState s = *state;
  if (out_array) out_array[s.out_index] = tok;
  s.pos += 1;
  s.len_lo = s.pos;
  s.len_hi = s.pos + 1;
  s.token = -1;
  s.out_index += 1;
  s.epoch += epoch_step;
  *state = s;
  *best = 0ull;
}

unsigned grid_for(int64_t n) { return (unsigned)std::max<int64_t>(1, std::min<int64_t>((n + 255) / 256, 65536)); }

}  // namespace

int launch_convert(const void* src, bool src_f32, void* dst, bool dst_f32, int64_t n, hipStream_t st) {
  AWQ_REQUIRE(src && dst && n > 0, "bad arguments");
  const dim3 g(grid_for(n)), b(256);
  if (src_f32 && dst_f32)
    hipLaunchKernelGGL((convert_kernel<float, float>), g, b, 0, st, (const float*)src, (float*)dst, n);
  else if (src_f32)
    hipLaunchKernelGGL((convert_kernel<float, bf16_t>), g, b, 0, st, (const float*)src, (bf16_t*)dst, n);
  else if (dst_f32)
    hipLaunchKernelGGL((convert_kernel<bf16_t, float>), g, b, 0, st, (const bf16_t*)src, (float*)dst, n);
  else
    hipLaunchKernelGGL((convert_kernel<bf16_t, bf16_t>), g, b, 0, st, (const bf16_t*)src, (bf16_t*)dst, n);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

int launch_embed_sinusoid(const void* table, bool f32, const int32_t* tokens, const int32_t* last, PassPos pos, int64_t M,
                          int64_t width, float scale, const double* freq, float* x, float* keep, hipStream_t st) {
  AWQ_REQUIRE(table && freq && x && (pos.dyn ? last != nullptr && M == 1 : tokens != nullptr), "bad arguments");
  AWQ_REQUIRE(M >= 1 && M <= 65535 && width >= 1 && width < (1 << 30), "bad shape");
  const dim3 g((unsigned)(((width + 1) / 2 + 255) / 256), (unsigned)M);
  if (f32)
    hipLaunchKernelGGL(embed_sinusoid_kernel<float>, g, dim3(256), 0, st, (const float*)table, tokens, last, pos, (int)width,
                       scale, freq, x, keep);
  else
    hipLaunchKernelGGL(embed_sinusoid_kernel<bf16_t>, g, dim3(256), 0, st, (const bf16_t*)table, tokens, last, pos,
                       (int)width, scale, freq, x, keep);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

int launch_norm_conv(const NormConvArgs& a, bool f32, hipStream_t st) {
  AWQ_REQUIRE(a.x && a.w1 && a.out1 && a.M >= 1 && a.M < (1 << 30), "bad arguments");
  AWQ_REQUIRE(a.groups >= 1 && a.groups <= 65535 && a.width >= a.groups && a.width % a.groups == 0 && a.ld >= a.width,
              "bad shape");
  AWQ_REQUIRE(!a.w2 || a.out2, "the second norm has no output");
  AWQ_REQUIRE(!a.conv || (a.taps >= 1 && a.taps <= 1024 && !a.rows && (a.taps == 1 || (a.state[0] && a.state[1]))),
              "bad convolution");
  if (f32 ? launch_norm4<float>(a, st) : launch_norm4<bf16_t>(a, st)) {
    AWQ_HIP_TRY(hipGetLastError());
    return AWQ_OK;
  }
  const dim3 g((unsigned)((a.M + kNormTokens - 1) / kNormTokens), (unsigned)a.groups);
  const size_t lds = sizeof(float) * (kNormTokens + (a.conv ? a.taps - 1 : 0));
  if (f32)
    hipLaunchKernelGGL(norm_conv_kernel<float>, g, dim3(256), lds, st, a);
  else
    hipLaunchKernelGGL(norm_conv_kernel<bf16_t>, g, dim3(256), lds, st, a);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

int launch_gated_norm(const float* o, int64_t ldo, const void* g, int64_t ldg, const float* w, void* y, int64_t ldy,
                      int64_t n, int64_t M, float eps, bool f32, hipStream_t st) {
  AWQ_REQUIRE(o && g && w && y && n >= 1 && n < (1 << 30) && M >= 1 && M < (1ll << 31), "bad arguments");
  if (n % 4 == 0 && ldo % 4 == 0 && ldg % 4 == 0 && ldy % 4 == 0 && ((uintptr_t)g & 15) == 0) {
    const dim3 b(M == 1 ? 1024 : 256);
    if (f32)
      hipLaunchKernelGGL(gated_norm4_kernel<float>, dim3((unsigned)M), b, 0, st, o, ldo, (const float*)g, ldg, w, (float*)y,
                         ldy, (int)n, eps);
    else
      hipLaunchKernelGGL(gated_norm4_kernel<bf16_t>, dim3((unsigned)M), b, 0, st, o, ldo, (const bf16_t*)g, ldg, w,
                         (bf16_t*)y, ldy, (int)n, eps);
    AWQ_HIP_TRY(hipGetLastError());
    return AWQ_OK;
  }
  if (f32)
    hipLaunchKernelGGL(gated_norm_kernel<float>, dim3((unsigned)M), dim3(256), 0, st, o, ldo, (const float*)g, ldg, w,
                       (float*)y, ldy, (int)n, eps);
  else
    hipLaunchKernelGGL(gated_norm_kernel<bf16_t>, dim3((unsigned)M), dim3(256), 0, st, o, ldo, (const bf16_t*)g, ldg, w,
                       (bf16_t*)y, ldy, (int)n, eps);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

int launch_add_rows(float* x, const float* y, int64_t n, hipStream_t st) {
  AWQ_REQUIRE(x && y && n > 0 && n < (1ll << 38), "bad arguments");
  hipLaunchKernelGGL(add_rows_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, st, x, y, n);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

int launch_take_best(unsigned long long* best, int32_t* out_token, int32_t* out_array, StepState* state,
                     int32_t epoch_step, hipStream_t st) {
  AWQ_REQUIRE(best && out_token && state, "bad arguments");
  hipLaunchKernelGGL(take_best_kernel, dim3(1), dim3(64), 0, st, best, out_token, out_array, state, epoch_step);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}
