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

// The same for head sizes that are whole 16-byte pieces: a group of lanes per row, 8 elements each.
__global__ __launch_bounds__(256) void window_append8_kernel(WindowAttnArgs a, int lanes) {
  const int items = a.heads + 2 * a.kv_heads;
  const int64_t at = (int64_t)blockIdx.x * (256 / lanes) + threadIdx.x / lanes;
  const int t = (int)(at / items), item = (int)(at - (int64_t)t * items), d0 = (threadIdx.x % lanes) * 8;
  if (t >= (int)a.M) return;
  bf16_t* row = reinterpret_cast<bf16_t*>(a.proj) + (int64_t)t * a.ldp;
  const int pos = a.pos.position() + t;
  const bool value = item >= a.heads + a.kv_heads;
  bf16_t* src = value ? row + (int64_t)(a.heads + a.kv_heads) * a.dim + (int64_t)(item - a.heads - a.kv_heads) * a.vdim
                      : row + (int64_t)item * a.dim;
  const int n = value ? a.vdim : a.dim;
  bf16x8_t x;
#pragma unroll
  for (int i = 0; i < 8; ++i) x[i] = (bf16_t)0.0f;
  if (d0 < n) x = *reinterpret_cast<const bf16x8_t*>(src + d0);
  float acc = 0.0f;
#pragma unroll
  for (int i = 0; i < 8; ++i) acc = __builtin_fmaf((float)x[i], (float)x[i], acc);
  for (int off = lanes >> 1; off > 0; off >>= 1) acc += __shfl_xor(acc, off, 64);
  if (value) {
    if (d0 < a.vl.row)
      *reinterpret_cast<bf16x8_t*>(reinterpret_cast<bf16_t*>(a.v_cache) +
                                   ring_row(a.vl, item - a.heads - a.kv_heads, pos % a.vl.slots) + d0) = x;
    return;
  }
  const float inv = 1.0f / sqrtf(acc / (float)a.dim + a.eps);
#pragma unroll
  for (int i = 0; i < 8; ++i) x[i] = (bf16_t)((float)x[i] * inv);
  if (item < a.heads) {
    if (d0 < a.dim) *reinterpret_cast<bf16x8_t*>(src + d0) = x;
  } else if (d0 < a.kl.row) {
    *reinterpret_cast<bf16x8_t*>(reinterpret_cast<bf16_t*>(a.k_cache) + ring_row(a.kl, item - a.heads, pos % a.kl.slots) + d0) = x;
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

// One token.  blockIdx.x: kv head and up to R of its query heads, blockIdx.y: 64 of the visible keys.  The rows a
// workgroup needs are requested before anything else; every lane group normalises the queries for itself, and the
// workgroup of the newest position takes its key and value from the projections and appends them.  A wavefront's
// lane holds the weight of one key.  With more than one part a second launch adds the parts up.
constexpr int kPartKeys = 64;

__host__ __device__ inline int window_parts(int64_t window, int64_t max_pos) {
  const int64_t n = window > 0 && window < max_pos ? window : max_pos;
  return (int)((n + kPartKeys - 1) / kPartKeys);
}

template <typename T>
struct Vec8;
template <>
struct Vec8<bf16_t> {
  bf16x8_t v;
};
template <>
struct Vec8<float> {
  typedef float f8 __attribute__((ext_vector_type(8)));
  f8 v;
};
// elements at .. at + 7 of a row of n, zeros behind it
template <typename T>
__device__ __forceinline__ void row_piece(const T* row, int at, int n, bool aligned, float (&x)[8]) {
  if (aligned && at + 8 <= n) {
    const Vec8<T> v = *reinterpret_cast<const Vec8<T>*>(row + at);
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = (float)v.v[i];
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = at + i < n ? (float)row[at + i] : 0.0f;
  }
}

// U: cache rows of a lane, row length / 32
template <typename T, int R, int U>
__global__ __launch_bounds__(256) void window_decode_kernel(WindowAttnArgs a, int chunks) {
  extern __shared__ float red[];      // [4][R][vw]
  __shared__ float sc[R][kPartKeys];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int g = blockIdx.x / chunks, rz = (blockIdx.x - g * chunks) * R;
  const int per_group = a.heads / a.kv_heads;
  const int nr = min(R, per_group - rz), h0 = g * per_group + rz;
  const int pos = a.pos.position();
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const int parts = (pos + 1 - lo + kPartKeys - 1) / kPartKeys;
  const int part = blockIdx.y;
  if (part >= parts) return;
  const int b = lo + part * kPartKeys, nk = min(kPartKeys, pos + 1 - b);
  const bool newest = part == parts - 1;
  const int kw = a.kl.row, vw = a.vl.row;
  // lanes of a key and of a value row: 8 elements each
  const int lpk = kw >> 3, sub = lane / lpk, d0 = (lane - sub * lpk) * 8, kpw = 64 / lpk, uk = kw >> 5;
  const int tpv = vw >> 3, c0 = (tid % tpv) * 8, first = tid / tpv, step = 256 / tpv, uv = vw >> 5;
  const T* const kc = reinterpret_cast<const T*>(a.k_cache);
  const T* const vc = reinterpret_cast<const T*>(a.v_cache);
  Vec8<T> kv[U], vv[U];
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int key = b + (u * 4 + wave) * kpw + sub;
    if (u < uk && key < pos) kv[u] = *reinterpret_cast<const Vec8<T>*>(kc + ring_row(a.kl, g, key % a.kl.slots) + d0);
  }
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int key = b + u * step + first;
    if (u < uv && key < pos) vv[u] = *reinterpret_cast<const Vec8<T>*>(vc + ring_row(a.vl, g, key % a.vl.slots) + c0);
  }
  const T* const proj = reinterpret_cast<const T*>(a.proj);
  const bool dim8 = (a.dim & 7) == 0, vdim8 = ((a.dim | a.vdim) & 7) == 0;
  auto normalised = [&](const T* row, float (&x)[8]) {
    row_piece(row, d0, a.dim, dim8, x);
    float acc = 0.0f;
#pragma unroll
    for (int i = 0; i < 8; ++i) acc = __builtin_fmaf(x[i], x[i], acc);
    for (int off = lpk >> 1; off > 0; off >>= 1) acc += __shfl_xor(acc, off, 64);
    const float inv = 1.0f / sqrtf(acc / (float)a.dim + a.eps);
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = (float)(T)(x[i] * inv);
  };
  float qv[R][8], kn[8] = {}, vn[8] = {};
#pragma unroll
  for (int r = 0; r < R; ++r) normalised(proj + (int64_t)(h0 + min(r, nr - 1)) * a.dim, qv[r]);
  if (newest) {
    normalised(proj + (int64_t)(a.heads + g) * a.dim, kn);
    row_piece(proj + (int64_t)(a.heads + a.kv_heads) * a.dim + (int64_t)g * a.vdim, c0, a.vdim, vdim8, vn);
    Vec8<T> out;
    if (rz == 0 && tid < lpk) {
#pragma unroll
      for (int i = 0; i < 8; ++i) out.v[i] = (T)kn[i];
      *reinterpret_cast<Vec8<T>*>(reinterpret_cast<T*>(a.k_cache) + ring_row(a.kl, g, pos % a.kl.slots) + d0) = out;
    }
    if (rz == 0 && tid < tpv) {
#pragma unroll
      for (int i = 0; i < 8; ++i) out.v[i] = (T)vn[i];
      *reinterpret_cast<Vec8<T>*>(reinterpret_cast<T*>(a.v_cache) + ring_row(a.vl, g, pos % a.vl.slots) + c0) = out;
    }
  }
  const float mul = a.scale * temperature(a, pos);
#pragma unroll
  for (int u = 0; u < U; ++u) {
    if (u >= uk) break;
    const int i = (u * 4 + wave) * kpw + sub, key = b + i;
    float x[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] = key < pos ? (float)kv[u].v[j] : kn[j];
#pragma unroll
    for (int r = 0; r < R; ++r) {
      float dot = 0.0f;
#pragma unroll
      for (int j = 0; j < 8; ++j) dot = __builtin_fmaf(qv[r][j], x[j], dot);
      for (int off = lpk >> 1; off > 0; off >>= 1) dot += __shfl_xor(dot, off, 64);
      if (d0 == 0) sc[r][i] = dot;
    }
  }
  __syncthreads();
  // every wavefront: lane = key
  float p[R], pm[R], pl[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const float s = lane < nk && r < nr ? sc[r][lane] * mul - a.slope[h0 + r] * (float)(pos - b - lane) : -INFINITY;
    float m = s;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) m = fmaxf(m, __shfl_xor(m, off, 64));
    const float e = r < nr ? expf(s - m) : 0.0f;
    float l = e;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) l += __shfl_xor(l, off, 64);
    p[r] = e;
    pm[r] = m;
    pl[r] = l;
  }
  float acc[R][8] = {};
#pragma unroll
  for (int u = 0; u < U; ++u) {
    if (u >= uv) break;
    const int i = u * step + first;
    float x[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] = b + i < pos ? (float)vv[u].v[j] : vn[j];
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const float w = __shfl(p[r], i, 64);
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[r][j] = __builtin_fmaf(w, i < nk ? x[j] : 0.0f, acc[r][j]);
    }
  }
  // lanes of a wavefront that share columns, then the wavefronts
#pragma unroll
  for (int r = 0; r < R; ++r)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      for (int off = tpv; off < 64; off <<= 1) acc[r][j] += __shfl_xor(acc[r][j], off, 64);
      if (lane < tpv) red[(wave * R + r) * vw + c0 + j] = acc[r][j];
    }
  __syncthreads();
  const int n_parts = gridDim.y;
#pragma unroll
  for (int r = 0; r < R; ++r) {
    if (r >= nr) break;
    float* const mine = a.parts + ((int64_t)(h0 + r) * n_parts + part) * (2 + a.vdim);
    for (int c = tid; c < a.vdim; c += 256) {
      const float x = (red[r * vw + c] + red[(R + r) * vw + c]) + (red[(2 * R + r) * vw + c] + red[(3 * R + r) * vw + c]);
      if (n_parts == 1)
        reinterpret_cast<T*>(a.ctx)[(int64_t)(h0 + r) * a.vdim + c] = (T)(x / pl[r]);
      else
        mine[2 + c] = x;
    }
    if (n_parts > 1 && tid == 0) mine[0] = pm[r], mine[1] = pl[r];
  }
}

// a workgroup per head; a part is [maximum, sum, context]
template <typename T>
__global__ __launch_bounds__(256) void window_combine_kernel(WindowAttnArgs a, int n_parts) {
  __shared__ float red[256];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63;
  const int pos = a.pos.position();
  const int parts = ((a.window > 0 ? min(a.window, pos + 1) : pos + 1) + kPartKeys - 1) / kPartKeys;
  const int64_t ps = 2 + a.vdim;
  const float* p = a.parts + (int64_t)h * n_parts * ps;
  float m = -INFINITY, l = 0.0f;
  for (int s = lane; s < parts; s += 64) m = fmaxf(m, p[s * ps]);
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) m = fmaxf(m, __shfl_xor(m, off, 64));
  for (int s = lane; s < parts; s += 64) l = __builtin_fmaf(expf(p[s * ps] - m), p[s * ps + 1], l);
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) l += __shfl_xor(l, off, 64);
  // columns, and as many runs of parts next to each other as there are threads left
  const int cols = min(256, a.vdim), runs = 256 / cols, run = tid / cols;
  for (int c = tid % cols; c < (a.vdim + cols - 1) / cols * cols; c += cols) {
    float x = 0.0f;
    if (run < runs && c < a.vdim)
#pragma unroll 4
      for (int s = run; s < parts; s += runs) x = __builtin_fmaf(expf(p[s * ps] - m), p[s * ps + 2 + c], x);
    red[tid] = x;
    __syncthreads();
    if (run == 0 && c < a.vdim) {
      for (int i = 1; i < runs; ++i) x += red[tid + i * cols];
      reinterpret_cast<T*>(a.ctx)[(int64_t)h * a.vdim + c] = (T)(x / l);
    }
    __syncthreads();
  }
}

template <typename T, int R>
int launch_decode_rows(const WindowAttnArgs& a, hipStream_t st) {
  const int chunks = (a.heads / a.kv_heads + R - 1) / R;
  const int parts = window_parts(a.window, a.len_bound);
  AWQ_REQUIRE(parts >= 1 && parts <= 65535, "too many keys");
  const dim3 g((unsigned)(a.kv_heads * chunks), (unsigned)parts);
  const size_t lds = sizeof(float) * 4 * R * a.vl.row;
  const int row = std::max(a.kl.row, a.vl.row);
  if (row == 64) hipLaunchKernelGGL((window_decode_kernel<T, R, 2>), g, dim3(256), lds, st, a, chunks);
  else if (row == 128) hipLaunchKernelGGL((window_decode_kernel<T, R, 4>), g, dim3(256), lds, st, a, chunks);
  else hipLaunchKernelGGL((window_decode_kernel<T, R, 8>), g, dim3(256), lds, st, a, chunks);
  AWQ_HIP_TRY(hipGetLastError());
  if (parts > 1) {
    hipLaunchKernelGGL(window_combine_kernel<T>, dim3((unsigned)a.heads), dim3(256), 0, st, a, parts);
    AWQ_HIP_TRY(hipGetLastError());
  }
  return AWQ_OK;
}

template <typename T>
int launch_decode(const WindowAttnArgs& a, hipStream_t st) {
  const int per = a.heads / a.kv_heads;
  if (per == 1) return launch_decode_rows<T, 1>(a, st);
  if (per == 2) return launch_decode_rows<T, 2>(a, st);
  if (per <= 4) return launch_decode_rows<T, 4>(a, st);
  return launch_decode_rows<T, 8>(a, st);
}

// Many tokens, bfloat16.  128 queries of one head per workgroup, 32 per wavefront; keys and values of 32 positions at
// a time go through LDS.  Operands of v_mfma_f32_32x32x16_bf16, lane (n, kh) = (lane % 32, lane / 32), queries as
// columns throughout:
//     S^T[key][query] = K Q^T,   O^T[c][query] += V^T P^T
// so that a query's maximum, sum and rescaling stay in a lane and its partner, and the weights a lane forms are the
// elements it supplies to the second product (slice j: keys 16 j + 8 (e / 4) + 4 kh + e % 4; V^T by the transposing
// LDS read).  Scores and weights are binary32; a weight enters the product as the sum of two bfloat16 terms.
typedef float f32x16_t __attribute__((ext_vector_type(16)));
typedef short short4_t __attribute__((ext_vector_type(4)));
constexpr int kTileQueries = 128, kTileKeys = 32;

template <int DK, int DV>
__global__ __launch_bounds__(256, (DK + DV > 256) ? 1 : 2) void window_tile_kernel(WindowAttnArgs a) {
  constexpr int KS = DK + 8, VS = DV + 16;
  constexpr int KP = DK / 64, VP = DV / 64;  // 16-byte pieces of a tile per thread
  __shared__ __attribute__((aligned(16))) bf16_t ks2[2 * kTileKeys * KS];
  __shared__ __attribute__((aligned(16))) bf16_t vs2[2 * kTileKeys * VS];
  const int h = blockIdx.x, g = h / (a.heads / a.kv_heads);
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n = lane & 31, kh = lane >> 5;
  const int M = (int)a.M, pos0 = a.pos.pos0;
  const int q_first = blockIdx.y * kTileQueries;
  const int qi = q_first + wave * 32 + n, qc = min(qi, M - 1);
  const int pq = pos0 + qc;  // this lane's position
  auto oldest = [&](int p) { return a.window > 0 ? max(0, p - a.window + 1) : 0; };
  const int w_first = pos0 + min(q_first + wave * 32, M - 1), w_last = pos0 + min(q_first + wave * 32 + 31, M - 1);
  const int lo_q = oldest(pq), lo_wave = oldest(w_first), lo_full = oldest(w_last);
  const int k_begin = oldest(pos0 + q_first) & ~(kTileKeys - 1);
  const int k_end = pos0 + min(q_first + kTileQueries - 1, M - 1) + 1;

  const bf16_t* q = reinterpret_cast<const bf16_t*>(a.proj) + (int64_t)qc * a.ldp + (int64_t)h * a.dim;
  bf16x8_t qop[DK / 16];
#pragma unroll
  for (int s = 0; s < DK / 16; ++s) {
    const int at = 16 * s + 8 * kh;
    if (a.dim == DK) {
      qop[s] = *reinterpret_cast<const bf16x8_t*>(q + at);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) qop[s][e] = at + e < a.dim ? q[at + e] : (bf16_t)0.0f;
    }
  }
  f32x16_t o[DV / 32];
#pragma unroll
  for (int d = 0; d < DV / 32; ++d)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[d][i] = 0.0f;
  float m_run = -1e30f, l_run = 0.0f;
  constexpr float kLog2e = 1.44269504088896340736f;
  const float mul = a.scale * temperature(a, pq) * kLog2e, slope = a.slope[h] * kLog2e;

  const bf16_t* const kc = reinterpret_cast<const bf16_t*>(a.k_cache);
  const bf16_t* const vc = reinterpret_cast<const bf16_t*>(a.v_cache);
  struct TileRegs {
    bf16x8_t k[KP > 0 ? KP : 1], v[VP > 0 ? VP : 1];
  };
  TileRegs ra, rb;
  auto load_tile = [&](int k0, TileRegs& r) __attribute__((always_inline)) {
    if (k0 >= k_end) return;
    const int slot = k0 % a.kl.slots;  // 32 positions from a multiple of 32 on never wrap
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int pc = tid + i * 256, key = pc / (DK / 8), at = (pc % (DK / 8)) * 8;
      r.k[i] = *reinterpret_cast<const bf16x8_t*>(kc + ring_row(a.kl, g, slot + key) + at);
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int pc = tid + i * 256, key = pc / (DV / 8), at = (pc % (DV / 8)) * 8;
      r.v[i] = *reinterpret_cast<const bf16x8_t*>(vc + ring_row(a.vl, g, slot + key) + at);
    }
  };
  auto store_tile = [&](int half, const TileRegs& r) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int pc = tid + i * 256, key = pc / (DK / 8), at = (pc % (DK / 8)) * 8;
      *reinterpret_cast<bf16x8_t*>(ks2 + (half * kTileKeys + key) * KS + at) = r.k[i];
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int pc = tid + i * 256, key = pc / (DV / 8), at = (pc % (DV / 8)) * 8;
      *reinterpret_cast<bf16x8_t*>(vs2 + (half * kTileKeys + key) * VS + at) = r.v[i];
    }
  };
  auto step = [&](int k0, int half) __attribute__((always_inline)) {
    if (k0 > w_last || k0 + kTileKeys <= lo_wave) return;  // no query of this wavefront sees a key of the tile
    const bf16_t* ks = ks2 + half * kTileKeys * KS;
    const bf16_t* vs = vs2 + half * kTileKeys * VS;
    f32x16_t s;
#pragma unroll
    for (int i = 0; i < 16; ++i) s[i] = 0.0f;
#pragma unroll
    for (int d = 0; d < DK / 16; ++d)
      s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8_t*>(ks + n * KS + 16 * d + 8 * kh), qop[d], s,
                                                  0, 0, 0);
    // s[i]: key k0 + 8 (i / 4) + 4 kh + i % 4 for this lane's query
    const int base = k0 + 4 * kh - pq;
#pragma unroll
    for (int i = 0; i < 16; ++i) s[i] = __builtin_fmaf(s[i], mul, slope * (float)(base + 8 * (i >> 2) + (i & 3)));
    if (k0 + kTileKeys - 1 > w_first || k0 < lo_full) {
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int key = k0 + 8 * (i >> 2) + 4 * kh + (i & 3);
        s[i] = key <= pq && key >= lo_q ? s[i] : -INFINITY;
      }
    }
    float mx = s[0];
#pragma unroll
    for (int i = 1; i < 16; ++i) mx = fmaxf(mx, s[i]);
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float m_new = fmaxf(m_run, mx);
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
    float rs = 0.0f;
    bf16x8_t hi[2], lo[2];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const float p = __builtin_amdgcn_exp2f(s[i] - m_new);
      rs += p;
      hi[i >> 3][i & 7] = (bf16_t)p;
      lo[i >> 3][i & 7] = (bf16_t)(p - (float)hi[i >> 3][i & 7]);
    }
    rs += __shfl_xor(rs, 32, 64);
    l_run = l_run * alpha + rs;
    m_run = m_new;
    if (__builtin_amdgcn_ballot_w64(alpha != 1.0f) != 0) {
#pragma unroll
      for (int d = 0; d < DV / 32; ++d)
#pragma unroll
        for (int i = 0; i < 16; ++i) o[d][i] *= alpha;
    }
    const int L16 = lane & 15;
    const bf16_t* vlane = vs + (4 * kh + (L16 >> 2)) * VS + 16 * ((lane >> 4) & 1) + 4 * (L16 & 3);
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int d = 0; d < DV / 32; ++d) {
        const bf16_t* vp = vlane + 16 * j * VS + d * 32;
        const short4_t l = __builtin_amdgcn_ds_read_tr16_b64_v4i16((short4_t __attribute__((address_space(3)))*)vp);
        const short4_t u = __builtin_amdgcn_ds_read_tr16_b64_v4i16((short4_t __attribute__((address_space(3)))*)(vp + 8 * VS));
        const bf16x4_t l4 = __builtin_bit_cast(bf16x4_t, l), u4 = __builtin_bit_cast(bf16x4_t, u);
        const bf16x8_t vv = {l4[0], l4[1], l4[2], l4[3], u4[0], u4[1], u4[2], u4[3]};
        o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vv, hi[j], o[d], 0, 0, 0);
        o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vv, lo[j], o[d], 0, 0, 0);
      }
  };
  load_tile(k_begin, ra);
  load_tile(k_begin + kTileKeys, rb);
  for (int k0 = k_begin; k0 < k_end; k0 += 2 * kTileKeys) {
    __syncthreads();  // the previous tiles' readers are done
    store_tile(0, ra);
    if (k0 + kTileKeys < k_end) store_tile(1, rb);
    __syncthreads();
    load_tile(k0 + 2 * kTileKeys, ra);
    load_tile(k0 + 3 * kTileKeys, rb);
    step(k0, 0);
    if (k0 + kTileKeys < k_end) step(k0 + kTileKeys, 1);
  }
  if (qi >= M) return;
  // o[d][i]: column 32 d + 8 (i / 4) + 4 kh + i % 4
  const float inv = 1.0f / l_run;
  bf16_t* out = reinterpret_cast<bf16_t*>(a.ctx) + (int64_t)qi * a.ldc + (int64_t)h * a.vdim;
#pragma unroll
  for (int d = 0; d < DV / 32; ++d)
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = 32 * d + 8 * u + 4 * kh;
      if (c + 3 < a.vdim && (a.vdim & 3) == 0) {
        bf16x4_t v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = (bf16_t)(o[d][4 * u + j] * inv);
        *reinterpret_cast<bf16x4_t*>(out + c) = v;
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c + j < a.vdim) out[c + j] = (bf16_t)(o[d][4 * u + j] * inv);
      }
    }
}

template <int DK>
void launch_tiles(const WindowAttnArgs& a, hipStream_t st) {
  const dim3 g((unsigned)a.heads, (unsigned)((a.M + kTileQueries - 1) / kTileQueries));
  if (a.vl.row == 64) hipLaunchKernelGGL((window_tile_kernel<DK, 64>), g, dim3(256), 0, st, a);
  else if (a.vl.row == 128) hipLaunchKernelGGL((window_tile_kernel<DK, 128>), g, dim3(256), 0, st, a);
  else hipLaunchKernelGGL((window_tile_kernel<DK, 256>), g, dim3(256), 0, st, a);
}

template <typename T>
int launch_append(const WindowAttnArgs& a, hipStream_t st) {
  const int row = std::max(a.kl.row, a.vl.row);
  if (sizeof(T) == 2 && ((a.dim | a.vdim) & 7) == 0 && row <= 256) {
    const int lanes = row / 8, per = 256 / lanes;
    const int64_t n = (int64_t)(a.heads + 2 * a.kv_heads) * a.M;
    hipLaunchKernelGGL(window_append8_kernel, dim3((unsigned)((n + per - 1) / per)), dim3(256), 0, st, a, lanes);
    AWQ_HIP_TRY(hipGetLastError());
    return AWQ_OK;
  }
  const dim3 g((unsigned)((a.heads + 2 * a.kv_heads + 3) / 4), (unsigned)a.M);
  hipLaunchKernelGGL(window_append_kernel<T>, g, dim3(256), 0, st, a);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

template <typename T>
int launch_queries(const WindowAttnArgs& a, hipStream_t st) {
  hipLaunchKernelGGL(window_query_kernel<T>, dim3((unsigned)a.heads, (unsigned)a.M), dim3(256),
                     (size_t)(a.dim + 256 + 4) * sizeof(float), st, a);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

}  // namespace

// the tiled and the one-token kernel have rows of 64, 128 or 256 elements; longer ones go a query at a time
int32_t window_row_padded(int32_t dim) { return dim <= 64 ? 64 : dim <= 128 ? 128 : (int32_t)round_up(dim, 256); }

int64_t window_parts_floats(int32_t heads, int32_t vdim, int64_t window, int64_t max_pos) {
  return (int64_t)heads * window_parts(window, max_pos) * (2 + vdim);
}

int launch_window_attention(const WindowAttnArgs& a, bool f32, hipStream_t st) {
  AWQ_REQUIRE(a.proj && a.k_cache && a.v_cache && a.ctx && a.slope && a.M >= 1 && a.M <= 65535, "bad arguments");
  AWQ_REQUIRE(a.heads >= 1 && a.kv_heads >= 1 && a.heads % a.kv_heads == 0, "heads must be a multiple of kv_heads");
  AWQ_REQUIRE(a.dim >= 1 && a.dim <= 1024 && a.vdim >= 1 && a.vdim <= 256 * kMaxColsPerThread, "head sizes must be at most 1024");
  AWQ_REQUIRE(a.kl.slots > 0 && a.kl.slots % 64 == 0 && a.vl.slots == a.kl.slots && a.kl.row == window_row_padded(a.dim) &&
                  a.vl.row == window_row_padded(a.vdim) && a.ldp % 8 == 0 && a.ldc % 8 == 0,
              "bad cache layout");
  const bool tiled = a.kl.row <= 256 && a.vl.row <= 256;
  if (a.M == 1 && tiled && a.parts && a.len_bound > 0)
    return f32 ? launch_decode<float>(a, st) : launch_decode<bf16_t>(a, st);
  if (int rc = f32 ? launch_append<float>(a, st) : launch_append<bf16_t>(a, st)) return rc;
  if (f32) return launch_queries<float>(a, st);
  if (!tiled || a.pos.dyn) return launch_queries<bf16_t>(a, st);
  if (a.kl.row == 64) launch_tiles<64>(a, st);
  else if (a.kl.row == 128) launch_tiles<128>(a, st);
  else launch_tiles<256>(a, st);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}
