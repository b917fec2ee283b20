// Attention over a shared latent (layers.hpp): keys and values of all heads are linear images of one cached vector per
// position, beside a rotated key part that the heads share; softmax with a learned score that has no key.
#include "layers.hpp"

namespace {

typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef float f32x16_t __attribute__((ext_vector_type(16)));
typedef short short4_t __attribute__((ext_vector_type(4)));
constexpr float kLog2e = 1.44269504088896340736f;

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
  return v;
}

// --- queries and cache rows ----------------------------------------------------------------------------------
// turn[rot / 2][2]: cosine and sine of the position's angles, brought into [-pi, pi] in binary64
__device__ __forceinline__ void turns_of(const LatentAttnArgs& a, int pos, float* turn) {
  for (int i = threadIdx.x; 2 * i < a.l.rot; i += 256) {
    const double turns = (double)pos * a.freq[i] * 0.15915494309189533577;  // 1 / 2 pi
    const float x = (float)((turns - rint(turns)) * 6.28318530717958647693);
    turn[2 * i] = cosf(x);
    turn[2 * i + 1] = sinf(x);
  }
  __syncthreads();
}

// `nh` heads' rotated parts, the first head's values at q.  INTO: to their place behind the latent entries of the queries
// ql, with zeros around them (entries rank .. row - 1); otherwise in place.
template <typename T, bool INTO>
__device__ __forceinline__ void rotate_queries(const LatentAttnArgs& a, T* q, T* ql, int nh, const float* turn) {
  const int rot = a.l.rot, rank = a.l.rank, rp = a.l.rank_padded(), row = a.l.row();
  const int tail = INTO ? row - rank : rot, skip = INTO ? rp - rank : 0;
  for (int i = threadIdx.x; i < nh * tail; i += 256) {
    const int h = i / tail, e = i - h * tail - skip;
    T* const src = q + (int64_t)h * (a.dim + rot) + a.dim;
    T* const dst = ql + (int64_t)h * row + rp;
    if (e >= 0 && e < rot) {
      if (e & 1) continue;
      const float u = (float)src[e], v = (float)src[e + 1], c = turn[e], s = turn[e + 1];
      T* const out = INTO ? dst : src;
      out[e] = (T)(u * c - v * s);
      out[e + 1] = (T)(v * c + u * s);
    } else if constexpr (INTO) {
      dst[e] = (T)0.0f;
    }
  }
}

// the cache row of token t of the pass
template <typename T>
__device__ __forceinline__ void append_row(const LatentAttnArgs& a, int t, int pos, const float* turn, float (&sums)[4]) {
  const int tid = threadIdx.x, rot = a.l.rot, rank = a.l.rank, rp = a.l.rank_padded(), row = a.l.row();
  const float* const d = a.down + t * a.ldd;
  float sq = 0.0f;
  for (int i = tid; i < rank; i += 256) sq = __builtin_fmaf(d[i], d[i], sq);
  sq = wave_sum(sq);
  if ((tid & 63) == 0) sums[tid >> 6] = sq;
  __syncthreads();
  const float inv = 1.0f / sqrtf(((sums[0] + sums[1]) + (sums[2] + sums[3])) / (float)rank + a.eps);
  T* const c = reinterpret_cast<T*>(a.cache) + (int64_t)pos * row;
  for (int i = tid; i < row; i += 256) {
    float v = 0.0f;
    const int e = i - rp;
    if (i < rank) {
      v = d[i] * inv * a.norm[i];
    } else if (e >= 0 && e < rot) {
      const float x = d[rank + e], other = d[rank + (e ^ 1)], cs = turn[e & ~1], sn = turn[e | 1];
      v = e & 1 ? x * cs + other * sn : x * cs - other * sn;
    }
    c[i] = (T)v;
  }
}

// blockIdx.x: token, blockIdx.y: `per` heads, and behind the last heads the token's cache row.  INTO: the
// unrotated parts go to qa, padded to `kq` inputs a head, the rotated ones to their place in ql; otherwise the rotated parts
// are rotated in place.
template <typename T, bool INTO>
__global__ __launch_bounds__(256) void latent_prepare_kernel(LatentAttnArgs a, int kq, int per) {
  extern __shared__ float turn[];
  __shared__ float sums[4];
  const int t = blockIdx.x, pos = a.pos.position() + t;
  turns_of(a, pos, turn);
  const int h0 = blockIdx.y * per;
  if (h0 >= a.heads) {
    append_row<T>(a, t, pos, turn, sums);
    return;
  }
  const int nh = min(per, a.heads - h0);
  T* const q = reinterpret_cast<T*>(a.q) + t * a.ldq + (int64_t)h0 * (a.dim + a.l.rot);
  if constexpr (INTO) {
    T* const qa = reinterpret_cast<T*>(a.qa) + ((int64_t)t * a.heads + h0) * kq;
    for (int i = threadIdx.x; i < nh * kq; i += 256) {
      const int h = i / kq, d = i - h * kq;
      qa[i] = d < a.dim ? q[(int64_t)h * (a.dim + a.l.rot) + d] : (T)0.0f;
    }
  }
  rotate_queries<T, INTO>(a, q, reinterpret_cast<T*>(a.ql) + ((int64_t)t * a.heads + h0) * a.l.row(), nh, turn);
}

// One token: the same and the product with W_uk in one launch.  blockIdx.x: head, blockIdx.y: 64 of its latent entries, 16 a
// wavefront (the first such workgroup of a head rotates, one more of the first head appends the cache row);
// v_mfma_f32_16x16x32_bf16 with the query in every column.
__global__ __launch_bounds__(256) void latent_query_one_kernel(LatentAttnArgs a, int64_t w_block, int chunks) {
  extern __shared__ float turn[];
  __shared__ float sums[4];
  const int h = blockIdx.x, part = blockIdx.y, pos = a.pos.position();
  if (part == chunks) {
    if (h != 0) return;
    turns_of(a, pos, turn);
    append_row<bf16_t>(a, 0, pos, turn, sums);
    return;
  }
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r = lane & 15, c = lane >> 4;
  const int row0 = part * 64 + wave * 16, rank = a.l.rank;
  bf16_t* const q = reinterpret_cast<bf16_t*>(a.q) + (int64_t)h * (a.dim + a.l.rot);
  bf16_t* const ql = reinterpret_cast<bf16_t*>(a.ql) + (int64_t)h * a.l.row();
  if (row0 < rank) {
    const bf16x8_t* w = reinterpret_cast<const bf16x8_t*>(reinterpret_cast<const bf16_t*>(a.w_uk) + h * w_block) +
                        ((int64_t)(row0 >> 5) * (a.dim >> 4) + (c >> 1)) * 64 + 32 * (c & 1) + (row0 & 16) + r;
    const bf16x8_t* x = reinterpret_cast<const bf16x8_t*>(q) + c;
    f32x4_t acc = {0.0f, 0.0f, 0.0f, 0.0f};
    constexpr int U = 8;
    const int steps = a.dim >> 5;
    bf16x8_t wv[U], xv[U];
#pragma unroll
    for (int i = 0; i < U; ++i)
      if (i < steps) wv[i] = w[(int64_t)i * 128], xv[i] = x[i * 4];
#pragma unroll
    for (int i = 0; i < U; ++i)
      if (i < steps) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[i], xv[i], acc, 0, 0, 0);
    for (int i = U; i < steps; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[(int64_t)i * 128], x[i * 4], acc, 0, 0, 0);
    if (r == 0)
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (row0 + 4 * c + j < rank) ql[row0 + 4 * c + j] = (bf16_t)acc[j];
  }
  if (part == 0) {
    turns_of(a, pos, turn);
    rotate_queries<bf16_t, true>(a, q, ql, 1, turn);
  }
}

// --- in the latent space, a query at a time --------------------------------------------------------------------
// A workgroup per (head, token), a thread per key, blocks of 256 keys with a running maximum.  Any sizes; the binary32
// form.  `kv_in`: padded inputs of the value product.
constexpr int kMaxColsPerThread = 4;
template <typename T>
__global__ __launch_bounds__(256) void latent_query_kernel(LatentAttnArgs a, int kv_in) {
  extern __shared__ float lds[];
  const int row = a.l.row(), rank = a.l.rank;
  float* q = lds;            // [row]
  float* p = lds + row;      // [256]
  float* red = p + 256;      // [4]
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x;
  const int pos = a.pos.position() + t;
  const T* const ql = reinterpret_cast<const T*>(a.ql) + ((int64_t)t * a.heads + h) * row;
  for (int d = tid; d < row; d += 256) q[d] = (float)ql[d];
  const T* const cache = reinterpret_cast<const T*>(a.cache);
  float m = a.sink ? a.sink[h] : -INFINITY, l = a.sink ? 1.0f : 0.0f, acc[kMaxColsPerThread] = {};
  __syncthreads();
  for (int k0 = 0; k0 <= pos; k0 += 256) {
    const int key = k0 + tid;
    float s = -INFINITY;
    if (key <= pos) {
      const T* kr = cache + (int64_t)key * row;
      float dot = 0.0f;
      for (int d = 0; d < row; ++d) dot = __builtin_fmaf(q[d], (float)kr[d], dot);
      s = dot * a.scale;
    }
    float mx = s;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float m_new = fmaxf(m, mx), alpha = expf(m - m_new), e = expf(s - m_new);
    p[tid] = e;
    const float sum = wave_sum(e);
    __syncthreads();
    if ((tid & 63) == 0) red[tid >> 6] = sum;
    __syncthreads();
    l = l * alpha + ((red[0] + red[1]) + (red[2] + red[3]));
    m = m_new;
    const int n = min(256, pos + 1 - k0);
#pragma unroll
    for (int c = 0; c < kMaxColsPerThread; ++c) {
      const int col = c * 256 + tid;
      if (col < rank) {
        float v = acc[c] * alpha;
        for (int j = 0; j < n; ++j) v = __builtin_fmaf(p[j], (float)cache[(int64_t)(k0 + j) * row + col], v);
        acc[c] = v;
      }
    }
    __syncthreads();
  }
  T* out = reinterpret_cast<T*>(a.ol) + ((int64_t)t * a.heads + h) * kv_in;
#pragma unroll
  for (int c = 0; c < kMaxColsPerThread; ++c)
    if (c * 256 + tid < kv_in) out[c * 256 + tid] = (T)(c * 256 + tid < rank ? acc[c] / l : 0.0f);
}

// --- in the latent space, on the matrix cores ------------------------------------------------------------------
// 32 query rows (token, head) of the pass per workgroup, row r = token * heads + head, against a share of the keys
// (blockIdx.y), 64 at a time from LDS, where they serve as keys and, their first entries, as values.
//     S^T[key][row] = K Q^T       v_mfma_f32_16x16x32_bf16, 16 keys per wavefront
//     O^T[c][row] += C^T P^T      v_mfma_f32_32x32x16_bf16, a quarter of the columns per wavefront; C^T by the transposing LDS
//                                 read, slice j taking keys 16 j + 8 (e / 4) + 4 kh + e % 4; weights as two bfloat16 terms
// A part is [maximum (binary logarithm), sum, -, -, columns].
constexpr int kRows = 32, kKeys = 64, kScoreStride = kKeys + 4, kWeightStride = kKeys + 8;
constexpr int kMaxParts = 128, kMaxRow = 640;

__host__ __device__ inline size_t rows_lds(int row) {
  return (size_t)(kKeys + kRows) * (row + 8) * 2 + kRows * kScoreStride * 4 + 2 * kRows * kWeightStride * 2 + kRows * 4;
}
// key tiles of a share, of all keys that the rows from `row0` on see
__device__ __forceinline__ int tiles_per_part(int row0, int rows, int heads, int pos0, int parts, int* tiles) {
  const int last = pos0 + min(row0 + kRows - 1, rows - 1) / heads;
  *tiles = last / kKeys + 1;
  return (*tiles + parts - 1) / parts;
}

template <int NT>
__global__ __launch_bounds__(256) void latent_rows_kernel(LatentAttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) char raw[];
  const int row = a.l.row(), rp = a.l.rank_padded(), KS = row + 8;
  bf16_t* const kt = reinterpret_cast<bf16_t*>(raw);                // [64][KS]
  bf16_t* const qt = kt + kKeys * KS;                               // [32][KS]
  float* const sc = reinterpret_cast<float*>(qt + kRows * KS);      // [32][kScoreStride]
  bf16_t* const ph = reinterpret_cast<bf16_t*>(sc + kRows * kScoreStride);  // [32][kWeightStride], twice
  bf16_t* const pl = ph + kRows * kWeightStride;
  float* const fade = reinterpret_cast<float*>(pl + kRows * kWeightStride);  // [32]
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int rows = (int)a.M * a.heads, row0 = blockIdx.x * kRows, parts = gridDim.y, part = blockIdx.y;
  const int pos0 = a.pos.position();
  int tiles;
  const int per = tiles_per_part(row0, rows, a.heads, pos0, parts, &tiles);
  const int first = part * per, end = min(tiles, first + per);
  if (first >= end) return;
  const bf16_t* const cache = reinterpret_cast<const bf16_t*>(a.cache);
  const bf16_t* const ql = reinterpret_cast<const bf16_t*>(a.ql);
  // four threads copy a key row, eight a query row, all loads in flight at once
  constexpr int kPieces = kMaxRow / 32;
  const int kr = tid >> 2, kf = (tid & 3) * 8, qr = tid >> 3, qf = (tid & 7) * 8;
  bf16x8_t kx[kPieces];
  auto load_keys = [&](int tile) __attribute__((always_inline)) {
    const bf16_t* const src = cache + ((int64_t)tile * kKeys + kr) * row + kf;  // the cache is whole tiles
#pragma unroll
    for (int i = 0; i < kPieces; ++i)
      if (32 * i < row) kx[i] = *reinterpret_cast<const bf16x8_t*>(src + 32 * i);
  };
  {
    const bf16_t* const src = ql + (int64_t)min(row0 + qr, rows - 1) * row + qf;
    bf16x8_t x[kPieces / 2];
#pragma unroll
    for (int i = 0; i < kPieces / 2; ++i)
      if (64 * i + qf < row) x[i] = *reinterpret_cast<const bf16x8_t*>(src + 64 * i);
    load_keys(first);
#pragma unroll
    for (int i = 0; i < kPieces / 2; ++i)
      if (64 * i + qf < row) *reinterpret_cast<bf16x8_t*>(qt + qr * KS + qf + 64 * i) = x[i];
  }
  f32x16_t o[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) o[i][e] = 0.0f;
  const int n16 = lane & 15, c16 = lane >> 4, n32 = lane & 31, kh = lane >> 5;
  // the softmax: eight threads per row, eight keys each
  const int sr = tid >> 3, sk = (tid & 7) * 8;
  const int sp = pos0 + min(row0 + sr, rows - 1) / a.heads;
  const float mul = a.scale * kLog2e;
  float m_run = -INFINITY, l_run = 0.0f;
  for (int tile = first; tile < end; ++tile) {
    __syncthreads();  // the previous tile's readers are done
#pragma unroll
    for (int i = 0; i < kPieces; ++i)
      if (32 * i < row) *reinterpret_cast<bf16x8_t*>(kt + kr * KS + kf + 32 * i) = kx[i];
    if (tile + 1 < end) load_keys(tile + 1);
    __syncthreads();
    f32x4_t s0 = {0.0f, 0.0f, 0.0f, 0.0f}, s1 = s0;
    const bf16_t* const kp = kt + (16 * wave + n16) * KS + 8 * c16;
    const bf16_t* const qp = qt + n16 * KS + 8 * c16;
    for (int d = 0; d < row; d += 32) {
      const bf16x8_t kv = *reinterpret_cast<const bf16x8_t*>(kp + d);
      s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kv, *reinterpret_cast<const bf16x8_t*>(qp + d), s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kv, *reinterpret_cast<const bf16x8_t*>(qp + 16 * KS + d), s1, 0, 0, 0);
    }
    *reinterpret_cast<f32x4_t*>(sc + n16 * kScoreStride + 16 * wave + 4 * c16) = s0;
    *reinterpret_cast<f32x4_t*>(sc + (16 + n16) * kScoreStride + 16 * wave + 4 * c16) = s1;
    __syncthreads();
    {
      float s[8];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const f32x4_t x = *reinterpret_cast<const f32x4_t*>(sc + sr * kScoreStride + sk + 4 * i);
#pragma unroll
        for (int e = 0; e < 4; ++e) s[4 * i + e] = tile * kKeys + sk + 4 * i + e <= sp ? x[e] * mul : -INFINITY;
      }
      float mx = s[0];
#pragma unroll
      for (int i = 1; i < 8; ++i) mx = fmaxf(mx, s[i]);
#pragma unroll
      for (int off = 1; off < 8; off <<= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
      const float m_new = fmaxf(m_run, mx), base = m_new == -INFINITY ? 0.0f : m_new;
      const float alpha = exp2f(m_run - base);
      float sum = 0.0f;
      bf16x8_t hi, lo;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float p = exp2f(s[i] - base);
        sum += p;
        hi[i] = (bf16_t)p;
        lo[i] = (bf16_t)(p - (float)hi[i]);
      }
#pragma unroll
      for (int off = 1; off < 8; off <<= 1) sum += __shfl_xor(sum, off, 64);
      l_run = l_run * alpha + sum;
      m_run = m_new;
      *reinterpret_cast<bf16x8_t*>(ph + sr * kWeightStride + sk) = hi;
      *reinterpret_cast<bf16x8_t*>(pl + sr * kWeightStride + sk) = lo;
      if (sk == 0) fade[sr] = alpha;
    }
    __syncthreads();
    const float alpha = fade[n32];
    const int L16 = lane & 15;
    const bf16_t* const vlane = kt + (4 * kh + (L16 >> 2)) * KS + 16 * ((lane >> 4) & 1) + 4 * (L16 & 3);
    bf16x8_t whi[4], wlo[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int at = n32 * kWeightStride + 16 * j + 4 * kh;
      const bf16x4_t h0 = *reinterpret_cast<const bf16x4_t*>(ph + at), h1 = *reinterpret_cast<const bf16x4_t*>(ph + at + 8);
      const bf16x4_t l0 = *reinterpret_cast<const bf16x4_t*>(pl + at), l1 = *reinterpret_cast<const bf16x4_t*>(pl + at + 8);
      whi[j] = bf16x8_t{h0[0], h0[1], h0[2], h0[3], h1[0], h1[1], h1[2], h1[3]};
      wlo[j] = bf16x8_t{l0[0], l0[1], l0[2], l0[3], l1[0], l1[1], l1[2], l1[3]};
    }
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int ct = wave + 4 * i;
      if (32 * ct >= rp) continue;
#pragma unroll
      for (int e = 0; e < 16; ++e) o[i][e] *= alpha;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bf16_t* vp = vlane + 16 * j * KS + ct * 32;
        const short4_t l = __builtin_amdgcn_ds_read_tr16_b64_v4i16((short4_t __attribute__((address_space(3)))*)vp);
        const short4_t u = __builtin_amdgcn_ds_read_tr16_b64_v4i16((short4_t __attribute__((address_space(3)))*)(vp + 8 * KS));
        const bf16x4_t l4 = __builtin_bit_cast(bf16x4_t, l), u4 = __builtin_bit_cast(bf16x4_t, u);
        const bf16x8_t vv = {l4[0], l4[1], l4[2], l4[3], u4[0], u4[1], u4[2], u4[3]};
        o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vv, whi[j], o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vv, wlo[j], o[i], 0, 0, 0);
      }
    }
  }
  const int ps = rp + 4;
  if (row0 + n32 < rows) {
    float* const mine = a.parts + ((int64_t)(row0 + n32) * parts + part) * ps + 4;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int ct = wave + 4 * i;
      if (32 * ct >= rp) continue;
#pragma unroll
      for (int u = 0; u < 4; ++u)
        *reinterpret_cast<f32x4_t*>(mine + 32 * ct + 8 * u + 4 * kh) =
            f32x4_t{o[i][4 * u], o[i][4 * u + 1], o[i][4 * u + 2], o[i][4 * u + 3]};
    }
  }
  if (sk == 0 && row0 + sr < rows) {
    float* const mine = a.parts + ((int64_t)(row0 + sr) * parts + part) * ps;
    mine[0] = m_run;
    mine[1] = l_run;
  }
}

// The parts of query row r and the sink: `scale` receives every part's factor; returns what the weighted parts are divided by
__device__ __forceinline__ float combine_factors(const LatentAttnArgs& a, int r, int parts, float* scale, int* used_parts) {
  const int tid = threadIdx.x, lane = tid & 63, ps = a.l.rank_padded() + 4;
  int tiles;
  const int per = tiles_per_part(r / kRows * kRows, (int)a.M * a.heads, a.heads, a.pos.position(), parts, &tiles);
  const int used = (tiles + per - 1) / per;
  const float* const p = a.parts + (int64_t)r * parts * ps;
  const float sink = a.sink ? a.sink[r % a.heads] * kLog2e : -INFINITY;
  float pm[kMaxParts / 64], pl[kMaxParts / 64], m = sink, l = 0.0f;
#pragma unroll
  for (int i = 0; i < kMaxParts / 64; ++i) {
    const int s = lane + 64 * i;
    pm[i] = s < used ? p[(int64_t)s * ps] : -INFINITY;
    pl[i] = s < used ? p[(int64_t)s * ps + 1] : 0.0f;
    m = fmaxf(m, pm[i]);
  }
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) m = fmaxf(m, __shfl_xor(m, off, 64));
#pragma unroll
  for (int i = 0; i < kMaxParts / 64; ++i) {
    const float e = exp2f(pm[i] - m);
    l = __builtin_fmaf(e, pl[i], l);
    if (tid < 64) scale[lane + 64 * i] = e;
  }
  l = wave_sum(l) + exp2f(sink - m);
  __syncthreads();
  *used_parts = used;
  return l;
}
__device__ __forceinline__ float combine_column(const LatentAttnArgs& a, int r, int parts, const float* scale, int used, int c) {
  const int ps = a.l.rank_padded() + 4;
  const float* const p = a.parts + (int64_t)r * parts * ps + 4 + c;
  float v = 0.0f;
#pragma unroll 8
  for (int s = 0; s < used; ++s) v = __builtin_fmaf(scale[s], p[(int64_t)s * ps], v);
  return v;
}

// a workgroup per query row
__global__ __launch_bounds__(256) void latent_combine_kernel(LatentAttnArgs a, int parts, int kv_in) {
  __shared__ float scale[kMaxParts];
  const int r = blockIdx.x;
  int used;
  const float inv = 1.0f / combine_factors(a, r, parts, scale, &used);
  bf16_t* const out = reinterpret_cast<bf16_t*>(a.ol) + (int64_t)r * kv_in;
  for (int c = threadIdx.x; c < kv_in; c += 256) out[c] = (bf16_t)(c < a.l.rank ? combine_column(a, r, parts, scale, used, c) * inv : 0.0f);
}

// One token: the same and the product with W_uv in one launch.  blockIdx.x: head, blockIdx.y: 64 of its values, 16 a
// wavefront; every workgroup combines for itself while its weights are on their way.
__global__ __launch_bounds__(256) void latent_value_one_kernel(LatentAttnArgs a, int parts, int kv_in, int64_t w_block) {
  extern __shared__ __attribute__((aligned(16))) bf16_t ol[];  // [kv_in]
  __shared__ float scale[kMaxParts];
  constexpr int U = 16;
  const int h = blockIdx.x, tid = threadIdx.x;
  const int lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), r = lane & 15, c = lane >> 4;
  const int row0 = blockIdx.y * 64 + wave * 16, steps = kv_in >> 5;
  const bool mine = row0 < a.vdim;
  const bf16x8_t* w = reinterpret_cast<const bf16x8_t*>(reinterpret_cast<const bf16_t*>(a.w_uv) + h * w_block) +
                      ((int64_t)(row0 >> 5) * (kv_in >> 4) + (c >> 1)) * 64 + 32 * (c & 1) + (row0 & 16) + r;
  bf16x8_t wv[U];
#pragma unroll
  for (int i = 0; i < U; ++i)
    if (mine && i < steps) wv[i] = w[(int64_t)i * 128];
  int used;
  const float inv = 1.0f / combine_factors(a, h, parts, scale, &used);
  for (int col = tid; col < kv_in; col += 256) ol[col] = (bf16_t)(col < a.l.rank ? combine_column(a, h, parts, scale, used, col) * inv : 0.0f);
  __syncthreads();
  if (!mine) return;
  const bf16x8_t* x = reinterpret_cast<const bf16x8_t*>(ol) + c;
  f32x4_t acc = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
  for (int i = 0; i < U; ++i)
    if (i < steps) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[i], x[i * 4], acc, 0, 0, 0);
  for (int i = U; i < steps; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[(int64_t)i * 128], x[i * 4], acc, 0, 0, 0);
  if (r != 0) return;
  bf16_t* const out = reinterpret_cast<bf16_t*>(a.ctx) + (int64_t)h * a.vdim + row0;
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (row0 + 4 * c + j < a.vdim) out[4 * c + j] = (bf16_t)acc[j];
}

// --- with keys and values formed first -------------------------------------------------------------------------
// 128 queries of one head per workgroup, 32 per wavefront, keys and values of 32 positions at a time through LDS; the
// operands as in window_attention.hip.  The sink is the state that a query's running maximum and sum start from.
constexpr int kTileQueries = 128, kTileKeys = 32;

template <int DK, int DV>
__global__ __launch_bounds__(256, (DK + DV > 256) ? 1 : 2) void latent_tile_kernel(LatentAttnArgs a) {
  constexpr int KS = DK + 8, VS = DV + 16;
  constexpr int KP = DK / 64, VP = DV / 64;  // 16-byte pieces of a tile per thread
  __shared__ __attribute__((aligned(16))) bf16_t ks2[2 * kTileKeys * KS];
  __shared__ __attribute__((aligned(16))) bf16_t vs2[2 * kTileKeys * VS];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n = lane & 31, kh = lane >> 5;
  const int M = (int)a.M, pos0 = a.pos.pos0;
  const int q_first = (gridDim.y - 1 - blockIdx.y) * kTileQueries;  // the longest rows first
  const int qi = q_first + wave * 32 + n, qc = min(qi, M - 1), pq = pos0 + qc;
  const int w_first = pos0 + min(q_first + wave * 32, M - 1), w_last = pos0 + min(q_first + wave * 32 + 31, M - 1);
  const int k_end = pos0 + min(q_first + kTileQueries - 1, M - 1) + 1;
  const int qk = a.dim + a.l.rot, row = a.l.row(), rp = a.l.rank_padded();
  const int64_t ldkv = (int64_t)a.heads * (a.dim + a.vdim);
  const bf16_t* const q = reinterpret_cast<const bf16_t*>(a.q) + (int64_t)qc * a.ldq + (int64_t)h * qk;
  const bf16_t* const kx = reinterpret_cast<const bf16_t*>(a.kv) + (int64_t)h * a.dim;
  const bf16_t* const vx = reinterpret_cast<const bf16_t*>(a.kv) + (int64_t)a.heads * a.dim + (int64_t)h * a.vdim;
  const bf16_t* const cache = reinterpret_cast<const bf16_t*>(a.cache) + rp;
  bf16x8_t zero;
#pragma unroll
  for (int e = 0; e < 8; ++e) zero[e] = (bf16_t)0.0f;
  bf16x8_t qop[DK / 16];
#pragma unroll
  for (int s = 0; s < DK / 16; ++s) {
    const int at = 16 * s + 8 * kh;
    qop[s] = at < qk ? *reinterpret_cast<const bf16x8_t*>(q + at) : zero;
  }
  f32x16_t o[DV / 32];
#pragma unroll
  for (int d = 0; d < DV / 32; ++d)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[d][i] = 0.0f;
  float m_run = a.sink ? a.sink[h] * kLog2e : -1e30f, l_run = a.sink ? 1.0f : 0.0f;
  const float mul = a.scale * kLog2e;
  struct TileRegs {
    bf16x8_t k[KP], v[VP];
  };
  TileRegs ra, rb;
  auto load_tile = [&](int k0, TileRegs& r) __attribute__((always_inline)) {
    if (k0 >= k_end) return;
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int pc = tid + i * 256, key = min(k0 + pc / (DK / 8), k_end - 1), at = (pc % (DK / 8)) * 8;
      r.k[i] = at < a.dim ? *reinterpret_cast<const bf16x8_t*>(kx + key * ldkv + at)
               : at < qk  ? *reinterpret_cast<const bf16x8_t*>(cache + (int64_t)key * row + at - a.dim)
                          : zero;
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int pc = tid + i * 256, key = min(k0 + pc / (DV / 8), k_end - 1), at = (pc % (DV / 8)) * 8;
      r.v[i] = at < a.vdim ? *reinterpret_cast<const bf16x8_t*>(vx + key * ldkv + at) : zero;
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
    if (k0 > w_last) return;  // no query of this wavefront sees a key of the tile
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
#pragma unroll
    for (int i = 0; i < 16; ++i) s[i] *= mul;
    if (k0 + kTileKeys - 1 > w_first) {
#pragma unroll
      for (int i = 0; i < 16; ++i) s[i] = k0 + 8 * (i >> 2) + 4 * kh + (i & 3) <= pq ? s[i] : -INFINITY;
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
  load_tile(0, ra);
  load_tile(kTileKeys, rb);
  for (int k0 = 0; k0 < k_end; k0 += 2 * kTileKeys) {
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
      if (c < a.vdim)  // vdim is a multiple of 8
        *reinterpret_cast<bf16x4_t*>(out + c) = bf16x4_t{(bf16_t)(o[d][4 * u] * inv), (bf16_t)(o[d][4 * u + 1] * inv),
                                                         (bf16_t)(o[d][4 * u + 2] * inv), (bf16_t)(o[d][4 * u + 3] * inv)};
    }
}

template <int DK>
void launch_tiles(const LatentAttnArgs& a, hipStream_t st) {
  const dim3 g((unsigned)a.heads, (unsigned)((a.M + kTileQueries - 1) / kTileQueries));
  if (a.vdim <= 64) hipLaunchKernelGGL((latent_tile_kernel<DK, 64>), g, dim3(256), 0, st, a);
  else if (a.vdim <= 128) hipLaunchKernelGGL((latent_tile_kernel<DK, 128>), g, dim3(256), 0, st, a);
  else hipLaunchKernelGGL((latent_tile_kernel<DK, 256>), g, dim3(256), 0, st, a);
}

int64_t q_inputs(const LatentAttnArgs& a) { return round_up(a.dim, kDenseKAlign); }
int64_t v_inputs(const LatentAttnArgs& a) { return round_up(a.l.rank, kDenseKAlign); }

// The rows kernel's shapes
bool on_matrix_cores(const LatentAttnArgs& a, bool f32) { return !f32 && a.l.rank_padded() <= 512 && a.l.row() <= kMaxRow; }

// Keys and values formed first: sizes the tiles have instances for, and enough queries that the products over dim and vdim
// instead of rank (twice) pay for forming them, per key and head rank * (dim + vdim)
bool can_form(const LatentAttnArgs& a, bool f32) {
  return !f32 && ((a.dim | a.l.rot | a.vdim) & 7) == 0 && a.dim + a.l.rot <= 256 && a.vdim <= 256;
}
int64_t form_from(const LatentAttnArgs& a) {
  const int64_t saved = 2 * a.l.rank - a.dim - a.vdim;
  if (saved <= 0) return INT64_MAX;
  return std::max<int64_t>(32, (int64_t)a.l.rank * (a.dim + a.vdim) / saved);
}

int parts_of(const LatentAttnArgs& a, int64_t M, int64_t keys) {
  const int64_t row_tiles = (M * a.heads + kRows - 1) / kRows, tiles = (keys + kKeys - 1) / kKeys;
  return (int)std::max<int64_t>(1, std::min<int64_t>(std::min<int64_t>(512 / row_tiles, tiles), kMaxParts));
}

template <typename T, bool INTO>
int launch_prepare(const LatentAttnArgs& a, hipStream_t st) {
  const int per = a.M >= 256 ? 32 : 4;  // heads of a workgroup: each forms the angles again
  const dim3 g((unsigned)a.M, (unsigned)((a.heads + per - 1) / per + (a.down ? 1 : 0)));
  hipLaunchKernelGGL((latent_prepare_kernel<T, INTO>), g, dim3(256), (size_t)(a.l.rot + 2) * 4, st, a, (int)q_inputs(a), per);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

static_assert((size_t)(kKeys + kRows) * (kMaxRow + 8) * 2 + kRows * kScoreStride * 4 + 4 * kRows * kWeightStride + kRows * 4 <= 160 * 1024,
              "more LDS than a compute unit has");
template <int NT>
int launch_rows(const LatentAttnArgs& a, int parts, hipStream_t st) {
  static bool raised = false;  // more LDS than the default limit of a launch
  if (!raised) {
    AWQ_HIP_TRY(hipFuncSetAttribute((const void*)latent_rows_kernel<NT>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
    raised = true;
  }
  hipLaunchKernelGGL(latent_rows_kernel<NT>, dim3((unsigned)((a.M * a.heads + kRows - 1) / kRows), (unsigned)parts), dim3(256),
                     rows_lds(a.l.row()), st, a);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

int heads_product(const LatentAttnArgs& a, const void* w, int64_t w_batch, int64_t k, const void* x, void* y, int64_t ldy,
                  int64_t y_batch, int64_t rows, bool f32, hipStream_t st) {
  DenseArgs d;
  d.w = w;
  d.k = k;
  d.M = a.M;
  d.batch = a.heads;
  d.w_batch = w_batch;
  d.x_batch = k;
  d.y_batch = y_batch;
  d.seg[0].x = x;
  d.seg[0].ldx = a.heads * k;
  d.seg[0].y = y;
  d.seg[0].ldy = ldy;
  d.seg[0].rows = (int32_t)rows;
  return launch_dense(d, f32, st);
}

}  // namespace

int64_t latent_uk_block(const LatentAttnArgs& a) { return round_up(a.l.rank, kDenseRowAlign) * q_inputs(a); }
int64_t latent_uv_block(const LatentAttnArgs& a) { return round_up(a.vdim, kDenseRowAlign) * v_inputs(a); }
int64_t latent_kv_rows(const LatentAttnArgs& a) { return round_up((int64_t)a.heads * (a.dim + a.vdim), kDenseRowAlign); }

bool latent_forms_keys(const LatentAttnArgs& a, int64_t max_tokens, bool f32) {
  return can_form(a, f32) && form_from(a) <= max_tokens;
}

LatentScratch latent_scratch(const LatentAttnArgs& a, int64_t max_tokens, bool f32) {
  const int64_t unit = f32 ? 4 : 2;
  const bool form = latent_forms_keys(a, max_tokens, f32);
  const int64_t M = form ? std::min<int64_t>(max_tokens, form_from(a)) : max_tokens;  // tokens taken into the latent space
  LatentScratch s;
  s.qa = M * a.heads * q_inputs(a) * unit;
  s.ql = M * a.heads * a.l.row() * unit;
  s.ol = M * a.heads * v_inputs(a) * unit;
  if (form) s.kv = a.max_pos * a.heads * (a.dim + a.vdim) * unit;
  if (on_matrix_cores(a, f32)) s.parts = std::max<int64_t>(512 * kRows, M * a.heads) * (a.l.rank_padded() + 4) * 4;
  return s;
}

int launch_latent_pack(const LatentAttnArgs& a, const void* uk, const void* uv, bool src_f32, void* w_uk, void* w_uv, void* w_kv,
                       bool f32, hipStream_t st) {
  const int64_t qk = q_inputs(a), vk = v_inputs(a), unit = src_f32 ? 4 : 2, keys = (int64_t)a.heads * a.dim;
  const int64_t uk_rows = latent_uk_block(a) / qk, uv_rows = latent_uv_block(a) / vk;
  for (int64_t h = 0; h < a.heads; ++h) {
    if (uk)
      if (int rc = launch_dense_pack((const char*)uk + h * a.dim * a.l.rank * unit, src_f32, a.dim, a.l.rank, w_uk, qk, h * uk_rows, 0,
                                     f32, st, PACK_TRANSPOSED))
        return rc;
    if (uv)
      if (int rc = launch_dense_pack((const char*)uv + h * a.vdim * a.l.rank * unit, src_f32, a.vdim, a.l.rank, w_uv, vk, h * uv_rows, 0,
                                     f32, st))
        return rc;
  }
  if (w_kv && uk)
    if (int rc = launch_dense_pack(uk, src_f32, keys, a.l.rank, w_kv, vk, 0, 0, f32, st)) return rc;
  if (w_kv && uv) return launch_dense_pack(uv, src_f32, (int64_t)a.heads * a.vdim, a.l.rank, w_kv, vk, keys, 0, f32, st);
  return AWQ_OK;
}

int launch_latent_attention(const LatentAttnArgs& a, bool f32, hipStream_t st) {
  AWQ_REQUIRE(a.q && a.freq && a.cache && a.w_uk && a.w_uv && a.ctx && a.qa && a.ql && a.ol && (!a.down || a.norm), "bad arguments");
  AWQ_REQUIRE(a.heads >= 1 && a.heads <= 65535 && a.dim >= 1 && a.vdim >= 1 && a.l.rank >= 1 && a.l.rank <= 256 * kMaxColsPerThread &&
                  a.l.rot >= 2 && a.l.rot % 2 == 0 && a.l.rot <= 1024,
              "bad shape");
  AWQ_REQUIRE(a.M >= 1 && a.M <= 65535 && a.M * a.heads < (1ll << 30) && a.ldq >= (int64_t)a.heads * (a.dim + a.l.rot) &&
                  (a.pos.dyn ? a.M == 1 : a.pos.pos0 + a.M <= a.max_pos),
              "bad tokens");
  if (can_form(a, f32) && !a.pos.dyn && a.M >= form_from(a)) {
    AWQ_REQUIRE(a.w_kv && a.kv && ((a.ldq | a.ldc) & 7) == 0, "a pass of this many tokens forms keys and values: w_kv, kv, rows of 8");
    if (int rc = launch_prepare<bf16_t, false>(a, st)) return rc;
    DenseArgs d;
    d.w = a.w_kv;
    d.k = v_inputs(a);  // behind rank: columns of weights that are zero
    d.M = a.pos.pos0 + a.M;
    d.workspace = a.dense_ws;
    d.workspace_floats = a.dense_ws_floats;
    d.seg[0].x = a.cache;
    d.seg[0].ldx = a.l.row();
    d.seg[0].y = a.kv;
    d.seg[0].ldy = (int64_t)a.heads * (a.dim + a.vdim);
    d.seg[0].rows = a.heads * (a.dim + a.vdim);
    if (int rc = launch_dense(d, false, st)) return rc;
    const int qk = a.dim + a.l.rot;
    if (qk <= 64) launch_tiles<64>(a, st);
    else if (qk <= 128) launch_tiles<128>(a, st);
    else if (qk <= 192) launch_tiles<192>(a, st);
    else launch_tiles<256>(a, st);
    AWQ_HIP_TRY(hipGetLastError());
    return AWQ_OK;
  }
  const bool cores = on_matrix_cores(a, f32);
  if (a.M == 1 && cores && a.dim % kDenseKAlign == 0 && ((a.dim + a.l.rot) & 7) == 0 && ((uintptr_t)a.q & 15) == 0) {
    const int chunks = (a.l.rank + 63) / 64;
    hipLaunchKernelGGL(latent_query_one_kernel, dim3((unsigned)a.heads, (unsigned)(chunks + (a.down ? 1 : 0))), dim3(256),
                       (size_t)(a.l.rot + 2) * 4, st, a, latent_uk_block(a), chunks);
    AWQ_HIP_TRY(hipGetLastError());
  } else {
    if (int rc = f32 ? launch_prepare<float, true>(a, st) : launch_prepare<bf16_t, true>(a, st)) return rc;
    if (int rc = heads_product(a, a.w_uk, latent_uk_block(a), q_inputs(a), a.qa, a.ql, (int64_t)a.heads * a.l.row(), a.l.row(),
                               a.l.rank, f32, st))
      return rc;
  }
  if (cores) {
    AWQ_REQUIRE(a.parts, "no scratch for the parts");
    const int parts = parts_of(a, a.M, a.pos.dyn ? a.max_pos : a.pos.pos0 + a.M);
    const int rp = a.l.rank_padded();
    if (int rc = rp <= 128 ? launch_rows<1>(a, parts, st) : rp <= 256 ? launch_rows<2>(a, parts, st) : launch_rows<4>(a, parts, st))
      return rc;
    if (a.M == 1) {
      hipLaunchKernelGGL(latent_value_one_kernel, dim3((unsigned)a.heads, (unsigned)((a.vdim + 63) / 64)), dim3(256),
                         (size_t)v_inputs(a) * 2, st, a, parts, (int)v_inputs(a), latent_uv_block(a));
      AWQ_HIP_TRY(hipGetLastError());
      return AWQ_OK;
    }
    hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)(a.M * a.heads)), dim3(256), 0, st, a, parts, (int)v_inputs(a));
  } else {
    const size_t lds = (size_t)(a.l.row() + 256 + 4) * 4;
    const dim3 g((unsigned)a.heads, (unsigned)a.M);
    if (f32) hipLaunchKernelGGL(latent_query_kernel<float>, g, dim3(256), lds, st, a, (int)v_inputs(a));
    else hipLaunchKernelGGL(latent_query_kernel<bf16_t>, g, dim3(256), lds, st, a, (int)v_inputs(a));
  }
  AWQ_HIP_TRY(hipGetLastError());
  return heads_product(a, a.w_uv, latent_uv_block(a), v_inputs(a), a.ol, a.ctx, a.ldc, a.vdim, a.vdim, f32, st);
}
