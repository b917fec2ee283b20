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

// The same for many tokens on the matrix cores, 128 tokens (a chunk) after the other.  With t, s counted inside the
// chunk and S the state ahead of it,
//     o_t = decay^(t+1) S^T q_t + sum over s <= t of decay^(t-s) (k_s . q_t) v_s
//     S  <- decay^n S + sum over t < n of k_t (decay^(n-1-t) v_t)^T
// A workgroup takes 32 columns of one head's state and all chunks in turn.  Wavefronts 0 .. 3 compute the outputs of 32
// tokens of a chunk each; wavefronts 4 .. 7 keep 32 (64 at dim 256) of the state's rows each in their accumulators and
// carry them over the chunk at the same time.  q, k and v
// are bfloat16 as projected, so their products are exact; the binary32 factors enter as sums of bfloat16 terms
// (three for the state and for the decayed values, two for the weights inside a chunk) and every accumulation is
// binary32.  Operands of v_mfma_f32_32x32x16_bf16, lane (n, kh) = (lane % 32, lane / 32):
//     W[s][t]   = K Q^T           K rows from LDS, Q in registers
//     O^T[v][t] = S^T Q^T         the state's terms from LDS as [v][d]
//     O^T[v][t] += V^T W          W's elements are already where the second operand wants them, if a 16-wide slice
//                                 j takes s = 16 j + 8 (e / 4) + 4 kh + e % 4; V^T from LDS as [v][t]
//     S[d][v]   += K^T V'         the same slices; K^T by the transposing LDS read
typedef float f32x16_t __attribute__((ext_vector_type(16)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef short short4_t __attribute__((ext_vector_type(4)));
constexpr int kChunk = 128;
constexpr int kVStride = kChunk + 8;  // elements per column of V^T

template <int D>
constexpr int linear_chunk_lds() {
  return (kChunk * (D + 16) + 4 * 32 * kVStride + 3 * 32 * (D + 8)) * 2;
}

// WHOLE: rows of q, k and v are 16-byte pieces
template <int D, bool WHOLE>
__global__ __launch_bounds__(512) void linear_chunk_kernel(LinearAttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) char lds_raw[];
  constexpr int KS = D + 16, SS = D + 8, NT = D / 32;  // NT tiles of 32 state rows, over four wavefronts
  constexpr int TPW = NT < 4 ? 1 : NT / 4;             // ... per wavefront
  constexpr int KP = D / 32;                           // 16-byte pieces of k per thread
  bf16_t* const ks = reinterpret_cast<bf16_t*>(lds_raw);       // [128][KS]
  bf16_t* const vt = ks + kChunk * KS;                         // [4][32][kVStride]: v, then three terms of v'
  bf16_t* const st = vt + 4 * 32 * kVStride;                   // [3][32][SS]
  const int head = blockIdx.x, v0 = blockIdx.y * 32;
  const int tid = threadIdx.x, lane = tid & 63, wave8 = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int wave = wave8 & 3;
  const bool outputs = wave8 < 4;
  const int n = lane & 31, kh = lane >> 5;
  const int M = (int)a.M;
  const bf16_t* const p = reinterpret_cast<const bf16_t*>(a.proj);
  const bf16_t* const q = p + (int64_t)head * a.dim;
  const bf16_t* const k = p + (int64_t)(a.heads + head) * a.dim;
  const bf16_t* const v = p + (int64_t)2 * a.heads * a.dim + (int64_t)head * a.vdim + v0;
  const int nv = min(32, a.vdim - v0);
  const float lg = a.log2_decay[head];
  const int dimp = (a.dim + 63) & ~63;
  float* const state = a.state + ((int64_t)head * a.vdim + v0 + n) * dimp;

  auto piece = [&](const bf16_t* row, int at, int len) __attribute__((always_inline)) {
    bf16x8_t r;
    if constexpr (WHOLE) {
      if (at < len) return *reinterpret_cast<const bf16x8_t*>(row + at);
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] = (bf16_t)0.0f;
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] = at + e < len ? row[at + e] : (bf16_t)0.0f;
    }
    return r;
  };

  // the state: rows 32 (wave + 4 i) + 8 g + 4 kh + j of column n in s[i][4 g + j]
  f32x16_t s[TPW];
  const bool holds = !outputs && wave < NT;
  const bool fresh = a.pos.position() == 0;
#pragma unroll
  for (int i = 0; i < TPW; ++i)
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const int d = 32 * (wave + 4 * i) + 8 * g + 4 * kh;
      f32x4_t x = {0.0f, 0.0f, 0.0f, 0.0f};
      if (!fresh && holds && d < dimp && n < nv) x = *reinterpret_cast<const f32x4_t*>(state + d);
#pragma unroll
      for (int j = 0; j < 4; ++j) s[i][4 * g + j] = x[j];
    }

  bf16x8_t kr[KP], vr[2];
  auto load = [&](int c0) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int pc = tid + 512 * i, row = pc / (D / 8), at = (pc % (D / 8)) * 8;
      kr[i] = piece(k + (int64_t)min(c0 + row, M - 1) * a.ldp, at, a.dim);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
      if (outputs) vr[i] = piece(v + (int64_t)min(c0 + 2 * lane + i, M - 1) * a.ldp, 8 * wave, nv);
  };
  // this lane's query: token 32 wave + n
  const int tq = 32 * wave + n;
  bf16x8_t qop[D / 16];
  auto load_q = [&](int c0) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < D / 16; ++i)
      qop[i] = piece(q + (int64_t)min(c0 + tq, M - 1) * a.ldp, 16 * i + 8 * kh, a.dim);
  };
  // decay^(31 - s) for this lane's rows s of a tile of 32
  float wr[16];
#pragma unroll
  for (int i = 0; i < 16; ++i) wr[i] = __builtin_amdgcn_exp2f((float)(31 - (8 * (i >> 2) + 4 * kh + (i & 3))) * lg);
  load(0);
  if (outputs) load_q(0);
  for (int c0 = 0; c0 < M; c0 += kChunk) {
    const int len = min(kChunk, M - c0);
    __syncthreads();  // the previous chunk's readers are done
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int pc = tid + 512 * i, row = pc / (D / 8), at = (pc % (D / 8)) * 8;
      *reinterpret_cast<bf16x8_t*>(ks + row * KS + at) = kr[i];
    }
    if (outputs) {
      // tokens 2 lane, 2 lane + 1, columns 8 wave ..; v' = decay^(len - 1 - t) v, nothing behind the last token
      float w[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int t = 2 * lane + i;
        w[i] = t < len ? __builtin_amdgcn_exp2f((float)(len - 1 - t) * lg) : 0.0f;
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        typedef bf16_t bf16x2_t __attribute__((ext_vector_type(2)));
        bf16x2_t out[4];
#pragma unroll
        for (int i = 0; i < 2; ++i) {
          float x = w[i] * (float)vr[i][e];
          out[0][i] = vr[i][e];
#pragma unroll
          for (int m = 1; m < 4; ++m) {
            out[m][i] = (bf16_t)x;
            x -= (float)out[m][i];
          }
        }
#pragma unroll
        for (int m = 0; m < 4; ++m)
          *reinterpret_cast<bf16x2_t*>(vt + (m * 32 + 8 * wave + e) * kVStride + 2 * lane) = out[m];
      }
    }
    if (holds) {
#pragma unroll
      for (int i = 0; i < TPW; ++i)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          bf16x4_t out[3];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            float x = s[i][4 * g + j];
#pragma unroll
            for (int m = 0; m < 3; ++m) {
              out[m][j] = (bf16_t)x;
              x -= (float)out[m][j];
            }
          }
#pragma unroll
          for (int m = 0; m < 3; ++m)
            *reinterpret_cast<bf16x4_t*>(st + (m * 32 + n) * SS + 32 * (wave + 4 * i) + 8 * g + 4 * kh) = out[m];
        }
    }
    __syncthreads();
    if (c0 + kChunk < M) load(c0 + kChunk);

    if (outputs && 32 * wave < len) {
      // one accumulator per term of the state: three independent chains of matrix instructions
      f32x16_t om[3];
#pragma unroll
      for (int m = 0; m < 3; ++m)
#pragma unroll
        for (int i = 0; i < 16; ++i) om[m][i] = 0.0f;
#pragma unroll
      for (int i = 0; i < D / 16; ++i)
#pragma unroll
        for (int m = 0; m < 3; ++m) {
          const bf16x8_t sv = *reinterpret_cast<const bf16x8_t*>(st + (m * 32 + n) * SS + 16 * i + 8 * kh);
          om[m] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sv, qop[i], om[m], 0, 0, 0);
        }
      const float wq = __builtin_amdgcn_exp2f((float)(tq + 1) * lg);
      f32x16_t o, o2;
#pragma unroll
      for (int i = 0; i < 16; ++i) o[i] = (om[0][i] + (om[1][i] + om[2][i])) * wq, o2[i] = 0.0f;
      for (int s0 = 0; s0 <= 32 * wave; s0 += 32) {
        f32x16_t w, w2;
#pragma unroll
        for (int i = 0; i < 16; ++i) w[i] = 0.0f, w2[i] = 0.0f;
#pragma unroll
        for (int i = 0; i < D / 16; i += 2) {
          const bf16_t* at = ks + (s0 + n) * KS + 16 * i + 8 * kh;
          w = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8_t*>(at), qop[i], w, 0, 0, 0);
          w2 = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8_t*>(at + 16), qop[i + 1], w2, 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) w[i] += w2[i];
        // decay^(t - s) = decay^(t - 31 - s0) decay^(31 + s0 - s); in the diagonal tile only s <= t counts
        if (s0 < 32 * wave) {
          const float wc = __builtin_amdgcn_exp2f((float)(tq - 31 - s0) * lg);
#pragma unroll
          for (int i = 0; i < 16; ++i) w[i] *= wr[i] * wc;
        } else {
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            const int back = tq - (s0 + 8 * (i >> 2) + 4 * kh + (i & 3));
            w[i] = back >= 0 ? w[i] * __builtin_amdgcn_exp2f((float)back * lg) : 0.0f;
          }
        }
        bf16x8_t hi[2], lo[2];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const float x = w[i];
          hi[i >> 3][i & 7] = (bf16_t)x;
          lo[i >> 3][i & 7] = (bf16_t)(x - (float)hi[i >> 3][i & 7]);
        }
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          const bf16_t* at = vt + n * kVStride + s0 + 16 * j + 4 * kh;
          const bf16x4_t l4 = *reinterpret_cast<const bf16x4_t*>(at), h4 = *reinterpret_cast<const bf16x4_t*>(at + 8);
          const bf16x8_t vv = {l4[0], l4[1], l4[2], l4[3], h4[0], h4[1], h4[2], h4[3]};
          o = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vv, hi[j], o, 0, 0, 0);
          o2 = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vv, lo[j], o2, 0, 0, 0);
        }
      }
#pragma unroll
      for (int i = 0; i < 16; ++i) o[i] += o2[i];
      if (c0 + kChunk < M) load_q(c0 + kChunk);
      if (tq < len) {
        float* out = a.o + (int64_t)(c0 + tq) * a.heads * a.vdim + (int64_t)head * a.vdim + v0;
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          const int c = 8 * g + 4 * kh;
          if (c + 3 < nv && (a.vdim & 3) == 0) {
            *reinterpret_cast<f32x4_t*>(out + c) = f32x4_t{o[4 * g], o[4 * g + 1], o[4 * g + 2], o[4 * g + 3]};
          } else {
#pragma unroll
            for (int j = 0; j < 4; ++j)
              if (c + j < nv) out[c + j] = o[4 * g + j];
          }
        }
      }
    }
    if (holds) {
      const float ws = __builtin_amdgcn_exp2f((float)len * lg);
      const int L16 = lane & 15;
      const bf16_t* const klane = ks + (4 * kh + (L16 >> 2)) * KS + 16 * ((lane >> 4) & 1) + 4 * (L16 & 3);
      f32x16_t sl[TPW];  // the smaller terms, apart: two chains
#pragma unroll
      for (int i = 0; i < TPW; ++i)
#pragma unroll
        for (int j = 0; j < 16; ++j) s[i][j] *= ws, sl[i][j] = 0.0f;
      for (int t0 = 0; t0 < len; t0 += 16) {
        bf16x8_t vv[3];
#pragma unroll
        for (int m = 0; m < 3; ++m) {
          const bf16_t* at = vt + ((m + 1) * 32 + n) * kVStride + t0 + 4 * kh;
          const bf16x4_t l4 = *reinterpret_cast<const bf16x4_t*>(at), h4 = *reinterpret_cast<const bf16x4_t*>(at + 8);
          vv[m] = bf16x8_t{l4[0], l4[1], l4[2], l4[3], h4[0], h4[1], h4[2], h4[3]};
        }
#pragma unroll
        for (int i = 0; i < TPW; ++i) {
          const bf16_t* at = klane + t0 * KS + 32 * (wave + 4 * i);
          const short4_t l = __builtin_amdgcn_ds_read_tr16_b64_v4i16((short4_t __attribute__((address_space(3)))*)at);
          const short4_t h = __builtin_amdgcn_ds_read_tr16_b64_v4i16((short4_t __attribute__((address_space(3)))*)(at + 8 * KS));
          const bf16x4_t l4 = __builtin_bit_cast(bf16x4_t, l), h4 = __builtin_bit_cast(bf16x4_t, h);
          const bf16x8_t kv = {l4[0], l4[1], l4[2], l4[3], h4[0], h4[1], h4[2], h4[3]};
#pragma unroll
          for (int m = 0; m < 3; ++m) {
            if (m == 0) s[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kv, vv[m], s[i], 0, 0, 0);
            else sl[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kv, vv[m], sl[i], 0, 0, 0);
          }
        }
      }
#pragma unroll
      for (int i = 0; i < TPW; ++i)
#pragma unroll
        for (int j = 0; j < 16; ++j) s[i][j] += sl[i][j];
    }
  }
  if (holds && n < nv)
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int d = 32 * (wave + 4 * i) + 8 * g + 4 * kh;
        if (d < dimp)
          *reinterpret_cast<f32x4_t*>(state + d) = f32x4_t{s[i][4 * g], s[i][4 * g + 1], s[i][4 * g + 2], s[i][4 * g + 3]};
      }
}

template <int D, bool WHOLE>
int launch_chunks(const LinearAttnArgs& a, hipStream_t st) {
  static bool raised = false;  // more LDS than the default limit of a launch
  if (!raised) {
    AWQ_HIP_TRY(hipFuncSetAttribute((const void*)linear_chunk_kernel<D, WHOLE>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                    linear_chunk_lds<D>()));
    raised = true;
  }
  hipLaunchKernelGGL((linear_chunk_kernel<D, WHOLE>), dim3((unsigned)a.heads, (unsigned)((a.vdim + 31) / 32)), dim3(512),
                     linear_chunk_lds<D>(), st, a);
  AWQ_HIP_TRY(hipGetLastError());
  return AWQ_OK;
}

// below this many tokens the token-by-token form is as fast
constexpr int kChunkFrom = 16;

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
  AWQ_REQUIRE(a.heads >= 1 && a.dim >= 1 && a.vdim >= 1 && a.vdim <= 65536 && a.ldp % 8 == 0 &&
                  a.ldp >= (int64_t)a.heads * (2 * a.dim + a.vdim),
              "bad shape");
  if (f32) return launch_step<float>(a, st);
  if (a.log2_decay && a.M >= kChunkFrom && a.M < (1 << 30) && a.dim <= 256) {
    const bool whole = ((a.dim | a.vdim) & 7) == 0;
    if (a.dim <= 64) return whole ? launch_chunks<64, true>(a, st) : launch_chunks<64, false>(a, st);
    if (a.dim <= 128) return whole ? launch_chunks<128, true>(a, st) : launch_chunks<128, false>(a, st);
    return whole ? launch_chunks<256, true>(a, st) : launch_chunks<256, false>(a, st);
  }
  return launch_step<bf16_t>(a, st);
}
