// Routed feed-forward (layers.hpp): which outputs of a router a token takes and with what weight, and the plan by which the
// tokens of a pass are brought to their experts' products.
#include "layers.hpp"

namespace {

// the lanes' LDS writes ahead of this are seen by all lanes' reads behind it
__device__ __forceinline__ void wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

// (value, lowest index) of the largest value of a wavefront
__device__ __forceinline__ void best_of_wave(float& v, int& i) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) {
    const float ov = __shfl_xor(v, off, 64);
    const int oi = __shfl_xor(i, off, 64);
    if (ov > v || (ov == v && oi < i)) v = ov, i = oi;
  }
}

// A wavefront per token.  LDS per wavefront: scores, choice scores, group scores.
template <int WAVES>
__global__ __launch_bounds__(WAVES * 64) void route_kernel(RouteArgs a) {
  extern __shared__ float lds[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, E = a.outputs;
  const int64_t t = (int64_t)blockIdx.x * WAVES + wave;
  float* const s = lds + wave * (2 * E + a.groups);
  float* const choice = s + E;
  float* const best = choice + E;
  if (t >= a.M) return;  // (no barrier below: a wavefront's LDS is its own)
  const float* const z = a.logits + t * a.ld;
  float m = -INFINITY, sum = 0.0f;
  for (int i = lane; i < E; i += 64) m = fmaxf(m, z[i]);
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) m = fmaxf(m, __shfl_xor(m, off, 64));
  for (int i = lane; i < E; i += 64) {
    const float e = expf(z[i] - m);
    s[i] = e;
    sum += e;
  }
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) sum += __shfl_xor(sum, off, 64);
  for (int i = lane; i < E; i += 64) {
    const float v = s[i] / sum;
    s[i] = v;
    choice[i] = a.correction ? v + a.correction[i] : v;
  }
  wave_sync();
  if (a.groups > 0) {
    const int size = E / a.groups;
    for (int g = lane; g < a.groups; g += 64) {
      float v = -INFINITY;
      for (int i = 0; i < size; ++i) v = fmaxf(v, choice[g * size + i]);
      best[g] = v;
    }
    wave_sync();
    // the groups that stay are marked with NaN, one after the other
    for (int k = 0; k < a.keep; ++k) {
      float v = -INFINITY;
      int at = 1 << 30;
      for (int g = lane; g < a.groups; g += 64)
        if (best[g] > v || (best[g] == v && g < at)) v = best[g], at = g;
      best_of_wave(v, at);
      if (lane == 0 && at < a.groups) best[at] = __builtin_nanf("");
      wave_sync();
    }
    for (int i = lane; i < E; i += 64) {
      const float b = best[i / size];
      if (b == b) choice[i] = -INFINITY;
    }
    wave_sync();
  }
  float total = 0.0f;
  for (int k = 0; k < a.top; ++k) {
    float v = -INFINITY;
    int at = 1 << 30;
    for (int i = lane; i < E; i += 64)
      if (choice[i] > v || (choice[i] == v && i < at && v != -INFINITY)) v = choice[i], at = i;
    best_of_wave(v, at);
    const bool found = at < E;
    const float w = found ? s[at] : 0.0f;
    total += w;
    if (lane == 0) {
      // (fewer finite choices than `top`: the place goes to an identity output of weight zero)
      a.ids[t * a.top + k] = found ? at : a.experts;
      a.weights[t * a.top + k] = w;
      if (found) choice[at] = -INFINITY;
    }
    wave_sync();
  }
  if (lane == 0)
    for (int k = 0; k < a.top; ++k) a.weights[t * a.top + k] /= total + 1e-20f;
}

// One workgroup.  Counts the tokens of every expert, lays their runs one behind the other in the list, cut into tiles.
__global__ __launch_bounds__(1024) void plan_kernel(RouteArgs a, int max_tiles) {
  extern __shared__ int counts[];  // [experts] counts, then [experts] next place
  __shared__ int wave_entries[16], wave_tiles[16], before[2];
  int* const next = counts + a.experts;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, E = a.experts;
  const int n = (int)a.M * a.top;
  for (int e = tid; e < E; e += 1024) counts[e] = 0;
  if (tid == 0) before[0] = before[1] = 0;
  __syncthreads();
  for (int p = tid; p < n; p += 1024) {
    const int e = a.ids[p];
    if (e < E) atomicAdd(&counts[e], 1);
  }
  __syncthreads();
  for (int e0 = 0; e0 < E; e0 += 1024) {
    const int e = e0 + tid, c = e < E ? counts[e] : 0, k = (c + a.tile_tokens - 1) / a.tile_tokens;
    int entries = c, tiles = k;  // sums up to and with this expert
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const int pe = __shfl_up(entries, off, 64), pt = __shfl_up(tiles, off, 64);
      if (lane >= off) entries += pe, tiles += pt;
    }
    if (lane == 63) wave_entries[wave] = entries, wave_tiles[wave] = tiles;
    __syncthreads();
    int base_e = before[0], base_t = before[1];
    for (int w = 0; w < wave; ++w) base_e += wave_entries[w], base_t += wave_tiles[w];
    const int at = base_e + entries - c, tile = base_t + tiles - k;
    if (e < E) {
      next[e] = at;
      for (int i = 0; i < k; ++i) {
        DenseTile d;
        d.group = e;
        d.first = at + i * a.tile_tokens;
        d.count = min(a.tile_tokens, c - i * a.tile_tokens);
        a.tiles[tile + i] = d;
      }
    }
    __syncthreads();
    if (tid == 1023) before[0] = base_e + entries, before[1] = base_t + tiles;
    __syncthreads();
  }
  for (int i = before[1] + tid; i < max_tiles; i += 1024) a.tiles[i] = DenseTile{0, 0, 0};
  for (int p = tid; p < n; p += 1024) {
    const int e = a.ids[p];
    if (e < E) a.list[atomicAdd(&next[e], 1)] = p;
  }
}

}  // namespace

// a run of each expert may end in a tile that is not full
int32_t route_max_tiles(int64_t M, int32_t top, int32_t experts, int32_t tile_tokens) {
  const int64_t pairs = M * top;
  return (int32_t)std::max<int64_t>(1, std::min<int64_t>(pairs, pairs / tile_tokens + std::min<int64_t>(experts, pairs)));
}

int32_t route_tile_tokens(int64_t M, int32_t top, int32_t outputs, bool f32) { return !f32 && M * top >= 128ll * outputs ? 128 : 64; }

int launch_route(const RouteArgs& a, hipStream_t st) {
  AWQ_REQUIRE(a.logits && a.ids && a.weights && a.M >= 1, "bad arguments");
  AWQ_REQUIRE(a.outputs >= 1 && a.outputs <= 4096 && a.experts >= 0 && a.experts <= a.outputs && a.top >= 1 && a.top <= a.outputs,
              "bad router");
  AWQ_REQUIRE(a.groups == 0 || (a.groups > 0 && a.outputs % a.groups == 0 && a.keep >= 1 && a.keep <= a.groups &&
                                a.keep * (a.outputs / a.groups) >= a.top),
              "bad groups");
  AWQ_REQUIRE(a.M * a.top < (1 << 30) && a.tile_tokens >= 1, "too many tokens");
  const size_t lds = sizeof(float) * (2 * a.outputs + a.groups);
  if (a.outputs <= 1024)
    hipLaunchKernelGGL(route_kernel<4>, dim3((unsigned)((a.M + 3) / 4)), dim3(256), 4 * lds, st, a);
  else
    hipLaunchKernelGGL(route_kernel<1>, dim3((unsigned)a.M), dim3(64), lds, st, a);
  AWQ_HIP_TRY(hipGetLastError());
  if (a.M > 1 && a.experts > 0) {
    AWQ_REQUIRE(a.tiles && a.list, "no place for the plan");
    hipLaunchKernelGGL(plan_kernel, dim3(1), dim3(1024), sizeof(int) * 2 * a.experts, st, a, route_max_tiles(a.M, a.top, a.experts, a.tile_tokens));
    AWQ_HIP_TRY(hipGetLastError());
  }
  return AWQ_OK;
}
