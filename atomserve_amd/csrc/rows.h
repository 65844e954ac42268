// Rows that stay in registers between their reductions: loads and stores of neighbouring values, sums over a workgroup,
// and how many threads take a row.
#pragma once
#include "common.h"

// VEC consecutive values at once (4: the address a multiple of 16 bytes for fp32, of 8 for bfloat16).
template <int VEC, typename T> __device__ __forceinline__ void load_vec(const T* p, float* v) {
  if constexpr (VEC == 1) {
    v[0] = to_f32(p[0]);
  } else if constexpr (sizeof(T) == 4) {
    const float4 r = *reinterpret_cast<const float4*>(p);
    v[0] = r.x; v[1] = r.y; v[2] = r.z; v[3] = r.w;
  } else {
    const uint2 r = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(r.x << 16); v[1] = __uint_as_float(r.x & 0xffff0000u);
    v[2] = __uint_as_float(r.y << 16); v[3] = __uint_as_float(r.y & 0xffff0000u);
  }
}
template <int VEC, typename T> __device__ __forceinline__ void store_vec(T* p, const float* v) {
  if constexpr (VEC == 1) {
    p[0] = from_f32<T>(v[0]);
  } else if constexpr (sizeof(T) == 4) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  } else {
    bf16 b[4] = {from_f32<bf16>(v[0]), from_f32<bf16>(v[1]), from_f32<bf16>(v[2]), from_f32<bf16>(v[3])};
    *reinterpret_cast<uint2*>(p) = *reinterpret_cast<const uint2*>(b);
  }
}

// N sums over the workgroup at once (up to 16 waves), in a fixed order; `red` is a __shared__ float[N * 16].
template <int N>
__device__ __forceinline__ void block_sums(float (&v)[N], float* red) {
  const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE, waves = blockDim.x / WAVE;
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = wave_sum(v[i]);
  if (waves == 1) return;
  __syncthreads();  // protects `red` against a previous use
  if (lane == 0) {
#pragma unroll
    for (int i = 0; i < N; ++i) red[i * 16 + wave] = v[i];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < N; ++i) {
    float s = 0.f;
    for (int w = 0; w < waves; ++w) s += red[i * 16 + w];
    v[i] = s;
  }
}

// How many threads take a row and in how many pieces each: few rows (a decode step) as wide as they come, many rows
// with more in a thread's registers.  False: the row is longer than the kernels keep.
static bool row_shape(int rows, int n, int vec, int* threads, int* pieces) {
  const int want = (n + vec - 1) / vec;
  int ch = rows >= 512 ? 4 : 1;
  while (ch > 1 && want <= 64 * ch / 2) ch /= 2;
  while (ch < (vec == 1 ? 32 : 8) && (want + ch - 1) / ch > 1024) ch *= 2;
  const int t = ((want + ch - 1) / ch + 63) / 64 * 64;
  if (t > 1024) return false;
  *threads = t;
  *pieces = ch;
  return true;
}
