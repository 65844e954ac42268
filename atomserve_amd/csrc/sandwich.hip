// Steps around sublayers whose output is normed again before it enters the stream, and two steps inside them.
//
//   post_norm_add   x += norm(y) * post; out = norm(x) * gain: the norm after a sublayer, the residual sum and the norm
//                   before the next sublayer in one pass over the row; y may be the sum of two outputs that are
//                   normed first, each with gains of its own
//   poly_norm       a N(z) + b N(z^2) + c N(z^3) + e over a row z, powers taken element by element and N the division
//                   by the row's root mean square
//   map_difference  two attention maps' heads a1 - lam a2, over its root mean square, times a factor
//
// A row stays in registers between its reductions.  Everything between the loads and the last rounding is fp32.
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

struct PostNorm {
  const float* bias1;  // [n] added to y1, y2 as they are read (null: none)
  const float* bias2;
  const float* gain1;  // PAIR: y = norm(y1) gain1 + norm(y2) gain2
  const float* gain2;
  float eps_in;
  const float* post;   // [n] gains of the norm after the sublayer
  float eps_post;
  const float* gain;   // [n] gains of the norm that follows (null: none is taken)
  float eps;
};

// A workgroup per row; a thread owns CH pieces of VEC neighbouring columns.
template <typename T, int VEC, int CH, bool PAIR>
__global__ __launch_bounds__(1024) void post_norm_add_kernel(float* __restrict__ x, const T* __restrict__ y1,
                                                             const T* __restrict__ y2, PostNorm p,
                                                             const int* __restrict__ rows, T* __restrict__ out, int n,
                                                             int update_x) {
  __shared__ float red[2 * 16];
  const int r = blockIdx.x;
  const size_t s = rows ? (size_t)rows[r] : (size_t)r;
  float d[CH][VEC], v[CH][VEC];
  float sums[PAIR ? 2 : 1] = {};
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
#pragma unroll
    for (int k = 0; k < VEC; ++k) d[c][k] = v[c][k] = 0.f;
    if (i < n) {
      float b[VEC];
      load_vec<VEC>(y1 + s * n + i, d[c]);
      if (p.bias1) {
        load_vec<VEC>(p.bias1 + i, b);
#pragma unroll
        for (int k = 0; k < VEC; ++k) d[c][k] += b[k];
      }
      if (PAIR) {
        load_vec<VEC>(y2 + s * n + i, v[c]);
        if (p.bias2) {
          load_vec<VEC>(p.bias2 + i, b);
#pragma unroll
          for (int k = 0; k < VEC; ++k) v[c][k] += b[k];
        }
      }
    }
#pragma unroll
    for (int k = 0; k < VEC; ++k) {
      sums[0] = fmaf(d[c][k], d[c][k], sums[0]);
      if (PAIR) sums[PAIR ? 1 : 0] = fmaf(v[c][k], v[c][k], sums[PAIR ? 1 : 0]);
    }
  }
  block_sums(sums, red);
  float one[1];
  if (PAIR) {
    const float inv1 = 1.0f / sqrtf(sums[0] / (float)n + p.eps_in), inv2 = 1.0f / sqrtf(sums[PAIR ? 1 : 0] / (float)n + p.eps_in);
    one[0] = 0.f;
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const int i = (c * blockDim.x + threadIdx.x) * VEC;
      if (i >= n) continue;
      float g1[VEC], g2[VEC];
      load_vec<VEC>(p.gain1 + i, g1);
      load_vec<VEC>(p.gain2 + i, g2);
#pragma unroll
      for (int k = 0; k < VEC; ++k) {
        d[c][k] = d[c][k] * inv1 * g1[k] + v[c][k] * inv2 * g2[k];
        one[0] = fmaf(d[c][k], d[c][k], one[0]);
      }
    }
    block_sums(one, red);
  } else {
    one[0] = sums[0];
  }
  const float inv_post = 1.0f / sqrtf(one[0] / (float)n + p.eps_post);
  one[0] = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
    if (i >= n) continue;
    float g[VEC];
    load_vec<VEC>(p.post + i, g);
    load_vec<VEC>(x + s * n + i, v[c]);
#pragma unroll
    for (int k = 0; k < VEC; ++k) {
      v[c][k] += d[c][k] * inv_post * g[k];
      one[0] = fmaf(v[c][k], v[c][k], one[0]);
    }
    if (update_x) store_vec<VEC>(x + s * n + i, v[c]);
  }
  if (!p.gain) return;
  block_sums(one, red);
  const float inv = 1.0f / sqrtf(one[0] / (float)n + p.eps);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
    if (i >= n) continue;
    float g[VEC];
    load_vec<VEC>(p.gain + i, g);
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[c][k] *= inv * g[k];
    store_vec<VEC>(out + (size_t)r * n + i, v[c]);
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

template <typename T, int VEC>
static int launch_post_norm(float* x, const void* y1, const void* y2, const PostNorm& p, const int* rows, void* out, int n_out,
                            int n, int update_x, hipStream_t stream) {
  int threads, ch;
  if (!row_shape(n_out, n, VEC, &threads, &ch)) return AS_BAD_SHAPE;
#define LAUNCH(CHV)                                                                                                    \
  if (y2) post_norm_add_kernel<T, VEC, CHV, true><<<n_out, threads, 0, stream>>>(x, (const T*)y1, (const T*)y2, p, rows, \
                                                                                 (T*)out, n, update_x);                \
  else post_norm_add_kernel<T, VEC, CHV, false><<<n_out, threads, 0, stream>>>(x, (const T*)y1, nullptr, p, rows, (T*)out, \
                                                                               n, update_x)
  switch (ch) {
    case 1: LAUNCH(1); break;
    case 2: LAUNCH(2); break;
    case 4: LAUNCH(4); break;
    case 8: LAUNCH(8); break;
    default:  // long rows of a width that is no multiple of four
      if constexpr (VEC == 1) {
        if (ch == 16) { LAUNCH(16); }
        else { LAUNCH(32); }
      }
      break;
  }
#undef LAUNCH
  return launch_status();
}

// x fp32 [T, n]; y1, y2 [T, n] and out [n_out, n] of `dtype`; row r of out comes from row rows[r] (or r) of the rest.
extern "C" int as_post_norm_add(float* x, const void* y1, const void* y2, int dtype, const float* bias1, const float* bias2,
                                const float* gain1, const float* gain2, float eps_in, const float* post, float eps_post,
                                const float* gain, float eps, const int* rows, void* out, int n_out, int n,
                                int update_x, hipStream_t stream) {
  if (n_out <= 0) return AS_OK;
  if (n <= 0 || !x || !y1 || !post || (gain && !out) || (y2 && (!gain1 || !gain2)) || (!y2 && bias2)) return AS_BAD_SHAPE;
  const PostNorm p = {bias1, bias2, gain1, gain2, eps_in, post, eps_post, gain, eps};
  if (dtype == DT_F32)
    return n % 4 ? launch_post_norm<float, 1>(x, y1, y2, p, rows, out, n_out, n, update_x, stream)
                 : launch_post_norm<float, 4>(x, y1, y2, p, rows, out, n_out, n, update_x, stream);
  if (dtype == DT_BF16)
    return n % 4 ? launch_post_norm<bf16, 1>(x, y1, y2, p, rows, out, n_out, n, update_x, stream)
                 : launch_post_norm<bf16, 4>(x, y1, y2, p, rows, out, n_out, n, update_x, stream);
  return AS_BAD_DTYPE;
}

// ---- a polynomial of normed powers ------------------------------------------------------------------------------
template <typename T, int VEC, int CH>
__global__ __launch_bounds__(1024) void poly_norm_kernel(const T* __restrict__ z, const float* __restrict__ coef, float eps,
                                                         T* __restrict__ out, int n) {
  __shared__ float red[3 * 16];
  const T* row = z + (size_t)blockIdx.x * n;
  float v[CH][VEC], s[3] = {0.f, 0.f, 0.f};
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[c][k] = 0.f;
    if (i < n) load_vec<VEC>(row + i, v[c]);
#pragma unroll
    for (int k = 0; k < VEC; ++k) {
      const float q = v[c][k] * v[c][k], w = q * v[c][k];
      s[0] += q;
      s[1] = fmaf(q, q, s[1]);
      s[2] = fmaf(w, w, s[2]);
    }
  }
  block_sums(s, red);
  const float a = coef[0] / sqrtf(s[0] / (float)n + eps), b = coef[1] / sqrtf(s[1] / (float)n + eps);
  const float cc = coef[2] / sqrtf(s[2] / (float)n + eps), e = coef[3];
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
    if (i >= n) continue;
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[c][k] = fmaf(fmaf(fmaf(cc, v[c][k], b), v[c][k], a), v[c][k], e);
    store_vec<VEC>(out + (size_t)blockIdx.x * n + i, v[c]);
  }
}

template <typename T, int VEC>
static int launch_poly_norm(const void* z, const float* coef, float eps, void* out, int num_tokens, int n, hipStream_t stream) {
  int threads, ch;
  if (!row_shape(num_tokens, n, VEC, &threads, &ch)) return AS_BAD_SHAPE;
#define LAUNCH(CHV) poly_norm_kernel<T, VEC, CHV><<<num_tokens, threads, 0, stream>>>((const T*)z, coef, eps, (T*)out, n)
  switch (ch) {
    case 1: LAUNCH(1); break;
    case 2: LAUNCH(2); break;
    case 4: LAUNCH(4); break;
    case 8: LAUNCH(8); break;
    default:  // long rows of a width that is no multiple of four
      if constexpr (VEC == 1) {
        if (ch == 16) { LAUNCH(16); }
        else { LAUNCH(32); }
      }
      break;
  }
#undef LAUNCH
  return launch_status();
}

// z, out [T, n] of `dtype`; coef fp32 [4]: a, b, c, e.
extern "C" int as_poly_norm(const void* z, int dtype, const float* coef, float eps, void* out, int num_tokens, int n,
                            hipStream_t stream) {
  if (num_tokens <= 0) return AS_OK;
  if (n <= 0 || !z || !coef || !out) return AS_BAD_SHAPE;
  if (dtype == DT_F32)
    return n % 4 ? launch_poly_norm<float, 1>(z, coef, eps, out, num_tokens, n, stream)
                 : launch_poly_norm<float, 4>(z, coef, eps, out, num_tokens, n, stream);
  if (dtype == DT_BF16)
    return n % 4 ? launch_poly_norm<bf16, 1>(z, coef, eps, out, num_tokens, n, stream)
                 : launch_poly_norm<bf16, 4>(z, coef, eps, out, num_tokens, n, stream);
  return AS_BAD_DTYPE;
}

// ---- the difference of two attention maps -------------------------------------------------------------------------
// heads [T, 2 H, Dp]: head h's first map at 2 h, its second at 2 h + 1, the first E of Dp coordinates count.  A wave per
// (token, head): o = a1 - lam a2; out[t, out_off + h E + j] = mult * o_j / sqrt(mean(o^2) + eps).  E <= 4 * WAVE * PIECES.
#define DIFF_PIECES 8

template <typename T, typename O, int VEC>
__global__ __launch_bounds__(256) void map_difference_kernel(const T* __restrict__ heads, int H, int E, int Dp, float lam,
                                                             float eps, float mult, O* __restrict__ out, int ld_out,
                                                             int out_off, int total) {
  const int item = blockIdx.x * 4 + threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  if (item >= total) return;
  const size_t t = item / H;
  const int h = item % H;
  const T* a1 = heads + (t * 2 * H + 2 * h) * Dp;
  const T* a2 = a1 + Dp;
  float o[DIFF_PIECES][VEC], ss = 0.f;
#pragma unroll
  for (int c = 0; c < DIFF_PIECES; ++c) {
    const int i = (c * WAVE + lane) * VEC;
    if (i < E) {
      float b[VEC];
      load_vec<VEC>(a1 + i, o[c]);
      load_vec<VEC>(a2 + i, b);
#pragma unroll
      for (int k = 0; k < VEC; ++k) {
        o[c][k] -= lam * b[k];
        ss = fmaf(o[c][k], o[c][k], ss);
      }
    }
  }
  ss = wave_sum(ss);
  const float f = mult / sqrtf(ss / (float)E + eps);
  O* dst = out + t * ld_out + out_off + h * E;
#pragma unroll
  for (int c = 0; c < DIFF_PIECES; ++c) {
    const int i = (c * WAVE + lane) * VEC;
    if (i < E) {
#pragma unroll
      for (int k = 0; k < VEC; ++k) o[c][k] *= f;
      store_vec<VEC>(dst + i, o[c]);
    }
  }
}

extern "C" int as_map_difference(const void* heads, int dtype, int H, int E, int Dp, float lam, float eps, float mult, void* out,
                                 int out_dtype, int ld_out, int out_off, int num_tokens, hipStream_t stream) {
  if (num_tokens <= 0) return AS_OK;
  if (H <= 0 || E <= 0 || Dp < E || out_off < 0 || out_off + H * E > ld_out) return AS_BAD_SHAPE;
  const bool four = E % 4 == 0 && Dp % 4 == 0 && ld_out % 4 == 0 && out_off % 4 == 0;
  if (E > (four ? 4 : 1) * WAVE * DIFF_PIECES) return AS_BAD_SHAPE;
  if ((long)num_tokens * H > 0x7fffffffL) return AS_BAD_SHAPE;
  const int total = num_tokens * H, blocks = (total + 3) / 4;
#define LAUNCH(T, O)                                                                                                              \
  if (four) map_difference_kernel<T, O, 4><<<blocks, 256, 0, stream>>>((const T*)heads, H, E, Dp, lam, eps, mult, (O*)out, ld_out, \
                                                                       out_off, total);                                          \
  else map_difference_kernel<T, O, 1><<<blocks, 256, 0, stream>>>((const T*)heads, H, E, Dp, lam, eps, mult, (O*)out, ld_out,      \
                                                                  out_off, total)
  if (dtype == DT_F32 && out_dtype == DT_F32) { LAUNCH(float, float); }
  else if (dtype == DT_F32 && out_dtype == DT_BF16) { LAUNCH(float, bf16); }
  else if (dtype == DT_BF16 && out_dtype == DT_BF16) { LAUNCH(bf16, bf16); }
  else return AS_BAD_DTYPE;
#undef LAUNCH
  return launch_status();
}
