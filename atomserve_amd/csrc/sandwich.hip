// Steps around sublayers whose output is normed again before it enters the stream, and two steps inside them.
//
//   post_norm_add   x += norm(y) * post; out = norm(x) * gain: the norm after a sublayer, the residual sum and the norm
//                   before the next sublayer in one pass over the row; y may be the sum of two outputs that are
//                   normed first, each with gains of its own; either norm divides by the root mean square or, centred,
//                   takes the mean off first; out may also be x as it is, rounded
//   poly_norm       a N(z) + b N(z^2) + c N(z^3) + e over a row z, powers taken element by element and N the division
//                   by the row's root mean square
//   token_gate      gelu(z) times a row of a table that the token names
//   map_difference  two attention maps' heads a1 - lam a2, over its root mean square, times a factor
//
// A row stays in registers between its reductions.  Everything between the loads and the last rounding is fp32.
#include "common.h"
#include "rows.h"

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
  int centre_post;     // CENTRED: the norm after the sublayer takes the mean off first (a layer norm)
  int centre;          // CENTRED: the norm that follows does
};

// A workgroup per row; a thread owns CH pieces of VEC neighbouring columns.
template <typename T, int VEC, int CH, bool PAIR, bool CENTRED>
__global__ __launch_bounds__(1024) void post_norm_add_kernel(float* __restrict__ x, const T* __restrict__ y1,
                                                             const T* __restrict__ y2, PostNorm p,
                                                             const int* __restrict__ rows, T* __restrict__ out, int n,
                                                             int update_x) {
  __shared__ float red[2 * 16];
  const int r = blockIdx.x;
  const size_t s = rows ? (size_t)rows[r] : (size_t)r;
  float d[CH][VEC], v[CH][VEC];
  float sums[PAIR ? 2 : 1] = {};
  // few rows (one piece a thread): everything the row needs is asked for at once, not a reduction later each
  constexpr bool EARLY = CH == 1 && !PAIR;
  [[maybe_unused]] float x_early[VEC], post_early[VEC], gain_early[VEC];
  if constexpr (EARLY) {
    const int i = min((int)threadIdx.x * VEC, n - VEC);
    load_vec<VEC>(x + s * n + i, x_early);
    load_vec<VEC>(p.post + i, post_early);
    if (p.gain) load_vec<VEC>(p.gain + i, gain_early);
  }
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
      if (CENTRED && !PAIR) sums[0] += p.centre_post ? d[c][k] : d[c][k] * d[c][k];
      else sums[0] = fmaf(d[c][k], d[c][k], sums[0]);
      if (PAIR) sums[PAIR ? 1 : 0] = fmaf(v[c][k], v[c][k], sums[PAIR ? 1 : 0]);
    }
  }
  block_sums(sums, red);
  float one[1];
  // a row's mean comes off: what `one` holds is the row's sum, and then the sum of the squared deviations
  auto centre = [&](float(&r)[CH][VEC]) {
    const float mean = one[0] / (float)n;
    one[0] = 0.f;
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      if ((int)(c * blockDim.x + threadIdx.x) * VEC >= n) continue;
#pragma unroll
      for (int k = 0; k < VEC; ++k) {
        r[c][k] -= mean;
        one[0] = fmaf(r[c][k], r[c][k], one[0]);
      }
    }
    block_sums(one, red);
  };
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
        if (CENTRED) one[0] += p.centre_post ? d[c][k] : d[c][k] * d[c][k];
        else one[0] = fmaf(d[c][k], d[c][k], one[0]);
      }
    }
    block_sums(one, red);
  } else {
    one[0] = sums[0];
  }
  if (CENTRED && p.centre_post) centre(d);
  const float inv_post = 1.0f / sqrtf(one[0] / (float)n + p.eps_post);
  one[0] = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
    if (i >= n) continue;
    float g[VEC];
    if constexpr (EARLY) {
#pragma unroll
      for (int k = 0; k < VEC; ++k) { g[k] = post_early[k]; v[c][k] = x_early[k]; }
    } else {
      load_vec<VEC>(p.post + i, g);
      load_vec<VEC>(x + s * n + i, v[c]);
    }
#pragma unroll
    for (int k = 0; k < VEC; ++k) {
      v[c][k] += d[c][k] * inv_post * g[k];
      if (CENTRED) one[0] += p.centre ? v[c][k] : v[c][k] * v[c][k];
      else one[0] = fmaf(v[c][k], v[c][k], one[0]);
    }
    if (update_x) store_vec<VEC>(x + s * n + i, v[c]);
    if (!p.gain && out) store_vec<VEC>(out + (size_t)r * n + i, v[c]);
  }
  if (!p.gain) return;
  block_sums(one, red);
  if (CENTRED && p.centre) centre(v);
  const float inv = 1.0f / sqrtf(one[0] / (float)n + p.eps);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
    if (i >= n) continue;
    float g[VEC];
    if constexpr (EARLY) {
#pragma unroll
      for (int k = 0; k < VEC; ++k) g[k] = gain_early[k];
    } else {
      load_vec<VEC>(p.gain + i, g);
    }
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[c][k] *= inv * g[k];
    store_vec<VEC>(out + (size_t)r * n + i, v[c]);
  }
}

template <typename T, int VEC>
static int launch_post_norm(float* x, const void* y1, const void* y2, const PostNorm& p, const int* rows, void* out, int n_out,
                            int n, int update_x, hipStream_t stream) {
  int threads, ch;
  if (!row_shape(n_out, n, VEC, &threads, &ch)) return AS_BAD_SHAPE;
#define LAUNCH2(CHV, PAIRV, CENTREDV)                                                                                       \
  post_norm_add_kernel<T, VEC, CHV, PAIRV, CENTREDV><<<n_out, threads, 0, stream>>>(x, (const T*)y1, (const T*)y2, p, rows, \
                                                                                    (T*)out, n, update_x)
#define LAUNCH(CHV)                                                                \
  if (y2 && (p.centre || p.centre_post)) LAUNCH2(CHV, true, true);                 \
  else if (y2) LAUNCH2(CHV, true, false);                                          \
  else if (p.centre || p.centre_post) LAUNCH2(CHV, false, true);                   \
  else LAUNCH2(CHV, false, false)
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
#undef LAUNCH2
  return launch_status();
}

// x fp32 [T, n]; y1, y2 [T, n] and out [n_out, n] of `dtype`; row r of out comes from row rows[r] (or r) of the rest.
// centre_post, centre: the norm after the sublayer, the one that follows, take the row's mean off first.  gain null with
// out given: out receives the stream itself.
extern "C" int as_post_norm_add(float* x, const void* y1, const void* y2, int dtype, const float* bias1, const float* bias2,
                                const float* gain1, const float* gain2, float eps_in, const float* post, float eps_post,
                                const float* gain, float eps, int centre_post, int centre, const int* rows, void* out,
                                int n_out, int n, int update_x, hipStream_t stream) {
  if (n_out <= 0) return AS_OK;
  if (n <= 0 || !x || !y1 || !post || (gain && !out) || (y2 && (!gain1 || !gain2)) || (!y2 && bias2)) return AS_BAD_SHAPE;
  const PostNorm p = {bias1, bias2, gain1, gain2, eps_in, post, eps_post, gain, eps, centre_post, centre};
  if (dtype == DT_F32)
    return n % 4 ? launch_post_norm<float, 1>(x, y1, y2, p, rows, out, n_out, n, update_x, stream)
                 : launch_post_norm<float, 4>(x, y1, y2, p, rows, out, n_out, n, update_x, stream);
  if (dtype == DT_BF16)
    return n % 4 ? launch_post_norm<bf16, 1>(x, y1, y2, p, rows, out, n_out, n, update_x, stream)
                 : launch_post_norm<bf16, 4>(x, y1, y2, p, rows, out, n_out, n, update_x, stream);
  return AS_BAD_DTYPE;
}

// ---- a layer norm of the stream, with a plain output still to be added ---------------------------------------------
// v = x[s] (+ y[s]), s = rows[r] or r; x receives v if update_x; out[r] = (v - mean) / sqrt(mean((v - mean)^2) + eps) * gain.
template <typename T, int VEC, int CH>
__global__ __launch_bounds__(1024) void layer_norm_kernel(float* __restrict__ x, const T* __restrict__ y,
                                                          const float* __restrict__ gain, float eps,
                                                          const int* __restrict__ rows, T* __restrict__ out, int n, int update_x) {
  __shared__ float red[16];
  const int r = blockIdx.x;
  const size_t s = rows ? (size_t)rows[r] : (size_t)r;
  float v[CH][VEC], one[1] = {0.f};
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[c][k] = 0.f;
    if (i >= n) continue;
    load_vec<VEC>(x + s * n + i, v[c]);
    if (y) {
      float d[VEC];
      load_vec<VEC>(y + s * n + i, d);
#pragma unroll
      for (int k = 0; k < VEC; ++k) v[c][k] += d[k];
      if (update_x) store_vec<VEC>(x + s * n + i, v[c]);
    }
#pragma unroll
    for (int k = 0; k < VEC; ++k) one[0] += v[c][k];
  }
  block_sums(one, red);
  const float mean = one[0] / (float)n;
  one[0] = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    if ((int)(c * blockDim.x + threadIdx.x) * VEC >= n) continue;
#pragma unroll
    for (int k = 0; k < VEC; ++k) {
      v[c][k] -= mean;
      one[0] = fmaf(v[c][k], v[c][k], one[0]);
    }
  }
  block_sums(one, red);
  const float inv = 1.0f / sqrtf(one[0] / (float)n + eps);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
    if (i >= n) continue;
    float g[VEC];
    load_vec<VEC>(gain + i, g);
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[c][k] *= inv * g[k];
    store_vec<VEC>(out + (size_t)r * n + i, v[c]);
  }
}

template <typename T, int VEC>
static int launch_layer_norm(float* x, const void* y, const float* gain, float eps, const int* rows, void* out, int n_out, int n,
                             int update_x, hipStream_t stream) {
  int threads, ch;
  if (!row_shape(n_out, n, VEC, &threads, &ch)) return AS_BAD_SHAPE;
#define LAUNCH(CHV) layer_norm_kernel<T, VEC, CHV><<<n_out, threads, 0, stream>>>(x, (const T*)y, gain, eps, rows, (T*)out, n, update_x)
  switch (ch) {
    case 1: LAUNCH(1); break;
    case 2: LAUNCH(2); break;
    case 4: LAUNCH(4); break;
    case 8: LAUNCH(8); break;
    default:
      if constexpr (VEC == 1) {
        if (ch == 16) { LAUNCH(16); }
        else { LAUNCH(32); }
      }
      break;
  }
#undef LAUNCH
  return launch_status();
}

extern "C" int as_layer_norm(float* x, const void* y, const float* gain, float eps, const int* rows, void* out, int dtype,
                             int n_out, int n, int update_x, hipStream_t stream) {
  if (n_out <= 0) return AS_OK;
  if (n <= 0 || !x || !gain || !out) return AS_BAD_SHAPE;
  if (dtype == DT_F32)
    return n % 4 ? launch_layer_norm<float, 1>(x, y, gain, eps, rows, out, n_out, n, update_x, stream)
                 : launch_layer_norm<float, 4>(x, y, gain, eps, rows, out, n_out, n, update_x, stream);
  if (dtype == DT_BF16)
    return n % 4 ? launch_layer_norm<bf16, 1>(x, y, gain, eps, rows, out, n_out, n, update_x, stream)
                 : launch_layer_norm<bf16, 4>(x, y, gain, eps, rows, out, n_out, n, update_x, stream);
  return AS_BAD_DTYPE;
}

// ---- the token's own input, gated ------------------------------------------------------------------------------------
// out[t, i] = gelu_tanh(z[t, i]) * table[ids[t], i], i < dim; z, table and out of one type, everything between fp32.
__device__ __forceinline__ float gelu_tanh(float v) {
  // (1 + tanh u) / 2 = 1 / (1 + e^(-2u)): nothing cancels for negative u, whose small gates a norm may enlarge again
  return v / (1.0f + expf(-2.0f * 0.7978845608028654f * (v + 0.044715f * v * v * v)));
}

template <typename T>
__global__ __launch_bounds__(256) void token_gate_kernel(const T* __restrict__ z, const T* __restrict__ table,
                                                         const int* __restrict__ ids, T* __restrict__ out, int dim, int total) {
  const int at = blockIdx.x * 256 + threadIdx.x;
  if (at >= total) return;
  const int t = at / dim, i = at - t * dim;
  const float v = to_f32(z[at]);
  out[at] = from_f32<T>(gelu_tanh(v) * to_f32(table[(size_t)ids[t] * dim + i]));
}

extern "C" int as_token_gate(const void* z, const void* table, const int* ids, int dtype, void* out, int dim, int num_tokens,
                             hipStream_t stream) {
  if (num_tokens <= 0) return AS_OK;
  if (dim <= 0 || (long)num_tokens * dim > 0x7fffff00L) return AS_BAD_SHAPE;
  const int total = num_tokens * dim, blocks = (total + 255) / 256;
  if (dtype == DT_F32)
    token_gate_kernel<float><<<blocks, 256, 0, stream>>>((const float*)z, (const float*)table, ids, (float*)out, dim, total);
  else if (dtype == DT_BF16)
    token_gate_kernel<bf16><<<blocks, 256, 0, stream>>>((const bf16*)z, (const bf16*)table, ids, (bf16*)out, dim, total);
  else return AS_BAD_DTYPE;
  return launch_status();
}

// The product before it too, for up to 16 rows of bfloat16: out[t, i] = gelu_tanh(x[t] . w[i]) * table[ids[t], i].  A workgroup of
// four waves per output i: their lanes share K, 16 bytes at a time, and hold a sum for every row; a wave's sums meet by lane swaps,
// each swap halving the rows that a lane still sums, so that a lane ends with one row's sum, and the four waves' in LDS.
template <int ROWS>
__global__ __launch_bounds__(256) void token_product_kernel(const bf16* __restrict__ x, const bf16* __restrict__ w,
                                                            const bf16* __restrict__ table, const int* __restrict__ ids,
                                                            bf16* __restrict__ out, int K, int dim, int num_tokens) {
  typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
  __shared__ float sums[4][ROWS];
  const int i = blockIdx.x, lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE, row = threadIdx.x;
  // what the gate needs is asked for first
  const float e = row < num_tokens ? (float)table[(size_t)ids[row] * dim + i] : 0.f;
  float acc[ROWS];
#pragma unroll
  for (int t = 0; t < ROWS; ++t) acc[t] = 0.f;
#pragma unroll 2
  for (int k = threadIdx.x * 8; k < K; k += 4 * WAVE * 8) {
    const bf16x8 wv = *reinterpret_cast<const bf16x8*>(w + (size_t)i * K + k);
#pragma unroll
    for (int t = 0; t < ROWS; ++t) {
      const bf16x8 xv = *reinterpret_cast<const bf16x8*>(x + (size_t)min(t, num_tokens - 1) * K + k);
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[t] = fmaf((float)wv[j], (float)xv[j], acc[t]);
    }
  }
#pragma unroll
  for (int n = ROWS, off = WAVE / 2; n > 1; n /= 2, off /= 2) {
#pragma unroll
    for (int t = 0; t < n / 2; ++t) {
      const float keep = lane & off ? acc[t + n / 2] : acc[t], give = lane & off ? acc[t] : acc[t + n / 2];
      acc[t] = keep + __shfl_xor(give, off, WAVE);
    }
  }
  constexpr int LANES = WAVE / ROWS;  // lanes that still hold parts of one row's sum: row lane / LANES
  float z = acc[0];
#pragma unroll
  for (int off = LANES / 2; off > 0; off /= 2) z += __shfl_xor(z, off, WAVE);
  if (lane % LANES == 0) sums[wave][lane / LANES] = z;
  __syncthreads();
  if (row < num_tokens) {
    z = (sums[0][row] + sums[1][row]) + (sums[2][row] + sums[3][row]);
    out[(size_t)row * dim + i] = (bf16)(gelu_tanh(z) * e);
  }
}

extern "C" int as_token_product(const void* x, const void* w, const void* table, const int* ids, void* out, int K, int dim,
                                int num_tokens, hipStream_t stream) {
  if (num_tokens <= 0) return AS_OK;
  if (K <= 0 || K % 8 || dim <= 0 || num_tokens > 16) return AS_BAD_SHAPE;
#define LAUNCH(R)                                                                                                          \
  token_product_kernel<R><<<dim, 256, 0, stream>>>((const bf16*)x, (const bf16*)w, (const bf16*)table, ids, (bf16*)out, \
                                                             K, dim, num_tokens)
  if (num_tokens == 1) LAUNCH(1);
  else if (num_tokens == 2) LAUNCH(2);
  else if (num_tokens <= 4) LAUNCH(4);
  else if (num_tokens <= 8) LAUNCH(8);
  else LAUNCH(16);
#undef LAUNCH
  return launch_status();
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
