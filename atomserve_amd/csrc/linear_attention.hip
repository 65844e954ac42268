// Linear attention with a decay: a state S [D, E] per head and request,
//
//   S_t = lam_h S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t         with a fixed lam per head, or
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T                        with a decay per token, head and key channel (`channel_*`),
//
// with q, k [D] and v [E] columns of one input product (an activation and a factor applied as they are read).
// The state is fp32 and lives in a slot per request; a row that starts its sequence starts from zero whatever its
// slot holds, a later row goes on from what the row before left.  Everything after the products is fp32.
//
//   decay_scan    token by token: a lane keeps a slice of one column of the state in registers for all of a row's tokens
//   decay_step    a step of single tokens: the state read and written in whole lines (keys of up to 128, values in fours)
//   decay_chunks  32 tokens at a time as four fp32 products on the matrix cores (keys of up to 128 coordinates)
//   decay_finish  o normed in groups (per head, or all heads together) with an optional gain, times act(gate)
//   channel_decays, channel_scan, channel_step, channel_chunks   the decays per channel, and the three with them
#include "common.h"

// Four consecutive values at once (the address a multiple of 16 bytes for fp32, of 8 for bfloat16).
__device__ __forceinline__ void load4(const float* p, float* v) {
  const float4 r = *reinterpret_cast<const float4*>(p);
  v[0] = r.x; v[1] = r.y; v[2] = r.z; v[3] = r.w;
}
__device__ __forceinline__ void load4(const bf16* p, float* v) {
  const uint2 r = *reinterpret_cast<const uint2*>(p);
  v[0] = __uint_as_float(r.x << 16); v[1] = __uint_as_float(r.x & 0xffff0000u);
  v[2] = __uint_as_float(r.y << 16); v[3] = __uint_as_float(r.y & 0xffff0000u);
}
__device__ __forceinline__ void store4(float* p, const float* v) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
__device__ __forceinline__ void store4(bf16* p, const float* v) {
  bf16 b[4] = {from_f32<bf16>(v[0]), from_f32<bf16>(v[1]), from_f32<bf16>(v[2]), from_f32<bf16>(v[3])};
  *reinterpret_cast<uint2*>(p) = *reinterpret_cast<const uint2*>(b);
}

#define ACT_NONE 0
#define ACT_SILU 1
#define ACT_SIGMOID 2

__device__ __forceinline__ float apply_act(float v, int act) {
  if (act == ACT_SILU) return v / (1.0f + expf(-v));
  if (act == ACT_SIGMOID) return 1.0f / (1.0f + expf(-v));
  return v;
}

// The same for inputs that arrive in bfloat16: the hardware's exponential and reciprocal (an ulp or two, far below
// what the inputs' own rounding left), a third of the instructions.
template <typename T> __device__ __forceinline__ float act_of(float v, int act) { return apply_act(v, act); }
template <> __device__ __forceinline__ float act_of<bf16>(float v, int act) {
  if (act == ACT_NONE) return v;
  const float s = __builtin_amdgcn_rcpf(1.0f + __expf(-v));
  return act == ACT_SILU ? v * s : s;
}

// ---- token by token ------------------------------------------------------------------------------------
// grid (column groups, heads, rows), one wave a workgroup.  The wave owns 64 / SL columns e of a head's state; a
// column's D rows are cut into SL slices of DPER in neighbouring lanes, whose partial sums meet by lane swaps.
#define SCAN_DPER 32

// CHAN: `decay` is [T, H, D], a decay per token and key channel; else [H].
template <typename T, bool CHAN>
__global__ __launch_bounds__(64) void decay_scan_kernel(const T* __restrict__ proj, int ld, int q_off, int k_off,
                                                        int v_off, int H, int D, int E, int act, float k_scale,
                                                        const float* __restrict__ decay, float* __restrict__ state,
                                                        const int* __restrict__ row_first,
                                                        const int* __restrict__ row_len,
                                                        const int* __restrict__ row_start,
                                                        const int* __restrict__ row_slots, float* __restrict__ out,
                                                        int SL, int writes) {
  const int lane = threadIdx.x, sl = lane % SL, col = lane / SL;
  const int cols = WAVE / SL;
  const int e = blockIdx.x * cols + col, h = blockIdx.y, r = blockIdx.z;
  const bool live = e < E;
  const int first = row_first[r], len = row_len[r], slot = row_slots[r];
  const float lam = CHAN ? 1.f : decay[h];
  const int d0 = sl * SCAN_DPER;
  float S[SCAN_DPER];
  float* kept = slot >= 0 ? state + (((size_t)slot * H + h) * D) * E : nullptr;
  const bool resume = kept && row_start[r] > 0;
#pragma unroll
  for (int i = 0; i < SCAN_DPER; ++i) S[i] = (resume && live && d0 + i < D) ? kept[(size_t)(d0 + i) * E + e] : 0.f;
  float qn[SCAN_DPER], kn[SCAN_DPER], an[CHAN ? SCAN_DPER : 1], vn = 0.f;
  auto fetch = [&](int t) {
    const T* row = proj + (size_t)t * ld;
#pragma unroll
    for (int i = 0; i < SCAN_DPER; ++i) {
      const bool in = d0 + i < D;
      qn[i] = in ? to_f32(row[q_off + h * D + d0 + i]) : 0.f;
      kn[i] = in ? to_f32(row[k_off + h * D + d0 + i]) : 0.f;
      if (CHAN) an[CHAN ? i : 0] = in ? decay[((size_t)t * H + h) * D + d0 + i] : 1.f;
    }
    vn = live ? to_f32(row[v_off + h * E + e]) : 0.f;
  };
  fetch(first);
  for (int t = first; t < first + len; ++t) {
    float q[SCAN_DPER], k[SCAN_DPER], a[CHAN ? SCAN_DPER : 1];
    const float v = apply_act(vn, act);
#pragma unroll
    for (int i = 0; i < SCAN_DPER; ++i) {
      q[i] = apply_act(qn[i], act);
      k[i] = apply_act(kn[i], act) * k_scale;
      if (CHAN) a[CHAN ? i : 0] = an[CHAN ? i : 0];
    }
    if (t + 1 < first + len) fetch(t + 1);
    float acc = 0.f;
#pragma unroll
    for (int i = 0; i < SCAN_DPER; ++i) {
      S[i] = fmaf(CHAN ? a[CHAN ? i : 0] : lam, S[i], k[i] * v);
      acc = fmaf(S[i], q[i], acc);
    }
    for (int off = 1; off < SL; off <<= 1) acc += __shfl_xor(acc, off, WAVE);
    if (live && sl == 0) out[((size_t)t * H + h) * E + e] = acc;
  }
  if (kept && writes && live) {
#pragma unroll
    for (int i = 0; i < SCAN_DPER; ++i)
      if (d0 + i < D) kept[(size_t)(d0 + i) * E + e] = S[i];
  }
}

template <bool CHAN>
static int launch_decay_scan(const void* proj, int dtype, int ld, int q_off, int k_off, int v_off, int H, int D, int E,
                             int act, float k_scale, const float* decay, float* state, const int* row_first,
                             const int* row_len, const int* row_start, const int* row_slots, int num_rows, float* out,
                             int writes, hipStream_t stream) {
  if (num_rows <= 0) return AS_OK;
  if (!decay || H <= 0 || D <= 0 || E <= 0 || D > 16 * SCAN_DPER || act < 0 || act > 2) return AS_BAD_SHAPE;
  int SL = 1;
  while (SL * SCAN_DPER < D) SL <<= 1;
  const int cols = WAVE / SL;
  dim3 grid((E + cols - 1) / cols, H, num_rows);
  if (grid.y > 65535 || grid.z > 65535) return AS_BAD_SHAPE;
  if (dtype == DT_F32)
    decay_scan_kernel<float, CHAN><<<grid, 64, 0, stream>>>((const float*)proj, ld, q_off, k_off, v_off, H, D, E, act, k_scale, decay,
                                                      state, row_first, row_len, row_start, row_slots, out, SL, writes);
  else if (dtype == DT_BF16)
    decay_scan_kernel<bf16, CHAN><<<grid, 64, 0, stream>>>((const bf16*)proj, ld, q_off, k_off, v_off, H, D, E, act, k_scale, decay,
                                                     state, row_first, row_len, row_start, row_slots, out, SL, writes);
  else return AS_BAD_DTYPE;
  return launch_status();
}

extern "C" int as_decay_scan(const void* proj, int dtype, int ld, int q_off, int k_off, int v_off, int H, int D, int E,
                             int act, float k_scale, const float* decay, float* state, const int* row_first,
                             const int* row_len, const int* row_start, const int* row_slots, int num_rows, float* out,
                             int writes, hipStream_t stream) {
  return launch_decay_scan<false>(proj, dtype, ld, q_off, k_off, v_off, H, D, E, act, k_scale, decay, state, row_first,
                                  row_len, row_start, row_slots, num_rows, out, writes, stream);
}

extern "C" int as_channel_scan(const void* proj, int dtype, int ld, int q_off, int k_off, int v_off, int H, int D, int E,
                               float k_scale, const float* alpha, float* state, const int* row_first, const int* row_len,
                               const int* row_start, const int* row_slots, int num_rows, float* out, int writes,
                               hipStream_t stream) {
  return launch_decay_scan<true>(proj, dtype, ld, q_off, k_off, v_off, H, D, E, ACT_NONE, k_scale, alpha, state, row_first,
                                 row_len, row_start, row_slots, num_rows, out, writes, stream);
}

// ---- one token a row (a decode step) ------------------------------------------------------------------------
// A step of single tokens is the state read once and written once: the wave's loads are whole 128-byte lines.  A
// lane owns four neighbouring columns e of sixteen rows d of one head's state (eight lanes a line of 32 columns,
// eight slices of d, whose partial sums meet by lane swaps).  Needs D <= 128 and E % 4 == 0.
#define STEP_DPER 16

template <typename T, bool CHAN>
__global__ __launch_bounds__(64) void decay_step_kernel(const T* __restrict__ proj, int ld, int q_off, int k_off,
                                                        int v_off, int H, int D, int E, int act, float k_scale,
                                                        const float* __restrict__ decay, float* __restrict__ state,
                                                        const int* __restrict__ row_first,
                                                        const int* __restrict__ row_start,
                                                        const int* __restrict__ row_slots, float* __restrict__ out,
                                                        int writes) {
  const int lane = threadIdx.x, quad = lane & 7, sl = lane >> 3;
  const int e = blockIdx.x * 32 + 4 * quad, h = blockIdx.y, r = blockIdx.z;
  const bool live = e < E;  // E % 4 == 0: a lane's four columns are all there or none
  const int t = row_first[r], slot = row_slots[r];
  const float lam = CHAN ? 1.f : decay[h];
  const int d0 = sl * STEP_DPER;
  float* kept = slot >= 0 ? state + (((size_t)slot * H + h) * D) * E : nullptr;
  const bool resume = kept && row_start[r] > 0;
  float S[STEP_DPER][4];
#pragma unroll
  for (int i = 0; i < STEP_DPER; ++i) {
    if (resume && live && d0 + i < D) load4(kept + (size_t)(d0 + i) * E + e, S[i]);
    else S[i][0] = S[i][1] = S[i][2] = S[i][3] = 0.f;
  }
  const T* row = proj + (size_t)t * ld;
  float q[STEP_DPER], k[STEP_DPER], a[CHAN ? STEP_DPER : 1], v[4];
#pragma unroll
  for (int i = 0; i < STEP_DPER; ++i) {
    const bool in = d0 + i < D;
    q[i] = in ? to_f32(row[q_off + h * D + d0 + i]) : 0.f;
    k[i] = in ? to_f32(row[k_off + h * D + d0 + i]) : 0.f;
    if (CHAN) a[CHAN ? i : 0] = in ? decay[((size_t)t * H + h) * D + d0 + i] : 1.f;
  }
#pragma unroll
  for (int c = 0; c < 4; ++c) v[c] = live ? apply_act(to_f32(row[v_off + h * E + e + c]), act) : 0.f;
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < STEP_DPER; ++i) {
    const float qa = apply_act(q[i], act), ka = apply_act(k[i], act) * k_scale;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      S[i][c] = fmaf(CHAN ? a[CHAN ? i : 0] : lam, S[i][c], ka * v[c]);
      acc[c] = fmaf(S[i][c], qa, acc[c]);
    }
  }
#pragma unroll
  for (int c = 0; c < 4; ++c)
    for (int off = 8; off < WAVE; off <<= 1) acc[c] += __shfl_xor(acc[c], off, WAVE);
  if (live && sl == 0) store4(out + ((size_t)t * H + h) * E + e, acc);
  if (kept && writes && live) {
#pragma unroll
    for (int i = 0; i < STEP_DPER; ++i)
      if (d0 + i < D) store4(kept + (size_t)(d0 + i) * E + e, S[i]);
  }
}

template <bool CHAN>
static int launch_decay_step(const void* proj, int dtype, int ld, int q_off, int k_off, int v_off, int H, int D, int E,
                             int act, float k_scale, const float* decay, float* state, const int* row_first,
                             const int* row_start, const int* row_slots, int num_rows, float* out, int writes,
                             hipStream_t stream) {
  if (num_rows <= 0) return AS_OK;
  if (H <= 0 || D <= 0 || E <= 0 || D > 8 * STEP_DPER || E % 4 || act < 0 || act > 2) return AS_BAD_SHAPE;
  dim3 grid((E + 31) / 32, H, num_rows);
  if (grid.y > 65535 || grid.z > 65535) return AS_BAD_SHAPE;
  if (dtype == DT_F32)
    decay_step_kernel<float, CHAN><<<grid, 64, 0, stream>>>((const float*)proj, ld, q_off, k_off, v_off, H, D, E, act, k_scale, decay,
                                                      state, row_first, row_start, row_slots, out, writes);
  else if (dtype == DT_BF16)
    decay_step_kernel<bf16, CHAN><<<grid, 64, 0, stream>>>((const bf16*)proj, ld, q_off, k_off, v_off, H, D, E, act, k_scale, decay,
                                                     state, row_first, row_start, row_slots, out, writes);
  else return AS_BAD_DTYPE;
  return launch_status();
}

extern "C" int as_decay_step(const void* proj, int dtype, int ld, int q_off, int k_off, int v_off, int H, int D, int E,
                             int act, float k_scale, const float* decay, float* state, const int* row_first,
                             const int* row_start, const int* row_slots, int num_rows, float* out, int writes,
                             hipStream_t stream) {
  return launch_decay_step<false>(proj, dtype, ld, q_off, k_off, v_off, H, D, E, act, k_scale, decay, state, row_first,
                                  row_start, row_slots, num_rows, out, writes, stream);
}

extern "C" int as_channel_step(const void* proj, int dtype, int ld, int q_off, int k_off, int v_off, int H, int D, int E,
                               float k_scale, const float* alpha, float* state, const int* row_first,
                               const int* row_start, const int* row_slots, int num_rows, float* out, int writes,
                               hipStream_t stream) {
  return launch_decay_step<true>(proj, dtype, ld, q_off, k_off, v_off, H, D, E, ACT_NONE, k_scale, alpha, state, row_first,
                                 row_start, row_slots, num_rows, out, writes, stream);
}

// ---- a row's tokens in chunks, on the matrix cores in fp32 ---------------------------------------------------
// Over a chunk of n <= 32 tokens that starts from the state S (token t counts from 0 within the chunk):
//
//   o_t = lam^(t+1) S^T q_t + sum_(j <= t) lam^(t-j) (q_t . k_j) v_j          S' = lam^n S + sum_j lam^(n-1-j) k_j v_j^T
//
// which is four products: A = Q K^T (masked and weighed), A V, Q S and K^T V, all of fp32 operands with fp32 sums
// (v_mfma_f32_32x32x2f32).  grid (column groups of 32, heads, rows), four waves a workgroup.  Wave w keeps rows
// 32 w .. 32 w + 31 of the state's 32 columns in its accumulator registers from the row's first token to its last,
// sums A and o over the same 32 key coordinates, and the waves' parts meet in LDS.  An accumulator register i of
// lane l is element (row 8 (i / 4) + 4 (l / 32) + i % 4, column l % 32); as the second operand of the next product
// it stands for exactly that row, so the state never leaves its registers.
#define CHUNK 32
#define CHUNK_DP 128  // keys are padded with zeros to this width: four waves of 32 coordinates
typedef float floatx16 __attribute__((ext_vector_type(16)));

template <typename T>
__global__ __launch_bounds__(256) void decay_chunk_kernel(const T* __restrict__ proj, int ld, int q_off, int k_off,
                                                         int v_off, int H, int D, int E, int act, float k_scale,
                                                         const float* __restrict__ decay, float* __restrict__ state,
                                                         const int* __restrict__ row_first,
                                                         const int* __restrict__ row_len,
                                                         const int* __restrict__ row_start,
                                                         const int* __restrict__ row_slots, float* __restrict__ out,
                                                         int writes) {
  __shared__ float Qs[CHUNK][CHUNK_DP + 1];
  __shared__ float Ks[CHUNK][CHUNK_DP + 1];
  __shared__ float Vs[CHUNK][CHUNK + 1];
  __shared__ float Part[4][CHUNK][CHUNK + 1];
  __shared__ float As[CHUNK][CHUNK + 1];
  __shared__ float pw[CHUNK + 1];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, col = lane & 31, half = lane >> 5;
  const int e0 = blockIdx.x * CHUNK, h = blockIdx.y, r = blockIdx.z;
  const int first = row_first[r], len = row_len[r], slot = row_slots[r];
  const float lam = decay[h];
  float* kept = slot >= 0 ? state + (((size_t)slot * H + h) * D) * E : nullptr;
  const bool resume = kept && row_start[r] > 0;
  const bool e_live = e0 + col < E;
  if (tid <= CHUNK) pw[tid] = powf(lam, (float)tid);
  floatx16 S;
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    const int d = 32 * w + 8 * (i / 4) + 4 * half + i % 4;
    S[i] = (resume && e_live && d < D) ? kept[(size_t)d * E + e0 + col] : 0.f;
  }
  // A chunk's inputs are asked for a chunk ahead and wait in registers as they were projected, so that the loads
  // run under the products of the chunk before.
  constexpr int QK_EACH = CHUNK * CHUNK_DP / 256, V_EACH = CHUNK * CHUNK / 256;
  T q_next[QK_EACH], k_next[QK_EACH], v_next[V_EACH];
  auto fetch = [&](int c0) {
    const int n = min(CHUNK, len - c0);
#pragma unroll
    for (int it = 0; it < QK_EACH; ++it) {
      const int idx = tid + 256 * it, t = idx / CHUNK_DP, d = idx % CHUNK_DP;
      const bool in = t < n && d < D;
      const T* row = proj + (size_t)(first + c0 + (in ? t : 0)) * ld + h * D + (in ? d : 0);
      q_next[it] = in ? row[q_off] : from_f32<T>(0.f);
      k_next[it] = in ? row[k_off] : from_f32<T>(0.f);
    }
#pragma unroll
    for (int it = 0; it < V_EACH; ++it) {
      const int idx = tid + 256 * it, t = idx / CHUNK, e = idx % CHUNK;
      const bool in = t < n && e0 + e < E;
      v_next[it] = in ? proj[(size_t)(first + c0 + t) * ld + v_off + h * E + e0 + e] : from_f32<T>(0.f);
    }
  };
  if (len > 0) fetch(0);
  for (int c0 = 0; c0 < len; c0 += CHUNK) {
    const int n = min(CHUNK, len - c0);
    __syncthreads();  // the chunk before has been read (and pw written)
#pragma unroll
    for (int it = 0; it < QK_EACH; ++it) {
      const int idx = tid + 256 * it, t = idx / CHUNK_DP, d = idx % CHUNK_DP;
      const bool in = t < n && d < D;
      Qs[t][d] = in ? act_of<T>(to_f32(q_next[it]), act) : 0.f;
      Ks[t][d] = in ? act_of<T>(to_f32(k_next[it]), act) * k_scale : 0.f;
    }
#pragma unroll
    for (int it = 0; it < V_EACH; ++it) {
      const int idx = tid + 256 * it, t = idx / CHUNK, e = idx % CHUNK;
      Vs[t][e] = (t < n && e0 + e < E) ? act_of<T>(to_f32(v_next[it]), act) : 0.f;
    }
    if (c0 + CHUNK < len) fetch(c0 + CHUNK);
    __syncthreads();
    // A = Q K^T over this wave's 32 coordinates
    floatx16 acc;
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int d = 32 * w + 8 * (i / 4) + 4 * half + i % 4;
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(Qs[col][d], Ks[col][d], acc, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) Part[w][8 * (i / 4) + 4 * half + i % 4][col] = acc[i];
    __syncthreads();
    for (int idx = tid; idx < CHUNK * CHUNK; idx += 256) {
      const int t = idx / CHUNK, j = idx % CHUNK;
      const float a = (Part[0][t][j] + Part[1][t][j]) + (Part[2][t][j] + Part[3][t][j]);
      As[t][j] = j <= t ? a * pw[t - j] : 0.f;
    }
    __syncthreads();
    // o = A V over this wave's 8 tokens, + lam^(t+1) Q S over its 32 coordinates
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] = 0.f;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int j = 8 * w + 2 * s + half;
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(As[col][j], Vs[j][col], acc, 0, 0, 0);
    }
    const float grow = pw[col + 1];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int d = 32 * w + 8 * (i / 4) + 4 * half + i % 4;
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(Qs[col][d] * grow, S[i], acc, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) Part[w][8 * (i / 4) + 4 * half + i % 4][col] = acc[i];
    // S = lam^n S + K^T V, key j weighed by lam^(n-1-j)
    const float shrink = pw[n];
#pragma unroll
    for (int i = 0; i < 16; ++i) S[i] *= shrink;
#pragma unroll
    for (int s = 0; s < 16; ++s) {
      const int j = 2 * s + half;
      const float kw = j < n ? Ks[j][32 * w + col] * pw[n - 1 - j] : 0.f;
      S = __builtin_amdgcn_mfma_f32_32x32x2f32(kw, Vs[j][col], S, 0, 0, 0);
    }
    __syncthreads();
    for (int idx = tid; idx < CHUNK * CHUNK; idx += 256) {
      const int t = idx / CHUNK, e = idx % CHUNK;
      if (t < n && e0 + e < E)
        out[((size_t)(first + c0 + t) * H + h) * E + e0 + e] = (Part[0][t][e] + Part[1][t][e]) + (Part[2][t][e] + Part[3][t][e]);
    }
  }
  if (kept && writes && e_live) {
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int d = 32 * w + 8 * (i / 4) + 4 * half + i % 4;
      if (d < D) kept[(size_t)d * E + e0 + col] = S[i];
    }
  }
}

extern "C" int as_decay_chunks(const void* proj, int dtype, int ld, int q_off, int k_off, int v_off, int H, int D, int E,
                               int act, float k_scale, const float* decay, float* state, const int* row_first,
                               const int* row_len, const int* row_start, const int* row_slots, int num_rows, float* out,
                               int writes, hipStream_t stream) {
  if (num_rows <= 0) return AS_OK;
  if (H <= 0 || D <= 0 || E <= 0 || D > CHUNK_DP || act < 0 || act > 2) return AS_BAD_SHAPE;
  dim3 grid((E + CHUNK - 1) / CHUNK, H, num_rows);
  if (grid.y > 65535 || grid.z > 65535) return AS_BAD_SHAPE;
  if (dtype == DT_F32)
    decay_chunk_kernel<float><<<grid, 256, 0, stream>>>((const float*)proj, ld, q_off, k_off, v_off, H, D, E, act, k_scale, decay,
                                                        state, row_first, row_len, row_start, row_slots, out, writes);
  else if (dtype == DT_BF16)
    decay_chunk_kernel<bf16><<<grid, 256, 0, stream>>>((const bf16*)proj, ld, q_off, k_off, v_off, H, D, E, act, k_scale, decay,
                                                       state, row_first, row_len, row_start, row_slots, out, writes);
  else return AS_BAD_DTYPE;
  return launch_status();
}

// ---- chunks with a decay per token and key channel ------------------------------------------------------------------
// With P(s..t) the product of the decays of tokens s .. t of a chunk, per channel (1 if empty):
//
//   o_t = (q_t P(0..t)) S + sum_(j <= t) [sum_d q_td k_jd P(j+1..t)_d] v_j,   S' = diag(P(0..n-1)) S + sum_j (k_j P(j+1..n-1)) v_j^T
//
// The bracket is a product of queries and keys only where P(j+1..t) splits into a factor of t and one of j.  It does at any
// token m between them, P(j+1..m-1) P(m..t), and both factors are at most 1: so the pairs (t, j) of a chunk are taken in
// five products of 16 x 16 by where they lie: t in the second half and j in the first (m = 16); t in the second 8 and j
// in the first 8 of a half (m = 8, 24; two blocks side by side); likewise within an 8 (m = 4, 12, 20, 28; four blocks);
// and the pairs within a 4, two products of eight blocks in all, whose factors are taken from the 4's first token on,
// q P(first+1..t) and k / P(first+1..j): at most three decays of at least CHANNEL_MIN each.  All factors are running
// products of the decays themselves; no logarithm or exponential is taken.  Otherwise as decay_chunk_kernel.
#define CHANNEL_MIN 1e-9f   // a smaller decay counts as this: what it leaves of the past is beyond the 32-bit sum's last digit
#define CHAN_LD (CHUNK_DP + 2)
typedef float floatx4 __attribute__((ext_vector_type(4)));

template <typename T>
__global__ __launch_bounds__(256) void channel_chunk_kernel(const T* __restrict__ proj, int ld, int q_off, int k_off,
                                                            int v_off, int H, int D, int E, float k_scale,
                                                            const float* __restrict__ alpha, float* __restrict__ state,
                                                            const int* __restrict__ row_first,
                                                            const int* __restrict__ row_len,
                                                            const int* __restrict__ row_start,
                                                            const int* __restrict__ row_slots, float* __restrict__ out,
                                                            int writes) {
  __shared__ float QF[CHUNK][CHAN_LD];  // q P(first of the half .. t)
  __shared__ float KB[CHUNK][CHAN_LD];  // k P(t + 1 .. last of the half)
  __shared__ float X8[CHUNK][CHAN_LD];  // first 8 of a half: k P(t + 1 .. the 8's last); second: q P(the 8's first .. t)
  __shared__ float X4[CHUNK][CHAN_LD];  // the same with the 4s of an 8
  __shared__ float QD[CHUNK][CHAN_LD];  // q P(the 4's second .. t)
  __shared__ float KD[CHUNK][CHAN_LD];  // k / P(the 4's second .. t)
  __shared__ float Vs[CHUNK][CHUNK + 1];
  __shared__ float Part[4][CHUNK][CHUNK + 1];
  __shared__ float As[CHUNK][CHUNK + 1];
  __shared__ float tot[2][CHUNK_DP];  // the product of a half's decays
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, col = lane & 31, half = lane >> 5;
  const int e0 = blockIdx.x * CHUNK, h = blockIdx.y, r = blockIdx.z;
  const int first = row_first[r], len = row_len[r], slot = row_slots[r];
  float* kept = slot >= 0 ? state + (((size_t)slot * H + h) * D) * E : nullptr;
  const bool resume = kept && row_start[r] > 0;
  const bool e_live = e0 + col < E;
  floatx16 S;
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    const int d = 32 * w + 8 * (i / 4) + 4 * half + i % 4;
    S[i] = (resume && e_live && d < D) ? kept[(size_t)d * E + e0 + col] : 0.f;
  }
  // A thread brings one channel of 16 tokens (a half of the chunk), a chunk ahead, and makes their running products.
  const int pd = tid & (CHUNK_DP - 1), ph = tid / CHUNK_DP;
  constexpr int V_EACH = CHUNK * CHUNK / 256;
  T q_next[16], k_next[16], v_next[V_EACH];
  float a_next[16];
  auto fetch = [&](int c0) {
    const int n = min(CHUNK, len - c0);
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int t = 16 * ph + i;
      const bool in = t < n && pd < D;
      const size_t at = first + c0 + (in ? t : 0);
      const T* row = proj + at * ld + h * D + (in ? pd : 0);
      q_next[i] = in ? row[q_off] : from_f32<T>(0.f);
      k_next[i] = in ? row[k_off] : from_f32<T>(0.f);
      a_next[i] = in ? alpha[(at * H + h) * D + pd] : 1.f;
    }
#pragma unroll
    for (int it = 0; it < V_EACH; ++it) {
      const int idx = tid + 256 * it, t = idx / CHUNK, e = idx % CHUNK;
      const bool in = t < n && e0 + e < E;
      v_next[it] = in ? proj[(size_t)(first + c0 + t) * ld + v_off + h * E + e0 + e] : from_f32<T>(0.f);
    }
  };
  if (len > 0) fetch(0);
  for (int c0 = 0; c0 < len; c0 += CHUNK) {
    const int n = min(CHUNK, len - c0);
    __syncthreads();  // the chunk before has been read
    {
      float q[16], k[16], a[16];
#pragma unroll
      for (int i = 0; i < 16; ++i) { q[i] = to_f32(q_next[i]); k[i] = to_f32(k_next[i]) * k_scale; a[i] = fmaxf(a_next[i], CHANNEL_MIN); }
      float p = 1.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) { p *= a[i]; QF[16 * ph + i][pd] = q[i] * p; }
      tot[ph][pd] = p;
      p = 1.f;
#pragma unroll
      for (int i = 15; i >= 0; --i) { KB[16 * ph + i][pd] = k[i] * p; p *= a[i]; }
      p = 1.f;
#pragma unroll
      for (int i = 7; i >= 0; --i) { X8[16 * ph + i][pd] = k[i] * p; p *= a[i]; }
      p = 1.f;
#pragma unroll
      for (int i = 8; i < 16; ++i) { p *= a[i]; X8[16 * ph + i][pd] = q[i] * p; }
#pragma unroll
      for (int g = 0; g < 16; g += 8) {
        p = 1.f;
#pragma unroll
        for (int i = 3; i >= 0; --i) { X4[16 * ph + g + i][pd] = k[g + i] * p; p *= a[g + i]; }
        p = 1.f;
#pragma unroll
        for (int i = 4; i < 8; ++i) { p *= a[g + i]; X4[16 * ph + g + i][pd] = q[g + i] * p; }
      }
#pragma unroll
      for (int g = 0; g < 16; g += 4) {
        p = 1.f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          if (i) p *= a[g + i];
          QD[16 * ph + g + i][pd] = q[g + i] * p;
          KD[16 * ph + g + i][pd] = i ? k[g + i] * __builtin_amdgcn_rcpf(p) : k[g];
        }
      }
    }
#pragma unroll
    for (int it = 0; it < V_EACH; ++it) {
      const int idx = tid + 256 * it;
      Vs[idx / CHUNK][idx % CHUNK] = to_f32(v_next[it]);
    }
    if (c0 + CHUNK < len) fetch(c0 + CHUNK);
    __syncthreads();
    {  // the pairs' weights over this wave's 32 coordinates, in five products
      const int rr = lane & 15, kk = lane >> 4;
      const int q8 = rr < 8 ? 8 + rr : 16 + rr, k8 = rr < 8 ? rr : 8 + rr;
      const int q4 = 8 * (rr >> 2) + 4 + (rr & 3), k4 = 8 * (rr >> 2) + (rr & 3);
      floatx4 acc[5];
#pragma unroll
      for (int m = 0; m < 5; ++m) acc[m] = floatx4{0.f, 0.f, 0.f, 0.f};
      if (32 * w < D) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const int d = 32 * w + 4 * i + kk;
          acc[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(QF[16 + rr][d], KB[rr][d], acc[0], 0, 0, 0);
          acc[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(X8[q8][d], X8[k8][d], acc[1], 0, 0, 0);
          acc[2] = __builtin_amdgcn_mfma_f32_16x16x4f32(X4[q4][d], X4[k4][d], acc[2], 0, 0, 0);
          acc[3] = __builtin_amdgcn_mfma_f32_16x16x4f32(QD[rr][d], KD[rr][d], acc[3], 0, 0, 0);
          acc[4] = __builtin_amdgcn_mfma_f32_16x16x4f32(QD[16 + rr][d], KD[16 + rr][d], acc[4], 0, 0, 0);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int row = 4 * kk + i;  // of the product: the query's place; its column rr: the key's
        Part[w][16 + row][rr] = acc[0][i];
        if ((row < 8) == (rr < 8)) Part[w][row < 8 ? 8 + row : 16 + row][k8] = acc[1][i];
        if ((row >> 2) == (rr >> 2)) {
          Part[w][8 * (row >> 2) + 4 + (row & 3)][k4] = acc[2][i];
          if (rr <= row) {
            Part[w][row][rr] = acc[3][i];
            Part[w][16 + row][16 + rr] = acc[4][i];
          }
        }
      }
    }
    __syncthreads();
    for (int idx = tid; idx < CHUNK * CHUNK; idx += 256) {
      const int t = idx / CHUNK, j = idx % CHUNK;
      As[t][j] = j <= t ? (Part[0][t][j] + Part[1][t][j]) + (Part[2][t][j] + Part[3][t][j]) : 0.f;
    }
    __syncthreads();
    // o = A V over this wave's 8 tokens, + (q P(0..t)) S over its 32 coordinates
    floatx16 acc;
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] = 0.f;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int j = 8 * w + 2 * s + half;
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(As[col][j], Vs[j][col], acc, 0, 0, 0);
    }
    if (32 * w < D) {
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int d = 32 * w + 8 * (i / 4) + 4 * half + i % 4;
        const float t0 = tot[0][d];
        acc = __builtin_amdgcn_mfma_f32_32x32x2f32(QF[col][d] * (col >= 16 ? t0 : 1.f), S[i], acc, 0, 0, 0);
        S[i] *= t0 * tot[1][d];
      }
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) Part[w][8 * (i / 4) + 4 * half + i % 4][col] = acc[i];
    if (32 * w < D) {  // S += (k P(j + 1 .. n - 1)) v
      const float t1 = tot[1][32 * w + col];
#pragma unroll
      for (int s = 0; s < 16; ++s) {
        const int j = 2 * s + half;
        S = __builtin_amdgcn_mfma_f32_32x32x2f32(KB[j][32 * w + col] * (s < 8 ? t1 : 1.f), Vs[j][col], S, 0, 0, 0);
      }
    }
    __syncthreads();
    for (int idx = tid; idx < CHUNK * CHUNK; idx += 256) {
      const int t = idx / CHUNK, e = idx % CHUNK;
      if (t < n && e0 + e < E)
        out[((size_t)(first + c0 + t) * H + h) * E + e0 + e] = (Part[0][t][e] + Part[1][t][e]) + (Part[2][t][e] + Part[3][t][e]);
    }
  }
  if (kept && writes && e_live) {
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int d = 32 * w + 8 * (i / 4) + 4 * half + i % 4;
      if (d < D) kept[(size_t)d * E + e0 + col] = S[i];
    }
  }
}

extern "C" int as_channel_chunks(const void* proj, int dtype, int ld, int q_off, int k_off, int v_off, int H, int D, int E,
                                 float k_scale, const float* alpha, float* state, const int* row_first, const int* row_len,
                                 const int* row_start, const int* row_slots, int num_rows, float* out, int writes,
                                 hipStream_t stream) {
  if (num_rows <= 0) return AS_OK;
  if (!alpha || H <= 0 || D <= 0 || E <= 0 || D > CHUNK_DP) return AS_BAD_SHAPE;
  dim3 grid((E + CHUNK - 1) / CHUNK, H, num_rows);
  if (grid.y > 65535 || grid.z > 65535) return AS_BAD_SHAPE;
  if (dtype == DT_F32)
    channel_chunk_kernel<float><<<grid, 256, 0, stream>>>((const float*)proj, ld, q_off, k_off, v_off, H, D, E, k_scale, alpha,
                                                          state, row_first, row_len, row_start, row_slots, out, writes);
  else if (dtype == DT_BF16)
    channel_chunk_kernel<bf16><<<grid, 256, 0, stream>>>((const bf16*)proj, ld, q_off, k_off, v_off, H, D, E, k_scale, alpha,
                                                         state, row_first, row_len, row_start, row_slots, out, writes);
  else return AS_BAD_DTYPE;
  return launch_status();
}

// ---- decays per channel from a two-step projection ---------------------------------------------------------------------
// low: columns low_off .. + rank of proj [T, ld] (the first step's result); up [C, rank] (T-typed), bias [C] fp32.
//   alpha[t, c] = max(sigmoid(z)^(1 / tau), CHANNEL_MIN),  z = sum_r low[t, r] up[c, r] + bias[c],  all of it in fp32.
// Two kernels: bfloat16 with rows on 16 bytes on the matrix cores (a wave 16 tokens of 64 channels: the products' sums are
// fp32 as they are), anything else with a thread per channel for DECAY_TOKENS tokens.
#define DECAY_TOKENS 16

// sigmoid(z)^(1 / tau); for bfloat16 inputs through the hardware's exponential and logarithm, whose error is that of the
// 32-bit result.
template <typename T> __device__ __forceinline__ float root_sigmoid(float z, float inv_tau) {
  const float log_s = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
  return fmaxf(expf(log_s * inv_tau), CHANNEL_MIN);
}
template <> __device__ __forceinline__ float root_sigmoid<bf16>(float z, float inv_tau) {
  const float z2 = z * 1.4426950408889634f;  // in base 2
  const float log_s = fminf(z2, 0.f) - __builtin_amdgcn_logf(1.f + __builtin_amdgcn_exp2f(-fabsf(z2)));
  return fmaxf(__builtin_amdgcn_exp2f(log_s * inv_tau), CHANNEL_MIN);
}

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
#define DECAY_STRIP 64
__global__ __launch_bounds__(256) void channel_decays_mfma_kernel(const bf16* __restrict__ proj, int ld, int low_off, int rank,
                                                                  const bf16* __restrict__ up, const float* __restrict__ bias,
                                                                  float inv_tau, float* __restrict__ alpha, int C,
                                                                  int num_tokens) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lr = lane & 15, lg = lane >> 4;
  const int t = (blockIdx.x * 4 + wave) * 16 + lr, c0 = blockIdx.y * DECAY_STRIP;
  if ((blockIdx.x * 4 + wave) * 16 >= num_tokens) return;
  const bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  floatx4 acc[4];
#pragma unroll
  for (int n = 0; n < 4; ++n) acc[n] = floatx4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < rank; k0 += 32) {
    const int k = k0 + lg * 8;
    const bf16x8 b = t < num_tokens && k < rank ? *reinterpret_cast<const bf16x8*>(proj + (size_t)t * ld + low_off + k) : zero;
#pragma unroll
    for (int n = 0; n < 4; ++n) {
      const int c = c0 + n * 16 + lr;
      const bf16x8 a = c < C && k < rank ? *reinterpret_cast<const bf16x8*>(up + (size_t)c * rank + k) : zero;
      acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[n], 0, 0, 0);
    }
  }
  if (t >= num_tokens) return;
#pragma unroll
  for (int n = 0; n < 4; ++n) {  // this lane: channels c .. c + 3 of token t
    const int c = c0 + n * 16 + 4 * lg;
    if (c >= C) continue;
    float b4[4], v[4];
    load4(bias + c, b4);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = root_sigmoid<bf16>(acc[n][i] + b4[i], inv_tau);
    store4(alpha + (size_t)t * C + c, v);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void channel_decays_kernel(const T* __restrict__ proj, int ld, int low_off, int rank,
                                                             const T* __restrict__ up, const float* __restrict__ bias,
                                                             float inv_tau, float* __restrict__ alpha, int C,
                                                             int num_tokens) {
  extern __shared__ float lows[];  // [rank][DECAY_TOKENS]
  const int t0 = blockIdx.x * DECAY_TOKENS, c = blockIdx.y * 256 + threadIdx.x;
  const int nt = min(DECAY_TOKENS, num_tokens - t0);
  for (int i = threadIdx.x; i < rank * DECAY_TOKENS; i += 256) {
    const int tq = i / rank, k = i % rank;
    lows[k * DECAY_TOKENS + tq] = tq < nt ? to_f32(proj[(size_t)(t0 + tq) * ld + low_off + k]) : 0.f;
  }
  __syncthreads();
  if (c >= C) return;
  float z[DECAY_TOKENS];
#pragma unroll
  for (int tq = 0; tq < DECAY_TOKENS; ++tq) z[tq] = bias[c];
  const T* row = up + (size_t)c * rank;
  auto take = [&](float u, int k) {
#pragma unroll
    for (int tq = 0; tq < DECAY_TOKENS; ++tq) z[tq] = fmaf(lows[k * DECAY_TOKENS + tq], u, z[tq]);
  };
  int k = 0;
  if (rank % 4 == 0) {
    for (; k < rank; k += 4) {
      float u[4];
      load4(row + k, u);
#pragma unroll
      for (int i = 0; i < 4; ++i) take(u[i], k + i);
    }
  } else {
    for (; k < rank; ++k) take(to_f32(row[k]), k);
  }
#pragma unroll
  for (int tq = 0; tq < DECAY_TOKENS; ++tq) {
    if (tq < nt) alpha[(size_t)(t0 + tq) * C + c] = root_sigmoid<T>(z[tq], inv_tau);
  }
}

extern "C" int as_channel_decays(const void* proj, int dtype, int ld, int low_off, int rank, const void* up,
                                 const float* bias, float tau, float* alpha, int C, int num_tokens, hipStream_t stream) {
  if (num_tokens <= 0) return AS_OK;
  if (rank <= 0 || rank > 960 || low_off < 0 || low_off + rank > ld || C <= 0 || !(tau > 0.f) || !up || !bias) return AS_BAD_SHAPE;
  dim3 grid((num_tokens + DECAY_TOKENS - 1) / DECAY_TOKENS, (C + 255) / 256);
  if (grid.y > 65535) return AS_BAD_SHAPE;
  const size_t lds = (size_t)rank * DECAY_TOKENS * sizeof(float);
  if (dtype == DT_BF16 && rank % 8 == 0 && ld % 8 == 0 && low_off % 8 == 0 && C % 4 == 0) {
    dim3 tiles((num_tokens + 63) / 64, (C + DECAY_STRIP - 1) / DECAY_STRIP);
    if (tiles.y > 65535) return AS_BAD_SHAPE;
    channel_decays_mfma_kernel<<<tiles, 256, 0, stream>>>((const bf16*)proj, ld, low_off, rank, (const bf16*)up, bias, 1.0f / tau, alpha, C, num_tokens);
    return launch_status();
  }
  if (dtype == DT_F32)
    channel_decays_kernel<float><<<grid, 256, lds, stream>>>((const float*)proj, ld, low_off, rank, (const float*)up, bias, 1.0f / tau, alpha, C, num_tokens);
  else if (dtype == DT_BF16)
    channel_decays_kernel<bf16><<<grid, 256, lds, stream>>>((const bf16*)proj, ld, low_off, rank, (const bf16*)up, bias, 1.0f / tau, alpha, C, num_tokens);
  else return AS_BAD_DTYPE;
  return launch_status();
}

// ---- the output's norm and gate ---------------------------------------------------------------------------
// o [T, n] fp32 is normed in `groups` equal parts (a head each, or 1: all heads together; eps inside the root),
// multiplied by gain [n] (null: none) and by act(gate[t, g_off + i]); out [T, n] in the compute dtype.
template <typename T>
__global__ __launch_bounds__(256) void decay_finish_kernel(const float* __restrict__ o, int n, int groups, float eps,
                                                           const float* __restrict__ gain, const T* __restrict__ proj,
                                                           int ld, int g_off, int gate_act, T* __restrict__ out) {
  extern __shared__ float inv[];  // [groups]
  const int t = blockIdx.x;
  const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE, waves = blockDim.x / WAVE;
  const float* row = o + (size_t)t * n;
  const int gs = n / groups;
  const bool by_four = gs % 4 == 0 && ld % 4 == 0 && g_off % 4 == 0;  // every row and group starts on 16 (8) bytes
  if (groups == 1) {
    __shared__ float red[17];
    float ss = 0.f;
    if (by_four) {
      for (int i = 4 * threadIdx.x; i < n; i += 4 * blockDim.x) {
        float v[4];
        load4(row + i, v);
#pragma unroll
        for (int c = 0; c < 4; ++c) ss = fmaf(v[c], v[c], ss);
      }
    } else {
      for (int i = threadIdx.x; i < n; i += blockDim.x) ss = fmaf(row[i], row[i], ss);
    }
    ss = block_sum(ss, red);
    if (threadIdx.x == 0) inv[0] = 1.0f / sqrtf(ss / (float)n + eps);
  } else {
    for (int g = wave; g < groups; g += waves) {
      float ss = 0.f;
      if (by_four) {
        for (int i = 4 * lane; i < gs; i += 4 * WAVE) {
          float v[4];
          load4(row + g * gs + i, v);
#pragma unroll
          for (int c = 0; c < 4; ++c) ss = fmaf(v[c], v[c], ss);
        }
      } else {
        for (int i = lane; i < gs; i += WAVE) ss = fmaf(row[g * gs + i], row[g * gs + i], ss);
      }
      ss = wave_sum(ss);
      if (lane == 0) inv[g] = 1.0f / sqrtf(ss / (float)gs + eps);
    }
  }
  __syncthreads();
  const T* gate = proj + (size_t)t * ld + g_off;
  if (by_four) {
    for (int i = 4 * threadIdx.x; i < n; i += 4 * blockDim.x) {
      float v[4], gt[4], gn[4] = {1.f, 1.f, 1.f, 1.f};
      load4(row + i, v);
      load4(gate + i, gt);
      if (gain) load4(gain + i, gn);
      const float scale = inv[i / gs];
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        float r = v[c] * scale;
        if (gain) r *= gn[c];
        v[c] = r * apply_act(gt[c], gate_act);
      }
      store4(out + (size_t)t * n + i, v);
    }
    return;
  }
  for (int i = threadIdx.x; i < n; i += blockDim.x) {
    float v = row[i] * inv[i / gs];
    if (gain) v *= gain[i];
    out[(size_t)t * n + i] = from_f32<T>(v * apply_act(to_f32(gate[i]), gate_act));
  }
}

extern "C" int as_decay_finish(const float* o, int n, int groups, float eps, const float* gain, const void* proj,
                               int dtype, int ld, int g_off, int gate_act, void* out, int num_tokens,
                               hipStream_t stream) {
  if (num_tokens <= 0) return AS_OK;
  if (n <= 0 || groups <= 0 || n % groups || groups > 8192 || gate_act < 0 || gate_act > 2) return AS_BAD_SHAPE;
  const size_t lds = (size_t)groups * sizeof(float);
  if (dtype == DT_F32)
    decay_finish_kernel<float><<<num_tokens, 256, lds, stream>>>(o, n, groups, eps, gain, (const float*)proj, ld, g_off, gate_act, (float*)out);
  else if (dtype == DT_BF16)
    decay_finish_kernel<bf16><<<num_tokens, 256, lds, stream>>>(o, n, groups, eps, gain, (const bf16*)proj, ld, g_off, gate_act, (bf16*)out);
  else return AS_BAD_DTYPE;
  return launch_status();
}
