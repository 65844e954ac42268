// A state space per head: a state S [N, E] per head and request,
//
//   dt_t = softplus(step_t + dt_bias_h),   a_t = exp(-exp(A_log_h) dt_t)
//   S_t = a_t S_(t-1) + dt_t B_t x_t^T,    y_t = S_t^T C_t + D_h x_t
//
// x [H, E], B and C [G, N] (head h reads group h / (H / G)) are columns of one fp32 array xbc [T, channels], laid out
// [x | B | C]: what the short convolution left.  The step sizes before their bias are columns of the input product.  The
// state is fp32 and lives in a slot per request; a row that starts its sequence starts from zero whatever its slot
// holds, a later row goes on from what the row before left.  Everything here is fp32.
//
//   state_space_scan    token by token: a lane keeps a slice of one column of the state in registers for all of a row's tokens
//   state_space_step    a step of single tokens: the state read and written in whole lines (N up to 128, E in fours)
//   state_space_chunks  32 tokens at a time as fp32 products on the matrix cores (N up to 128); long rows in segments
//                       that run at once
//   gated_group_norm    y times silu(z), in groups over its root mean square, times a gain
#include "common.h"
#include "rows.h"

__device__ __forceinline__ float softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// The exponential of weights and gates: the hardware's where the inputs came in bfloat16.
template <typename T> __device__ __forceinline__ float quick_exp(float v) { return expf(v); }
template <> __device__ __forceinline__ float quick_exp<bf16>(float v) { return __expf(v); }

struct Space {
  const float* xbc;  // [T, channels]
  int channels, H, G, N, E;
  const void* proj;  // [T, ld]: the steps at column step_off
  int ld, step_off;
  const float* dt_bias;  // [H]
  const float* a_log;    // [H]
  const float* skip;     // [H]: D
  float* state;          // [slots, H, N, E]
  const int* row_first;
  const int* row_len;
  const int* row_start;
  const int* row_slots;
  int num_rows;
  float* out;  // [T, H E]
  int writes;
  // segments of long rows (`state_space_chunks`)
  int seg_len;       // 0: a row is one segment
  float* seg_state;  // [segments + 1][H][E blocks][N tiles][16][64]: what a segment starts from, in accumulator order
  float* seg_decay;  // [segments + 1][H]: the logarithm of a segment's whole decay
};

__device__ __forceinline__ size_t state_at(const Space& s, int slot, int h, int n, int e) {
  return (((size_t)slot * s.H + h) * s.N + n) * s.E + e;
}

// ---- token by token --------------------------------------------------------------------------------------------
// grid (column groups, heads, rows), one wave a workgroup.  The wave owns 64 / SL columns e of a head's state; a column's
// N rows are cut into SL slices of SCAN_PER in neighbouring lanes, whose partial sums meet by lane swaps.
#define SCAN_PER 32

template <typename T>
__global__ __launch_bounds__(64) void state_space_scan_kernel(Space s, int SL) {
  const int lane = threadIdx.x, sl = lane % SL, cols = WAVE / SL;
  const int e = blockIdx.x * cols + lane / SL, h = blockIdx.y, r = blockIdx.z, n0 = sl * SCAN_PER;
  const bool live = e < s.E;
  const int first = s.row_first[r], len = s.row_len[r], slot = s.row_slots[r];
  const int g = h / (s.H / s.G), b_off = s.H * s.E + g * s.N, c_off = b_off + s.G * s.N;
  const bool resume = slot >= 0 && s.row_start[r] > 0;
  const float rate = expf(s.a_log[h]), bias = s.dt_bias[h], skip = s.skip[h];
  float S[SCAN_PER];
#pragma unroll
  for (int i = 0; i < SCAN_PER; ++i) S[i] = resume && live && n0 + i < s.N ? s.state[state_at(s, slot, h, n0 + i, e)] : 0.f;
  for (int t = first; t < first + len; ++t) {
    const float* row = s.xbc + (size_t)t * s.channels;
    const float dt = softplus(to_f32(((const T*)s.proj)[(size_t)t * s.ld + s.step_off + h]) + bias), a = expf(-rate * dt);
    const float x = live ? row[h * s.E + e] : 0.f, u = dt * x;
    float acc = 0.f;
#pragma unroll
    for (int i = 0; i < SCAN_PER; ++i) {
      const bool in = n0 + i < s.N;
      S[i] = fmaf(a, S[i], (in ? row[b_off + n0 + i] : 0.f) * u);
      acc = fmaf(S[i], in ? row[c_off + n0 + i] : 0.f, acc);
    }
    for (int off = 1; off < SL; off <<= 1) acc += __shfl_xor(acc, off, WAVE);
    if (live && sl == 0) s.out[(size_t)t * s.H * s.E + h * s.E + e] = fmaf(skip, x, acc);
  }
  if (slot >= 0 && s.writes && live) {
#pragma unroll
    for (int i = 0; i < SCAN_PER; ++i)
      if (n0 + i < s.N) s.state[state_at(s, slot, h, n0 + i, e)] = S[i];
  }
}

// ---- one token a row (a decode step) -------------------------------------------------------------------------------
// The state read once and written once: the wave's loads are whole 128-byte lines.  A lane owns four neighbouring columns e
// of sixteen rows n of one head's state (eight lanes a line of 32 columns, eight slices of n, whose partial sums meet by
// lane swaps).  Needs N <= 128 and E % 4 == 0.
#define STEP_PER 16

template <typename T>
__global__ __launch_bounds__(64) void state_space_step_kernel(Space s) {
  const int lane = threadIdx.x, quad = lane & 7, sl = lane >> 3;
  const int e = blockIdx.x * 32 + 4 * quad, h = blockIdx.y, r = blockIdx.z, n0 = sl * STEP_PER;
  const bool live = e < s.E;
  const int t = s.row_first[r], slot = s.row_slots[r];
  const int g = h / (s.H / s.G), b_off = s.H * s.E + g * s.N, c_off = b_off + s.G * s.N;
  const bool resume = slot >= 0 && s.row_start[r] > 0;
  float* kept = s.state + state_at(s, slot < 0 ? 0 : slot, h, 0, e);
  float S[STEP_PER][4];
#pragma unroll
  for (int i = 0; i < STEP_PER; ++i) {
    if (resume && live && n0 + i < s.N) load_vec<4>(kept + (size_t)(n0 + i) * s.E, S[i]);
    else S[i][0] = S[i][1] = S[i][2] = S[i][3] = 0.f;
  }
  const float* row = s.xbc + (size_t)t * s.channels;
  float B[STEP_PER], C[STEP_PER], x[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < STEP_PER; ++i) {
    const bool in = n0 + i < s.N;
    B[i] = in ? row[b_off + n0 + i] : 0.f;
    C[i] = in ? row[c_off + n0 + i] : 0.f;
  }
#pragma unroll
  for (int c = 0; c < 4; ++c) x[c] = live ? row[h * s.E + e + c] : 0.f;
  const float dt = softplus(to_f32(((const T*)s.proj)[(size_t)t * s.ld + s.step_off + h]) + s.dt_bias[h]);
  const float a = expf(-expf(s.a_log[h]) * dt), skip = s.skip[h];
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < STEP_PER; ++i) {
    const float b = B[i] * dt;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      S[i][c] = fmaf(a, S[i][c], b * x[c]);
      acc[c] = fmaf(S[i][c], C[i], acc[c]);
    }
  }
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    for (int off = 8; off < WAVE; off <<= 1) acc[c] += __shfl_xor(acc[c], off, WAVE);
    acc[c] = fmaf(skip, x[c], acc[c]);
  }
  if (live && sl == 0) {
#pragma unroll
    for (int c = 0; c < 4; ++c) s.out[(size_t)t * s.H * s.E + h * s.E + e + c] = acc[c];
  }
  if (slot >= 0 && s.writes && live) {
#pragma unroll
    for (int i = 0; i < STEP_PER; ++i)
      if (n0 + i < s.N) store_vec<4>(kept + (size_t)(n0 + i) * s.E, S[i]);
  }
}

// ---- a row's tokens in chunks, on the matrix cores in fp32 ------------------------------------------------------------
// Over a chunk of n <= 32 tokens that starts from the state S, with l_t = sum_(i <= t) log a_i within the chunk:
//
//   y_t = e^(l_t) S^T C_t + sum_(j <= t) M_tj x_j,   M_tj = e^(l_t - l_j) dt_j (B_j . C_t) + [t = j] D
//   S' = e^(l_(n-1)) S + sum_j e^(l_(n-1) - l_j) dt_j B_j x_j^T
//
// No factor exceeds what the recurrence itself multiplies by: l falls, and every exponent is at most 0.  The l are summed and
// subtracted in 64 bits, so a token whose decay is tiny costs its neighbours in the chunk no accuracy.
//
// grid (quads of units, groups, segments), four waves a workgroup.  A unit is 32 columns of one head's state; the four waves
// take units of one group, so they read the same B and C, which come into LDS once for all of them, a chunk ahead.  A wave
// keeps its unit's N x 32 state in accumulator registers; an accumulator register i of lane l is element (row
// 8 (i / 4) + 4 (l / 32) + i % 4, column l % 32), and stands for exactly that row as the second operand of a product and, of a
// transposed product, as the first: the pairs' matrix is made as B C^T (its column the query's place t), so neither it nor the
// state ever leaves its registers.  The products B_j . C_t are the same for all heads of a group: each wave sums 32 of the N
// coordinates, and the parts meet in LDS.
//
// A long row is cut into segments of seg_len tokens so that few rows fill the GPU: first every segment but a row's last sums
// what it adds to a state of zero (STATES), then `state_space_pass_kernel` turns these into what each segment starts from, then
// all segments run at once.
#define CHUNK 32
typedef float floatx16 __attribute__((ext_vector_type(16)));

__device__ __forceinline__ int acc_row(int i, int half) { return 8 * (i / 4) + 4 * half + i % 4; }

// The row and the number within it of segment z; false: there are not so many.
__device__ __forceinline__ bool find_segment(const Space& s, int z, int* row, int* nth, int* count) {
  if (s.seg_len == 0) {
    *row = z;
    *nth = 0;
    *count = 1;
    return true;
  }
  for (int r = 0; r < s.num_rows; ++r) {
    const int n = max(1, (s.row_len[r] + s.seg_len - 1) / s.seg_len);
    if (z < n) {
      *row = r;
      *nth = z;
      *count = n;
      return true;
    }
    z -= n;
  }
  return false;
}

template <typename T, int NT, bool STATES>
__global__ __launch_bounds__(256, 2) void state_space_chunk_kernel(Space s) {
  constexpr int NP = 32 * NT, LD = NP + 4, QUADS = NP / 4, EACH = CHUNK * QUADS / 256;
  __shared__ __attribute__((aligned(16))) float Bs[CHUNK][LD];
  __shared__ __attribute__((aligned(16))) float Cs[STATES ? 1 : CHUNK][LD];
  __shared__ __attribute__((aligned(16))) float part[STATES ? 1 : NT][4][WAVE][4];
  __shared__ __attribute__((aligned(16))) double log_sum[4][CHUNK];  // per wave: l
  __shared__ __attribute__((aligned(16))) float step[4][CHUNK];      // dt
  __shared__ __attribute__((aligned(16))) float grow[4][CHUNK];      // e^l
  __shared__ __attribute__((aligned(16))) float to_end[4][CHUNK];    // e^(l_last - l) dt
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, col = lane & 31, half = lane >> 5;
  int r, nth, count;
  if (!find_segment(s, blockIdx.z, &r, &nth, &count)) return;
  if (STATES && nth + 1 == count) return;
  const int g = blockIdx.y, per_group = s.H / s.G, blocks = (s.E + 31) / 32;
  const int unit = blockIdx.x * 4 + w;
  const bool working = unit < per_group * blocks;
  const int h = g * per_group + (working ? unit / blocks : 0), e0 = (working ? unit % blocks : 0) * 32;
  const int first = s.row_first[r] + nth * s.seg_len, len = s.seg_len ? min(s.seg_len, s.row_len[r] - nth * s.seg_len) : s.row_len[r];
  const int slot = s.row_slots[r];
  const int b_off = s.H * s.E + g * s.N, c_off = b_off + s.G * s.N;
  const bool whole = ((s.channels | s.N | b_off | c_off) & 3) == 0;  // every B and C starts on 16 bytes
  const bool e_live = working && e0 + col < s.E;
  const float rate = expf(s.a_log[h]), bias = s.dt_bias[h], skip = s.skip[h];
  auto segment_state = [&](int seg, int tile, int i) {
    return ((((size_t)seg * s.H + h) * blocks + e0 / 32) * NT + tile) * 1024 + i * 64 + lane;
  };
  floatx16 S[NT];
  const bool resume = !STATES && count == 1 && slot >= 0 && s.row_start[r] > 0;
  if (!STATES && count > 1 && working) {
#pragma unroll
    for (int tile = 0; tile < NT; ++tile)
#pragma unroll
      for (int i = 0; i < 16; ++i) S[tile][i] = s.seg_state[segment_state(blockIdx.z, tile, i)];
  } else if (resume) {
    const float* kept = s.state + state_at(s, slot, h, 0, 0);
#pragma unroll
    for (int tile = 0; tile < NT; ++tile)
#pragma unroll
      for (int i = 0; i < 16; ++i) {  // a place beyond the state is read as the nearest one within and counts as zero
        const int n = 32 * tile + acc_row(i, half);
        const float v = kept[min(n, s.N - 1) * s.E + min(e0 + col, s.E - 1)];
        S[tile][i] = e_live && n < s.N ? v : 0.f;
      }
  } else {
#pragma unroll
    for (int tile = 0; tile < NT; ++tile)
#pragma unroll
      for (int i = 0; i < 16; ++i) S[tile][i] = 0.f;
  }
  // B and C of a chunk are asked for while the chunk before updates the state and wait in registers; x while this chunk's first
  // products run.
  float4 b_next[EACH], c_next[STATES ? 1 : EACH];
  float step_next = 0.f;
  auto fetch = [&](int c0) {
    const int n = min(CHUNK, len - c0);
    const float* base = s.xbc + (size_t)(first + c0) * s.channels;  // one address for the wave, 32-bit offsets for its lanes
#pragma unroll
    for (int it = 0; it < EACH; ++it) {
      const int idx = tid + 256 * it, t = idx / QUADS, d = (idx % QUADS) * 4;
      float4 b, c = make_float4(0.f, 0.f, 0.f, 0.f);
      if (whole) {
        const int at = min(t, n - 1) * s.channels + min(d, s.N - 4);
        b = *reinterpret_cast<const float4*>(base + b_off + at);
        if (!STATES) c = *reinterpret_cast<const float4*>(base + c_off + at);
      } else {
        const int at = min(t, n - 1) * s.channels, d1 = min(d, s.N - 1), d2 = min(d + 1, s.N - 1), d3 = min(d + 2, s.N - 1), d4 = min(d + 3, s.N - 1);
        b = make_float4(base[b_off + at + d1], base[b_off + at + d2], base[b_off + at + d3], base[b_off + at + d4]);
        if (!STATES) c = make_float4(base[c_off + at + d1], base[c_off + at + d2], base[c_off + at + d3], base[c_off + at + d4]);
        if (d + 1 >= s.N) b.y = c.y = 0.f;
        if (d + 2 >= s.N) b.z = c.z = 0.f;
        if (d + 3 >= s.N) b.w = c.w = 0.f;
      }
      if (t >= n || d >= s.N) b = c = make_float4(0.f, 0.f, 0.f, 0.f);
      b_next[it] = b;
      if (!STATES) c_next[STATES ? 0 : it] = c;
    }
    step_next = to_f32(((const T*)s.proj)[(size_t)(first + c0 + min(col, n - 1)) * s.ld + s.step_off + h]);
  };
  double decayed = 0.0;  // STATES: the segment's whole log decay
  fetch(0);
  for (int c0 = 0; c0 < len; c0 += CHUNK) {
    const int n = min(CHUNK, len - c0);
    // this head's steps and decays: both halves of the wave do the same
    const float dt = col < n ? softplus(step_next + bias) : 0.f;
    double l = -(double)rate * (double)dt;
#pragma unroll
    for (int off = 1; off < CHUNK; off <<= 1) {
      const double before = __shfl_up(l, off, 32);
      if (col >= off) l += before;
    }
    const double last = __shfl(l, 31, 32);  // tokens beyond the row decay by nothing
    decayed += last;
    __syncthreads();  // the chunk before has been read
#pragma unroll
    for (int it = 0; it < EACH; ++it) {
      const int idx = tid + 256 * it, t = idx / QUADS, d = (idx % QUADS) * 4;
      *reinterpret_cast<float4*>(&Bs[t][d]) = b_next[it];
      if (!STATES) *reinterpret_cast<float4*>(&Cs[STATES ? 0 : t][d]) = c_next[STATES ? 0 : it];
    }
    if (lane < CHUNK) {
      to_end[w][lane] = quick_exp<T>((float)(last - l)) * dt;
      if (!STATES) {
        log_sum[w][lane] = l;
        step[w][lane] = dt;
        grow[w][lane] = quick_exp<T>((float)l);
      }
    }
    float x[16];
    {
      const float* base = s.xbc + (size_t)(first + c0) * s.channels + h * s.E;
      const int e = min(e0 + col, s.E - 1);
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int j = acc_row(i, half);
        const float v = base[min(j, n - 1) * s.channels + e];
        x[i] = j < n && e_live ? v : 0.f;
      }
    }
    __syncthreads();
    floatx16 y;
    if (!STATES) {
      float pairs[16];  // B_j . C_t, j this register's row, t = col
      if (w < NT) {
        floatx16 acc;
#pragma unroll
        for (int i = 0; i < 16; ++i) acc[i] = 0.f;
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const float4 b = *reinterpret_cast<const float4*>(&Bs[col][32 * w + 8 * q + 4 * half]);
          const float4 c = *reinterpret_cast<const float4*>(&Cs[STATES ? 0 : col][32 * w + 8 * q + 4 * half]);
          acc = __builtin_amdgcn_mfma_f32_32x32x2f32(b.x, c.x, acc, 0, 0, 0);
          acc = __builtin_amdgcn_mfma_f32_32x32x2f32(b.y, c.y, acc, 0, 0, 0);
          acc = __builtin_amdgcn_mfma_f32_32x32x2f32(b.z, c.z, acc, 0, 0, 0);
          acc = __builtin_amdgcn_mfma_f32_32x32x2f32(b.w, c.w, acc, 0, 0, 0);
        }
#pragma unroll
        for (int q = 0; q < 4; ++q)
          *reinterpret_cast<float4*>(part[STATES ? 0 : w][q][lane]) = make_float4(acc[4 * q], acc[4 * q + 1], acc[4 * q + 2], acc[4 * q + 3]);
      }
      __builtin_amdgcn_sched_barrier(0);  // or the operands of everything that follows are asked for at once
      // meanwhile: y = e^(l_t) S^T C
#pragma unroll
      for (int i = 0; i < 16; ++i) y[i] = 0.f;
#pragma unroll
      for (int tile = 0; tile < NT; ++tile) {
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const float4 c = *reinterpret_cast<const float4*>(&Cs[STATES ? 0 : col][32 * tile + 8 * q + 4 * half]);
          y = __builtin_amdgcn_mfma_f32_32x32x2f32(c.x, S[tile][4 * q], y, 0, 0, 0);
          y = __builtin_amdgcn_mfma_f32_32x32x2f32(c.y, S[tile][4 * q + 1], y, 0, 0, 0);
          y = __builtin_amdgcn_mfma_f32_32x32x2f32(c.z, S[tile][4 * q + 2], y, 0, 0, 0);
          y = __builtin_amdgcn_mfma_f32_32x32x2f32(c.w, S[tile][4 * q + 3], y, 0, 0, 0);
        }
        if (tile & 1) __builtin_amdgcn_sched_barrier(0);
      }
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const float4 f = *reinterpret_cast<const float4*>(&grow[w][8 * q + 4 * half]);
        y[4 * q] *= f.x; y[4 * q + 1] *= f.y; y[4 * q + 2] *= f.z; y[4 * q + 3] *= f.w;
      }
      __syncthreads();
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        float4 sum = *reinterpret_cast<const float4*>(part[0][q][lane]);
#pragma unroll
        for (int o = 1; o < NT; ++o) {
          const float4 v = *reinterpret_cast<const float4*>(part[STATES ? 0 : o][q][lane]);
          sum.x += v.x; sum.y += v.y; sum.z += v.z; sum.w += v.w;
        }
        pairs[4 * q] = sum.x; pairs[4 * q + 1] = sum.y; pairs[4 * q + 2] = sum.z; pairs[4 * q + 3] = sum.w;
      }
      const double mine = log_sum[w][col];
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int j = acc_row(i, half);
        float m = quick_exp<T>(fminf((float)(mine - log_sum[w][j]), 0.f)) * step[w][j] * pairs[i];
        m = j < col ? m : j == col ? m + skip : 0.f;
        y = __builtin_amdgcn_mfma_f32_32x32x2f32(m, x[i], y, 0, 0, 0);
      }
    }
    __builtin_amdgcn_sched_barrier(0);
    if (c0 + CHUNK < len) fetch(c0 + CHUNK);
    const float shrink = quick_exp<T>((float)last);
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const float4 f = *reinterpret_cast<const float4*>(&to_end[w][8 * q + 4 * half]);
      x[4 * q] *= f.x; x[4 * q + 1] *= f.y; x[4 * q + 2] *= f.z; x[4 * q + 3] *= f.w;
    }
#pragma unroll
    for (int tile = 0; tile < NT; ++tile) {
#pragma unroll
      for (int i = 0; i < 16; ++i) S[tile][i] *= shrink;
#pragma unroll
      for (int i = 0; i < 16; ++i)
        S[tile] = __builtin_amdgcn_mfma_f32_32x32x2f32(Bs[acc_row(i, half)][32 * tile + col], x[i], S[tile], 0, 0, 0);
      if (tile & 1) __builtin_amdgcn_sched_barrier(0);
    }
    if (!STATES && e_live) {
      float* to = s.out + (size_t)(first + c0) * s.H * s.E + h * s.E + e0 + col;
      const int ld = s.H * s.E;
      if (n == CHUNK) {
#pragma unroll
        for (int i = 0; i < 16; ++i) to[acc_row(i, half) * ld] = y[i];
      } else {
#pragma unroll
        for (int i = 0; i < 16; ++i)
          if (acc_row(i, half) < n) to[acc_row(i, half) * ld] = y[i];
      }
    }
  }
  if (STATES) {
    if (working) {
#pragma unroll
      for (int tile = 0; tile < NT; ++tile)
#pragma unroll
        for (int i = 0; i < 16; ++i) s.seg_state[segment_state(blockIdx.z + 1, tile, i)] = S[tile][i];
      if (e0 == 0 && lane == 0) s.seg_decay[(size_t)blockIdx.z * s.H + h] = (float)decayed;
    }
    return;
  }
  if (slot >= 0 && s.writes && e_live && nth + 1 == count) {
    float* kept = s.state + state_at(s, slot, h, 0, e0 + col);
    int hf = half;
    asm volatile("" : "+v"(hf));  // or the addresses of the state's first read are kept through the loop for this
#pragma unroll
    for (int tile = 0; tile < NT; ++tile)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int n = 32 * tile + acc_row(i, hf);
        if (n < s.N) kept[n * s.E] = S[tile][i];
      }
  }
}

// What the segments of a row add to a state -> what each of them starts from.  grid (blocks of 256 values of a state in
// accumulator order, rows).
template <int NT>
__global__ __launch_bounds__(256) void state_space_pass_kernel(Space s) {
  const int r = blockIdx.y, blocks = (s.E + 31) / 32, per = s.H * blocks * NT * 1024;
  const int at = blockIdx.x * 256 + threadIdx.x;
  if (at >= per) return;
  int z = 0;
  for (int i = 0; i < r; ++i) z += max(1, (s.row_len[i] + s.seg_len - 1) / s.seg_len);
  const int count = max(1, (s.row_len[r] + s.seg_len - 1) / s.seg_len);
  if (count == 1) return;
  const int lane = at & 63, i = (at >> 6) & 15, tile = at / 1024 % NT, block = at / (1024 * NT) % blocks, h = at / (1024 * NT * blocks);
  const int n = 32 * tile + acc_row(i, lane >> 5), e = 32 * block + (lane & 31), slot = s.row_slots[r];
  float v = 0.f;
  if (slot >= 0 && s.row_start[r] > 0 && n < s.N && e < s.E) v = s.state[state_at(s, slot, h, n, e)];
  // the first segment's too: the last one may have written the slot before the first one starts
  s.seg_state[(size_t)z * per + at] = v;
  for (int k = 0; k + 1 < count; ++k) {
    float* next = s.seg_state + (size_t)(z + k + 1) * per + at;
    v = fmaf(expf(s.seg_decay[(size_t)(z + k) * s.H + h]), v, *next);
    *next = v;
  }
}

// kernel 0: token by token; 1: every row one token; 2: in chunks, rows of more than seg_len tokens (0: none) in segments:
// seg_state [max_segments + 1, H, ceil(E / 32), ceil(N / 32), 1024] and seg_decay [max_segments + 1, H] fp32, max_segments at
// least sum over the rows of ceil(len / seg_len).
extern "C" int as_state_space(const float* xbc, int channels, int H, int G, int N, int E, const void* proj, int dtype, int ld,
                              int step_off, const float* dt_bias, const float* a_log, const float* skip, float* state,
                              const int* row_first, const int* row_len, const int* row_start, const int* row_slots,
                              int num_rows, float* out, int writes, int kernel, int seg_len, int max_segments,
                              float* seg_state, float* seg_decay, hipStream_t stream) {
  if (num_rows <= 0) return AS_OK;
  if (H <= 0 || G <= 0 || H % G || N <= 0 || E <= 0 || channels < H * E + 2 * G * N || step_off < 0 || step_off + H > ld ||
      H > 65535 || num_rows > 65535)
    return AS_BAD_SHAPE;
  if (dtype != DT_F32 && dtype != DT_BF16) return AS_BAD_DTYPE;
  Space s = {xbc, channels, H, G, N, E, proj, ld, step_off, dt_bias, a_log, skip, state, row_first, row_len, row_start,
             row_slots, num_rows, out, writes, 0, seg_state, seg_decay};
  if (kernel == 0) {
    if (N > 16 * SCAN_PER) return AS_BAD_SHAPE;
    int SL = 1;
    while (SL * SCAN_PER < N) SL <<= 1;
    const int cols = WAVE / SL;
    dim3 grid((E + cols - 1) / cols, H, num_rows);
    if (dtype == DT_F32) state_space_scan_kernel<float><<<grid, 64, 0, stream>>>(s, SL);
    else state_space_scan_kernel<bf16><<<grid, 64, 0, stream>>>(s, SL);
    return launch_status();
  }
  if (N > 128) return AS_BAD_SHAPE;
  if (kernel == 1) {
    if (E % 4) return AS_BAD_SHAPE;
    dim3 grid((E + 31) / 32, H, num_rows);
    if (dtype == DT_F32) state_space_step_kernel<float><<<grid, 64, 0, stream>>>(s);
    else state_space_step_kernel<bf16><<<grid, 64, 0, stream>>>(s);
    return launch_status();
  }
  if (kernel != 2 || seg_len < 0 || seg_len % CHUNK) return AS_BAD_SHAPE;
  if (seg_len && (!seg_state || !seg_decay || max_segments < 1 || max_segments > 65534)) return AS_BAD_SHAPE;
  const int blocks = (E + 31) / 32, units = H / G * blocks, NT = (N + 31) / 32;
  s.seg_len = seg_len;
  dim3 grid((units + 3) / 4, G, seg_len ? max_segments : num_rows);
  dim3 pass((unsigned)(((long)H * blocks * NT * 1024 + 255) / 256), num_rows);
#define LAUNCH2(T, NTV)                                                          \
  if (seg_len) {                                                                 \
    state_space_chunk_kernel<T, NTV, true><<<grid, 256, 0, stream>>>(s);         \
    state_space_pass_kernel<NTV><<<pass, 256, 0, stream>>>(s);                   \
  }                                                                              \
  state_space_chunk_kernel<T, NTV, false><<<grid, 256, 0, stream>>>(s)
#define LAUNCH(T)                      \
  switch (NT) {                        \
    case 1: LAUNCH2(T, 1); break;      \
    case 2: LAUNCH2(T, 2); break;      \
    case 3: LAUNCH2(T, 3); break;      \
    default: LAUNCH2(T, 4); break;     \
  }
  if (dtype == DT_F32) {
    LAUNCH(float)
  } else {
    LAUNCH(bf16)
  }
#undef LAUNCH
#undef LAUNCH2
  return launch_status();
}

// ---- the output's gate and norm ------------------------------------------------------------------------------------------
// v = y * silu(z), z columns z_off .. z_off + n of proj [T, ld]; every one of `groups` equal parts of v over its own root mean
// square (eps inside), times gain [n]; out [T, n] of proj's type.  grid (tokens, groups); a part stays in registers.
template <typename T, int VEC, int CH>
__global__ __launch_bounds__(1024) void gated_group_norm_kernel(const float* __restrict__ y, const T* __restrict__ proj, int ld,
                                                                int z_off, const float* __restrict__ gain, float eps, int n,
                                                                int size, T* __restrict__ out) {
  __shared__ float red[16];
  const size_t t = blockIdx.x;
  const int from = blockIdx.y * size;
  float v[CH][VEC], ss[1] = {0.f};
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
    if (i >= size) continue;
    float z[VEC];
    load_vec<VEC>(y + t * n + from + i, v[c]);
    load_vec<VEC>(proj + t * ld + z_off + from + i, z);
#pragma unroll
    for (int k = 0; k < VEC; ++k) {
      v[c][k] *= z[k] / (1.0f + quick_exp<T>(-z[k]));
      ss[0] = fmaf(v[c][k], v[c][k], ss[0]);
    }
  }
  block_sums(ss, red);
  const float inv = 1.0f / sqrtf(ss[0] / (float)size + eps);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (c * blockDim.x + threadIdx.x) * VEC;
    if (i >= size) continue;
    float g[VEC];
    load_vec<VEC>(gain + from + i, g);
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[c][k] *= inv * g[k];
    store_vec<VEC>(out + t * n + from + i, v[c]);
  }
}

template <typename T, int VEC>
static int launch_gated_group_norm(const float* y, const void* proj, int ld, int z_off, const float* gain, float eps, int n, int groups,
                                   void* out, int num_tokens, hipStream_t stream) {
  int threads, ch;
  const int size = n / groups;
  if (!row_shape(num_tokens * groups, size, VEC, &threads, &ch)) return AS_BAD_SHAPE;
  dim3 grid(num_tokens, groups);
#define LAUNCH(CHV) \
  gated_group_norm_kernel<T, VEC, CHV><<<grid, threads, 0, stream>>>(y, (const T*)proj, ld, z_off, gain, eps, n, size, (T*)out)
  switch (ch) {
    case 1: LAUNCH(1); break;
    case 2: LAUNCH(2); break;
    case 4: LAUNCH(4); break;
    case 8: LAUNCH(8); break;
    default:  // long parts of a width that is no multiple of four
      if constexpr (VEC == 1) {
        if (ch == 16) { LAUNCH(16); }
        else { LAUNCH(32); }
      }
      break;
  }
#undef LAUNCH
  return launch_status();
}

extern "C" int as_gated_group_norm(const float* y, const void* proj, int dtype, int ld, int z_off, const float* gain, float eps,
                                   int n, int groups, void* out, int num_tokens, hipStream_t stream) {
  if (num_tokens <= 0) return AS_OK;
  if (n <= 0 || groups <= 0 || n % groups || groups > 65535 || z_off < 0 || z_off + n > ld) return AS_BAD_SHAPE;
  const bool four = ((n / groups) | ld | z_off) % 4 == 0;
  if (dtype == DT_F32)
    return four ? launch_gated_group_norm<float, 4>(y, proj, ld, z_off, gain, eps, n, groups, out, num_tokens, stream)
                : launch_gated_group_norm<float, 1>(y, proj, ld, z_off, gain, eps, n, groups, out, num_tokens, stream);
  if (dtype == DT_BF16)
    return four ? launch_gated_group_norm<bf16, 4>(y, proj, ld, z_off, gain, eps, n, groups, out, num_tokens, stream)
                : launch_gated_group_norm<bf16, 1>(y, proj, ld, z_off, gain, eps, n, groups, out, num_tokens, stream);
  return AS_BAD_DTYPE;
}
