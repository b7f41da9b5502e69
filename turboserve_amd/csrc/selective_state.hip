// A selective state space: per head and request a 32-bit state S [N, P] that every token decays by one number and
// adds an outer product to,
//     dt = softplus(d + dt_bias)        a = exp(-exp(A_log) dt)
//     S <- a S + dt B x^T               y = S^T C + D x,
// with x [P] of the head, B and C [N] of the head's group (heads / groups neighbouring heads share one).
// dt, a, S, y and everything between them are 32-bit.  The state lies in the slot as [P][N], a column's N elements
// side by side.
//
// `u` [T, H P + 2 G N] (x | B | C, of type U) is the convolved part of the projection; `proj` is the fused projection
// [T, width] of the run's type, or `splits` 32-bit partial sums, of which the H columns from dt_at on are d.
//
// ts_selective_walk   per (request, head, stretch of columns): the request's tokens one behind the other, the state in
//                     registers.  Single tokens, short portions, and every 32-bit run.
// Long portions of bfloat16 runs are cut into pieces of SS_PIECE tokens that run side by side on the matrix cores.  With
// c_i the sum of log a over the piece's tokens up to and including i,
//     S_end = exp(c_last) S_before + sum_j exp(c_last - c_j) dt_j B_j x_j^T
//     y_i   = exp(c_i) S_before^T C_i + sum_{j <= i} exp(c_i - c_j) dt_j (C_i . B_j) x_j + D x_i,
// (the blocked form of Dao and Gu, "Transformers are SSMs: Generalized Models and Efficient Algorithms Through
// Structured State Space Duality"), in three launches: ts_selective_pieces mode 0 (every piece's own S_end from a zero
// state), ts_selective_carry (the state before each piece, elementwise; the last one goes to the slot),
// mode 1 (y).  x, B and C are bfloat16 numbers, so C . B is exact products summed in 32-bit; every other factor is a
// 32-bit number that is cut into three bfloat16 numbers whose sum it is exactly, and the three products are summed
// in 32-bit: nothing of the recurrence is rounded to 16 bits.
//
// ts_gated_group_norm: y silu(z), every one of `parts` equal parts of a row divided by its own root mean square, times
// a gain, rounded once.
#include "vec.hpp"

#define SS_PIECE 128
#define SS_STRETCH 32
#define SS_PARTS 8  // lanes that share a column of the state in the walk

typedef __bf16 ss_bf16x8 __attribute__((ext_vector_type(8)));
typedef float ss_f32x4 __attribute__((ext_vector_type(4)));
typedef unsigned int ss_u32x2 __attribute__((ext_vector_type(2)));

template <typename P>
__device__ __forceinline__ float ss_input(const P* p, int splits, size_t stride) {
  if (splits == 1) return to_float(p[0]);
  float s = 0.f;
  for (int first = 0; first < splits; first += 8) {
    float v[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = to_float(p[(size_t)min(first + j, splits - 1) * stride]);
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (first + j < splits) s += v[j];
  }
  return s;
}

__device__ __forceinline__ float ss_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// ---------------------------------------------------------------------------------------------
// the walk
// ---------------------------------------------------------------------------------------------

// NR: state rows a thread holds (of every stretch of 4 SS_PARTS rows the four from 4 part on); COLS: columns of a
// workgroup; BATCH: tokens staged in LDS at a time.
template <typename U, typename P, int NR, int BATCH, int COLS>
__global__ void __launch_bounds__(SS_PARTS * COLS)
selective_walk_kernel(float* __restrict__ y, float* __restrict__ state, const U* __restrict__ u, const P* __restrict__ proj, int splits,
                      size_t split_stride, int width, int dt_at, const float* __restrict__ dt_bias, const float* __restrict__ a_log,
                      const float* __restrict__ skip, const int* __restrict__ state_slots, const int* __restrict__ query_start_loc,
                      int first_seq, int heads, int groups, int n, int p) {
  constexpr int ROWS = SS_PARTS * NR, THREADS = SS_PARTS * COLS;
  __shared__ __attribute__((aligned(16))) float bs[BATCH][ROWS];
  __shared__ __attribute__((aligned(16))) float cs[BATCH][ROWS];
  __shared__ float xs[BATCH][COLS];
  __shared__ float dts[BATCH], as[BATCH];
  const int seq = first_seq + blockIdx.x, h = blockIdx.y, g = h / (heads / groups);
  const int tid = threadIdx.x, part = tid % SS_PARTS, col_in = tid / SS_PARTS;
  const int c0 = blockIdx.z * COLS, c = c0 + col_in;
  const bool live = c < p;
  const int row0 = query_start_loc[seq], count = query_start_loc[seq + 1] - row0;
  const size_t u_width = (size_t)heads * p + (size_t)2 * groups * n;
  const size_t b_at = (size_t)heads * p + (size_t)g * n, c_at = b_at + (size_t)groups * n;
  float* held = state + (((size_t)state_slots[seq] * heads + h) * p + (live ? c : 0)) * n;
  const bool quads = n % 4 == 0;
  float s[NR];
#pragma unroll
  for (int x = 0; x < NR / 4; ++x) {
    const int d = x * 4 * SS_PARTS + part * 4;
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (live && quads) {
      if (d < n) v = *reinterpret_cast<const float4*>(held + d);
    } else if (live) {
      if (d < n) v.x = held[d];
      if (d + 1 < n) v.y = held[d + 1];
      if (d + 2 < n) v.z = held[d + 2];
      if (d + 3 < n) v.w = held[d + 3];
    }
    s[4 * x] = v.x; s[4 * x + 1] = v.y; s[4 * x + 2] = v.z; s[4 * x + 3] = v.w;
  }
  const float rate = expf(a_log[h]), bias = dt_bias[h], d_skip = skip[h];
  for (int base = 0; base < count; base += BATCH) {
    const int batch = min(BATCH, count - base);
    if (base > 0) __syncthreads();  // the batch before is done with what is staged
    for (int i = tid; i < batch * ROWS; i += THREADS) {
      const int j = i / ROWS, d = i % ROWS;
      const U* row = u + (size_t)(row0 + base + j) * u_width;
      bs[j][d] = d < n ? to_float(row[b_at + d]) : 0.f;
      cs[j][d] = d < n ? to_float(row[c_at + d]) : 0.f;
    }
    for (int i = tid; i < batch * COLS; i += THREADS) {
      const int j = i / COLS, cc = c0 + i % COLS;
      xs[j][i % COLS] = cc < p ? to_float(u[(size_t)(row0 + base + j) * u_width + (size_t)h * p + cc]) : 0.f;
    }
    if (tid < batch) {
      const float dt = ss_softplus(ss_input(proj + (size_t)(row0 + base + tid) * width + dt_at + h, splits, split_stride) + bias);
      dts[tid] = dt;
      as[tid] = expf(-rate * dt);
    }
    __syncthreads();
    for (int j = 0; j < batch; ++j) {
      const float a = as[j], xv = xs[j][col_in], dx = dts[j] * xv;
      float r[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int x = 0; x < NR / 4; ++x) {
        const float4 b4 = *reinterpret_cast<const float4*>(&bs[j][x * 4 * SS_PARTS + part * 4]);
        const float4 c4 = *reinterpret_cast<const float4*>(&cs[j][x * 4 * SS_PARTS + part * 4]);
        const int i = 4 * x;
        s[i] = fmaf(a, s[i], b4.x * dx); s[i + 1] = fmaf(a, s[i + 1], b4.y * dx);
        s[i + 2] = fmaf(a, s[i + 2], b4.z * dx); s[i + 3] = fmaf(a, s[i + 3], b4.w * dx);
        r[0] = fmaf(s[i], c4.x, r[0]); r[1] = fmaf(s[i + 1], c4.y, r[1]);
        r[2] = fmaf(s[i + 2], c4.z, r[2]); r[3] = fmaf(s[i + 3], c4.w, r[3]);
      }
      float sum = (r[0] + r[1]) + (r[2] + r[3]);
      // Over the eight lanes of the column.
      sum += lanes_moved<0xB1, 0xF>(0.f, sum);
      sum += lanes_moved<0x4E, 0xF>(0.f, sum);
      sum += lanes_moved<0x141, 0xF>(0.f, sum);
      if (live && part == 0) y[((size_t)(row0 + base + j) * heads + h) * p + c] = fmaf(d_skip, xv, sum);
    }
  }
  if (!live || count < 1) return;
#pragma unroll
  for (int x = 0; x < NR / 4; ++x) {
    const int d = x * 4 * SS_PARTS + part * 4;
    if (quads) {
      if (d < n) *reinterpret_cast<float4*>(held + d) = make_float4(s[4 * x], s[4 * x + 1], s[4 * x + 2], s[4 * x + 3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (d + e < n) held[d + e] = s[4 * x + e];
    }
  }
}

// ---------------------------------------------------------------------------------------------
// pieces side by side on the matrix cores
// ---------------------------------------------------------------------------------------------

struct SsPiece {
  int seq;    // request of the step
  int first;  // first row
  int count;  // rows, at most SS_PIECE
  int pad;
};

// v = the sum of three bfloat16 numbers, exactly (each takes the next eight bits of the mantissa); returned as bits in
// the upper halves of the words.
__device__ __forceinline__ void ss_cut(float v, uint32_t& top, uint32_t& mid, uint32_t& low) {
  top = __float_as_uint(v) & 0xffff0000u;
  const float r1 = v - __uint_as_float(top);
  mid = __float_as_uint(r1) & 0xffff0000u;
  low = __float_as_uint(r1 - __uint_as_float(mid));
}

// The upper halves of two words side by side.
__device__ __forceinline__ uint32_t ss_pair(uint32_t lower, uint32_t upper) { return __builtin_amdgcn_perm(upper, lower, 0x07060302u); }

__device__ __forceinline__ ss_f32x4 ss_mfma(ts_u32x4 a, ts_u32x4 b, ss_f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(ss_bf16x8, a), __builtin_bit_cast(ss_bf16x8, b), c, 0, 0, 0);
}

// What a piece's tokens need of the decays: dt and the running sum of log a as two 32-bit numbers (formed in 64-bit, so
// that a difference of two of them is good to 32-bit however long the piece has decayed).
struct SsSteps {
  float dt[SS_PIECE];
  float top[SS_PIECE];
  float low[SS_PIECE];
};

// By the first wavefront: lane l takes the tokens 2 l and 2 l + 1 (beyond the piece: dt 0, nothing added).
template <typename P>
__device__ __forceinline__ void ss_steps(SsSteps& at, const P* proj, int splits, size_t split_stride, int width, int dt_at, float bias,
                                         float rate, SsPiece piece) {
  const int lane = threadIdx.x;
  float dt[2];
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const int j = 2 * lane + e;
    const float z = ss_input(proj + (size_t)(piece.first + min(j, piece.count - 1)) * width + dt_at, splits, split_stride) + bias;
    dt[e] = j < piece.count ? ss_softplus(z) : 0.f;
  }
  const double own = -(double)rate * ((double)dt[0] + (double)dt[1]);
  double sum = own;
#pragma unroll
  for (int d = 1; d < TS_WAVE; d <<= 1) {
    const double other = __shfl_up(sum, d);
    if (lane >= d) sum += other;
  }
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const double c = e == 1 ? sum : sum - own - (double)rate * (double)dt[0];
    at.dt[2 * lane + e] = dt[e];
    const float top = (float)c;
    at.top[2 * lane + e] = top;
    at.low[2 * lane + e] = (float)(c - (double)top);
  }
}

// Rows 4 q .. 4 q + 3 (from row r0 of u, rows beyond `count` zero) of the eight columns from `col` on, turned: element
// (column e, row i) of the result.
__device__ __forceinline__ void ss_load_rows(const bf16_t* u, size_t u_width, int first, int r0, int count, size_t col, bool in, ts_u32x4 (&raw)[4]) {
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    raw[i] = ts_u32x4{0u, 0u, 0u, 0u};
    if (in && r0 + i < count) raw[i] = *reinterpret_cast<const ts_u32x4*>(u + (size_t)(first + r0 + i) * u_width + col);
  }
}

__device__ __forceinline__ uint32_t ss_half(ts_u32x4 v, int e) { return e & 1 ? v[e / 2] & 0xffff0000u : v[e / 2] << 16; }  // as the bits of a float

// Where mode 0 keeps token j of row r in LDS.  Rows are SS_STRETCH + 8 apart; the four chunks of eight tokens change
// places by the row's group of eight, and groups of 32 rows are 16 words further apart: so the threads that turn tokens
// and rows over, whose rows are eight apart, write to different banks.
__device__ __forceinline__ int ss_place(int r, int j) {
  return r * (SS_STRETCH + 8) + (r >> 5) * 32 + ((((j >> 3) ^ (r >> 3)) & 3) << 3) + (j & 7);
}

constexpr int ss_rows_size(int rows) { return rows * (SS_STRETCH + 8) + ((rows + 31) >> 5) * 32; }

// Mode 0.  NK: stretches of 32 state rows; PT: stretches of 16 columns.  A wavefront owns every fourth stretch of 16
// state rows and all columns: S_end^T (rows n, columns p) = sum over j of B^T (exact, LDS, tokens side by side) times
// the weighted x (three planes, LDS).  The piece is taken in stretches of
// SS_STRETCH tokens, so that four workgroups and more fit a compute unit.
template <typename P, int NK, int PT>
__global__ void __launch_bounds__(256)
selective_piece_state_kernel(float* __restrict__ piece_state, float* __restrict__ piece_decay, const bf16_t* __restrict__ u,
                             const P* __restrict__ proj, int splits, size_t split_stride, int width, int dt_at,
                             const float* __restrict__ dt_bias, const float* __restrict__ a_log, const SsPiece* __restrict__ pieces,
                             int heads, int groups, int n, int p) {
  constexpr int NP = 32 * NK, PP = 16 * PT;
  constexpr int TILES = (2 * NK + 3) / 4;  // stretches of 16 state rows a wavefront owns
  extern __shared__ __attribute__((aligned(16))) uint16_t ss_lds[];
  uint16_t* bt = ss_lds;                          // NP rows: B, tokens side by side
  uint16_t* const xw[3] = {ss_lds + ss_rows_size(NP), ss_lds + ss_rows_size(NP) + ss_rows_size(PP),
                           ss_lds + ss_rows_size(NP) + 2 * ss_rows_size(PP)};  // PP rows each: the weighted x in three planes
  __shared__ SsSteps steps;
  const int item = blockIdx.x, h = blockIdx.y, g = h / (heads / groups);
  const SsPiece piece = pieces[item];
  const int tid = threadIdx.x, wave = tid / TS_WAVE, lane = tid % TS_WAVE;
  const int lo = lane % 16, quad = lane / 16;
  const int c0 = blockIdx.z * PP;
  const size_t u_width = (size_t)heads * p + (size_t)2 * groups * n;
  const size_t b_at = (size_t)heads * p + (size_t)g * n, x_at = (size_t)h * p + c0;
  if (wave == 0) ss_steps(steps, proj, splits, split_stride, width, dt_at + h, dt_bias[h], expf(a_log[h]), piece);
  ss_f32x4 acc[TILES][PT];
#pragma unroll
  for (int a = 0; a < TILES; ++a)
#pragma unroll
    for (int b = 0; b < PT; ++b) acc[a][b] = ss_f32x4{0.f, 0.f, 0.f, 0.f};
  for (int j0 = 0; j0 < piece.count; j0 += SS_STRETCH) {
    __syncthreads();  // the steps are there; the stretch before has been read
    for (int i = tid; i < (SS_STRETCH / 4) * (NP / 8); i += 256) {
      const int q = i / (NP / 8), d = (i % (NP / 8)) * 8;
      ts_u32x4 raw[4];
      ss_load_rows(u, u_width, piece.first, j0 + 4 * q, piece.count, b_at + d, d < n, raw);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const ss_u32x2 four = {ss_pair(ss_half(raw[0], e), ss_half(raw[1], e)), ss_pair(ss_half(raw[2], e), ss_half(raw[3], e))};
        *reinterpret_cast<ss_u32x2*>(&bt[ss_place(d + e, 4 * q)]) = four;
      }
    }
    const float end_top = steps.top[SS_PIECE - 1], end_low = steps.low[SS_PIECE - 1];
    for (int i = tid; i < (SS_STRETCH / 2) * (PP / 8); i += 256) {  // two tokens by eight columns a thread
      const int q = i / (PP / 8), d = (i % (PP / 8)) * 8;
      ts_u32x4 raw[2];
      float w[2];
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const int j = j0 + 2 * q + k;
        raw[k] = ts_u32x4{0u, 0u, 0u, 0u};
        if (c0 + d < p && j < piece.count) raw[k] = *reinterpret_cast<const ts_u32x4*>(u + (size_t)(piece.first + j) * u_width + x_at + d);
        w[k] = steps.dt[j] * expf((end_top - steps.top[j]) + (end_low - steps.low[j]));
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        uint32_t top[2], mid[2], low[2];
#pragma unroll
        for (int k = 0; k < 2; ++k) ss_cut(w[k] * __uint_as_float(ss_half(raw[k], e)), top[k], mid[k], low[k]);
        const int at = ss_place(d + e, 2 * q);
        *reinterpret_cast<uint32_t*>(&xw[0][at]) = ss_pair(top[0], top[1]);
        *reinterpret_cast<uint32_t*>(&xw[1][at]) = ss_pair(mid[0], mid[1]);
        *reinterpret_cast<uint32_t*>(&xw[2][at]) = ss_pair(low[0], low[1]);
      }
    }
    __syncthreads();
    ts_u32x4 bf[TILES];
#pragma unroll
    for (int a = 0; a < TILES; ++a)
      bf[a] = *reinterpret_cast<const ts_u32x4*>(&bt[ss_place(16 * min(wave + 4 * a, 2 * NK - 1) + lo, 8 * quad)]);
#pragma unroll
    for (int plane = 2; plane >= 0; --plane)  // (the small planes first)
#pragma unroll
      for (int b = 0; b < PT; ++b) {
        const ts_u32x4 xf = *reinterpret_cast<const ts_u32x4*>(&xw[plane][ss_place(16 * b + lo, 8 * quad)]);
#pragma unroll
        for (int a = 0; a < TILES; ++a) acc[a][b] = ss_mfma(bf[a], xf, acc[a][b]);
      }
  }
#pragma unroll
  for (int a = 0; a < TILES; ++a) {
    const int d = 16 * (wave + 4 * a) + 4 * quad;
#pragma unroll
    for (int b = 0; b < PT; ++b) {
      const int c = c0 + 16 * b + lo;
      if (d < n && c < p)
        *reinterpret_cast<ss_f32x4*>(piece_state + (((size_t)item * heads + h) * p + c) * n + d) = acc[a][b];
    }
  }
  if (blockIdx.z == 0 && tid == 0) piece_decay[(size_t)item * heads + h] = expf(steps.top[SS_PIECE - 1] + steps.low[SS_PIECE - 1]);
}

// Between the modes.  A thread takes four neighbouring elements of a head's state through its request's pieces.
struct SsCarry {
  int slot_seq;
  int first;
  int count;
  int pad;
};

__global__ void __launch_bounds__(256)
selective_carry_kernel(float* __restrict__ state, const int* __restrict__ state_slots, const SsCarry* __restrict__ carries,
                       float* __restrict__ piece_state, const float* __restrict__ piece_decay, int heads, int per_head) {
  const SsCarry carry = carries[blockIdx.x];
  const int h = blockIdx.y;
  const int e = 4 * (blockIdx.z * blockDim.x + threadIdx.x);
  if (e >= per_head) return;
  float* slot = state + ((size_t)state_slots[carry.slot_seq] * heads + h) * per_head + e;
  float4 s = *reinterpret_cast<const float4*>(slot);
  constexpr int AHEAD = 8;  // pieces in flight
  for (int i0 = 0; i0 < carry.count; i0 += AHEAD) {
    float4 own[AHEAD];
    float decay[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const size_t at = (size_t)(carry.first + min(i0 + i, carry.count - 1)) * heads + h;
      own[i] = *reinterpret_cast<const float4*>(piece_state + at * per_head + e);
      decay[i] = piece_decay[at];
    }
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      if (i0 + i < carry.count) {
        *reinterpret_cast<float4*>(piece_state + ((size_t)(carry.first + i0 + i) * heads + h) * per_head + e) = s;
        s.x = fmaf(decay[i], s.x, own[i].x); s.y = fmaf(decay[i], s.y, own[i].y);
        s.z = fmaf(decay[i], s.z, own[i].z); s.w = fmaf(decay[i], s.w, own[i].w);
      }
    }
  }
  *reinterpret_cast<float4*>(slot) = s;
}

// Mode 1.  Wavefront w owns the tokens of the stretches w and 7 - w of sixteen (together they see as many tokens as any
// other's two).  Everything is computed turned, y^T (rows p, columns i): the weights (C_i . B_j) exp(c_i - c_j) dt_j come
// out of one product with token i on the lane and four tokens j in its registers, which is what the next product wants of
// its second operand if the tokens j are counted in that order; they never leave the registers.
// Of the tokens j before the stretch the factor is exp(c_i - c_r) times exp(c_r - c_j) dt_j, r the last token before
// the stretch: the first is applied to a stretch's sums once, the second comes from a table that the workgroup makes once
// (`before`: both exponents are at most zero, so nothing overflows however strong the decays are).
template <typename P, int NK, int PT>
__global__ void __launch_bounds__(256, NK <= 4 ? 4 : 2)
selective_piece_out_kernel(float* __restrict__ y, const float* __restrict__ piece_state, const bf16_t* __restrict__ u,
                           const P* __restrict__ proj, int splits, size_t split_stride, int width, int dt_at,
                           const float* __restrict__ dt_bias, const float* __restrict__ a_log, const float* __restrict__ skip,
                           const SsPiece* __restrict__ pieces, int heads, int groups, int n, int p) {
  constexpr int NP = 32 * NK, PP = 16 * PT, SROW = NP + 8, XROW = SS_PIECE + 4, HALF = SS_PIECE / 2;
  extern __shared__ __attribute__((aligned(16))) uint16_t ss_lds[];
  uint16_t* planes = ss_lds;           // [2][PP][SROW]: the state before the piece, its two lower planes, then its upper one
  uint16_t* br = ss_lds;               // then [HALF][SROW]: B of half the tokens at a time
  uint16_t* xt = ss_lds + HALF * SROW; // and [PP][XROW]: x, tokens side by side
  __shared__ __attribute__((aligned(16))) SsSteps steps;
  __shared__ __attribute__((aligned(16))) float before[SS_PIECE / 16][SS_PIECE];  // [stretch of i][j]
  const int item = blockIdx.x, h = blockIdx.y, g = h / (heads / groups);
  const SsPiece piece = pieces[item];
  const int tid = threadIdx.x, wave = tid / TS_WAVE, lane = tid % TS_WAVE;
  const int lo = lane % 16, quad = lane / 16;
  const int c0 = blockIdx.z * PP;
  const size_t u_width = (size_t)heads * p + (size_t)2 * groups * n;
  const size_t b_at = (size_t)heads * p + (size_t)g * n, c_at = b_at + (size_t)groups * n, x_at = (size_t)h * p + c0;
  const int tiles[2] = {wave, 7 - wave};
  if (wave == 0) ss_steps(steps, proj, splits, split_stride, width, dt_at + h, dt_bias[h], expf(a_log[h]), piece);
  const float* entering = piece_state + (((size_t)item * heads + h) * p + c0) * n;
  ts_u32x4 cf[2][NK];  // C of the wavefront's tokens: columns i, eight state rows a lane
  ss_f32x4 acc[PT][2];
#pragma unroll
  for (int b = 0; b < PT; ++b)
#pragma unroll
    for (int a = 0; a < 2; ++a) acc[b][a] = ss_f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int ITEMS = (PP * (NP / 8) + 255) / 256;
  ts_u32x4 upper[ITEMS];  // the upper plane of what the thread has read of the state, while the lower ones are multiplied
#pragma unroll
  for (int turn = 0; turn < 2; ++turn) {  // the two lower planes first, then the upper one in their place
    if (turn > 0) __syncthreads();
#pragma unroll
    for (int x = 0; x < ITEMS; ++x) {
      const int i = tid + 256 * x;
      if (i >= PP * (NP / 8)) continue;
      const int c = i / (NP / 8), d = (i % (NP / 8)) * 8;
      if (turn > 0) {
        *reinterpret_cast<ts_u32x4*>(&planes[c * SROW + d]) = upper[x];
        continue;
      }
      float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      if (c0 + c < p && d < n) {
        const float4 v0 = *reinterpret_cast<const float4*>(entering + (size_t)c * n + d);
        const float4 v1 = *reinterpret_cast<const float4*>(entering + (size_t)c * n + d + 4);
        v[0] = v0.x; v[1] = v0.y; v[2] = v0.z; v[3] = v0.w;
        v[4] = v1.x; v[5] = v1.y; v[6] = v1.z; v[7] = v1.w;
      }
      ts_u32x4 middle, lower;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        uint32_t top[2], mid[2], low[2];
        ss_cut(v[2 * e], top[0], mid[0], low[0]);
        ss_cut(v[2 * e + 1], top[1], mid[1], low[1]);
        upper[x][e] = ss_pair(top[0], top[1]);
        middle[e] = ss_pair(mid[0], mid[1]);
        lower[e] = ss_pair(low[0], low[1]);
      }
      *reinterpret_cast<ts_u32x4*>(&planes[c * SROW + d]) = middle;
      *reinterpret_cast<ts_u32x4*>(&planes[(PP + c) * SROW + d]) = lower;
    }
    if (turn == 0) {
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        const int i = 16 * tiles[a] + lo;
#pragma unroll
        for (int k = 0; k < NK; ++k) {
          const int d = 32 * k + 8 * quad;
          cf[a][k] = ts_u32x4{0u, 0u, 0u, 0u};
          if (i < piece.count && d < n) cf[a][k] = *reinterpret_cast<const ts_u32x4*>(u + (size_t)(piece.first + i) * u_width + c_at + d);
        }
      }
    }
    __syncthreads();
    if (turn == 0) {
#pragma unroll 1
      for (int i = tid; i < SS_PIECE / 16 * SS_PIECE; i += 256) {
        const int tile = i / SS_PIECE, j = i % SS_PIECE, r = 16 * tile - 1;
        if (j <= r) before[tile][j] = steps.dt[j] * __expf((steps.top[r] - steps.top[j]) + (steps.low[r] - steps.low[j]));
      }
    }
#pragma unroll
    for (int plane = 1 - turn; plane >= 0; --plane)
#pragma unroll
      for (int k = 0; k < NK; ++k)
#pragma unroll
        for (int b = 0; b < PT; ++b) {
          const ts_u32x4 sf = *reinterpret_cast<const ts_u32x4*>(&planes[(plane * PP + 16 * b + lo) * SROW + 32 * k + 8 * quad]);
#pragma unroll
          for (int a = 0; a < 2; ++a) acc[b][a] = ss_mfma(sf, cf[a][k], acc[b][a]);
        }
  }
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    const float by = tiles[a] > 0 ? expf(steps.top[16 * tiles[a] - 1] + steps.low[16 * tiles[a] - 1]) : 1.f;
#pragma unroll
    for (int b = 0; b < PT; ++b) acc[b][a] *= by;
  }
  for (int half = 0; half * HALF < piece.count; ++half) {
    __syncthreads();  // the planes, or B of the first half, have been read: their place takes what follows
#pragma unroll 2
    for (int i = tid; i < HALF * (NP / 8); i += 256) {
      const int j = i / (NP / 8), d = (i % (NP / 8)) * 8;
      ts_u32x4 raw = {0u, 0u, 0u, 0u};
      if (half * HALF + j < piece.count && d < n)
        raw = *reinterpret_cast<const ts_u32x4*>(u + (size_t)(piece.first + half * HALF + j) * u_width + b_at + d);
      *reinterpret_cast<ts_u32x4*>(&br[j * SROW + d]) = raw;
    }
#pragma unroll 1
    for (int i = tid; half == 0 && i < (SS_PIECE / 2) * (PP / 8); i += 256) {  // two tokens by eight columns a thread
      const int q = i / (PP / 8), d = (i % (PP / 8)) * 8;
      ts_u32x4 raw[2];
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        raw[k] = ts_u32x4{0u, 0u, 0u, 0u};
        if (c0 + d < p && 2 * q + k < piece.count)
          raw[k] = *reinterpret_cast<const ts_u32x4*>(u + (size_t)(piece.first + 2 * q + k) * u_width + x_at + d);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e)
        *reinterpret_cast<uint32_t*>(&xt[(d + e) * XROW + 2 * q]) = ss_pair(ss_half(raw[0], e), ss_half(raw[1], e));
    }
    __syncthreads();
#pragma unroll
    for (int a = 0; a < 2; ++a) {
      const int tile = tiles[a];
      if (16 * tile >= piece.count) continue;
#pragma unroll 1
      for (int jb = 2 * half; jb < 2 * half + 2 && 2 * jb <= tile; ++jb) {
        ss_f32x4 s[2] = {ss_f32x4{0.f, 0.f, 0.f, 0.f}, ss_f32x4{0.f, 0.f, 0.f, 0.f}};  // by stretch of 16 tokens j
#pragma unroll
        for (int k = 0; k < NK; ++k)
#pragma unroll
          for (int t = 0; t < 2; ++t)
            s[t] = ss_mfma(*reinterpret_cast<const ts_u32x4*>(&br[(32 * (jb - 2 * half) + 16 * t + lo) * SROW + 32 * k + 8 * quad]), cf[a][k], s[t]);
        const int j0 = 32 * jb + 4 * quad;
        if (2 * jb + 1 < tile) {
#pragma unroll
          for (int t = 0; t < 2; ++t) s[t] *= *reinterpret_cast<const ss_f32x4*>(&before[tile][j0 + 16 * t]);
        } else {
          // The stretch's own tokens (and, of an odd one, the sixteen before it): from here on the sums are y's own.
          const int i = 16 * tile + lo;
          const float mine_top = steps.top[i], mine_low = steps.low[i];
          const float by = tile > 0 ? expf((mine_top - steps.top[16 * tile - 1]) + (mine_low - steps.low[16 * tile - 1])) : expf(mine_top + mine_low);
#pragma unroll
          for (int b = 0; b < PT; ++b) acc[b][a] *= by;
#pragma unroll
          for (int t = 0; t < 2; ++t) {
            const ss_f32x4 tops = *reinterpret_cast<const ss_f32x4*>(&steps.top[j0 + 16 * t]);
            const ss_f32x4 lows = *reinterpret_cast<const ss_f32x4*>(&steps.low[j0 + 16 * t]);
            const ss_f32x4 dts = *reinterpret_cast<const ss_f32x4*>(&steps.dt[j0 + 16 * t]);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              // (A later token's decay is never formed: its exponent would be positive.)
              const bool seen = j0 + 16 * t + r <= i;
              const float gone = seen ? (mine_top - tops[r]) + (mine_low - lows[r]) : 0.f;
              s[t][r] = seen ? s[t][r] * dts[r] * __expf(gone) : 0.f;
            }
          }
        }
        ts_u32x4 wf[3];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          uint32_t top[2], mid[2], low[2];
#pragma unroll
          for (int k = 0; k < 2; ++k) ss_cut(s[e / 2][2 * (e % 2) + k], top[k], mid[k], low[k]);
          wf[0][e] = ss_pair(top[0], top[1]);
          wf[1][e] = ss_pair(mid[0], mid[1]);
          wf[2][e] = ss_pair(low[0], low[1]);
        }
#pragma unroll
        for (int b = 0; b < PT; ++b) {
          const uint16_t* row = &xt[(16 * b + lo) * XROW + j0];
          const ss_u32x2 first = *reinterpret_cast<const ss_u32x2*>(row), second = *reinterpret_cast<const ss_u32x2*>(row + 16);
          const ts_u32x4 xf = {first[0], first[1], second[0], second[1]};
#pragma unroll
          for (int plane = 2; plane >= 0; --plane) acc[b][a] = ss_mfma(xf, wf[plane], acc[b][a]);
        }
      }
    }
  }
  const float d_skip = skip[h];
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    const int i = 16 * tiles[a] + lo;
    if (i >= piece.count) continue;
#pragma unroll
    for (int b = 0; b < PT; ++b) {
      const int c = 16 * b + 4 * quad;
      if (c0 + c >= p) continue;
      float x[4];
      load_vec<bf16_t, 4>(u + (size_t)(piece.first + i) * u_width + x_at + c, x);
      float v[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = fmaf(d_skip, x[e], acc[b][a][e]);
      store_vec<float, 4>(y + ((size_t)(piece.first + i) * heads + h) * p + c0 + c, v);
    }
  }
}

// ---------------------------------------------------------------------------------------------
// the gated norm in parts
// ---------------------------------------------------------------------------------------------
template <typename T, typename P, int VEC, int CHUNKS>
__global__ void __launch_bounds__(1024)
gated_group_norm_kernel(T* __restrict__ out, const float* __restrict__ y, const P* __restrict__ proj, int splits, size_t split_stride,
                        int width, int z_at, const T* __restrict__ gain, float eps, int parts, int size) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, part = blockIdx.y;
  const size_t row = ((size_t)t * parts + part) * size;
  const P* z = proj + (size_t)t * width + z_at + (size_t)part * size;
  float v[CHUNKS][VEC];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int i = (int)(c * blockDim.x + threadIdx.x) * VEC;
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[c][e] = 0.f;
    if (i < size) {
      float gate[VEC];
      load_vec<P, VEC>(z + i, gate);
      load_vec<float, VEC>(y + row + i, v[c]);
      for (int first = 1; first < splits; first += 8) {
        float more[8][VEC];
#pragma unroll
        for (int j = 0; j < 8; ++j) load_vec<P, VEC>(z + (size_t)min(first + j, splits - 1) * split_stride + i, more[j]);
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (first + j < splits) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) gate[e] += more[j][e];
          }
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        v[c][e] *= gate[e] / (1.f + expf(-gate[e]));
        ss = fmaf(v[c][e], v[c][e], ss);
      }
    }
  }
  const float by = rsqrtf(block_sum(ss, scratch) / (float)size + eps);
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int i = (int)(c * blockDim.x + threadIdx.x) * VEC;
    if (i < size) {
      float w[VEC];
      load_vec<T, VEC>(gain + (size_t)part * size + i, w);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[c][e] *= by * w[e];
      store_vec<T, VEC>(out + row + i, v[c]);
    }
  }
}

// ---------------------------------------------------------------------------------------------
// entry points
// ---------------------------------------------------------------------------------------------

static bool ss_sizes_ok(int heads, int groups, int n, int p, int width, int dt_at, int splits) {
  return heads >= 1 && heads <= 65535 && groups >= 1 && heads % groups == 0 && n >= 1 && n <= 512 && p >= 1 && p <= 65535 && splits >= 1 &&
         dt_at >= 0 && dt_at + heads <= width;
}

// u_f32: u is 32-bit (else bfloat16); dtype, in_f32: as everywhere (the projection's type).
extern "C" int ts_selective_walk(float* y, float* state, const void* u, int u_f32, const void* proj, int in_f32, int splits,
                                 long split_stride, int width, int dt_at, const float* dt_bias, const float* a_log, const float* skip,
                                 const int* state_slots, const int* query_start_loc, int first_seq, int num_seqs, int heads, int groups,
                                 int n, int p, int dtype, hipStream_t stream) {
  if (num_seqs == 0) return TS_OK;
  if (!y || !state || !u || !proj || !dt_bias || !a_log || !skip || !state_slots || !query_start_loc) return TS_ERR_ARG;
  if (!ss_sizes_ok(heads, groups, n, p, width, dt_at, splits)) return TS_ERR_SHAPE;
#define SS_GO(U, P, NR, BATCH, COLS)                                                                                                \
  hipLaunchKernelGGL((selective_walk_kernel<U, P, NR, BATCH, COLS>), dim3(num_seqs, heads, (p + COLS - 1) / COLS),                  \
                     dim3(SS_PARTS * COLS), 0, stream, y, state, (const U*)u, (const P*)proj, splits, (size_t)split_stride, width, \
                     dt_at, dt_bias, a_log, skip, state_slots, query_start_loc, first_seq, heads, groups, n, p)
#define SS_SIZES(U, P)                                     \
  do {                                                     \
    if (n <= 32) SS_GO(U, P, 4, 8, 32);                    \
    else if (n <= 64) SS_GO(U, P, 8, 8, 32);               \
    else if (n <= 128) SS_GO(U, P, 16, 8, 32);             \
    else if (n <= 256) SS_GO(U, P, 32, 4, 32);             \
    else SS_GO(U, P, 64, 4, 32);                           \
  } while (0)
  if (dtype == TS_F32) SS_SIZES(float, float);
  else if (dtype == TS_BF16 && in_f32 && !u_f32) SS_SIZES(bf16_t, float);
  else if (dtype == TS_BF16 && !u_f32) SS_SIZES(bf16_t, bf16_t);
  else return TS_ERR_DTYPE;
#undef SS_SIZES
#undef SS_GO
  return ts_launch_status();
}

// bfloat16 runs; mode 0: every piece's own end state and decay; mode 1: y from the state before each piece.
extern "C" int ts_selective_pieces(float* y, float* piece_state, float* piece_decay, const void* u, const void* proj, int in_f32, int splits,
                                   long split_stride, int width, int dt_at, const float* dt_bias, const float* a_log, const float* skip,
                                   const void* pieces, int num_pieces, int heads, int groups, int n, int p, int mode, hipStream_t stream) {
  if (num_pieces == 0) return TS_OK;
  if (!piece_state || !piece_decay || !u || !proj || !dt_bias || !a_log || !skip || !pieces || (mode == 1 && !y) || mode < 0 || mode > 1)
    return TS_ERR_ARG;
  if (!ss_sizes_ok(heads, groups, n, p, width, dt_at, splits) || n > 256 || n % 8 != 0 || p % 8 != 0) return TS_ERR_SHAPE;
  if (((uintptr_t)u | (uintptr_t)piece_state | (uintptr_t)y) % 16 != 0) return TS_ERR_ARG;
  bool refused = false;
#define SS_PIECES(P, NK, PT)                                                                                                         \
  do {                                                                                                                               \
    const dim3 grid(num_pieces, heads, (p + 16 * PT - 1) / (16 * PT));                                                               \
    constexpr int state_lds = (ss_rows_size(32 * NK) + 3 * ss_rows_size(16 * PT)) * 2;                                                                      \
    constexpr int planes = 2 * 16 * PT * (32 * NK + 8) * 2, rows = (SS_PIECE / 2 * (32 * NK + 8) + 16 * PT * (SS_PIECE + 4)) * 2;    \
    constexpr int out_lds = planes > rows ? planes : rows;                                                                           \
    if (mode == 0) {                                                                                                                 \
      static const bool ready = hipFuncSetAttribute((const void*)selective_piece_state_kernel<P, NK, PT>,                            \
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, state_lds) == hipSuccess;            \
      refused = !ready;                                                                                                              \
      if (ready)                                                                                                                     \
        hipLaunchKernelGGL((selective_piece_state_kernel<P, NK, PT>), grid, dim3(256), state_lds, stream, piece_state, piece_decay,  \
                           (const bf16_t*)u, (const P*)proj, splits, (size_t)split_stride, width, dt_at, dt_bias, a_log,             \
                           (const SsPiece*)pieces, heads, groups, n, p);                                                             \
    } else {                                                                                                                         \
      static const bool ready = hipFuncSetAttribute((const void*)selective_piece_out_kernel<P, NK, PT>,                              \
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, out_lds) == hipSuccess;              \
      refused = !ready;                                                                                                              \
      if (ready)                                                                                                                     \
        hipLaunchKernelGGL((selective_piece_out_kernel<P, NK, PT>), grid, dim3(256), out_lds, stream, y, piece_state,                \
                           (const bf16_t*)u, (const P*)proj, splits, (size_t)split_stride, width, dt_at, dt_bias, a_log, skip,       \
                           (const SsPiece*)pieces, heads, groups, n, p);                                                             \
    }                                                                                                                                \
  } while (0)
#define SS_SIZES(P, PT)                          \
  do {                                           \
    if (n <= 32) SS_PIECES(P, 1, PT);            \
    else if (n <= 64) SS_PIECES(P, 2, PT);       \
    else if (n <= 128) SS_PIECES(P, 4, PT);      \
    else SS_PIECES(P, 8, PT);                    \
  } while (0)
  if (in_f32) {
    if (p <= 32) SS_SIZES(float, 2);
    else SS_SIZES(float, 4);
  } else {
    if (p <= 32) SS_SIZES(bf16_t, 2);
    else SS_SIZES(bf16_t, 4);
  }
#undef SS_SIZES
#undef SS_PIECES
  return refused ? TS_ERR_LAUNCH : ts_launch_status();
}

extern "C" int ts_selective_carry(float* state, const int* state_slots, const void* carries, float* piece_state, const float* piece_decay,
                                  int requests, int heads, int n, int p, hipStream_t stream) {
  if (requests == 0) return TS_OK;
  if (!state || !state_slots || !carries || !piece_state || !piece_decay) return TS_ERR_ARG;
  if (heads < 1 || heads > 65535 || n < 1 || p < 1 || n > 512 || p > 65535 || (n * p) % 4 != 0) return TS_ERR_SHAPE;
  const dim3 grid(requests, heads, (n * p / 4 + 255) / 256);
  hipLaunchKernelGGL(selective_carry_kernel, grid, dim3(256), 0, stream, state, state_slots, (const SsCarry*)carries, piece_state,
                     piece_decay, heads, n * p);
  return ts_launch_status();
}

template <typename T, typename P>
static int launch_gated_group_norm(void* out, const float* y, const void* proj, int splits, long split_stride, int width, int z_at,
                                   const void* gain, float eps, int tokens, int parts, int size, hipStream_t stream) {
  const bool wide = size % 4 == 0 && width % 4 == 0 && z_at % 4 == 0 && split_stride % 4 == 0 &&
                    ((uintptr_t)out | (uintptr_t)y | (uintptr_t)proj | (uintptr_t)gain) % 16 == 0;
#define GN_GO(VEC, CHUNKS, THREADS)                                                                                                    \
  hipLaunchKernelGGL((gated_group_norm_kernel<T, P, VEC, CHUNKS>), dim3(tokens, parts), dim3(THREADS), 0, stream, (T*)out, y,          \
                     (const P*)proj, splits, (size_t)split_stride, width, z_at, (const T*)gain, eps, parts, size)
  if (wide) {
    const int pieces = size / 4;
    const bool few = (long)tokens * parts < 256;
    if (pieces <= 256 || (few && pieces <= 1024)) GN_GO(4, 1, (pieces + 63) / 64 * 64);
    else if (pieces <= 1024) GN_GO(4, 4, 256);
    else if (pieces <= 4096) GN_GO(4, 4, 1024);
    else if (pieces <= 16384) GN_GO(4, 16, 1024);
    else return TS_ERR_SHAPE;
  } else {
    if (size <= 1024) GN_GO(1, 1, (size + 63) / 64 * 64);
    else if (size <= 16384) GN_GO(1, 16, 1024);
    else return TS_ERR_SHAPE;
  }
#undef GN_GO
  return ts_launch_status();
}

extern "C" int ts_gated_group_norm(void* out, const float* y, const void* proj, int in_f32, int splits, long split_stride, int width,
                                   int z_at, const void* gain, float eps, int tokens, int parts, int size, int dtype, hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!out || !y || !proj || !gain) return TS_ERR_ARG;
  if (parts < 1 || parts > 65535 || size < 1 || z_at < 0 || (long)z_at + (long)parts * size > width || splits < 1) return TS_ERR_SHAPE;
  if (dtype == TS_F32)
    return launch_gated_group_norm<float, float>(out, y, proj, splits, split_stride, width, z_at, gain, eps, tokens, parts, size, stream);
  if (dtype == TS_BF16 && in_f32)
    return launch_gated_group_norm<bf16_t, float>(out, y, proj, splits, split_stride, width, z_at, gain, eps, tokens, parts, size, stream);
  if (dtype == TS_BF16)
    return launch_gated_group_norm<bf16_t, bf16_t>(out, y, proj, splits, split_stride, width, z_at, gain, eps, tokens, parts, size, stream);
  return TS_ERR_DTYPE;
}
