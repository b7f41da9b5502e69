// States that decay by one number per head and token: per head and request a 32-bit state S [N, P] that every token
// takes as
//     S <- a S + w B x^T        y = S^T C,
// with x [P] of the head, B and C [N] of the head's group (heads / groups neighbouring heads share one).  Three rules
// make a and w:
//   selective  dt = softplus(d + dt_bias), a = exp(-exp(A_log) dt), w = dt; y gets D x added   (a selective state space)
//   fixed      a is one number per head, w = 1                                                   (retention)
//   gated      log input gate i = cap tanh((i' + i_bias) / cap), log forget gate f = log sigmoid(cap tanh((f' + f_bias) /
//              cap)), a running maximum m (it starts at 0) that keeps the exponentials small: m' = max(f + m, i), a = exp(f +
//              m - m'), w = exp(i - m').  Beside S a sum n [N] takes every token as n <- a n + w B, and n . C and m' leave
//              with y: the read-out's denominator.  n is one more column of the state, whose x is 1.
// a, w, S, n, m, y and everything between them are 32-bit.  A column's N elements of the state lie side by side in the
// slot ([P][N]); n and m lie in slots of their own.
//
// x, B and C are columns of the rows `u` (type U, 32-bit partial sums where a projection left such); d, i' and f' are H
// columns each of the fused projection `proj` [T, width] of the run's type, or `splits` 32-bit partial sums.
//
// ts_decaying_walk    per (request, head, stretch of columns): the request's tokens one behind the other, the state in
//                     registers.  Single tokens, short portions, and every 32-bit run.
// Long portions of bfloat16 runs are cut into pieces of SS_PIECE tokens that run side by side on the matrix cores.  With
// c_i the sum of log a over the piece's tokens up to and including i, token j's write weighs w_j exp(s_j - t_i) at token i:
// s = t = -c for the first two rules; s_j = i_j - c_j, t_i = max(m before the piece, s_1 .. s_i), w = 1 for the third
// (m_i = c_i + t_i).  No exponent is above zero.  With t_0 what the state before the piece stands against (0, or m),
//     S_end = exp(t_0 - t_last) S_before + sum_j w_j exp(s_j - t_last) B_j x_j^T
//     y_i   = exp(t_0 - t_i) S_before^T C_i + sum_{j <= i} w_j exp(s_j - t_i) (C_i . B_j) x_j,
// (the blocked form of Dao and Gu, "Transformers are SSMs: Generalized Models and Efficient Algorithms Through
// Structured State Space Duality"), in three launches: ts_decaying_pieces mode 0 (every piece's own S_end from a zero
// state), ts_decaying_carry (the state before each piece, elementwise; the last one goes to the slot),
// mode 1 (y).  x, B and C are bfloat16 numbers, so C . B is exact products summed in 32-bit; every other factor is a
// 32-bit number that is cut into three bfloat16 numbers whose sum it is exactly, and the three products are summed
// in 32-bit: nothing of the recurrence is rounded to 16 bits.
//
// ts_heads_finish: every head's y (over its denominator) divided by its root mean square, times a gain, times a gate,
// rounded once; it also leaves the running maximum of a request's last token in the request's slot.
//
// ts_gated_group_norm: y silu(z), every one of `parts` equal parts of a row divided by its own root mean square, times
// a gain, rounded once.
#include "vec.hpp"

#define SS_PIECE 128
#define SS_STRETCH 32
#define SS_PARTS 8  // lanes that share a column of the state in the walk

#define SS_SELECTIVE 0
#define SS_FIXED 1
#define SS_GATED 2
#define SS_NEVER -1e30  // the exponent of a token that is not there

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

// Two at once, twice as many loads in flight.
template <typename P>
__device__ __forceinline__ void ss_input_two(const P* p, const P* q, int splits, size_t stride, float& a, float& b) {
  if (splits == 1) {
    a = to_float(p[0]);
    b = to_float(q[0]);
    return;
  }
  a = b = 0.f;
  for (int first = 0; first < splits; first += 8) {
    float v[8], w[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      v[j] = to_float(p[(size_t)min(first + j, splits - 1) * stride]);
      w[j] = to_float(q[(size_t)min(first + j, splits - 1) * stride]);
    }
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (first + j < splits) {
        a += v[j];
        b += w[j];
      }
  }
}

// The same of VEC neighbouring elements.
template <typename P, int VEC>
__device__ __forceinline__ void ss_input_vec(const P* p, int splits, size_t stride, float (&v)[VEC]) {
  load_vec<P, VEC>(p, v);
  for (int first = 1; first < splits; first += 8) {
    float more[8][VEC];
#pragma unroll
    for (int j = 0; j < 8; ++j) load_vec<P, VEC>(p + (size_t)min(first + j, splits - 1) * stride, more[j]);
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (first + j < splits) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] += more[j][e];
      }
  }
}

__device__ __forceinline__ float ss_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// Where a token's vectors lie in its row of `u`: x of head h from x_at + h P on, B and C of group g from b_at + g N and
// c_at + g N on.
struct SsRows {
  int splits;
  long stride;
  int width;
  int x_at, b_at, c_at;
};

// What a and w are made from: the H columns of the projection from `first` on (gated: 2 H, i' then f'), and a number
// or two per head (selective: dt_bias, A_log; fixed: the decays; gated: the two gates' biases).
struct SsGates {
  int splits;
  long stride;
  int width;
  int first;
  const float* one;
  const float* two;
  float cap;
};

__device__ __forceinline__ float ss_capped(float z, float cap) { return cap * tanhf(z / cap); }

__device__ __forceinline__ float ss_log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// The log gates of head h at row t.
template <typename P>
__device__ __forceinline__ void ss_log_gates(const P* proj, const SsGates& gates, int t, int h, int heads, float& in, float& forget) {
  const P* row = proj + (size_t)t * gates.width + gates.first + h;
  float i, f;
  ss_input_two(row, row + heads, gates.splits, gates.stride, i, f);
  in = ss_capped(i + gates.one[h], gates.cap);
  forget = ss_log_sigmoid(ss_capped(f + gates.two[h], gates.cap));
}

// ---------------------------------------------------------------------------------------------
// the walk
// ---------------------------------------------------------------------------------------------

// NR: state rows a thread holds (of every stretch of 4 SS_PARTS rows the four from 4 part on); COLS: columns of a
// workgroup; BATCH: tokens staged in LDS at a time.  norm [T, H, 2] (gated): n . C and the running maximum.
template <typename U, typename P, int RULE, int NR, int BATCH, int COLS>
__global__ void __launch_bounds__(SS_PARTS * COLS, NR <= 32 ? 5 : 2)
decaying_walk_kernel(float* __restrict__ y, float* __restrict__ norm, float* __restrict__ state, float* __restrict__ sums,
                     const float* __restrict__ tops, const U* __restrict__ u, SsRows rows, const P* __restrict__ proj, SsGates gates,
                     const float* __restrict__ skip, float scale, const int* __restrict__ state_slots,
                     const int* __restrict__ query_start_loc, int first_seq, int heads, int groups, int n, int p) {
  constexpr int ROWS = SS_PARTS * NR, THREADS = SS_PARTS * COLS;
  __shared__ __attribute__((aligned(16))) float bs[BATCH][ROWS];
  __shared__ __attribute__((aligned(16))) float cs[BATCH][ROWS];
  __shared__ float xs[BATCH][COLS];
  __shared__ float ws[BATCH], as[BATCH], ms[BATCH];
  const int seq = first_seq + blockIdx.x, h = blockIdx.y, g = h / (heads / groups);
  const int tid = threadIdx.x, part = tid % SS_PARTS, col_in = tid / SS_PARTS;
  const int c0 = blockIdx.z * COLS, c = c0 + col_in;
  const bool summing = RULE == SS_GATED && c == p;  // the column of n
  const bool live = c < p || summing;
  const int row0 = query_start_loc[seq], count = query_start_loc[seq + 1] - row0;
  const size_t b_at = (size_t)rows.b_at + (size_t)g * n, c_at = (size_t)rows.c_at + (size_t)g * n, x_at = (size_t)rows.x_at + (size_t)h * p;
  const size_t owner = (size_t)state_slots[seq] * heads + h;
  float* held = summing ? sums + owner * n : state + (owner * p + (live ? c : 0)) * n;
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
  float rate = 0.f, bias = 0.f, d_skip = 0.f, top = 0.f;
  if (RULE == SS_SELECTIVE) {
    rate = expf(gates.two[h]);
    bias = gates.one[h];
    d_skip = skip[h];
  }
  if (RULE == SS_FIXED) rate = gates.one[h];
  if (RULE == SS_GATED) top = tops[owner];
  for (int base = 0; base < count; base += BATCH) {
    const int batch = min(BATCH, count - base);
    if (base > 0) __syncthreads();  // the batch before is done with what is staged
    // The gates are the second wavefront's, x the last ones': a step of one token waits for them side by side.
    const int lane = tid - TS_WAVE;
    if (RULE == SS_SELECTIVE && lane >= 0 && lane < batch) {
      const float dt = ss_softplus(ss_input(proj + (size_t)(row0 + base + lane) * gates.width + gates.first + h, gates.splits, gates.stride) + bias);
      ws[lane] = dt;
      as[lane] = expf(-rate * dt);
    }
    if (RULE == SS_FIXED && lane >= 0 && lane < batch) {
      ws[lane] = 1.f;
      as[lane] = rate;
    }
    if (RULE == SS_GATED && lane >= 0 && lane < TS_WAVE) {  // lane j takes token j's gates; the maximum passes from token to token
      float in, forget;
      ss_log_gates(proj, gates, row0 + base + min(lane, batch - 1), h, heads, in, forget);
      for (int j = 0; j < batch; ++j) {
        const float i = __shfl(in, j), f = __shfl(forget, j), next = fmaxf(f + top, i);
        if (lane == j) {
          ws[j] = expf(i - next);
          as[j] = expf(f + top - next);
          ms[j] = next;
        }
        top = next;
      }
    }
    for (int i = THREADS - 1 - tid; i < batch * COLS; i += THREADS) {
      const int j = i / COLS, cc = c0 + i % COLS;
      float v = RULE == SS_GATED && cc == p ? 1.f : 0.f;
      if (cc < p) v = ss_input(u + (size_t)(row0 + base + j) * rows.width + x_at + cc, rows.splits, rows.stride);
      xs[j][i % COLS] = v;
    }
    for (int i = tid; i < batch * ROWS; i += THREADS) {
      const int j = i / ROWS, d = i % ROWS;
      const U* row = u + (size_t)(row0 + base + j) * rows.width;
      float vb = 0.f, vc = 0.f;
      if (d < n) ss_input_two(row + b_at + d, row + c_at + d, rows.splits, rows.stride, vb, vc);
      bs[j][d] = vb;
      cs[j][d] = vc;
    }
    __syncthreads();
    for (int j = 0; j < batch; ++j) {
      const float a = as[j], xv = xs[j][col_in], dx = ws[j] * xv;
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
      if (live && part == 0) {
        const size_t at = (size_t)(row0 + base + j) * heads + h;
        if (summing) {
          norm[2 * at] = sum * scale;
          norm[2 * at + 1] = ms[j];
        } else {
          y[at * p + c] = RULE == SS_SELECTIVE ? fmaf(d_skip, xv, sum) : sum * scale;
        }
      }
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

// What a piece's tokens need of the decays: w, and the exponents s and t as two 32-bit numbers each (formed in 64-bit, so
// that a difference of two of them is good to 32-bit however long the piece has decayed).  Where s = t it is kept once.
template <int RULE>
struct SsSteps {
  static constexpr int OWN = RULE == SS_GATED ? SS_PIECE : 1;
  float w[SS_PIECE];
  float top[SS_PIECE];  // s
  float low[SS_PIECE];
  float to_top[OWN];    // t
  float to_low[OWN];
  float m[OWN];         // the running maximum
  float total;          // the sum of log a over the piece
  __device__ __forceinline__ float t_top(int i) const { return RULE == SS_GATED ? to_top[i] : top[i]; }
  __device__ __forceinline__ float t_low(int i) const { return RULE == SS_GATED ? to_low[i] : low[i]; }
  // s_j - t_i, and t_r - t_i.
  __device__ __forceinline__ float from(int j, int i) const { return (top[j] - t_top(i)) + (low[j] - t_low(i)); }
  __device__ __forceinline__ float passed(int r, int i) const { return (t_top(r) - t_top(i)) + (t_low(r) - t_low(i)); }
};

// By the first wavefront: lane l takes the tokens 2 l and 2 l + 1 (beyond the piece: nothing decays, nothing is added).
// `floor`: what t starts from (gated).
template <int RULE, typename P>
__device__ __forceinline__ void ss_steps(SsSteps<RULE>& at, const P* proj, const SsGates& gates, int h, int heads, double floor, SsPiece piece) {
  const int lane = threadIdx.x;
  float w[2];
  double gone[2], in[2] = {0., 0.};  // log a; the log input gate
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const int j = 2 * lane + e, t = piece.first + min(j, piece.count - 1);
    const bool there = j < piece.count;
    if (RULE == SS_SELECTIVE) {
      const float z = ss_input(proj + (size_t)t * gates.width + gates.first + h, gates.splits, gates.stride) + gates.one[h];
      w[e] = there ? ss_softplus(z) : 0.f;
      gone[e] = -(double)expf(gates.two[h]) * (double)w[e];
    } else if (RULE == SS_FIXED) {
      w[e] = there ? 1.f : 0.f;
      gone[e] = there ? log((double)gates.one[h]) : 0.;
    } else {
      float i, f;
      ss_log_gates(proj, gates, t, h, heads, i, f);
      w[e] = there ? 1.f : 0.f;
      gone[e] = there ? (double)f : 0.;
      in[e] = (double)i;
    }
  }
  const double own = gone[0] + gone[1];
  double sum = own;
#pragma unroll
  for (int d = 1; d < TS_WAVE; d <<= 1) {
    const double other = __shfl_up(sum, d);
    if (lane >= d) sum += other;
  }
  const double c[2] = {sum - own + gone[0], sum};
  double s[2] = {-c[0], -c[1]};
  if (RULE == SS_GATED) {
#pragma unroll
    for (int e = 0; e < 2; ++e) s[e] = 2 * lane + e < piece.count ? in[e] + s[e] : SS_NEVER;
    double most = fmax(s[0], s[1]);
#pragma unroll
    for (int d = 1; d < TS_WAVE; d <<= 1) {
      const double other = __shfl_up(most, d);
      if (lane >= d) most = fmax(most, other);
    }
    const double before = __shfl_up(most, 1);
    const double t[2] = {fmax(fmax(lane > 0 ? before : SS_NEVER, s[0]), floor), fmax(most, floor)};
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      const float top = (float)t[e];
      at.to_top[2 * lane + e] = top;
      at.to_low[2 * lane + e] = (float)(t[e] - (double)top);
      at.m[2 * lane + e] = (float)(c[e] + t[e]);
    }
  }
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const float top = (float)s[e];
    at.w[2 * lane + e] = w[e];
    at.top[2 * lane + e] = top;
    at.low[2 * lane + e] = (float)(s[e] - (double)top);
  }
  if (lane == TS_WAVE - 1) at.total = (float)c[1];
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
// piece_state [pieces][H][P (gated: + 1, n)][N]; piece_decay [pieces][H]: the product of the piece's decays (gated: [..][2], the
// sum of log a, and the piece's own m).
template <typename P, int RULE, int NK, int PT>
__global__ void __launch_bounds__(256)
decaying_piece_state_kernel(float* __restrict__ piece_state, float* __restrict__ piece_decay, const bf16_t* __restrict__ u, SsRows rows,
                            const P* __restrict__ proj, SsGates gates, const SsPiece* __restrict__ pieces, int heads, int groups, int n,
                            int p) {
  constexpr int NP = 32 * NK, PP = 16 * PT;
  constexpr int TILES = (2 * NK + 3) / 4;  // stretches of 16 state rows a wavefront owns
  extern __shared__ __attribute__((aligned(16))) uint16_t ss_lds[];
  uint16_t* bt = ss_lds;                          // NP rows: B, tokens side by side
  uint16_t* const xw[3] = {ss_lds + ss_rows_size(NP), ss_lds + ss_rows_size(NP) + ss_rows_size(PP),
                           ss_lds + ss_rows_size(NP) + 2 * ss_rows_size(PP)};  // PP rows each: the weighted x in three planes
  __shared__ SsSteps<RULE> steps;
  __shared__ __attribute__((aligned(16))) float ends[RULE == SS_GATED ? SS_STRETCH : 4];  // the stretch's weights at the piece's end
  const int item = blockIdx.x, h = blockIdx.y, g = h / (heads / groups);
  const SsPiece piece = pieces[item];
  const int tid = threadIdx.x, wave = tid / TS_WAVE, lane = tid % TS_WAVE;
  const int lo = lane % 16, quad = lane / 16;
  const int c0 = blockIdx.z * PP;
  const size_t u_width = rows.width;
  const size_t b_at = (size_t)rows.b_at + (size_t)g * n, x_at = (size_t)rows.x_at + (size_t)h * p + c0;
  const bool summing = RULE == SS_GATED && blockIdx.z == 0;  // this workgroup also makes the piece's n, thread d row d
  float own_sum = 0.f;
  if (wave == 0) ss_steps<RULE>(steps, proj, gates, h, heads, SS_NEVER, piece);
  const size_t columns = RULE == SS_GATED ? p + 1 : p;
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
    for (int i = tid; i < (SS_STRETCH / 2) * (PP / 8); i += 256) {  // two tokens by eight columns a thread
      const int q = i / (PP / 8), d = (i % (PP / 8)) * 8;
      ts_u32x4 raw[2];
      float w[2];
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const int j = j0 + 2 * q + k;
        raw[k] = ts_u32x4{0u, 0u, 0u, 0u};
        if (c0 + d < p && j < piece.count) raw[k] = *reinterpret_cast<const ts_u32x4*>(u + (size_t)(piece.first + j) * u_width + x_at + d);
        w[k] = steps.w[j] * expf(steps.from(j, SS_PIECE - 1));
        if (RULE == SS_GATED && d == 0) ends[2 * q + k] = w[k];
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
    if (summing && tid < NP) {
#pragma unroll
      for (int j = 0; j < SS_STRETCH; j += 8) {
        const ts_u32x4 row = *reinterpret_cast<const ts_u32x4*>(&bt[ss_place(tid, j)]);
#pragma unroll
        for (int e = 0; e < 8; ++e) own_sum = fmaf(ends[j + e], __uint_as_float(ss_half(row, e)), own_sum);
      }
    }
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
        *reinterpret_cast<ss_f32x4*>(piece_state + (((size_t)item * heads + h) * columns + c) * n + d) = acc[a][b];
    }
  }
  if (summing && tid < n) piece_state[(((size_t)item * heads + h) * columns + p) * n + tid] = own_sum;
  if (blockIdx.z == 0 && tid == 0) {
    const size_t at = (size_t)item * heads + h;
    if (RULE == SS_GATED) {
      piece_decay[2 * at] = steps.total;
      piece_decay[2 * at + 1] = steps.m[SS_PIECE - 1];
    } else {
      piece_decay[at] = expf(steps.total);
    }
  }
}

// Between the modes.  A thread takes four neighbouring elements of a head's state (gated: or of n) through its request's
// pieces, and leaves what the pieces start from (gated: also m before each, in piece_top; the slot's own m stays until the
// finish, since every workgroup here reads it).
struct SsCarry {
  int slot_seq;
  int first;
  int count;
  int pad;
};

template <int RULE>
__global__ void __launch_bounds__(256)
decaying_carry_kernel(float* __restrict__ state, float* __restrict__ sums, const float* __restrict__ tops, const int* __restrict__ state_slots,
                      const SsCarry* __restrict__ carries, float* __restrict__ piece_state, const float* __restrict__ piece_decay,
                      float* __restrict__ piece_top, int heads, int n, int p) {
  const SsCarry carry = carries[blockIdx.x];
  const int h = blockIdx.y;
  const int e = 4 * (blockIdx.z * blockDim.x + threadIdx.x);
  const int own_state = n * p, per_head = RULE == SS_GATED ? own_state + n : own_state;
  if (e >= per_head) return;
  const size_t owner = (size_t)state_slots[carry.slot_seq] * heads + h;
  float* slot = RULE == SS_GATED && e >= own_state ? sums + owner * n + (e - own_state) : state + owner * own_state + e;
  float4 s = *reinterpret_cast<const float4*>(slot);
  float top = RULE == SS_GATED ? tops[owner] : 0.f;
  constexpr int AHEAD = 8;  // pieces in flight
  for (int i0 = 0; i0 < carry.count; i0 += AHEAD) {
    float4 own[AHEAD];
    float decay[AHEAD], most[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const size_t at = (size_t)(carry.first + min(i0 + i, carry.count - 1)) * heads + h;
      own[i] = *reinterpret_cast<const float4*>(piece_state + at * per_head + e);
      if (RULE == SS_GATED) {
        decay[i] = piece_decay[2 * at];
        most[i] = piece_decay[2 * at + 1];
      } else {
        decay[i] = piece_decay[at];
      }
    }
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      if (i0 + i < carry.count) {
        const size_t at = (size_t)(carry.first + i0 + i) * heads + h;
        *reinterpret_cast<float4*>(piece_state + at * per_head + e) = s;
        float a = decay[i], w = 1.f;
        if (RULE == SS_GATED) {
          if (e == 0) piece_top[at] = top;
          const float next = fmaxf(decay[i] + top, most[i]);
          a = expf(decay[i] + top - next);
          w = expf(most[i] - next);
          top = next;
        }
        s.x = fmaf(a, s.x, w * own[i].x); s.y = fmaf(a, s.y, w * own[i].y);
        s.z = fmaf(a, s.z, w * own[i].z); s.w = fmaf(a, s.w, w * own[i].w);
      }
    }
  }
  *reinterpret_cast<float4*>(slot) = s;
}

// Mode 1.  Wavefront w owns the tokens of the stretches w and 7 - w of sixteen (together they see as many tokens as any
// other's two).  Everything is computed turned, y^T (rows p, columns i): the weights (C_i . B_j) exp(c_i - c_j) dt_j come
// out of one product with token i on the lane and four tokens j in its registers, which is what the next product wants of
// its second operand if the tokens j are counted in that order; they never leave the registers.
// Of the tokens j before the stretch the factor is exp(t_r - t_i) times w_j exp(s_j - t_r), r the last token before
// the stretch: the first is applied to a stretch's sums once, the second comes from a table that the workgroup makes once
// (`before`: both exponents are at most zero, so nothing overflows however strong the decays are).
// n . C (gated) is the same sum without x: of the weights that a lane holds, and of n before the piece against C.
template <typename P, int RULE, int NK, int PT>
__global__ void __launch_bounds__(256, NK <= 4 ? 4 : 2)
decaying_piece_out_kernel(float* __restrict__ y, float* __restrict__ norm, const float* __restrict__ piece_state,
                          const float* __restrict__ piece_top, const bf16_t* __restrict__ u, SsRows rows, const P* __restrict__ proj,
                          SsGates gates, const float* __restrict__ skip, float scale, const SsPiece* __restrict__ pieces, int heads,
                          int groups, int n, int p) {
  constexpr int NP = 32 * NK, PP = 16 * PT, SROW = NP + 8, XROW = SS_PIECE + 4, HALF = SS_PIECE / 2;
  extern __shared__ __attribute__((aligned(16))) uint16_t ss_lds[];
  uint16_t* planes = ss_lds;           // [2][PP][SROW]: the state before the piece, its two lower planes, then its upper one
  uint16_t* br = ss_lds;               // then [HALF][SROW]: B of half the tokens at a time
  uint16_t* xt = ss_lds + HALF * SROW; // and [PP][XROW]: x, tokens side by side
  __shared__ __attribute__((aligned(16))) SsSteps<RULE> steps;
  __shared__ __attribute__((aligned(16))) float before[SS_PIECE / 16][SS_PIECE];  // [stretch of i][j]
  const int item = blockIdx.x, h = blockIdx.y, g = h / (heads / groups);
  const SsPiece piece = pieces[item];
  const int tid = threadIdx.x, wave = tid / TS_WAVE, lane = tid % TS_WAVE;
  const int lo = lane % 16, quad = lane / 16;
  const int c0 = blockIdx.z * PP;
  const size_t u_width = rows.width;
  const size_t b_at = (size_t)rows.b_at + (size_t)g * n, c_at = (size_t)rows.c_at + (size_t)g * n, x_at = (size_t)rows.x_at + (size_t)h * p + c0;
  const int tiles[2] = {wave, 7 - wave};
  const bool summing = RULE == SS_GATED && blockIdx.z == 0;
  const float enter = RULE == SS_GATED ? piece_top[(size_t)item * heads + h] : 0.f;  // t before the piece
  if (wave == 0) ss_steps<RULE>(steps, proj, gates, h, heads, enter, piece);
  const size_t head_state = ((size_t)item * heads + h) * (RULE == SS_GATED ? p + 1 : p);
  const float* entering = piece_state + (head_state + c0) * n;
  float sum_of[2] = {0.f, 0.f};  // this lane's share of n . C of its tokens
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
        if (j <= r) before[tile][j] = steps.w[j] * __expf(steps.from(j, r));
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
  if (summing) {
    const float* held = piece_state + (head_state + p) * n;
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      const int d = 32 * k + 8 * quad;
      if (d >= n) continue;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float v = held[d + e];
#pragma unroll
        for (int a = 0; a < 2; ++a) sum_of[a] = fmaf(v, __uint_as_float(ss_half(cf[a][k], e)), sum_of[a]);
      }
    }
  }
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    const int r = 16 * tiles[a] - 1;
    const float by = tiles[a] > 0 ? expf((enter - steps.t_top(r)) - steps.t_low(r)) : 1.f;
#pragma unroll
    for (int b = 0; b < PT; ++b) acc[b][a] *= by;
    sum_of[a] *= by;
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
          const float mine_top = steps.t_top(i), mine_low = steps.t_low(i);
          const float by = tile > 0 ? expf(steps.passed(16 * tile - 1, i)) : expf((enter - mine_top) - mine_low);
#pragma unroll
          for (int b = 0; b < PT; ++b) acc[b][a] *= by;
          sum_of[a] *= by;
#pragma unroll
          for (int t = 0; t < 2; ++t) {
            const ss_f32x4 tops = *reinterpret_cast<const ss_f32x4*>(&steps.top[j0 + 16 * t]);
            const ss_f32x4 lows = *reinterpret_cast<const ss_f32x4*>(&steps.low[j0 + 16 * t]);
            const ss_f32x4 ws = *reinterpret_cast<const ss_f32x4*>(&steps.w[j0 + 16 * t]);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              // (A later token's decay is never formed: its exponent would be positive.)
              const bool seen = j0 + 16 * t + r <= i;
              const float gone = seen ? (tops[r] - mine_top) + (lows[r] - mine_low) : 0.f;
              s[t][r] = seen ? s[t][r] * ws[r] * __expf(gone) : 0.f;
            }
          }
        }
        if (summing) {
#pragma unroll
          for (int t = 0; t < 2; ++t) sum_of[a] += (s[t][0] + s[t][1]) + (s[t][2] + s[t][3]);
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
  if (summing) {
#pragma unroll
    for (int a = 0; a < 2; ++a) {
      const int i = 16 * tiles[a] + lo;
      float sum = sum_of[a];  // over the four lanes of the token
      sum += __shfl_xor(sum, 16);
      sum += __shfl_xor(sum, 32);
      if (quad == 0 && i < piece.count) {
        const size_t at = (size_t)(piece.first + i) * heads + h;
        norm[2 * at] = sum * scale;
        norm[2 * at + 1] = steps.m[i];
      }
    }
  }
  const float d_skip = RULE == SS_SELECTIVE ? skip[h] : 0.f;
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    const int i = 16 * tiles[a] + lo;
    if (i >= piece.count) continue;
#pragma unroll
    for (int b = 0; b < PT; ++b) {
      const int c = 16 * b + 4 * quad;
      if (c0 + c >= p) continue;
      float v[4];
      if (RULE == SS_SELECTIVE) {
        float x[4];
        load_vec<bf16_t, 4>(u + (size_t)(piece.first + i) * u_width + x_at + c, x);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = fmaf(d_skip, x[e], acc[b][a][e]);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = acc[b][a][e] * scale;
      }
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
      ss_input_vec<P, VEC>(z + i, splits, split_stride, gate);
      load_vec<float, VEC>(y + row + i, v[c]);
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
// the finish
// ---------------------------------------------------------------------------------------------

// One wavefront per (token, head): o = y / (max(|n . C|, exp(-m)) + 1e-6) where `norm` holds (n . C, m) (else o = y), divided
// by its root mean square, times a gain [H P] (null: none), times silu or sigmoid of the gate (columns gate_at + h P of the
// projection), times scale.  m of a request's last token goes to the request's slot.
template <typename T, typename P, int VEC>
__global__ void __launch_bounds__(256)
heads_finish_kernel(T* __restrict__ out, size_t out_stride, const float* __restrict__ y, const float* __restrict__ norm,
                    const P* __restrict__ proj, int splits, size_t split_stride, int width, int gate_at, const T* __restrict__ gain,
                    int sigmoid, float eps, float scale, float* __restrict__ tops, const int* __restrict__ state_slots,
                    const int* __restrict__ token_seq, const int* __restrict__ query_start_loc, long items, int heads, int p) {
  const long item = (long)blockIdx.x * 4 + threadIdx.x / TS_WAVE;
  const int lane = threadIdx.x % TS_WAVE;
  if (item >= items) return;  // a whole wavefront leaves: the sums below are per wavefront
  const int t = (int)(item / heads), h = (int)(item % heads);
  float inv = 1.f;
  if (norm) {
    const float m = norm[2 * item + 1];
    inv = 1.f / (fmaxf(fabsf(norm[2 * item]), expf(-m)) + 1e-6f);
    const int seq = token_seq[t];
    if (lane == 0 && t + 1 == query_start_loc[seq + 1]) tops[(size_t)state_slots[seq] * heads + h] = m;
  }
  const float* row = y + (size_t)item * p;
  const P* gates = proj + (size_t)t * width + gate_at + (size_t)h * p;
  T* to = out + (size_t)t * out_stride + (size_t)h * p;
  // A wavefront's first HELD turns stay in registers, the gates asked for before the sum is waited for.
  constexpr int HELD = 2;
  float v[HELD][VEC], z[HELD][VEC];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < HELD; ++c) {
    const int i = (c * TS_WAVE + lane) * VEC;
    if (i >= p) continue;
    load_vec<float, VEC>(row + i, v[c]);
    ss_input_vec<P, VEC>(gates + i, splits, split_stride, z[c]);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss = fmaf(v[c][e] * inv, v[c][e] * inv, ss);
  }
  for (int i = (HELD * TS_WAVE + lane) * VEC; i < p; i += TS_WAVE * VEC) {
    float more[VEC];
    load_vec<float, VEC>(row + i, more);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss = fmaf(more[e] * inv, more[e] * inv, ss);
  }
  const float by = inv * rsqrtf(wave_sum(ss) / (float)p + eps) * scale;
  auto leave = [&](int i, float (&value)[VEC], const float (&gate)[VEC]) __attribute__((always_inline)) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) value[e] *= by * ((sigmoid ? 1.f : gate[e]) / (1.f + expf(-gate[e])));
    if (gain) {
      float w[VEC];
      load_vec<T, VEC>(gain + (size_t)h * p + i, w);
#pragma unroll
      for (int e = 0; e < VEC; ++e) value[e] *= w[e];
    }
    store_vec<T, VEC>(to + i, value);
  };
#pragma unroll
  for (int c = 0; c < HELD; ++c) {
    const int i = (c * TS_WAVE + lane) * VEC;
    if (i < p) leave(i, v[c], z[c]);
  }
  for (int i = (HELD * TS_WAVE + lane) * VEC; i < p; i += TS_WAVE * VEC) {
    float more[VEC], gate[VEC];
    load_vec<float, VEC>(row + i, more);
    ss_input_vec<P, VEC>(gates + i, splits, split_stride, gate);
    leave(i, more, gate);
  }
}

// ---------------------------------------------------------------------------------------------
// entry points
// ---------------------------------------------------------------------------------------------

static bool ss_sizes_ok(int rule, const SsRows& rows, const SsGates& gates, int heads, int groups, int n, int p) {
  if (heads < 1 || heads > 65535 || groups < 1 || heads % groups != 0 || n < 1 || n > 512 || p < 1 || p > 65534) return false;
  if (rows.splits < 1 || rows.x_at < 0 || rows.b_at < 0 || rows.c_at < 0 || (long)rows.x_at + (long)heads * p > rows.width ||
      (long)rows.b_at + (long)groups * n > rows.width || (long)rows.c_at + (long)groups * n > rows.width)
    return false;
  const int columns = rule == SS_FIXED ? 0 : rule == SS_GATED ? 2 * heads : heads;
  return gates.splits >= 1 && gates.first >= 0 && (long)gates.first + columns <= gates.width;
}

static bool ss_rule_ok(int rule, const SsGates& gates, const void* proj, const void* skip, const void* norm, const void* sums, const void* tops) {
  if (!gates.one || (rule != SS_FIXED && (!gates.two || !proj))) return false;
  if (rule == SS_SELECTIVE) return skip != nullptr;
  if (rule == SS_GATED) return norm && sums && tops && gates.cap > 0.f;
  return rule == SS_FIXED;
}

// u_f32: u is 32-bit (`u_splits` partial sums of it), else bfloat16; dtype, in_f32: as everywhere (the projection's type).
// rule: SS_SELECTIVE, SS_FIXED (reads no projection), SS_GATED (norm, sums, tops).
extern "C" int ts_decaying_walk(float* y, float* norm, float* state, float* sums, const float* tops, const void* u, int u_f32, int u_splits,
                                long u_stride, int u_width, int x_at, int b_at, int c_at, const void* proj, int in_f32, int splits,
                                long split_stride, int width, int first_gate, const float* one, const float* two, float cap,
                                const float* skip, float scale, const int* state_slots, const int* query_start_loc, int first_seq,
                                int num_seqs, int heads, int groups, int n, int p, int rule, int dtype, hipStream_t stream) {
  if (num_seqs == 0) return TS_OK;
  const SsRows rows = {u_splits, u_stride, u_width, x_at, b_at, c_at};
  const SsGates gates = {splits, split_stride, width, first_gate, one, two, cap};
  if (!y || !state || !u || !state_slots || !query_start_loc || !ss_rule_ok(rule, gates, proj, skip, norm, sums, tops)) return TS_ERR_ARG;
  if (!ss_sizes_ok(rule, rows, gates, heads, groups, n, p)) return TS_ERR_SHAPE;
  const int columns = rule == SS_GATED ? p + 1 : p;
#define SS_GO(U, P, RULE, NR, BATCH, COLS)                                                                                            \
  hipLaunchKernelGGL((decaying_walk_kernel<U, P, RULE, NR, BATCH, COLS>), dim3(num_seqs, heads, (columns + COLS - 1) / COLS),         \
                     dim3(SS_PARTS * COLS), 0, stream, y, norm, state, sums, tops, (const U*)u, rows, (const P*)proj, gates, skip,   \
                     scale, state_slots, query_start_loc, first_seq, heads, groups, n, p)
#define SS_SIZES(U, P, RULE)                                     \
  do {                                                           \
    if (n <= 32) SS_GO(U, P, RULE, 4, 8, 32);                    \
    else if (n <= 64) SS_GO(U, P, RULE, 8, 8, 32);               \
    else if (n <= 128) SS_GO(U, P, RULE, 16, 8, 32);             \
    else if (n <= 256) SS_GO(U, P, RULE, 32, 4, 32);             \
    else SS_GO(U, P, RULE, 64, 4, 32);                           \
  } while (0)
  const bool half = dtype == TS_BF16 && !u_f32;
  if (dtype != TS_F32 && dtype != TS_BF16) return TS_ERR_DTYPE;
  if (dtype == TS_F32 && !u_f32) return TS_ERR_DTYPE;
  if (half && u_splits != 1) return TS_ERR_ARG;
  if (rule == SS_SELECTIVE) {
    if (dtype == TS_F32) SS_SIZES(float, float, SS_SELECTIVE);
    else if (half && in_f32) SS_SIZES(bf16_t, float, SS_SELECTIVE);
    else if (half) SS_SIZES(bf16_t, bf16_t, SS_SELECTIVE);
    else return TS_ERR_DTYPE;
  } else if (rule == SS_FIXED) {
    if (u_f32) SS_SIZES(float, float, SS_FIXED);
    else SS_SIZES(bf16_t, bf16_t, SS_FIXED);
  } else {  // (the vectors and the gates' inputs lie in one projection)
    if (u_f32 != (in_f32 || dtype == TS_F32)) return TS_ERR_DTYPE;
    if (u_f32) SS_SIZES(float, float, SS_GATED);
    else SS_SIZES(bf16_t, bf16_t, SS_GATED);
  }
#undef SS_SIZES
#undef SS_GO
  return ts_launch_status();
}

template <typename P, int RULE, int NK, int PT>
static int ss_pieces_launch(int mode, float* y, float* norm, float* piece_state, float* piece_decay, const float* piece_top, const void* u,
                            SsRows rows, const void* proj, SsGates gates, const float* skip, float scale, const void* pieces,
                            int num_pieces, int heads, int groups, int n, int p, hipStream_t stream) {
  const dim3 grid(num_pieces, heads, (p + 16 * PT - 1) / (16 * PT));
  if (mode == 0) {
    constexpr int lds = (ss_rows_size(32 * NK) + 3 * ss_rows_size(16 * PT)) * 2;
    static const bool ready = hipFuncSetAttribute((const void*)decaying_piece_state_kernel<P, RULE, NK, PT>,
                                                  hipFuncAttributeMaxDynamicSharedMemorySize, lds) == hipSuccess;
    if (!ready) return TS_ERR_LAUNCH;
    hipLaunchKernelGGL((decaying_piece_state_kernel<P, RULE, NK, PT>), grid, dim3(256), lds, stream, piece_state, piece_decay,
                       (const bf16_t*)u, rows, (const P*)proj, gates, (const SsPiece*)pieces, heads, groups, n, p);
  } else {
    constexpr int planes = 2 * 16 * PT * (32 * NK + 8) * 2, half = (SS_PIECE / 2 * (32 * NK + 8) + 16 * PT * (SS_PIECE + 4)) * 2;
    constexpr int lds = planes > half ? planes : half;
    static const bool ready = hipFuncSetAttribute((const void*)decaying_piece_out_kernel<P, RULE, NK, PT>,
                                                  hipFuncAttributeMaxDynamicSharedMemorySize, lds) == hipSuccess;
    if (!ready) return TS_ERR_LAUNCH;
    hipLaunchKernelGGL((decaying_piece_out_kernel<P, RULE, NK, PT>), grid, dim3(256), lds, stream, y, norm, piece_state, piece_top,
                       (const bf16_t*)u, rows, (const P*)proj, gates, skip, scale, (const SsPiece*)pieces, heads, groups, n, p);
  }
  return ts_launch_status();
}

// bfloat16 runs; mode 0: every piece's own end state and decay; mode 1: y from the state before each piece.
extern "C" int ts_decaying_pieces(float* y, float* norm, float* piece_state, float* piece_decay, const float* piece_top, const void* u,
                                  int u_width, int x_at, int b_at, int c_at, const void* proj, int in_f32, int splits, long split_stride,
                                  int width, int first_gate, const float* one, const float* two, float cap, const float* skip, float scale,
                                  const void* pieces, int num_pieces, int heads, int groups, int n, int p, int rule, int mode,
                                  hipStream_t stream) {
  if (num_pieces == 0) return TS_OK;
  const SsRows rows = {1, 0, u_width, x_at, b_at, c_at};
  const SsGates gates = {splits, split_stride, width, first_gate, one, two, cap};
  if (!piece_state || !piece_decay || !u || !pieces || (mode == 1 && !y) || mode < 0 || mode > 1) return TS_ERR_ARG;
  if (!ss_rule_ok(rule, gates, proj, skip, norm, piece_state, piece_top)) return TS_ERR_ARG;
  if (!ss_sizes_ok(rule, rows, gates, heads, groups, n, p) || n > 256 || n % 8 != 0 || p % 8 != 0) return TS_ERR_SHAPE;
  if (u_width % 8 != 0 || x_at % 8 != 0 || b_at % 8 != 0 || c_at % 8 != 0) return TS_ERR_SHAPE;  // 16-byte accesses
  if (((uintptr_t)u | (uintptr_t)piece_state | (uintptr_t)y) % 16 != 0) return TS_ERR_ARG;
#define SS_GO(P, RULE, NK, PT)                                                                                                     \
  return ss_pieces_launch<P, RULE, NK, PT>(mode, y, norm, piece_state, piece_decay, piece_top, u, rows, proj, gates, skip, scale,  \
                                           pieces, num_pieces, heads, groups, n, p, stream)
#define SS_SIZES(P, RULE, PT)                 \
  do {                                        \
    if (n <= 32) SS_GO(P, RULE, 1, PT);       \
    if (n <= 64) SS_GO(P, RULE, 2, PT);       \
    if (n <= 128) SS_GO(P, RULE, 4, PT);      \
    SS_GO(P, RULE, 8, PT);                    \
  } while (0)
#define SS_WIDTHS(P, RULE)                    \
  do {                                        \
    if (p <= 32) SS_SIZES(P, RULE, 2);        \
    SS_SIZES(P, RULE, 4);                     \
  } while (0)
  if (rule == SS_SELECTIVE && in_f32) SS_WIDTHS(float, SS_SELECTIVE);
  if (rule == SS_SELECTIVE) SS_WIDTHS(bf16_t, SS_SELECTIVE);
  if (rule == SS_FIXED) SS_WIDTHS(bf16_t, SS_FIXED);
  if (in_f32) SS_WIDTHS(float, SS_GATED);
  SS_WIDTHS(bf16_t, SS_GATED);
#undef SS_WIDTHS
#undef SS_SIZES
#undef SS_GO
}

extern "C" int ts_decaying_carry(float* state, float* sums, const float* tops, const int* state_slots, const void* carries,
                                 float* piece_state, const float* piece_decay, float* piece_top, int requests, int heads, int n, int p,
                                 int rule, hipStream_t stream) {
  if (requests == 0) return TS_OK;
  if (!state || !state_slots || !carries || !piece_state || !piece_decay) return TS_ERR_ARG;
  if (rule == SS_GATED && (!sums || !tops || !piece_top)) return TS_ERR_ARG;
  if (heads < 1 || heads > 65535 || n < 1 || p < 1 || n > 512 || p > 65534 || n % 4 != 0) return TS_ERR_SHAPE;
  const int columns = rule == SS_GATED ? p + 1 : p;
  const dim3 grid(requests, heads, (n * columns / 4 + 255) / 256);
  if (rule == SS_GATED)
    hipLaunchKernelGGL(decaying_carry_kernel<SS_GATED>, grid, dim3(256), 0, stream, state, sums, tops, state_slots, (const SsCarry*)carries,
                       piece_state, piece_decay, piece_top, heads, n, p);
  else  // (the other rules carry alike)
    hipLaunchKernelGGL(decaying_carry_kernel<SS_FIXED>, grid, dim3(256), 0, stream, state, sums, tops, state_slots, (const SsCarry*)carries,
                       piece_state, piece_decay, piece_top, heads, n, p);
  return ts_launch_status();
}

template <typename T, typename P>
static int launch_heads_finish(void* out, long out_stride, const float* y, const float* norm, const void* proj, int splits, long split_stride,
                               int width, int gate_at, const void* gain, int sigmoid, float eps, float scale, float* tops,
                               const int* state_slots, const int* token_seq, const int* query_start_loc, long items, int heads, int p,
                               hipStream_t stream) {
  const dim3 grid((unsigned)((items + 3) / 4)), block(256);
  const bool wide = p % 4 == 0 && width % 4 == 0 && gate_at % 4 == 0 && split_stride % 4 == 0 && out_stride % 4 == 0 &&
                    ((uintptr_t)out % (4 * sizeof(T))) == 0 && (((uintptr_t)y | (uintptr_t)proj | (uintptr_t)gain) % 16) == 0;
#define HF_GO(VEC)                                                                                                                   \
  hipLaunchKernelGGL((heads_finish_kernel<T, P, VEC>), grid, block, 0, stream, (T*)out, (size_t)out_stride, y, norm, (const P*)proj, \
                     splits, (size_t)split_stride, width, gate_at, (const T*)gain, sigmoid, eps, scale, tops, state_slots, token_seq, \
                     query_start_loc, items, heads, p)
  if (wide) HF_GO(4);
  else HF_GO(1);
#undef HF_GO
  return ts_launch_status();
}

extern "C" int ts_heads_finish(void* out, long out_stride, const float* y, const float* norm, const void* proj, int in_f32, int splits,
                               long split_stride, int width, int gate_at, const void* gain, int sigmoid, float eps, float scale, float* tops,
                               const int* state_slots, const int* token_seq, const int* query_start_loc, int tokens, int heads, int p,
                               int dtype, hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!out || !y || !proj || (norm && (!tops || !state_slots || !token_seq || !query_start_loc))) return TS_ERR_ARG;
  if (heads < 1 || p < 1 || gate_at < 0 || (long)gate_at + (long)heads * p > width || splits < 1 || out_stride < (long)heads * p) return TS_ERR_SHAPE;
  const long items = (long)tokens * heads;
#define HF_ARGS out, out_stride, y, norm, proj, splits, split_stride, width, gate_at, gain, sigmoid, eps, scale, tops, state_slots, token_seq, \
                query_start_loc, items, heads, p, stream
  if (dtype == TS_F32) return launch_heads_finish<float, float>(HF_ARGS);
  if (dtype == TS_BF16 && in_f32) return launch_heads_finish<bf16_t, float>(HF_ARGS);
  if (dtype == TS_BF16) return launch_heads_finish<bf16_t, bf16_t>(HF_ARGS);
#undef HF_ARGS
  return TS_ERR_DTYPE;
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
