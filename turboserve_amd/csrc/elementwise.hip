// Row-wise kernels of the decoder: embedding gather, RMSNorm (with the residual sum fused in),
// SwiGLU, and rotary encoding fused with the scatter of keys and values into cache pages.
//
// Formulas restate src/turboserve/engine/model/layers.py:202-208 (RMSNorm), :214-222 and
// :290-302 (rotary, half-split pairs), :437-440 (SwiGLU) and
// src/turboserve/engine/core/kv_cache.py:601-631 (cache write at slot = block * BS + offset).
// Reductions, the residual sum and the rotation are computed in 32-bit whatever T is.
#include <type_traits>

#include "common.hpp"

// ---------------------------------------------------------------------------------------------
// embedding: residual[t, :] = float(table[ids[t], :])
// ---------------------------------------------------------------------------------------------
template <typename T>
__global__ void embed_kernel(float* __restrict__ residual, const T* __restrict__ table,
                             const int* __restrict__ ids, int hidden, int vocab, float scale) {
  const int t = blockIdx.x;
  int id = ids[t];
  const bool valid = id >= 0 && id < vocab;
  const T* row = table + (size_t)(valid ? id : 0) * hidden;
  float* out = residual + (size_t)t * hidden;
  for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
    // An id outside the table is a host error; it yields NaN instead of a read out of bounds.
    out[i] = valid ? to_float(row[i]) * scale : __uint_as_float(0x7fc00000u);
  }
}

extern "C" int ts_embed(void* residual, const void* table, const int* ids, int tokens, int hidden,
                        int vocab, float scale, int dtype, hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!residual || !table || !ids || hidden < 1 || vocab < 1) return TS_ERR_ARG;
  dim3 grid(tokens), block(256);
  if (dtype == TS_F32)
    hipLaunchKernelGGL(embed_kernel<float>, grid, block, 0, stream, (float*)residual, (const float*)table, ids, hidden, vocab, scale);
  else if (dtype == TS_BF16)
    hipLaunchKernelGGL(embed_kernel<bf16_t>, grid, block, 0, stream, (float*)residual, (const bf16_t*)table, ids, hidden, vocab, scale);
  else
    return TS_ERR_DTYPE;
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// RMSNorm.  y = w * round_T(x * rsqrt(mean(x^2) + eps)): the normalised value is rounded to the
// storage type before the gain, as the reference does (layers.py:208).
//
// add_rmsnorm: s = residual + pending (32-bit); residual = s; y = norm(s).  With `rows` the
// kernel reads rows[i] and writes y[i] only (residual untouched): the final norm at the wanted
// positions.
// ---------------------------------------------------------------------------------------------
// The gain: `one_rounding == 0` is the rule above, w * round_T(n); otherwise the whole norm is
// 32-bit arithmetic with one rounding at the end, round_T(n * (gain_offset + w)) (a gain stored
// around zero has gain_offset 1).
template <typename T>
__device__ __forceinline__ float with_gain(float normalised, float gain, float gain_offset, int one_rounding) {
  return one_rounding ? normalised * (gain_offset + gain) : gain * round_to<T>(normalised);
}

template <typename T>
__global__ void rmsnorm_kernel(T* __restrict__ y, const T* __restrict__ x, const T* __restrict__ w,
                               float eps, int hidden, float gain_offset, int one_rounding) {
  __shared__ float scratch[16];
  const size_t base = (size_t)blockIdx.x * hidden;
  float ss = 0.f;
  for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
    const float v = to_float(x[base + i]);
    ss += v * v;
  }
  ss = block_sum(ss, scratch);
  const float rstd = rsqrtf(ss / (float)hidden + eps);
  for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
    y[base + i] = from_float<T>(with_gain<T>(to_float(x[base + i]) * rstd, to_float(w[i]), gain_offset, one_rounding));
  }
}

// `init` plus the `splits` values that lie `stride` elements apart, added in split order; the loads
// of up to eight splits are in flight together (see add_splits4).
template <typename P>
__device__ __forceinline__ float add_splits(const P* p, int splits, size_t stride, float init) {
  float s = init;
  if (splits == 1) return s + to_float(p[0]);
  int sp0 = 0;
  do {
    float v[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = to_float(p[(size_t)min(sp0 + j, splits - 1) * stride]);
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (sp0 + j < splits) s += v[j];
    sp0 += 8;
  } while (sp0 < splits);
  return s;
}

// P is the type of `pending`: T, or float for `splits` partial sums of a product that are
// `split_stride` elements apart and are added up here.
// A pending output may carry a norm of its own (`post`): it is then divided by its root mean square,
// multiplied by `post.gain` and by `post.scale`, all in 32-bit, before it is added (a block that
// normalises a part's output before the residual sum).  `also` does not go with it.
template <typename T>
struct PostNorm {
  const T* gain;  // null: the pending output is added as it is
  float eps;
  float scale;
};

template <typename T, typename P>
__global__ void add_rmsnorm_kernel(T* __restrict__ y, float* __restrict__ residual,
                                   const P* __restrict__ pending, int splits, size_t split_stride,
                                   const T* __restrict__ w, const int* __restrict__ rows, float eps,
                                   int hidden, float gain_offset, int one_rounding,
                                   const float* __restrict__ also, int also_splits, size_t also_stride,
                                   PostNorm<T> post) {
  __shared__ float scratch[16];
  const int src = rows ? rows[blockIdx.x] : blockIdx.x;
  const size_t in_base = (size_t)src * hidden;
  const size_t out_base = (size_t)blockIdx.x * hidden;
  float ss = 0.f;
  if (post.gain) {
    float pss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
      const float v = add_splits(pending + in_base + i, splits, split_stride, 0.f);
      pss += v * v;
    }
    pss = block_sum(pss, scratch);
    const float by = rsqrtf(pss / (float)hidden + post.eps) * post.scale;
    // Without `rows` the sum is left in the residual stream; with `rows` it is formed again below.
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
      const float v = add_splits(pending + in_base + i, splits, split_stride, 0.f);
      const float s = residual[in_base + i] + v * by * to_float(post.gain[i]);
      if (!rows) residual[in_base + i] = s;
      ss += s * s;
    }
    ss = block_sum(ss, scratch);
    const float rstd = rsqrtf(ss / (float)hidden + eps);
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
      float s = residual[in_base + i];
      if (rows) s += add_splits(pending + in_base + i, splits, split_stride, 0.f) * by * to_float(post.gain[i]);
      y[out_base + i] = from_float<T>(with_gain<T>(s * rstd, to_float(w[i]), gain_offset, one_rounding));
    }
    return;
  }
  for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
    float s = residual[in_base + i];
    if (pending) s = add_splits(pending + in_base + i, splits, split_stride, s);
    if (also) s = add_splits(also + in_base + i, also_splits, also_stride, s);
    if ((pending || also) && !rows) residual[in_base + i] = s;  // re-read below by this same thread
    ss += s * s;
  }
  ss = block_sum(ss, scratch);
  const float rstd = rsqrtf(ss / (float)hidden + eps);
  for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
    float s = residual[in_base + i];
    if (rows && pending) s = add_splits(pending + in_base + i, splits, split_stride, s);
    if (rows && also) s = add_splits(also + in_base + i, also_splits, also_stride, s);
    y[out_base + i] = from_float<T>(with_gain<T>(s * rstd, to_float(w[i]), gain_offset, one_rounding));
  }
}

extern "C" int ts_rmsnorm(void* y, const void* x, const void* w, float eps, int tokens, int hidden,
                          float gain_offset, int one_rounding, int dtype, hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!y || !x || !w || hidden < 1) return TS_ERR_ARG;
  dim3 grid(tokens), block(hidden <= 1024 ? 256 : 1024);
  if (dtype == TS_F32)
    hipLaunchKernelGGL(rmsnorm_kernel<float>, grid, block, 0, stream, (float*)y, (const float*)x, (const float*)w, eps, hidden, gain_offset, one_rounding);
  else if (dtype == TS_BF16)
    hipLaunchKernelGGL(rmsnorm_kernel<bf16_t>, grid, block, 0, stream, (bf16_t*)y, (const bf16_t*)x, (const bf16_t*)w, eps, hidden, gain_offset, one_rounding);
  else
    return TS_ERR_DTYPE;
  return ts_launch_status();
}

// The same, four elements per thread per item and the row kept in registers between the two
// passes: for hidden sizes that are a multiple of 4 and at most 16 * blockDim.x.  A decode step
// has few rows, so each row gets a large block and the loads of all splits are in flight at once.
template <typename T>
struct Vec4Of;
template <>
struct Vec4Of<float> {
  typedef float4 type;
  static __device__ __forceinline__ void load(const float* p, float (&v)[4]) {
    const float4 x = *reinterpret_cast<const float4*>(p);
    v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
  }
  static __device__ __forceinline__ void store(float* p, const float (&v)[4]) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  }
};
template <>
struct Vec4Of<bf16_t> {
  static __device__ __forceinline__ void load(const bf16_t* p, float (&v)[4]) {
    const uint2 x = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(x.x << 16); v[1] = __uint_as_float(x.x & 0xffff0000u);
    v[2] = __uint_as_float(x.y << 16); v[3] = __uint_as_float(x.y & 0xffff0000u);
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float (&v)[4]) {
    uint2 x;
    x.x = (uint32_t)from_float<bf16_t>(v[0]).bits | ((uint32_t)from_float<bf16_t>(v[1]).bits << 16);
    x.y = (uint32_t)from_float<bf16_t>(v[2]).bits | ((uint32_t)from_float<bf16_t>(v[3]).bits << 16);
    *reinterpret_cast<uint2*>(p) = x;
  }
};

// Partial sums of a product lie `stride` elements apart.  The loads of a batch of splits are
// issued together and only then added, in split order: a loop that loads and adds one split at a
// time makes every split wait a full trip to memory, and these kernels are nothing but such
// trips.  Up to 16 splits are one batch in straight-line code (so that the caller's own loads,
// issued before, are waited for only where they are used); more go in batches of 8.  A value
// that is not split (splits == 1) takes the one load.
template <int N, typename P>
__device__ __forceinline__ void add_split_batch4(const P* p, int first, int splits, size_t stride, float (&s)[4]) {
  float v[N][4];
#pragma unroll
  for (int j = 0; j < N; ++j) Vec4Of<P>::load(p + (size_t)min(first + j, splits - 1) * stride, v[j]);
#pragma unroll
  for (int j = 0; j < N; ++j) {
    if (first + j < splits) {
#pragma unroll
      for (int e = 0; e < 4; ++e) s[e] += v[j][e];
    }
  }
}

template <typename P>
__device__ __forceinline__ void add_splits4(const P* p, int splits, size_t stride, float (&s)[4]) {
  if (splits == 1) {
    add_split_batch4<1>(p, 0, 1, stride, s);
  } else if (splits <= 4) {
    add_split_batch4<4>(p, 0, splits, stride, s);
  } else if (splits <= 8) {
    add_split_batch4<8>(p, 0, splits, stride, s);
  } else if (splits <= 16) {
    add_split_batch4<16>(p, 0, splits, stride, s);
  } else {
    for (int first = 0; first < splits; first += 8) add_split_batch4<8>(p, first, splits, stride, s);
  }
}

#define NORM_ITEMS 4

template <typename T, typename P, bool POST>
__global__ void add_rmsnorm_vec4_kernel(T* __restrict__ y, float* __restrict__ residual,
                                        const P* __restrict__ pending, int splits, size_t split_stride,
                                        const T* __restrict__ w, const int* __restrict__ rows, float eps,
                                        int hidden, float gain_offset, int one_rounding,
                                        const float* __restrict__ also, int also_splits, size_t also_stride,
                                        PostNorm<T> post) {
  __shared__ float scratch[16];
  const int src = rows ? rows[blockIdx.x] : blockIdx.x;
  const size_t in_base = (size_t)src * hidden;
  const size_t out_base = (size_t)blockIdx.x * hidden;
  const int quads = hidden / 4;
  float s[NORM_ITEMS][4], g[NORM_ITEMS][4];
  float ss = 0.f;
  if (POST) {
    // The pending output with its own norm: its sum of squares first, then the residual sum.
    float p[NORM_ITEMS][4], pg[NORM_ITEMS][4];
    float pss = 0.f;
#pragma unroll
    for (int it = 0; it < NORM_ITEMS; ++it) {
      const int qd = threadIdx.x + it * blockDim.x;
      if (qd < quads) {
        Vec4Of<float>::load(residual + in_base + 4 * qd, s[it]);
        Vec4Of<T>::load(w + 4 * qd, g[it]);
        Vec4Of<T>::load(post.gain + 4 * qd, pg[it]);
#pragma unroll
        for (int e = 0; e < 4; ++e) p[it][e] = 0.f;
        add_splits4(pending + in_base + 4 * qd, splits, split_stride, p[it]);
#pragma unroll
        for (int e = 0; e < 4; ++e) pss += p[it][e] * p[it][e];
      }
    }
    pss = block_sum(pss, scratch);
    const float by = rsqrtf(pss / (float)hidden + post.eps) * post.scale;
#pragma unroll
    for (int it = 0; it < NORM_ITEMS; ++it) {
      const int qd = threadIdx.x + it * blockDim.x;
      if (qd < quads) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          s[it][e] += p[it][e] * by * pg[it][e];
          ss += s[it][e] * s[it][e];
        }
        if (!rows) Vec4Of<float>::store(residual + in_base + 4 * qd, s[it]);
      }
    }
  }
#pragma unroll
  for (int it = 0; it < NORM_ITEMS; ++it) {
    const int qd = threadIdx.x + it * blockDim.x;
    if (!POST && qd < quads) {
      Vec4Of<float>::load(residual + in_base + 4 * qd, s[it]);
      Vec4Of<T>::load(w + 4 * qd, g[it]);  // with the other loads, not behind the reduction's barriers
      if (pending) add_splits4(pending + in_base + 4 * qd, splits, split_stride, s[it]);
      if (also) add_splits4(also + in_base + 4 * qd, also_splits, also_stride, s[it]);
      if ((pending || also) && !rows) Vec4Of<float>::store(residual + in_base + 4 * qd, s[it]);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss += s[it][e] * s[it][e];
    }
  }
  ss = block_sum(ss, scratch);
  const float rstd = rsqrtf(ss / (float)hidden + eps);
#pragma unroll
  for (int it = 0; it < NORM_ITEMS; ++it) {
    const int qd = threadIdx.x + it * blockDim.x;
    if (qd < quads) {
      float o[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = with_gain<T>(s[it][e] * rstd, g[it][e], gain_offset, one_rounding);
      Vec4Of<T>::store(y + out_base + 4 * qd, o);
    }
  }
}

template <typename T, typename P>
static void launch_add_rmsnorm(void* y, float* residual, const void* pending, int splits, long split_stride,
                               const void* w, const int* rows, float eps, int out_rows, int hidden,
                               float gain_offset, int one_rounding, const float* also, int also_splits,
                               long also_stride, const void* post_gain, float post_eps, float post_scale,
                               hipStream_t stream) {
  // Few rows (decode): one large block per row; many rows (prefill): just enough threads.
  int threads = out_rows <= 256 ? 1024 : 256;
  const int need = (hidden / 4 + NORM_ITEMS - 1) / NORM_ITEMS;
  if (threads < need) threads = ((need + 63) / 64) * 64;
  const PostNorm<T> post = {(const T*)post_gain, post_eps, post_scale};
  if (hidden % 4 == 0 && threads <= 1024 && post_gain) {
    hipLaunchKernelGGL((add_rmsnorm_vec4_kernel<T, P, true>), dim3(out_rows), dim3(threads), 0, stream, (T*)y, residual,
                       (const P*)pending, splits, (size_t)split_stride, (const T*)w, rows, eps, hidden, gain_offset,
                       one_rounding, also, also_splits, (size_t)also_stride, post);
  } else if (hidden % 4 == 0 && threads <= 1024) {
    hipLaunchKernelGGL((add_rmsnorm_vec4_kernel<T, P, false>), dim3(out_rows), dim3(threads), 0, stream, (T*)y, residual,
                       (const P*)pending, splits, (size_t)split_stride, (const T*)w, rows, eps, hidden, gain_offset,
                       one_rounding, also, also_splits, (size_t)also_stride, post);
  } else {
    hipLaunchKernelGGL((add_rmsnorm_kernel<T, P>), dim3(out_rows), dim3(hidden <= 1024 ? 256 : 1024), 0, stream,
                       (T*)y, residual, (const P*)pending, splits, (size_t)split_stride, (const T*)w, rows, eps,
                       hidden, gain_offset, one_rounding, also, also_splits, (size_t)also_stride, post);
  }
}

// `out_rows` = rows of y written: the number of entries of `rows` if given, else the tokens.
// pending_f32 != 0: `pending` holds `splits` 32-bit partial sums, `split_stride` elements apart.
// `also`: a second addend, `also_splits` 32-bit partial sums `also_stride` apart (a block whose two parts
// both add to the stream), or null.  `post_gain` [hidden] of the run type, or null: the pending output is
// divided by its root mean square (`post_eps` inside the root) and multiplied by the gain and by
// `post_scale` before it is added.
extern "C" int ts_add_rmsnorm(void* y, float* residual, const void* pending, int pending_f32, int splits,
                              long split_stride, const void* w, const int* rows, float eps, int out_rows,
                              int hidden, float gain_offset, int one_rounding, int dtype, const float* also,
                              int also_splits, long also_stride, const void* post_gain, float post_eps,
                              float post_scale, hipStream_t stream) {
  if (out_rows == 0) return TS_OK;
  if (!y || !residual || !w || hidden < 1 || splits < 1 || (also && also_splits < 1)) return TS_ERR_ARG;
  if (post_gain && (!pending || also)) return TS_ERR_ARG;
  if (dtype == TS_F32)
    launch_add_rmsnorm<float, float>(y, residual, pending, splits, split_stride, w, rows, eps, out_rows, hidden, gain_offset, one_rounding, also, also_splits, also_stride, post_gain, post_eps, post_scale, stream);
  else if (dtype == TS_BF16 && pending_f32)
    launch_add_rmsnorm<bf16_t, float>(y, residual, pending, splits, split_stride, w, rows, eps, out_rows, hidden, gain_offset, one_rounding, also, also_splits, also_stride, post_gain, post_eps, post_scale, stream);
  else if (dtype == TS_BF16)
    launch_add_rmsnorm<bf16_t, bf16_t>(y, residual, pending, splits, split_stride, w, rows, eps, out_rows, hidden, gain_offset, one_rounding, also, also_splits, also_stride, post_gain, post_eps, post_scale, stream);
  else
    return TS_ERR_DTYPE;
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// Gated unit over the fused gate|up projection [T, 2 I]: out[t, i] = gated_unit(gate[t, i], up[t, i])
// (common.hpp; silu(gate) * up is the rule {1, 0, 0}), with
// gate in the first I columns and up in the last (paired == 0), or alternating: gate i in column
// 2 i, up i in column 2 i + 1 (paired != 0).
// ---------------------------------------------------------------------------------------------
// P: type of the projection output: T, or float for `splits` partial sums to be added up.
template <typename T, typename P>
__global__ void swiglu_kernel(T* __restrict__ out, const P* __restrict__ gate_up, int splits,
                              size_t split_stride, int inter, size_t total, int paired, GluRule rule) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const size_t t = idx / inter;
  const int i = (int)(idx - t * inter);
  const size_t gate_at = t * 2 * inter + (paired ? 2 * i : i);
  const size_t up_at = paired ? gate_at + 1 : gate_at + inter;
  const float g = add_splits(gate_up + gate_at, splits, split_stride, 0.f);
  const float u = add_splits(gate_up + up_at, splits, split_stride, 0.f);
  out[idx] = from_float<T>(gated_unit(g, u, rule));
}

// Four outputs per thread with 8- or 16-byte loads: for I a multiple of 4.
template <typename T, typename P>
__global__ void swiglu_vec4_kernel(T* __restrict__ out, const P* __restrict__ gate_up, int splits,
                                   size_t split_stride, int inter, size_t quads, int paired, GluRule rule) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= quads) return;
  const int per_row = inter / 4;
  const size_t t = idx / per_row;
  const int i = (int)(idx - t * per_row) * 4;
  float g[4], u[4];
  float a[4] = {0.f, 0.f, 0.f, 0.f}, b[4] = {0.f, 0.f, 0.f, 0.f};
  if (paired) {  // eight consecutive columns: g0 u0 g1 u1 | g2 u2 g3 u3
    add_splits4(gate_up + t * 2 * inter + 2 * i, splits, split_stride, a);
    add_splits4(gate_up + t * 2 * inter + 2 * i + 4, splits, split_stride, b);
    g[0] = a[0]; u[0] = a[1]; g[1] = a[2]; u[1] = a[3];
    g[2] = b[0]; u[2] = b[1]; g[3] = b[2]; u[3] = b[3];
  } else {
    add_splits4(gate_up + t * 2 * inter + i, splits, split_stride, a);
    add_splits4(gate_up + t * 2 * inter + inter + i, splits, split_stride, b);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      g[e] = a[e];
      u[e] = b[e];
    }
  }
  float o[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) o[e] = gated_unit(g[e], u[e], rule);
  Vec4Of<T>::store(out + t * inter + i, o);
}

// Eight outputs per thread with 16-byte loads and stores: bfloat16 in and out, one split, I a
// multiple of 8 (the many-row case: a product of the library's, then this).  The same arithmetic
// per element as above.
__global__ void swiglu_bf16x8_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ gate_up, int inter,
                                     size_t octets, int paired, GluRule rule) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= octets) return;
  const int per_row = inter / 8;
  const size_t t = idx / per_row;
  const int i = (int)(idx - t * per_row) * 8;
  const bf16_t* row = gate_up + t * 2 * inter;
  // paired: sixteen consecutive columns g0 u0 .. g7 u7; else eight of the gate and eight of the up half
  const uint4 a = *reinterpret_cast<const uint4*>(paired ? row + 2 * i : row + i);
  const uint4 b = *reinterpret_cast<const uint4*>(paired ? row + 2 * i + 8 : row + inter + i);
  const uint32_t wa[4] = {a.x, a.y, a.z, a.w}, wb[4] = {b.x, b.y, b.z, b.w};
  float g[8], u[8];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float a_lo = __uint_as_float(wa[e] << 16), a_hi = __uint_as_float(wa[e] & 0xffff0000u);
    const float b_lo = __uint_as_float(wb[e] << 16), b_hi = __uint_as_float(wb[e] & 0xffff0000u);
    if (paired) {
      g[e] = a_lo; u[e] = a_hi; g[4 + e] = b_lo; u[4 + e] = b_hi;
    } else {
      g[2 * e] = a_lo; g[2 * e + 1] = a_hi; u[2 * e] = b_lo; u[2 * e + 1] = b_hi;
    }
  }
  float o[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) o[e] = gated_unit(g[e], u[e], rule);
  uint32_t w[4];
#pragma unroll
  for (int e = 0; e < 4; ++e)
    w[e] = (uint32_t)from_float<bf16_t>(o[2 * e]).bits | ((uint32_t)from_float<bf16_t>(o[2 * e + 1]).bits << 16);
  *reinterpret_cast<uint4*>(out + t * inter + i) = make_uint4(w[0], w[1], w[2], w[3]);
}

template <typename T, typename P>
static void launch_swiglu(void* out, const void* gate_up, int splits, long split_stride, int tokens, int inter,
                          int paired, GluRule rule, hipStream_t stream) {
  if (std::is_same<T, bf16_t>::value && std::is_same<P, bf16_t>::value && splits == 1 && inter % 8 == 0) {
    const size_t octets = (size_t)tokens * (inter / 8);
    hipLaunchKernelGGL(swiglu_bf16x8_kernel, dim3((unsigned)((octets + 255) / 256)), dim3(256), 0, stream,
                       (bf16_t*)out, (const bf16_t*)gate_up, inter, octets, paired, rule);
  } else if (inter % 4 == 0) {
    const size_t quads = (size_t)tokens * (inter / 4);
    hipLaunchKernelGGL((swiglu_vec4_kernel<T, P>), dim3((unsigned)((quads + 255) / 256)), dim3(256), 0, stream,
                       (T*)out, (const P*)gate_up, splits, (size_t)split_stride, inter, quads, paired, rule);
  } else {
    const size_t total = (size_t)tokens * inter;
    hipLaunchKernelGGL((swiglu_kernel<T, P>), dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream, (T*)out,
                       (const P*)gate_up, splits, (size_t)split_stride, inter, total, paired, rule);
  }
}

extern "C" int ts_swiglu(void* out, const void* gate_up, int in_f32, int splits, long split_stride,
                         int tokens, int inter, int paired, float steepness, float limit, float up_shift, float cubic,
                         int dtype, hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!out || !gate_up || inter < 1 || splits < 1) return TS_ERR_ARG;
  const GluRule rule = {steepness, limit, up_shift, cubic};
  if (dtype == TS_F32)
    launch_swiglu<float, float>(out, gate_up, splits, split_stride, tokens, inter, paired, rule, stream);
  else if (dtype == TS_BF16 && in_f32)
    launch_swiglu<bf16_t, float>(out, gate_up, splits, split_stride, tokens, inter, paired, rule, stream);
  else if (dtype == TS_BF16)
    launch_swiglu<bf16_t, bf16_t>(out, gate_up, splits, split_stride, tokens, inter, paired, rule, stream);
  else
    return TS_ERR_DTYPE;
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// Rotary encoding + cache write.  The projection output is [T, (Hq + 2 Hkv) * D]: q heads, then
// k heads, then v heads; it is either of type T, or `splits` 32-bit partial sums that are added
// up here.  One block per (token, head).  q and k are rotated by the angles of the token's
// position (cos/sin tables are 32-bit, [capacity, D/2]; pair (i, i + D/2)); the rotated q goes
// to q_out (rows q_stride apart; with a projection of type T this may be the projection itself:
// rotation in place); k (rotated) and v go to the pages at slot = block * BS + offset.  Key
// pages are [NB, Hkv, BS, D]; value pages are transposed, [NB, Hkv, D, BS], so that the
// attention kernels read eight consecutive keys' values of one head dimension with a single
// 16-byte load.  rotate == 0 skips the rotation (a position encoding that only stores).
// slots == nullptr or a negative slot: nothing is stored for that token.
// ---------------------------------------------------------------------------------------------
// One rotation, written out so that every kernel rounds it the same way.
__device__ __forceinline__ void rotate_pair(float x1, float x2, float c, float s, float& o1, float& o2) {
  o1 = __builtin_fmaf(x1, c, -(x2 * s));
  o2 = __builtin_fmaf(x2, c, x1 * s);
}

template <typename T, typename P>
__global__ void rope_store_kernel(T* q_out, long q_stride, const P* proj, int splits,
                                  size_t split_stride, T* __restrict__ k_pages, T* __restrict__ v_pages,
                                  const float* __restrict__ cos_table, const float* __restrict__ sin_table,
                                  const int* __restrict__ positions, const int* __restrict__ slots,
                                  int heads, int kv_heads, int dim, int block_size, int rotate) {
  const int t = blockIdx.x;
  const int h = blockIdx.y;
  const int half = dim / 2;
  const int width = (heads + 2 * kv_heads) * dim;
  const P* row = proj + (size_t)t * width + (size_t)h * dim;
  const int pos = positions[t];
  const int slot = slots ? slots[t] : -1;
  T* page = nullptr;   // this token's row of a key page
  T* vpage = nullptr;  // this token's column of a value page (elements block_size apart)
  if (h >= heads && slot >= 0) {
    const int kvh = (h - heads) % kv_heads;
    const size_t blk = (size_t)(slot / block_size);
    const int off = slot % block_size;
    const size_t head_base = (blk * kv_heads + kvh) * (size_t)block_size * dim;
    if (h < heads + kv_heads)
      page = k_pages + head_base + (size_t)off * dim;
    else
      vpage = v_pages + head_base + off;
  }
  T* qrow = (h < heads) ? q_out + (size_t)t * q_stride + (size_t)h * dim : nullptr;
  if (h < heads + kv_heads) {
    const float* c = cos_table + (size_t)pos * half;
    const float* s = sin_table + (size_t)pos * half;
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
      float x1 = add_splits(row + i, splits, split_stride, 0.f);
      float x2 = add_splits(row + i + half, splits, split_stride, 0.f);
      float r1 = x1, r2 = x2;
      if (rotate) rotate_pair(x1, x2, c[i], s[i], r1, r2);
      const T o1 = from_float<T>(r1);
      const T o2 = from_float<T>(r2);
      if (qrow) {
        qrow[i] = o1;
        qrow[i + half] = o2;
      }
      if (page) {
        page[i] = o1;
        page[i + half] = o2;
      }
    }
  } else if (vpage) {
    for (int i = threadIdx.x; i < dim; i += blockDim.x) {
      const float x = add_splits(row + i, splits, split_stride, 0.f);
      vpage[(size_t)i * block_size] = from_float<T>(x);
    }
  }
}

// The same for many tokens at once (prompt portions): bfloat16 in and out, no partial sums, head
// size a multiple of 16.  One block per (group of 8 consecutive tokens, head).  q and k heads: a
// thread rotates 8 pairs with 16-byte loads and stores.  v heads: a thread collects one head
// dimension of the 8 tokens; when the group's slots are 8 consecutive ones starting at a multiple
// of 8 (the usual case inside a prompt: they lie in one page, block_size being a multiple of 8)
// that is one 16-byte store into the transposed value page, else one 2-byte store per token.
constexpr int ROPE_GROUP = 8;

__global__ void __launch_bounds__(64)
rope_store_group_kernel(bf16_t* q_out, long q_stride, const bf16_t* proj, bf16_t* __restrict__ k_pages,
                        bf16_t* __restrict__ v_pages, const float* __restrict__ cos_table,
                        const float* __restrict__ sin_table, const int* __restrict__ positions,
                        const int* __restrict__ slots, int tokens, int heads, int kv_heads, int dim,
                        int block_size, int rotate) {
  typedef uint16_t u16x8 __attribute__((ext_vector_type(8)));
  typedef float f32x4v __attribute__((ext_vector_type(4)));
  const int t0 = blockIdx.x * ROPE_GROUP;
  const int h = blockIdx.y;
  const int half = dim / 2;
  const int width = (heads + 2 * kv_heads) * dim;
  const int count = min(ROPE_GROUP, tokens - t0);
  if (h < heads + kv_heads) {
    const bool is_key = h >= heads;
    const int kvh = h - heads;
    const int vectors = half / 8;  // 16-byte pieces of a half row
    for (int item = threadIdx.x; item < ROPE_GROUP * vectors; item += blockDim.x) {
      const int j = item / vectors, i = (item % vectors) * 8;
      if (j >= count) continue;
      const int t = t0 + j;
      const bf16_t* row = proj + (size_t)t * width + (size_t)h * dim;
      const u16x8 a = *reinterpret_cast<const u16x8*>(row + i);
      const u16x8 b = *reinterpret_cast<const u16x8*>(row + i + half);
      u16x8 o1 = a, o2 = b;
      if (rotate) {
        const float* c = cos_table + (size_t)positions[t] * half + i;
        const float* s = sin_table + (size_t)positions[t] * half + i;
        const f32x4v c0 = *reinterpret_cast<const f32x4v*>(c), c1 = *reinterpret_cast<const f32x4v*>(c + 4);
        const f32x4v s0 = *reinterpret_cast<const f32x4v*>(s), s1 = *reinterpret_cast<const f32x4v*>(s + 4);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float cv = e < 4 ? c0[e & 3] : c1[e & 3], sv = e < 4 ? s0[e & 3] : s1[e & 3];
          float r1, r2;
          rotate_pair(to_float(bf16_t{a[e]}), to_float(bf16_t{b[e]}), cv, sv, r1, r2);
          o1[e] = from_float<bf16_t>(r1).bits;
          o2[e] = from_float<bf16_t>(r2).bits;
        }
      }
      if (!is_key) {
        bf16_t* qrow = q_out + (size_t)t * q_stride + (size_t)h * dim;
        *reinterpret_cast<u16x8*>(qrow + i) = o1;
        *reinterpret_cast<u16x8*>(qrow + i + half) = o2;
      } else {
        const int slot = slots ? slots[t] : -1;
        if (slot < 0) continue;
        bf16_t* page = k_pages + (((size_t)(slot / block_size) * kv_heads + kvh) * block_size + slot % block_size) * dim;
        *reinterpret_cast<u16x8*>(page + i) = o1;
        *reinterpret_cast<u16x8*>(page + i + half) = o2;
      }
    }
    return;
  }
  if (!slots) return;
  const int kvh = h - heads - kv_heads;
  int slot[ROPE_GROUP];
#pragma unroll
  for (int j = 0; j < ROPE_GROUP; ++j) slot[j] = j < count ? slots[t0 + j] : -1;
  bool run = count == ROPE_GROUP && slot[0] >= 0 && (slot[0] & 7) == 0 && (block_size & 7) == 0;
#pragma unroll
  for (int j = 1; j < ROPE_GROUP; ++j) run = run && slot[j] == slot[0] + j;
  const bf16_t* column = proj + (size_t)t0 * width + (size_t)h * dim;
  for (int d = threadIdx.x; d < dim; d += blockDim.x) {
    u16x8 v;
#pragma unroll
    for (int j = 0; j < ROPE_GROUP; ++j) v[j] = j < count ? column[(size_t)j * width + d].bits : (uint16_t)0;
    if (run) {
      bf16_t* dst = v_pages + (((size_t)(slot[0] / block_size) * kv_heads + kvh) * dim + d) * block_size + slot[0] % block_size;
      *reinterpret_cast<u16x8*>(dst) = v;
    } else {
#pragma unroll
      for (int j = 0; j < ROPE_GROUP; ++j) {
        if (slot[j] < 0) continue;
        v_pages[(((size_t)(slot[j] / block_size) * kv_heads + kvh) * dim + d) * block_size + slot[j] % block_size] = bf16_t{v[j]};
      }
    }
  }
}

extern "C" int ts_rope_store(void* q_out, long q_stride, const void* proj, int in_f32, int splits,
                             long split_stride, void* k_pages, void* v_pages, const float* cos_table,
                             const float* sin_table, const int* positions, const int* slots, int tokens,
                             int heads, int kv_heads, int dim, int block_size, int rotate, int dtype,
                             hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!q_out || !proj || !positions || heads < 1 || kv_heads < 1 || dim < 2 || (dim & 1) || block_size < 1 ||
      splits < 1)
    return TS_ERR_ARG;
  if (rotate && (!cos_table || !sin_table)) return TS_ERR_ARG;
  if (slots && (!k_pages || !v_pages)) return TS_ERR_ARG;
  dim3 grid(tokens, heads + 2 * kv_heads), block(64);
  const bool aligned = ((uintptr_t)q_out | (uintptr_t)proj | (uintptr_t)k_pages | (uintptr_t)v_pages |
                        (uintptr_t)cos_table | (uintptr_t)sin_table) % 16 == 0 && q_stride % 8 == 0;
  if (dtype == TS_BF16 && !in_f32 && splits == 1 && dim % 16 == 0 && tokens >= 4 * ROPE_GROUP && aligned) {
    dim3 groups((tokens + ROPE_GROUP - 1) / ROPE_GROUP, heads + 2 * kv_heads);
    hipLaunchKernelGGL(rope_store_group_kernel, groups, block, 0, stream, (bf16_t*)q_out, q_stride, (const bf16_t*)proj, (bf16_t*)k_pages, (bf16_t*)v_pages, cos_table, sin_table, positions, slots, tokens, heads, kv_heads, dim, block_size, rotate);
    return ts_launch_status();
  }
  if (dtype == TS_F32)
    hipLaunchKernelGGL((rope_store_kernel<float, float>), grid, block, 0, stream, (float*)q_out, q_stride, (const float*)proj, splits, (size_t)split_stride, (float*)k_pages, (float*)v_pages, cos_table, sin_table, positions, slots, heads, kv_heads, dim, block_size, rotate);
  else if (dtype == TS_BF16 && in_f32)
    hipLaunchKernelGGL((rope_store_kernel<bf16_t, float>), grid, block, 0, stream, (bf16_t*)q_out, q_stride, (const float*)proj, splits, (size_t)split_stride, (bf16_t*)k_pages, (bf16_t*)v_pages, cos_table, sin_table, positions, slots, heads, kv_heads, dim, block_size, rotate);
  else if (dtype == TS_BF16)
    hipLaunchKernelGGL((rope_store_kernel<bf16_t, bf16_t>), grid, block, 0, stream, (bf16_t*)q_out, q_stride, (const bf16_t*)proj, splits, (size_t)split_stride, (bf16_t*)k_pages, (bf16_t*)v_pages, cos_table, sin_table, positions, slots, heads, kv_heads, dim, block_size, rotate);
  else
    return TS_ERR_DTYPE;
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// gather rows: out[i, :] = x[rows[i], :]
// ---------------------------------------------------------------------------------------------
template <typename T>
__global__ void gather_rows_kernel(T* __restrict__ out, const T* __restrict__ x,
                                   const int* __restrict__ rows, int width) {
  const size_t src = (size_t)rows[blockIdx.x] * width;
  const size_t dst = (size_t)blockIdx.x * width;
  for (int i = threadIdx.x; i < width; i += blockDim.x) out[dst + i] = x[src + i];
}

extern "C" int ts_gather_rows(void* out, const void* x, const int* rows, int n, int width,
                              int dtype, hipStream_t stream) {
  if (n == 0) return TS_OK;
  if (!out || !x || !rows || width < 1) return TS_ERR_ARG;
  dim3 grid(n), block(256);
  if (dtype == TS_F32)
    hipLaunchKernelGGL(gather_rows_kernel<float>, grid, block, 0, stream, (float*)out, (const float*)x, rows, width);
  else if (dtype == TS_BF16)
    hipLaunchKernelGGL(gather_rows_kernel<bf16_t>, grid, block, 0, stream, (bf16_t*)out, (const bf16_t*)x, rows, width);
  else
    return TS_ERR_DTYPE;
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// patch_tokens: token_ids[i] = source[patch[i]] where patch[i] >= 0 (else left as it is).  A step
// that is launched before the host has read the tokens the step before sampled takes them from
// the sampler's device buffer this way.  patch[i] must be below `sources`; a value at or beyond
// it is ignored (nothing is read out of bounds).
// ---------------------------------------------------------------------------------------------
__global__ void patch_tokens_kernel(int* __restrict__ token_ids, const int* __restrict__ patch,
                                    const int* __restrict__ source, int n, int sources) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n) return;
  const int from = patch[i];
  if (from >= 0 && from < sources) token_ids[i] = source[from];
}

extern "C" int ts_patch_tokens(int* token_ids, const int* patch, const int* source, int n, int sources,
                               hipStream_t stream) {
  if (n == 0) return TS_OK;
  if (!token_ids || !patch || !source || n < 0 || sources < 1) return TS_ERR_ARG;
  hipLaunchKernelGGL(patch_tokens_kernel, dim3((n + 255) / 256), dim3(256), 0, stream, token_ids, patch, source, n,
                     sources);
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// embedding with a position vector: residual[t, :] = float(table[ids[t], :]) + at[positions[t], :]
// (`at` is 32-bit, [capacity, hidden]; the host keeps positions below its capacity).
// ---------------------------------------------------------------------------------------------
template <typename T>
__global__ void embed_positions_kernel(float* __restrict__ residual, const T* __restrict__ table,
                                       const int* __restrict__ ids, const int* __restrict__ positions,
                                       const float* __restrict__ at, int hidden, int vocab) {
  const int t = blockIdx.x;
  const int id = ids[t];
  const bool valid = id >= 0 && id < vocab;
  const T* row = table + (size_t)(valid ? id : 0) * hidden;
  const float* place = at + (size_t)positions[t] * hidden;
  float* out = residual + (size_t)t * hidden;
  for (int i = threadIdx.x; i < hidden; i += blockDim.x)
    out[i] = valid ? to_float(row[i]) + place[i] : __uint_as_float(0x7fc00000u);
}

extern "C" int ts_embed_positions(void* residual, const void* table, const int* ids, const int* positions,
                                  const float* at, int tokens, int hidden, int vocab, int dtype, hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!residual || !table || !ids || !positions || !at || hidden < 1 || vocab < 1) return TS_ERR_ARG;
  dim3 grid(tokens), block(256);
  if (dtype == TS_F32)
    hipLaunchKernelGGL(embed_positions_kernel<float>, grid, block, 0, stream, (float*)residual, (const float*)table, ids, positions, at, hidden, vocab);
  else if (dtype == TS_BF16)
    hipLaunchKernelGGL(embed_positions_kernel<bf16_t>, grid, block, 0, stream, (float*)residual, (const bf16_t*)table, ids, positions, at, hidden, vocab);
  else
    return TS_ERR_DTYPE;
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// stream offset: residual[t, :] += origin[t, :] (where given) + offset[:] (where given), 32-bit.
// ---------------------------------------------------------------------------------------------
template <typename T>
__global__ void stream_offset_kernel(float* __restrict__ residual, const float* __restrict__ origin,
                                     const T* __restrict__ offset, int hidden, size_t total) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  float s = residual[idx];
  if (origin) s += origin[idx];
  if (offset) s += to_float(offset[idx % hidden]);
  residual[idx] = s;
}

extern "C" int ts_stream_offset(float* residual, const float* origin, const void* offset, int tokens, int hidden,
                                int dtype, hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!residual || hidden < 1) return TS_ERR_ARG;
  const size_t total = (size_t)tokens * hidden;
  dim3 grid((unsigned)((total + 255) / 256)), block(256);
  if (dtype == TS_F32)
    hipLaunchKernelGGL(stream_offset_kernel<float>, grid, block, 0, stream, residual, origin, (const float*)offset, hidden, total);
  else if (dtype == TS_BF16)
    hipLaunchKernelGGL(stream_offset_kernel<bf16_t>, grid, block, 0, stream, residual, origin, (const bf16_t*)offset, hidden, total);
  else
    return TS_ERR_DTYPE;
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// copy of 32-bit values by a kernel (a recorded step holds kernels only, no copy nodes).
// ---------------------------------------------------------------------------------------------
__global__ void copy_f32_kernel(float* __restrict__ out, const float* __restrict__ in, size_t total) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx < total) out[idx] = in[idx];
}

extern "C" int ts_copy_f32(float* out, const float* in, long total, hipStream_t stream) {
  if (total == 0) return TS_OK;
  if (!out || !in || total < 0) return TS_ERR_ARG;
  hipLaunchKernelGGL(copy_f32_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream, out, in, (size_t)total);
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// An activation over a projection output [T, I] (of type T, or `splits` 32-bit partial sums that are
// added up here): out[t, i] = act(x[t, i]), computed in 32-bit and rounded once.  For feed-forwards
// without a gate: down(act(up(x))).
//   kind 0: relu(x)^2     kind 1: relu(x)     kind 2: x sigmoid(x)
//   kind 3: the tanh form of GELU, 0.5 x (1 + tanh(sqrt(2 / pi) (x + 0.044715 x^3)))
// ---------------------------------------------------------------------------------------------
__device__ __forceinline__ float activation(float x, int kind) {
  if (kind == 0) {
    const float r = fmaxf(x, 0.f);
    return r * r;
  }
  if (kind == 1) return fmaxf(x, 0.f);
  if (kind == 2) return x / (1.f + expf(-x));
  return x / (1.f + expf(-1.5957691216057308f * fmaf(0.044715f * x * x, x, x)));
}

template <typename T, typename P>
__global__ void activate_kernel(T* __restrict__ out, const P* __restrict__ x, int splits, size_t split_stride,
                                size_t total, int kind) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  out[idx] = from_float<T>(activation(add_splits(x + idx, splits, split_stride, 0.f), kind));
}

template <typename T, typename P>
__global__ void activate_vec4_kernel(T* __restrict__ out, const P* __restrict__ x, int splits, size_t split_stride,
                                     size_t quads, int kind) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= quads) return;
  float s[4] = {0.f, 0.f, 0.f, 0.f};
  add_splits4(x + 4 * idx, splits, split_stride, s);
  float o[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) o[e] = activation(s[e], kind);
  Vec4Of<T>::store(out + 4 * idx, o);
}

template <typename T, typename P>
static void launch_activate(void* out, const void* x, int splits, long split_stride, size_t total, int kind,
                            hipStream_t stream) {
  if (total % 4 == 0 && ((uintptr_t)out | (uintptr_t)x) % 16 == 0 && split_stride % 4 == 0) {
    const size_t quads = total / 4;
    hipLaunchKernelGGL((activate_vec4_kernel<T, P>), dim3((unsigned)((quads + 255) / 256)), dim3(256), 0, stream, (T*)out,
                       (const P*)x, splits, (size_t)split_stride, quads, kind);
  } else {
    hipLaunchKernelGGL((activate_kernel<T, P>), dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream, (T*)out,
                       (const P*)x, splits, (size_t)split_stride, total, kind);
  }
}

extern "C" int ts_activate(void* out, const void* x, int in_f32, int splits, long split_stride, int tokens, int inter,
                           int kind, int dtype, hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!out || !x || inter < 1 || splits < 1 || kind < 0 || kind > 3) return TS_ERR_ARG;
  const size_t total = (size_t)tokens * inter;
  if (dtype == TS_F32)
    launch_activate<float, float>(out, x, splits, split_stride, total, kind, stream);
  else if (dtype == TS_BF16 && in_f32)
    launch_activate<bf16_t, float>(out, x, splits, split_stride, total, kind, stream);
  else if (dtype == TS_BF16)
    launch_activate<bf16_t, bf16_t>(out, x, 1, 0, total, kind, stream);
  else
    return TS_ERR_DTYPE;
  return ts_launch_status();
}

// ---------------------------------------------------------------------------------------------
// clearing the state of requests that start: rows `slots` of every state tensor, one launch
// ---------------------------------------------------------------------------------------------
#define ZERO_SLOTS 32

struct ZeroSlots {
  int at[ZERO_SLOTS];
};

// table [n][2]: a state tensor's address and the bytes of one of its rows (a multiple of 4).
__global__ void __launch_bounds__(256) zero_state_rows_kernel(const long long* __restrict__ table, ZeroSlots slots) {
  const size_t words = (size_t)table[2 * blockIdx.y + 1] / 4;
  uint32_t* row = reinterpret_cast<uint32_t*>(table[2 * blockIdx.y]) + (size_t)slots.at[blockIdx.x] * words;
  const size_t step = (size_t)gridDim.z * blockDim.x, from = (size_t)blockIdx.z * blockDim.x + threadIdx.x;
  if (words % 4 == 0 && ((uintptr_t)row & 15) == 0) {
    for (size_t i = from; i < words / 4; i += step) reinterpret_cast<uint4*>(row)[i] = make_uint4(0u, 0u, 0u, 0u);
  } else {
    for (size_t i = from; i < words; i += step) row[i] = 0u;
  }
}

// `slots` is host memory.
extern "C" int ts_zero_state_rows(const long long* table, int n, const int* slots, int count, hipStream_t stream) {
  if (n == 0 || count == 0) return TS_OK;
  if (!table || !slots || n < 0 || n > 65535 || count < 0) return TS_ERR_ARG;
  for (int first = 0; first < count; first += ZERO_SLOTS) {
    const int here = count - first < ZERO_SLOTS ? count - first : ZERO_SLOTS;
    ZeroSlots some;
    for (int i = 0; i < ZERO_SLOTS; ++i) some.at[i] = slots[first + (i < here ? i : 0)];
    hipLaunchKernelGGL(zero_state_rows_kernel, dim3(here, n, 32), dim3(256), 0, stream, table, some);
  }
  return ts_launch_status();
}
