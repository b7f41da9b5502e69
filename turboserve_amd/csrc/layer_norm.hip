// Layer norm where it carries the residual sum.
//
// ts_add_layer_norm, per row:
//     p = pending                                   (type T, or `splits` 32-bit partial sums added up here)
//     p = scale * (layer_norm(p) * post_w + post_b)  where a norm of the pending output is given
//     s = residual + p;  residual = s
//     y = round_T(layer_norm(s) * w + b)             where a norm of the sum is given, else round_T(s)
// with layer_norm(v) = (v - mean) / sqrt(variance + eps), the variance being the mean of the squared deviations
// (two passes over registers), all in 32-bit with one rounding.  A norm without a bias has a null one.  With `rows` the kernel reads rows[i] and writes
// y[i] only (residual untouched): the final norm at the wanted positions.  So one launch serves a block with a
// norm in front of its parts, one with a norm behind them, and the head.
//
// A row is one workgroup's; a thread keeps its CHUNKS pieces of VEC neighbouring elements in registers.
#include "vec.hpp"

template <typename T>
struct LayerNormRule {
  const T* w;  // null: no norm
  const T* b;  // null: nothing is added
  float eps;
  float scale;
};

template <typename T, int VEC, int CHUNKS>
__device__ __forceinline__ void ln_apply(float (&s)[CHUNKS][VEC], LayerNormRule<T> rule, int hidden, float* scratch) {
  float sum = 0.f;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c)
#pragma unroll
    for (int e = 0; e < VEC; ++e) sum += s[c][e];  // (places beyond the row hold zeros)
  const float mean = block_sum(sum, scratch) / (float)hidden;
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const bool in = (int)(c * blockDim.x + threadIdx.x) * VEC < hidden;
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      s[c][e] -= mean;
      if (in) ss = fmaf(s[c][e], s[c][e], ss);
    }
  }
  const float rstd = rsqrtf(block_sum(ss, scratch) / (float)hidden + rule.eps);
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int i = (int)(c * blockDim.x + threadIdx.x) * VEC;
    if (i < hidden) {
      float w[VEC], b[VEC];
      load_vec<T, VEC>(rule.w + i, w);
      if (rule.b) {
        load_vec<T, VEC>(rule.b + i, b);
      } else {
#pragma unroll
        for (int e = 0; e < VEC; ++e) b[e] = 0.f;
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) s[c][e] = rule.scale * fmaf(s[c][e] * rstd, w[e], b[e]);
    }
  }
}

template <typename T, typename P, int VEC, int CHUNKS>
__global__ void __launch_bounds__(1024)
add_layer_norm_kernel(T* __restrict__ y, float* __restrict__ residual, const P* __restrict__ pending, int splits,
                      size_t split_stride, LayerNormRule<T> post, LayerNormRule<T> last, const int* __restrict__ rows, int hidden) {
  __shared__ float scratch[16];
  const int src = rows ? rows[blockIdx.x] : blockIdx.x;
  const size_t in_base = (size_t)src * hidden, out_base = (size_t)blockIdx.x * hidden;
  float s[CHUNKS][VEC], held[CHUNKS][VEC];
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int i = (int)(c * blockDim.x + threadIdx.x) * VEC;
#pragma unroll
    for (int e = 0; e < VEC; ++e) s[c][e] = held[c][e] = 0.f;
    if (i < hidden) {
      load_vec<float, VEC>(residual + in_base + i, held[c]);
      if (pending) load_vec<P, VEC>(pending + in_base + i, s[c]);
    }
  }
  for (int first = 1; first < splits; first += 8) {  // the other partial sums, eight loads in flight, added in split order
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
      const int i = (int)(c * blockDim.x + threadIdx.x) * VEC;
      if (i < hidden) {
        float v[8][VEC];
#pragma unroll
        for (int j = 0; j < 8; ++j) load_vec<P, VEC>(pending + (size_t)min(first + j, splits - 1) * split_stride + in_base + i, v[j]);
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (first + j < splits) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) s[c][e] += v[j][e];
          }
      }
    }
  }
  if (post.w) ln_apply<T, VEC, CHUNKS>(s, post, hidden, scratch);
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int i = (int)(c * blockDim.x + threadIdx.x) * VEC;
    const bool in = i < hidden;
#pragma unroll
    for (int e = 0; e < VEC; ++e) s[c][e] = in ? held[c][e] + s[c][e] : 0.f;
    if (in && pending && !rows) store_vec<float, VEC>(residual + in_base + i, s[c]);
  }
  if (last.w) ln_apply<T, VEC, CHUNKS>(s, last, hidden, scratch);
#pragma unroll
  for (int c = 0; c < CHUNKS; ++c) {
    const int i = (int)(c * blockDim.x + threadIdx.x) * VEC;
    if (i >= hidden) continue;
    store_vec<T, VEC>(y + out_base + i, s[c]);
  }
}

template <typename T, typename P>
static int launch_add_layer_norm(void* y, float* residual, const void* pending, int splits, long split_stride, const void* post_w,
                                 const void* post_b, float post_eps, float post_scale, const void* w, const void* b, float eps,
                                 const int* rows, int out_rows, int hidden, hipStream_t stream) {
  const LayerNormRule<T> post = {(const T*)post_w, (const T*)post_b, post_eps, post_scale};
  const LayerNormRule<T> last = {(const T*)w, (const T*)b, eps, 1.f};
  const bool wide = hidden % 4 == 0 && ((uintptr_t)y | (uintptr_t)residual | (uintptr_t)pending | (uintptr_t)post_w | (uintptr_t)post_b |
                                        (uintptr_t)w | (uintptr_t)b) % 16 == 0;
#define LN_GO(VEC, CHUNKS, THREADS)                                                                                           \
  hipLaunchKernelGGL((add_layer_norm_kernel<T, P, VEC, CHUNKS>), dim3(out_rows), dim3(THREADS), 0, stream, (T*)y, residual,   \
                     (const P*)pending, splits, (size_t)split_stride, post, last, rows, hidden)
  if (wide) {
    // Steps of few rows spread a row over as many wavefronts as it has pieces for; prompts keep 256 threads a row.
    const int pieces = hidden / 4;
    const bool few = out_rows < 64;
    if (pieces <= 256) LN_GO(4, 1, (pieces + 63) / 64 * 64);
    else if (few && pieces <= 1024) LN_GO(4, 1, (pieces + 63) / 64 * 64);
    else if (pieces <= 512) LN_GO(4, 2, 256);
    else if (pieces <= 1024) LN_GO(4, 4, 256);
    else if (pieces <= 2048) LN_GO(4, 4, 512);
    else if (pieces <= 4096) LN_GO(4, 4, 1024);
    else return TS_ERR_SHAPE;
  } else {
    if (hidden <= 1024) LN_GO(1, 1, (hidden + 63) / 64 * 64);
    else if (hidden <= 4096) LN_GO(1, 4, 1024);
    else if (hidden <= 16384) LN_GO(1, 16, 1024);
    else return TS_ERR_SHAPE;
  }
#undef LN_GO
  return ts_launch_status();
}

extern "C" int ts_add_layer_norm(void* y, float* residual, const void* pending, int pending_f32, int splits, long split_stride,
                                 const void* post_w, const void* post_b, float post_eps, float post_scale, const void* w,
                                 const void* b, float eps, const int* rows, int out_rows, int hidden, int dtype, hipStream_t stream) {
  if (out_rows == 0) return TS_OK;
  if (!y || !residual || hidden < 1 || splits < 1 || (splits > 1 && !pending) || (post_w && !pending)) return TS_ERR_ARG;
  if ((!post_w && post_b) || (!w && b)) return TS_ERR_ARG;
  if (dtype == TS_F32)
    return launch_add_layer_norm<float, float>(y, residual, pending, splits, split_stride, post_w, post_b, post_eps, post_scale, w, b, eps, rows, out_rows, hidden, stream);
  if (dtype == TS_BF16 && pending_f32)
    return launch_add_layer_norm<bf16_t, float>(y, residual, pending, splits, split_stride, post_w, post_b, post_eps, post_scale, w, b, eps, rows, out_rows, hidden, stream);
  if (dtype == TS_BF16)
    return launch_add_layer_norm<bf16_t, bf16_t>(y, residual, pending, splits, split_stride, post_w, post_b, post_eps, post_scale, w, b, eps, rows, out_rows, hidden, stream);
  return TS_ERR_DTYPE;
}
