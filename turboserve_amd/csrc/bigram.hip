// A token's start from two tables.
//
// ts_embed_bigram, per token: row ids[t] of a table plus row (prev * mul_prev + id * mul_cur) mod buckets of a second
// table, `prev` the token before it in its request; a request's first token takes the row `buckets`.  The token before
// a step's first comes from the request's state slot (held [slots, 1]: the last token id plus one, 0 for a request
// that starts).  In a step of single tokens the same launch moves the slot on; otherwise ts_embed_bigram_carry does.
#include "vec.hpp"

// The multipliers come in reduced modulo `buckets`, so every product fits 64 bits.
template <typename T>
__global__ void __launch_bounds__(256)
embed_bigram_kernel(float* __restrict__ out, const T* __restrict__ table, const T* __restrict__ pairs, const int* __restrict__ ids,
                    int* held, const int* __restrict__ state_slots, const int* __restrict__ token_seq,
                    const int* __restrict__ query_start_loc, int hidden, int vocab, int buckets, unsigned mul_prev, unsigned mul_cur,
                    int single, int wide) {
  const int t = blockIdx.x;
  const int seq = single ? t : token_seq[t];
  const int row0 = single ? t : query_start_loc[seq];
  const int id = ids[t];
  const int prev = t > row0 ? ids[t - 1] : held[state_slots[seq]] - 1;
  const bool valid = id >= 0 && id < vocab;  // an id outside the table is a host error; it yields NaN
  const unsigned row = prev < 0 || !valid ? (unsigned)buckets
                                : (unsigned)(((uint64_t)prev * mul_prev + (uint64_t)id * mul_cur) % (unsigned)buckets);
  if (single) {
    __syncthreads();  // the workgroup has read the slot
    if (threadIdx.x == 0) held[state_slots[seq]] = id + 1;
  }
  const T* one = table + (size_t)(valid ? id : 0) * hidden;
  const T* other = pairs + (size_t)row * hidden;
  float* to = out + (size_t)t * hidden;
  if (wide && valid) {
    for (int i = 4 * threadIdx.x; i < hidden; i += 4 * blockDim.x) {
      float a[4], b[4];
      load_vec<T, 4>(one + i, a);
      load_vec<T, 4>(other + i, b);
      *reinterpret_cast<float4*>(to + i) = make_float4(a[0] + b[0], a[1] + b[1], a[2] + b[2], a[3] + b[3]);
    }
    return;
  }
  for (int i = threadIdx.x; i < hidden; i += blockDim.x)
    to[i] = valid ? to_float(one[i]) + to_float(other[i]) : __uint_as_float(0x7fc00000u);
}

__global__ void embed_bigram_carry_kernel(int* __restrict__ held, const int* __restrict__ ids, const int* __restrict__ state_slots,
                                          const int* __restrict__ query_start_loc, int num_seqs) {
  const int seq = blockIdx.x * blockDim.x + threadIdx.x;
  if (seq < num_seqs && query_start_loc[seq + 1] > query_start_loc[seq]) held[state_slots[seq]] = ids[query_start_loc[seq + 1] - 1] + 1;
}

extern "C" int ts_embed_bigram(float* out, const void* table, const void* pairs, const int* ids, int* held, const int* state_slots,
                               const int* token_seq, const int* query_start_loc, int tokens, int num_seqs, int hidden, int vocab,
                               int buckets, int mul_prev, int mul_cur, int dtype, hipStream_t stream) {
  if (tokens == 0) return TS_OK;
  if (!out || !table || !pairs || !ids || !held || !state_slots || !token_seq || !query_start_loc) return TS_ERR_ARG;
  if (hidden < 1 || vocab < 1 || buckets < 1 || mul_prev < 0 || mul_cur < 0 || num_seqs < 1) return TS_ERR_SHAPE;
  const int single = tokens == num_seqs;
  const int wide = hidden % 4 == 0 && ((uintptr_t)out | (uintptr_t)table | (uintptr_t)pairs) % 16 == 0;
#define EB_GO(T)                                                                                                               \
  hipLaunchKernelGGL((embed_bigram_kernel<T>), dim3(tokens), dim3(256), 0, stream, out, (const T*)table, (const T*)pairs, ids, \
                     held, state_slots, token_seq, query_start_loc, hidden, vocab, buckets, (unsigned)mul_prev, (unsigned)mul_cur, single, wide)
  if (dtype == TS_F32) EB_GO(float);
  else if (dtype == TS_BF16) EB_GO(bf16_t);
  else return TS_ERR_DTYPE;
#undef EB_GO
  if (!single)
    hipLaunchKernelGGL(embed_bigram_carry_kernel, dim3((num_seqs + 63) / 64), dim3(64), 0, stream, held, ids, state_slots,
                       query_start_loc, num_seqs);
  return ts_launch_status();
}
