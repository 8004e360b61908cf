// What the single-row product kernels share: a block of 256 threads owns a few rows of a weight, thread t
// takes their 16-byte chunks t, t + 256, ..., and the waves' sums meet in LDS.
#pragma once

#include "common.h"

namespace iron {

// Block-wide sum through LDS (one barrier); every thread gets the total.
__device__ __forceinline__ float block_sum(float v, float* scratch4) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) scratch4[threadIdx.x >> 6] = v;
  __syncthreads();
  return scratch4[0] + scratch4[1] + scratch4[2] + scratch4[3];
}

// A weight row's chunks of this thread (zeros past the row's end), streamed past the caches.
template <int CH>
__device__ __forceinline__ void load_row(const bf16_t* __restrict__ row, int K, uint4 (&w)[CH]) {
  const __amdgpu_buffer_rsrc_t run = bounded_bytes(row, 2 * K);
#pragma unroll
  for (int i = 0; i < CH; ++i) w[i] = load_bounded_stream(run, 16 * ((int)threadIdx.x + 256 * i));
}

// A row's chunks times the activation's: two-element dot products of the bf16 pairs as they were
// loaded (v_dot2c_f32_bf16: exact products, float32 sums) -- a quarter of the instructions of
// widening both sides and a multiply-add an element, and what a resident block does after its
// loads have landed is time its CU's share of the memory system idles.
typedef __bf16 bf16x2_t __attribute__((ext_vector_type(2)));
template <int CH>
__device__ __forceinline__ float dot_row(const uint4 (&w)[CH], const uint4 (&xp)[CH]) {
  float acc = 0.f;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2_t, w[i].x), __builtin_bit_cast(bf16x2_t, xp[i].x), acc, false);
    acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2_t, w[i].y), __builtin_bit_cast(bf16x2_t, xp[i].y), acc, false);
    acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2_t, w[i].z), __builtin_bit_cast(bf16x2_t, xp[i].z), acc, false);
    acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2_t, w[i].w), __builtin_bit_cast(bf16x2_t, xp[i].w), acc, false);
  }
  return acc;
}

}  // namespace iron
