// The gates of a memory that fades and is written by one forget gate, as its token-by-token, chunked and decode forms take them.
#pragma once

#include "rows.h"

namespace iron {

// Rows [q | f | v | ..], heads * dim columns of q and of f, heads * vdim of v; a channel's bias, and the bound its gate keeps above.
struct FadeGates {
  const bf16_t *bias, *lower;
};

// f = l + (1 - l) sigmoid(z + bias), and 1 - f without a difference of near numbers.
struct Fade {
  float keep, write;
};
// (T: the rows' type; the hardware's exponential, reciprocal and logarithm, an ulp or two off, where they are bf16)
template <typename T>
__device__ __forceinline__ float logistic(float z) {
  if constexpr (sizeof(T) == 2) return __builtin_amdgcn_rcpf(1.f + __expf(-z));
  else return 1.f / (1.f + expf(-z));
}
template <typename T>
__device__ __forceinline__ Fade fade_of(float z, float bias, float lower) {
  z += bias;
  const float rest = 1.f - lower;
  return Fade{lower + rest * logistic<T>(z), rest * logistic<T>(-z)};
}
// log2 f, finite: a gate that has closed altogether counts as one that is as good as closed.
template <typename T>
__device__ __forceinline__ float log2_fade(const Fade& f) {
  if constexpr (sizeof(T) == 2) return __builtin_amdgcn_logf(fmaxf(f.keep, 1e-37f));
  else return f.keep > 0.5f ? log1pf(-f.write) * 1.4426950408889634f : log2f(fmaxf(f.keep, 1e-37f));
}
template <typename T>
__device__ __forceinline__ float silu_read(float q) { return q * logistic<T>(q); }

}  // namespace iron
