// The gates of a matrix memory, as its token-by-token and its chunked form take them.
#pragma once

#include "rows.h"

namespace iron {

struct MemoryGates {
  const bf16_t *i_bias, *f_bias;
  int i_at, f_at;                        // columns of a row
  float cap;
};

// log(sigmoid(z)) without a difference of large numbers.
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float capped(float z, float cap) { return cap * tanhf(z / cap); }

}  // namespace iron
