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
__device__ __forceinline__ Fade fade_of(float z, float bias, float lower) {
  z += bias;
  const float rest = 1.f - lower;
  return Fade{lower + rest / (1.f + expf(-z)), rest / (1.f + expf(z))};
}
// log f, finite: a gate that has closed altogether counts as one that is as good as closed.
__device__ __forceinline__ float log_fade(const Fade& f) { return f.keep > 0.5f ? log1pf(-f.write) : logf(fmaxf(f.keep, 1e-37f)); }
__device__ __forceinline__ float silu_read(float q) { return q / (1.f + expf(-q)); }

}  // namespace iron
