// What latent attention's kernels and the fused decode kernels share: its sizes, and a position's row.
#pragma once

#include "rows.h"

namespace iron {

struct LatentShape {
  int slots, rows;                       // the batch's
  int heads, dim, rot, vdim, rank;
  int turned, angle_rows;                // columns of the rot ones that turn, and rows of the table of angles
  int window, ring;
  int cap;                               // expanded key rows there is room for
  float scale;
};

// A row [query latent | latent | shared key part] by a block of 256: both latents over their root mean square, the key
// part turned; in 16-byte pieces, at most CH a thread, held between the sums and the stores.
struct LatentRow {
  const bf16_t *q_gain, *c_gain;
  const float* angles;
  int q_rank;
  float eps;
};
// QUERY false: xr begins at the latent, and the query's part is somebody else's.
template <typename T, int CH, bool QUERY>
__device__ __forceinline__ void latent_row(const T* __restrict__ xr, const LatentRow& g, const LatentShape& a, int slot, int pos,
                                           T* __restrict__ q_out, T* __restrict__ latents, T* __restrict__ shared_keys, float (*part)[4]) {
  const int t = threadIdx.x, qn = QUERY ? g.q_rank >> 3 : 0, cn = qn + (a.rank >> 3), n = cn + (a.rot >> 3), at = pos % a.ring;
  float f[CH][8], gain[CH][8], qs = 0.f, cs = 0.f;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int e = t + 256 * i;
    if (e < n) load_vec<8>(xr + e * 8, f[i]);
    if (e < cn) load_vec<8>(QUERY && e < qn ? g.q_gain + e * 8 : g.c_gain + (e - qn) * 8, gain[i]);
  }
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int e = t + 256 * i;
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) sum = e < cn ? fmaf(f[i][j], f[i][j], sum) : 0.f;
    qs += e < qn ? sum : 0.f;
    cs += e < qn ? 0.f : sum;
  }
  qs = wave_sum(qs);
  cs = wave_sum(cs);
  if ((t & 63) == 0) {
    part[0][t >> 6] = qs;
    part[1][t >> 6] = cs;
  }
  __syncthreads();
  const float qi = 1.0f / sqrtf((part[0][0] + part[0][1] + part[0][2] + part[0][3]) / (float)g.q_rank + g.eps);
  const float ci = 1.0f / sqrtf((part[1][0] + part[1][1] + part[1][2] + part[1][3]) / (float)a.rank + g.eps);
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int e = t + 256 * i;
    if (e >= n) break;
    if (e < cn) {
#pragma unroll
      for (int j = 0; j < 8; ++j) f[i][j] *= (e < qn ? qi : ci) * gain[i][j];
      store_vec<8>(QUERY && e < qn ? q_out + e * 8 : latents + ((size_t)slot * a.ring + at) * a.rank + (e - qn) * 8, f[i]);
    } else {
      const int c = (e - cn) * 8;
      if (c < a.turned) {
        const float* turn = g.angles + (size_t)min(pos, a.angle_rows - 1) * a.turned + c;
#pragma unroll
        for (int j = 0; j < 8; j += 2) {
          const float u = f[i][j], v = f[i][j + 1];
          f[i][j] = u * turn[j] - v * turn[j + 1];
          f[i][j + 1] = v * turn[j] + u * turn[j + 1];
        }
      }
      store_vec<8>(shared_keys + ((size_t)slot * a.ring + at) * a.rot + c, f[i]);
    }
  }
}

static bool latent_row_wide(const LatentShape& a, int stride, int q_rank) {
  return (stride | q_rank | a.rank | a.rot | a.turned) % 8 == 0 && q_rank + a.rank + a.rot <= 4 * 2048;
}

}  // namespace iron
