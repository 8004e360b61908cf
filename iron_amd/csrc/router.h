// How a router's logits become a row's experts and their shares.
#pragma once

#include "rows.h"

namespace iron {

constexpr int ROUTER_MAX = 1024;   // experts

// The `top` largest of n logits in LDS by one wave, in order, the first of equal ones first; their shares.
__device__ __forceinline__ void choose(float* __restrict__ z, int n, int top, int* __restrict__ ids, float* __restrict__ shares) {
  const int lane = threadIdx.x & 63;
  float first = 0.f, total = 0.f, mine = 0.f;
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int at = n;
    for (int i = lane; i < n; i += 64)
      if (z[i] > best) {
        best = z[i];
        at = i;
      }
    const float most = wave_max(best);
    // (no logit above -inf, or none that is a number: the first expert)
    const unsigned long long here = __builtin_amdgcn_ballot_w64(best == most && at < n);
    int id = n;
    for (unsigned long long left = here; left != 0; left &= left - 1) id = min(id, __shfl(at, __builtin_ctzll(left), 64));
    if (id >= n) id = 0;
    if (k == 0) first = most;
    const float e = expf(most - first);
    total += e;
    if (lane == k) mine = e;
    if (lane == 0) {
      ids[k] = id;
      z[id] = -INFINITY;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  if (lane < top) shares[lane] = mine / total;
}

// The `top` largest of the n scores (a softmax over the logits z) plus corrections by one wave, in order, the first of equal ones
// first; their shares, the scores over their sum.  z and by: LDS.
__device__ __forceinline__ void choose_scored(float* __restrict__ z, float* __restrict__ by, const bf16_t* __restrict__ correction, int n, int top,
                                              int* __restrict__ ids, float* __restrict__ shares) {
  const int lane = threadIdx.x & 63;
  if (n <= 64) {   // a logit a lane
    const float logit = lane < n ? z[lane] : -INFINITY, e = expf(logit - wave_max(logit)), score = e / wave_sum(e);
    float key = lane < n ? score + (correction != nullptr ? bf16_to_f32(correction[lane]) : 0.f) : -INFINITY, sum = 0.f, mine = 0.f;
    for (int k = 0; k < top; ++k) {
      const unsigned long long here = __builtin_amdgcn_ballot_w64(key == wave_max(key) && key > -INFINITY);
      const int id = here != 0 ? __builtin_ctzll(here) : 0;   // (none that is a number: the first)
      const float chosen = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, score), id));
      sum += chosen;
      if (lane == k) mine = chosen;
      if (lane == 0) ids[k] = id;
      if (lane == id) key = -INFINITY;
    }
    if (lane < top) shares[lane] = mine / (sum + 1e-20f);
    return;
  }
  float most = -INFINITY, total = 0.f;
  for (int i = lane; i < n; i += 64) most = fmaxf(most, z[i]);
  most = wave_max(most);
  for (int i = lane; i < n; i += 64) total += expf(z[i] - most);
  total = wave_sum(total);
  for (int i = lane; i < n; i += 64) {   // (a lane reads what it wrote)
    z[i] = expf(z[i] - most) / total;
    by[i] = z[i] + (correction != nullptr ? bf16_to_f32(correction[i]) : 0.f);
  }
  float sum = 0.f, mine = 0.f;
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY, score = 0.f;
    int at = n;
    for (int i = lane; i < n; i += 64)
      if (by[i] > best) {
        best = by[i];
        score = z[i];
        at = i;
      }
    const float largest = wave_max(best);
    int id = n, from = 0;
    for (unsigned long long left = __builtin_amdgcn_ballot_w64(best == largest && at < n); left != 0; left &= left - 1) {
      const int l = __builtin_ctzll(left), other = __shfl(at, l, 64);
      if (other < id) {
        id = other;
        from = l;
      }
    }
    score = __shfl(score, from, 64);
    if (id >= n) id = 0;   // (none that is a number: the first)
    sum += score;
    if (lane == k) mine = score;
    if (lane == 0) ids[k] = id;
    if (lane == (id & 63)) by[id] = -INFINITY;
  }
  if (lane < top) shares[lane] = mine / (sum + 1e-20f);
}

// A row's choice from logits another launch left, by the block's first wave; z and by: LDS, ROUTER_MAX floats each.
struct RouterChoice {
  const float* z;            // NULL: there is none to make
  const bf16_t* correction;
  int logits, top;
  int* ids;
  float* shares;
};
__device__ __forceinline__ void choose_row(const RouterChoice& a, float* __restrict__ z, float* __restrict__ by) {
  if (threadIdx.x >= 64) return;
  for (int i = threadIdx.x; i < a.logits; i += 64) z[i] = a.z[i];   // (a lane reads what it wrote)
  choose_scored(z, by, a.correction, a.logits, a.top, a.ids, a.shares);
}
#define IRON_ROUTER_CHOICE_REQUIRE(name)                                                                                             \
  IRON_REQUIRE(z == nullptr || (slots == 1 && ids && shares && logits > 0 && logits <= ROUTER_MAX && top > 0 && top <= logits && top <= 64), \
               name ": one slot's choice of %d of %d logits", top, logits)

// The expert an id names, -1 for one of the identities behind the last.
__device__ __forceinline__ int expert_of(int id, int experts, int identity) { return identity > 0 && id >= experts ? -1 : min(max(id, 0), experts - 1); }

}  // namespace iron
