// What attention kernels over packed projections and a ring a slot share.
#pragma once

#include "rows.h"

namespace iron {

// A call's rows are [q heads | k heads | v heads]; position p's key and value live in row p % ring of the slot's ring.
struct PackedHeads {
  int rows, stride;                      // the packed rows, and their length
  int heads, kv_heads, dim, vdim;
  int ring;
};

// The span's last rows into the ring: a block a row, from the span's last one back.
template <typename T>
__global__ __launch_bounds__(256) void ring_store_kernel(const T* __restrict__ x, T* __restrict__ keys, T* __restrict__ values,
                                                         const int* __restrict__ spans, PackedHeads a) {
  const Span s = span_of(spans, blockIdx.y, a.rows);
  const int i = s.rows - 1 - (int)blockIdx.x;
  if (i < 0 || (int)blockIdx.x >= a.ring) return;
  const int at = (s.start + i) % a.ring, nk = a.kv_heads * a.dim, nv = a.kv_heads * a.vdim;
  const T* row = x + (size_t)(s.row0 + i) * a.stride + a.heads * a.dim;
  T* kd = keys + ((size_t)blockIdx.y * a.ring + at) * nk;
  T* vd = values + ((size_t)blockIdx.y * a.ring + at) * nv;
  for (int c = threadIdx.x; c < nk; c += 256) kd[c] = row[c];
  for (int c = threadIdx.x; c < nv; c += 256) vd[c] = row[nk + c];
}

template <typename T>
static void launch_ring_store(const void* x, void* keys, void* values, const int* spans, const PackedHeads& a, int slots, hipStream_t s) {
  hipLaunchKernelGGL((ring_store_kernel<T>), dim3(a.rows < a.ring ? a.rows : a.ring, slots), dim3(256), 0, s, (const T*)x, (T*)keys, (T*)values,
                     spans, a);
}

// The slot whose span holds `row` (every lane of a wave gets it), or -1.
__device__ __forceinline__ int slot_of_row(const int* __restrict__ spans, int slots, int rows, int row) {
  for (int first = 0; first < slots; first += 64) {
    const int i = first + ((int)threadIdx.x & 63);
    bool here = false;
    if (i < slots) {
      const Span s = span_of(spans, i, rows);
      here = row >= s.row0 && row < s.row0 + s.rows;
    }
    const unsigned long long found = __builtin_amdgcn_ballot_w64(here);
    if (found != 0) return first + __builtin_ctzll(found);
  }
  return -1;
}

// The spans cut into tiles of `size` rows, one span's after the other's in the order of the slots: the slot of tile `index` and its
// first row within the span.  False past the last.
__device__ __forceinline__ bool tile_of(const int* __restrict__ spans, int slots, int rows, int size, int index, int& slot, int& first) {
  const int lane = (int)threadIdx.x & 63;
  for (int f = 0; f < slots; f += 64) {
    int n = 0;
    if (f + lane < slots) n = (span_of(spans, f + lane, rows).rows + size - 1) / size;
    int sum = n;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const int v = __shfl_up(sum, d, 64);
      if (lane >= d) sum += v;
    }
    const unsigned long long past = __builtin_amdgcn_ballot_w64(index < sum);
    if (past != 0) {
      const int at = __builtin_ctzll(past);
      slot = __builtin_amdgcn_readfirstlane(f + at);
      first = __builtin_amdgcn_readfirstlane((index - (__shfl(sum, at, 64) - __shfl(n, at, 64))) * size);
      return true;
    }
    index -= __shfl(sum, 63, 64);
  }
  return false;
}

}  // namespace iron
