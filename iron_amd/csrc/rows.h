// Rows of either activation type -- bf16, or float where a model runs in 32 bits throughout -- read
// and written as floats, and the spans that say which rows belong to which sequence.
#pragma once

#include "common.h"

namespace iron {

// VEC consecutive elements: 8 at 16-byte alignment, or one.
template <int VEC, typename T>
__device__ __forceinline__ void load_vec(const T* __restrict__ p, float (&f)[VEC]) {
  static_assert(VEC == 8 || VEC == 1, "eight elements or one");
  if constexpr (VEC == 1) {
    if constexpr (sizeof(T) == 2) f[0] = bf16_to_f32(*p);
    else f[0] = *p;
  } else if constexpr (sizeof(T) == 2) {
    unpack8(*reinterpret_cast<const uint4*>(p), f);
  } else {
    const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
    f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
  }
}
template <int VEC, typename T>
__device__ __forceinline__ void store_vec(T* __restrict__ p, const float (&f)[VEC]) {
  if constexpr (VEC == 1) {
    if constexpr (sizeof(T) == 2) *p = f32_to_bf16(f[0]);
    else *p = f[0];
  } else if constexpr (sizeof(T) == 2) {
    *reinterpret_cast<uint4*>(p) = pack8(f);
  } else {
    reinterpret_cast<float4*>(p)[0] = make_float4(f[0], f[1], f[2], f[3]);
    reinterpret_cast<float4*>(p)[1] = make_float4(f[4], f[5], f[6], f[7]);
  }
}
template <typename T>
__device__ __forceinline__ float load_one(const T* __restrict__ p) {
  float f[1];
  load_vec<1>(p, f);
  return f[0];
}
template <typename T>
__device__ __forceinline__ void store_one(T* __restrict__ p, float v) {
  const float f[1] = {v};
  store_vec<1>(p, f);
}

// act(g) * u.  kind: 0 the limited gate, min(g, limit) through x sigmoid(1.702 x), times one more than u held within the limit;
// 1 SiLU; 2 GELU (tanh form); 3 ReLU.
__device__ __forceinline__ float gated_value(int kind, float limit, float g, float u) {
  if (kind == 0) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.f + expf(-1.702f * g)) * (u + 1.f);
  }
  return (kind == 3 ? fmaxf(g, 0.f) : (kind == 1 ? g / (1.f + expf(-g)) : gelu_tanh_f32(g))) * u;
}

// One sequence's part of a batch of rows: `rows` rows from `row0` on are its tokens at positions
// `start`, `start + 1`, ...  The table has an entry a slot; an idle slot's has no rows.  Held inside
// the batch here, so that no table can lead a kernel outside its buffers.
struct Span {
  int row0, rows, start;
};
__device__ __forceinline__ Span span_of(const int* __restrict__ spans, int slot, int batch_rows) {
  const int4 v = reinterpret_cast<const int4*>(spans)[slot];
  Span s;
  s.row0 = v.x < 0 ? 0 : (v.x > batch_rows ? batch_rows : v.x);
  const int left = batch_rows - s.row0;
  s.rows = v.y < 0 ? 0 : (v.y > left ? left : v.y);
  s.start = v.z < 0 ? 0 : v.z;
  return s;
}

// A batch's spans cut into chunks of `chunk` rows, one after the other in the order of their rows, each span
// from a chunk of its own: a span's first chunk, and how many there can be.
__device__ __forceinline__ int first_chunk(const int* __restrict__ spans, int slots, int slot, int rows, int chunk) {
  const Span mine = span_of(spans, slot, rows);
  int rank = 0;
  for (int i = 0; i < slots; ++i) {
    const Span s = span_of(spans, i, rows);
    rank += s.rows > 0 && s.row0 < mine.row0;
  }
  return mine.row0 / chunk + rank;
}
__host__ __device__ inline long chunks_of(int rows, int slots, int chunk) { return (rows + chunk - 1) / chunk + slots; }

// A barrier for what the block exchanges through LDS: waits for its LDS traffic, not (as __syncthreads does)
// for the loads from memory in flight.
__device__ __forceinline__ void block_barrier_lds() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

}  // namespace iron
