// A feed-forward of routed experts: each row's `top` experts by its router's logits, shares by a softmax over the chosen
// ones, and the shares' sum of what they make of the row, down (act(gate h) * (up h)).
//
//   router:   float32 logits, a row a block
//   pairs:    a (row, chosen expert) at a time, the weights' rows dealt to waves (few rows; either type)
//   grouped:  pairs dealt to their experts, each expert's padded to whole row tiles, two grouped products and a row's sum (bf16)
#include "../../include/iron_hip.h"
#include "grouped.h"
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

template <typename T, int VEC, int NW>
__global__ __launch_bounds__(NW * 64) void router_kernel(const T* __restrict__ h, const bf16_t* __restrict__ w, const bf16_t* __restrict__ bias,
                                                     int* __restrict__ ids, float* __restrict__ shares, int rows, int cols, int experts,
                                                     int top, const int* __restrict__ valid) {
  __shared__ float z[ROUTER_MAX];
  const int row = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  if (row >= bound_or(valid, rows)) return;
  const T* hr = h + (size_t)row * cols;
  for (int e = wave; e < experts; e += NW) {
    const bf16_t* wr = w + (size_t)e * cols;
    float sum = 0.f;
#pragma unroll 4
    for (int c = lane * VEC; c < cols; c += 64 * VEC) {
      float a[VEC], b[VEC];
      load_vec<VEC>(hr + c, a);
      load_vec<VEC>(wr + c, b);
#pragma unroll
      for (int j = 0; j < VEC; ++j) sum = fmaf(a[j], b[j], sum);
    }
    sum = wave_sum(sum);
    if (lane == 0) z[e] = sum + bf16_to_f32(bias[e]);
  }
  __syncthreads();
  if (wave == 0) choose(z, experts, top, ids + (size_t)row * top, shares + (size_t)row * top);
}

__device__ __forceinline__ float act_exact(int kind, float g) {
  return kind == 3 ? fmaxf(g, 0.f) : (kind == 1 ? g / (1.f + expf(-g)) : gelu_tanh_f32(g));
}

// a[pair] = act(gate_e h) * (up_e h): a wave PER rows of each matrix.
template <typename T, int VEC, int PER>
__global__ __launch_bounds__(256) void expert_pairs_kernel(const T* __restrict__ h, const bf16_t* __restrict__ gate, const bf16_t* __restrict__ up,
                                                           const int* __restrict__ ids, T* __restrict__ a, int rows, int cols, int ff, int experts,
                                                           int top, int kind, const int* __restrict__ valid) {
  const int pair = blockIdx.y, lane = threadIdx.x & 63, f0 = (blockIdx.x * 4 + (threadIdx.x >> 6)) * PER;
  if (pair / top >= bound_or(valid, rows) || f0 >= ff) return;
  const int e = min(max(ids[pair], 0), experts - 1);
  const T* hr = h + (size_t)(pair / top) * cols;
  float g[PER], u[PER];
#pragma unroll
  for (int p = 0; p < PER; ++p) g[p] = u[p] = 0.f;
  const bf16_t *gr[PER], *ur[PER];
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const size_t at = ((size_t)e * ff + min(f0 + p, ff - 1)) * cols;
    gr[p] = gate + at;
    ur[p] = up + at;
  }
#pragma unroll 4
  for (int c = lane * VEC; c < cols; c += 64 * VEC) {
    float x[VEC], b[PER][VEC], d[PER][VEC];
    load_vec<VEC>(hr + c, x);
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      load_vec<VEC>(gr[p] + c, b[p]);
      load_vec<VEC>(ur[p] + c, d[p]);
    }
#pragma unroll
    for (int p = 0; p < PER; ++p)
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        g[p] = fmaf(x[j], b[p][j], g[p]);
        u[p] = fmaf(x[j], d[p][j], u[p]);
      }
  }
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const float gs = wave_sum(g[p]), us = wave_sum(u[p]);
    if (lane == 0 && f0 + p < ff) store_one(a + (size_t)pair * ff + f0 + p, act_exact(kind, gs) * us);
  }
}

// y[row] = sum over its experts of share * down_e a[pair]: a block PER rows of down, a wave every fourth of the experts.
template <typename T, int VEC, int PER>
__global__ __launch_bounds__(256) void expert_sums_kernel(const T* __restrict__ a, const bf16_t* __restrict__ down, const int* __restrict__ ids,
                                                          const float* __restrict__ shares, T* __restrict__ y, int rows, int cols, int ff,
                                                          int experts, int top, const int* __restrict__ valid) {
  __shared__ float red[4][PER];
  const int row = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c0 = blockIdx.x * PER;
  if (row >= bound_or(valid, rows)) return;
  float sum[PER];
#pragma unroll
  for (int p = 0; p < PER; ++p) sum[p] = 0.f;
  for (int k = wave; k < top; k += 4) {
    const int pair = row * top + k, e = min(max(ids[pair], 0), experts - 1);
    const float share = shares[pair];
    const T* ar = a + (size_t)pair * ff;
    const bf16_t* dr[PER];
    float part[PER];
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      part[p] = 0.f;
      dr[p] = down + ((size_t)e * cols + min(c0 + p, cols - 1)) * ff;
    }
#pragma unroll 4
    for (int f = lane * VEC; f < ff; f += 64 * VEC) {
      float x[VEC], b[PER][VEC];
#pragma unroll
      for (int p = 0; p < PER; ++p) load_vec<VEC>(dr[p] + f, b[p]);
      load_vec<VEC>(ar + f, x);
#pragma unroll
      for (int p = 0; p < PER; ++p)
#pragma unroll
        for (int j = 0; j < VEC; ++j) part[p] = fmaf(x[j], b[p][j], part[p]);
    }
#pragma unroll
    for (int p = 0; p < PER; ++p) sum[p] = fmaf(share, part[p], sum[p]);
  }
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const float v = wave_sum(sum[p]);
    if (lane == 0) red[wave][p] = v;
  }
  __syncthreads();
  const int p = threadIdx.x;
  if (p < PER && c0 + p < cols) store_one(y + (size_t)row * cols + c0 + p, red[0][p] + red[1][p] + red[2][p] + red[3][p]);
}

// ------------------------------------------------------------- many rows
// A call's workspace behind these offsets (in bytes): what the plan leaves, the activated rows, the experts' rows.
struct GroupedPlan {
  int most;                    // row tiles there can be
  size_t which, place, rows, acts, outs, bytes;
  GroupedPlan(int pairs, int experts, int cols, int ff) {
    auto up = [](size_t n) { return (n + 255) & ~(size_t)255; };
    most = pairs / 128 + (pairs < experts ? pairs : experts);
    which = 256;                                     // (the count stands first)
    place = which + up((size_t)most * 4);            // a pair's place among the sorted
    rows = place + up((size_t)pairs * 4);            // a place's row
    acts = rows + up((size_t)most * 128 * 4);
    outs = acts + up((size_t)most * 128 * ff * 2);
    bytes = outs + up((size_t)most * 128 * cols * 2);
  }
};

// One block: how many pairs each expert has, where its tiles begin, and every pair's place.
__global__ __launch_bounds__(1024) void expert_plan_kernel(const int* __restrict__ ids, int* __restrict__ count, int* __restrict__ which,
                                                           int* __restrict__ place, int* __restrict__ rows_of, int rows, int experts, int top,
                                                           int most, const int* __restrict__ valid) {
  __shared__ int held[ROUTER_MAX], first[ROUTER_MAX], scan[2][ROUTER_MAX];
  const int t = threadIdx.x, pairs = bound_or(valid, rows) * top;
  held[t] = 0;
  for (int i = t; i < most * 128; i += 1024) rows_of[i] = 0;   // a tile's places past its expert's pairs
  __syncthreads();
  for (int p = t; p < pairs; p += 1024) atomicAdd(&held[min(max(ids[p], 0), experts - 1)], 1);
  __syncthreads();
  const int tiles = (held[t] + 127) / 128;
  scan[0][t] = tiles;
  __syncthreads();
  int at = 0;
  for (int d = 1; d < ROUTER_MAX; d <<= 1, at ^= 1) {
    scan[at ^ 1][t] = scan[at][t] + (t >= d ? scan[at][t - d] : 0);
    __syncthreads();
  }
  const int begin = scan[at][t] - tiles;
  first[t] = begin * 128;
  for (int i = 0; i < tiles; ++i)
    if (begin + i < most) which[begin + i] = t;
  if (t == 0) *count = min(scan[at][ROUTER_MAX - 1], most);
  __syncthreads();
  for (int p = t; p < pairs; p += 1024) {
    const int to = min(atomicAdd(&first[min(max(ids[p], 0), experts - 1)], 1), most * 128 - 1);
    place[p] = to;
    rows_of[to] = p / top;
  }
}

// y[row] = sum over its pairs of share * what the pair's expert left.
__global__ __launch_bounds__(256) void expert_gather_kernel(const bf16_t* __restrict__ outs, const int* __restrict__ place,
                                                            const float* __restrict__ shares, bf16_t* __restrict__ y, int rows, int cols,
                                                            int top, const int* __restrict__ valid) {
  const int row = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 8;
  if (row >= bound_or(valid, rows) || c >= cols) return;
  float sum[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) sum[j] = 0.f;
#pragma unroll 4
  for (int k = 0; k < top; ++k) {
    float f[8];
    load_vec<8>(outs + (size_t)place[row * top + k] * cols + c, f);
    const float share = shares[row * top + k];
#pragma unroll
    for (int j = 0; j < 8; ++j) sum[j] = fmaf(share, f[j], sum[j]);
  }
  store_vec<8>(y + (size_t)row * cols + c, sum);
}

// Rows from which a portion's pairs are grouped.
static bool grouped_pays(int rows, int cols, int ff, int is_float) { return !is_float && rows >= 64 && cols % 64 == 0 && ff % 64 == 0; }

}  // namespace iron

using namespace iron;

extern "C" int iron_router(const void* h, const uint16_t* w, const uint16_t* bias, int* ids, float* shares, int rows, int cols, int experts,
                           int top, int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(h && w && bias && ids && shares, "router: null operand");
  IRON_REQUIRE(rows > 0 && cols > 0 && experts > 0 && experts <= ROUTER_MAX, "router: rows (%d), cols (%d) positive, experts (%d) from 1 to %d",
               rows, cols, experts, ROUTER_MAX);
  IRON_REQUIRE(top > 0 && top <= experts && top <= 64, "router: top (%d) from 1 to the experts (%d), 64 at most", top, experts);
  const bool vec = cols % 8 == 0 && (((uintptr_t)h | (uintptr_t)w) & 15) == 0;
  // Few rows: a wave an expert, so that a row's weights are all on their way at once.
#define IRON_ROUTER(T, VEC)                                                                                                                \
  {                                                                                                                                        \
    if (rows < 256)                                                                                                                        \
      hipLaunchKernelGGL((router_kernel<T, VEC, 16>), dim3(rows), dim3(1024), 0, (hipStream_t)stream, (const T*)h, w, bias, ids, shares,   \
                         rows, cols, experts, top, valid);                                                                                 \
    else                                                                                                                                   \
      hipLaunchKernelGGL((router_kernel<T, VEC, 4>), dim3(rows), dim3(256), 0, (hipStream_t)stream, (const T*)h, w, bias, ids, shares,     \
                         rows, cols, experts, top, valid);                                                                                 \
  }
  if (is_float) { if (vec) IRON_ROUTER(float, 8) else IRON_ROUTER(float, 1) }
  else { if (vec) IRON_ROUTER(bf16_t, 8) else IRON_ROUTER(bf16_t, 1) }
#undef IRON_ROUTER
  IRON_LAUNCH_CHECK();
}

extern "C" int64_t iron_experts_workspace_bytes(int rows, int cols, int ff, int experts, int top, int is_float) {
  if (grouped_pays(rows, cols, ff, is_float)) return (int64_t)GroupedPlan(rows * top, experts, cols, ff).bytes;
  return (int64_t)rows * top * ff * (is_float ? 4 : 2);
}

extern "C" int iron_experts(const void* h, const uint16_t* gate, const uint16_t* up, const uint16_t* down, const int* ids, const float* shares,
                            void* y, void* workspace, int rows, int cols, int ff, int experts, int top, int activation, int is_float,
                            const int* valid, void* stream) {
  IRON_REQUIRE(h && gate && up && down && ids && shares && y && workspace, "experts: null operand");
  IRON_REQUIRE(rows > 0 && cols > 0 && ff > 0 && experts > 0 && top > 0 && top <= experts, "experts: sizes must be positive, top (%d) of %d experts",
               top, experts);
  IRON_REQUIRE(activation >= 1 && activation <= 3, "experts: activation (%d) is 1 (SiLU), 2 (GELU, tanh form) or 3 (ReLU)", activation);
  hipStream_t s = (hipStream_t)stream;
  if (grouped_pays(rows, cols, ff, is_float)) {
    IRON_REQUIRE(experts <= ROUTER_MAX && rows <= 65535 && (long)rows * top <= (1 << 24) && (long)rows * cols < (1L << 30),
                 "experts: %d rows, %d of %d experts", rows, top, experts);
    IRON_REQUIRE((((uintptr_t)h | (uintptr_t)gate | (uintptr_t)up | (uintptr_t)down | (uintptr_t)workspace | (uintptr_t)y) & 15) == 0,
                 "experts: operands must be 16-byte aligned");
    const GroupedPlan p(rows * top, experts, cols, ff);
    char* w = (char*)workspace;
    int *count = (int*)w, *which = (int*)(w + p.which), *place = (int*)(w + p.place), *rows_of = (int*)(w + p.rows);
    const GroupedTiles g{count, which, p.most};
    bf16_t *acts = (bf16_t*)(w + p.acts), *outs = (bf16_t*)(w + p.outs);
    hipLaunchKernelGGL(expert_plan_kernel, dim3(1), dim3(1024), 0, s, ids, count, which, place, rows_of, rows, experts, top, p.most, valid);
    if (int e = launch_grouped_pair((const bf16_t*)h, gate, up, acts, ff, cols, g, rows_of, activation, s)) return e;
    if (int e = launch_grouped(acts, down, outs, cols, ff, g, s)) return e;
    hipLaunchKernelGGL(expert_gather_kernel, dim3((cols + 2047) / 2048, rows), dim3(256), 0, s, outs, place, shares, (bf16_t*)y, rows, cols, top, valid);
    IRON_LAUNCH_CHECK();
  }
  IRON_REQUIRE((long)rows * top <= 65535, "experts: %d rows of %d experts exceed the grid's y extent", rows, top);
  const bool vec = cols % 8 == 0 && ff % 8 == 0 &&
                   (((uintptr_t)h | (uintptr_t)gate | (uintptr_t)up | (uintptr_t)down | (uintptr_t)workspace | (uintptr_t)y) & 15) == 0;
#define IRON_PAIRS(T, VEC)                                                                                                                    \
  {                                                                                                                                           \
    hipLaunchKernelGGL((expert_pairs_kernel<T, VEC, 1>), dim3((ff + 3) / 4, rows * top), dim3(256), 0, s, (const T*)h, gate, up, ids,         \
                       (T*)workspace, rows, cols, ff, experts, top, activation, valid);                                                       \
    hipLaunchKernelGGL((expert_sums_kernel<T, VEC, 2>), dim3((cols + 1) / 2, rows), dim3(256), 0, s, (const T*)workspace, down, ids, shares, \
                       (T*)y, rows, cols, ff, experts, top, valid);                                                                           \
  }
  if (is_float) { if (vec) IRON_PAIRS(float, 8) else IRON_PAIRS(float, 1) }
  else { if (vec) IRON_PAIRS(bf16_t, 8) else IRON_PAIRS(bf16_t, 1) }
#undef IRON_PAIRS
  IRON_LAUNCH_CHECK();
}
