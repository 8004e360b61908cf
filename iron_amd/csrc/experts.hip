// A feed-forward of routed experts: each row's `top` experts by its router's logits, shares by a softmax over the chosen
// ones -- or by a softmax over all, chosen by scores with corrections and shared by those without -- and the shares' sum of
// what they make of the row, down (act(gate h) * (up h)).  Ids behind the experts' last are identities: they hand on the row.
//
//   router:   float32 logits, a row a block
//   pairs:    a (row, chosen expert) at a time, or all of an expert's at once, the weights' rows dealt to waves (few rows; either type)
//   grouped:  pairs dealt to their experts, each expert's padded to whole row tiles, two grouped products and a row's sum (bf16)
#include "../../include/iron_hip.h"
#include "grouped.h"
#include "row_products.h"
#include "router.h"

namespace iron {

template <typename T, int VEC, int NW>
__global__ __launch_bounds__(NW * 64) void router_kernel(const T* __restrict__ h, const bf16_t* __restrict__ w, const bf16_t* __restrict__ bias,
                                                     const bf16_t* __restrict__ correction, int scored, int* __restrict__ ids,
                                                     float* __restrict__ shares, int rows, int cols, int experts, int top,
                                                     const int* __restrict__ valid) {
  __shared__ float z[ROUTER_MAX], by[ROUTER_MAX];
  const int row = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  if (row >= bound_or(valid, rows)) return;
  const T* hr = h + (size_t)row * cols;
  constexpr int AT_ONCE = NW >= 16 ? 2 : 4;   // experts whose weights meet a piece of the row
  for (int e0 = wave; e0 < experts; e0 += NW * AT_ONCE) {
    float sum[AT_ONCE];
    const bf16_t* wr[AT_ONCE];
#pragma unroll
    for (int k = 0; k < AT_ONCE; ++k) {
      sum[k] = 0.f;
      wr[k] = w + (size_t)min(e0 + k * NW, experts - 1) * cols;
    }
#pragma unroll 4
    for (int c = lane * VEC; c < cols; c += 64 * VEC) {
      float a[VEC];
      load_vec<VEC>(hr + c, a);
#pragma unroll
      for (int k = 0; k < AT_ONCE; ++k) {
        float b[VEC];
        load_vec<VEC>(wr[k] + c, b);
#pragma unroll
        for (int j = 0; j < VEC; ++j) sum[k] = fmaf(a[j], b[j], sum[k]);
      }
    }
#pragma unroll
    for (int k = 0; k < AT_ONCE; ++k) {
      const float total = wave_sum(sum[k]);
      const int e = e0 + k * NW;
      if (lane == 0 && e < experts) z[e] = total + (bias != nullptr ? bf16_to_f32(bias[e]) : 0.f);
    }
  }
  __syncthreads();
  if (wave != 0) return;
  if (scored) choose_scored(z, by, correction, experts, top, ids + (size_t)row * top, shares + (size_t)row * top);
  else choose(z, experts, top, ids + (size_t)row * top, shares + (size_t)row * top);
}

__device__ __forceinline__ float act_exact(int kind, float g) {
  return kind == 3 ? fmaxf(g, 0.f) : (kind == 1 ? g / (1.f + expf(-g)) : gelu_tanh_f32(g));
}

// VEC elements of a row and of a weight's row, and their product: bf16 pairs as they were loaded, or floats.
template <typename T, int VEC>
struct Run {
  float f[VEC];
  template <typename U>
  __device__ __forceinline__ void load(const U* __restrict__ p) { load_vec<VEC>(p, f); }
  template <typename U>
  __device__ __forceinline__ void stream(const U* __restrict__ p) { load_vec<VEC>(p, f); }
};
template <>
struct Run<bf16_t, 8> {
  uint4 v;
  __device__ __forceinline__ void load(const bf16_t* __restrict__ p) { v = *reinterpret_cast<const uint4*>(p); }
  __device__ __forceinline__ void stream(const bf16_t* __restrict__ p) { v = load_stream(reinterpret_cast<const uint4*>(p)); }
};
template <typename T, int VEC>
__device__ __forceinline__ float add_product(const Run<T, VEC>& a, const Run<T, VEC>& b, float sum) {
  if constexpr (sizeof(T) == 2 && VEC == 8) {
    const uint4 x[1] = {a.v}, y[1] = {b.v};
    return sum + dot_row<1>(x, y);
  } else {
#pragma unroll
    for (int j = 0; j < VEC; ++j) sum = fmaf(a.f[j], b.f[j], sum);
    return sum;
  }
}

// a[pair] = act(gate_e h) * (up_e h): a wave a row of each matrix.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void expert_pairs_kernel(const T* __restrict__ h, const bf16_t* __restrict__ gate, const bf16_t* __restrict__ up,
                                                           const int* __restrict__ ids, T* __restrict__ a, int rows, int cols, int ff, int experts,
                                                           int identity, int top, int kind, const int* __restrict__ valid) {
  const int lane = threadIdx.x & 63, f = blockIdx.x * 4 + (threadIdx.x >> 6), pairs = f < ff ? bound_or(valid, rows) * top : 0;
  for (int pair = blockIdx.y; pair < pairs; pair += gridDim.y) {
    const int e = expert_of(ids[pair], experts, identity);
    if (e < 0) continue;
    const size_t at = ((size_t)e * ff + f) * cols;
    const T* hr = h + (size_t)(pair / top) * cols;
    float g = 0.f, u = 0.f;
#pragma unroll 4
    for (int c = lane * VEC; c < cols; c += 64 * VEC) {
      Run<T, VEC> x, b, d;
      b.stream(gate + at + c);
      d.stream(up + at + c);
      x.load(hr + c);
      g = add_product(b, x, g);
      u = add_product(d, x, u);
    }
    g = wave_sum(g);
    u = wave_sum(u);
    if (lane == 0) store_one(a + (size_t)pair * ff + f, act_exact(kind, g) * u);
  }
}

// The same, a block one expert: its weights' rows meet all of its pairs, four at a time (several rows of a step).
constexpr int SHARED_PAIRS = 4096;
template <typename T, int VEC, int N>
__device__ __forceinline__ void expert_rows(const T* __restrict__ h, const bf16_t* __restrict__ gr, const bf16_t* __restrict__ ur,
                                            const int* __restrict__ list, T* __restrict__ a, int f, int cols, int ff, int top, int kind) {
  const int lane = threadIdx.x & 63;
  const T* hr[N];
  float g[N], u[N];
#pragma unroll
  for (int p = 0; p < N; ++p) {
    hr[p] = h + (size_t)(__builtin_amdgcn_readfirstlane(list[p]) / top) * cols;
    g[p] = u[p] = 0.f;
  }
#pragma unroll 2
  for (int c = lane * VEC; c < cols; c += 64 * VEC) {
    Run<T, VEC> x[N], b, d;
    b.load(gr + c);
    d.load(ur + c);
#pragma unroll
    for (int p = 0; p < N; ++p) x[p].load(hr[p] + c);
#pragma unroll
    for (int p = 0; p < N; ++p) {
      g[p] = add_product(b, x[p], g[p]);
      u[p] = add_product(d, x[p], u[p]);
    }
  }
#pragma unroll
  for (int p = 0; p < N; ++p) {
    const float gs = wave_sum(g[p]), us = wave_sum(u[p]);
    if (lane == 0) store_one(a + (size_t)list[p] * ff + f, act_exact(kind, gs) * us);
  }
}
template <typename T, int VEC>
__global__ __launch_bounds__(256) void expert_shared_kernel(const T* __restrict__ h, const bf16_t* __restrict__ gate, const bf16_t* __restrict__ up,
                                                            const int* __restrict__ ids, T* __restrict__ a, int rows, int cols, int ff,
                                                            int experts, int identity, int top, int kind, const int* __restrict__ valid) {
  __shared__ int list[SHARED_PAIRS], held;
  const int e = blockIdx.y, f = blockIdx.x * 4 + (threadIdx.x >> 6), pairs = bound_or(valid, rows) * top;
  if (threadIdx.x == 0) held = 0;
  __syncthreads();
  for (int p = threadIdx.x; p < pairs; p += 256)
    if (expert_of(ids[p], experts, identity) == e) list[atomicAdd(&held, 1)] = p;
  __syncthreads();
  const int n = held;
  if (n == 0 || f >= ff) return;
  const size_t at = ((size_t)e * ff + f) * cols;
  int p = 0;
  for (; p + 4 <= n; p += 4) expert_rows<T, VEC, 4>(h, gate + at, up + at, list + p, a, f, cols, ff, top, kind);
  if (n - p == 3) expert_rows<T, VEC, 3>(h, gate + at, up + at, list + p, a, f, cols, ff, top, kind);
  else if (n - p == 2) expert_rows<T, VEC, 2>(h, gate + at, up + at, list + p, a, f, cols, ff, top, kind);
  else if (n - p == 1) expert_rows<T, VEC, 1>(h, gate + at, up + at, list + p, a, f, cols, ff, top, kind);
}

// y[row] = sum over its experts of share * down_e a[pair]: a block PER rows of down, a wave every fourth of the experts.
template <typename T, int VEC, int PER>
__global__ __launch_bounds__(256) void expert_sums_kernel(const T* __restrict__ a, const bf16_t* __restrict__ down, const int* __restrict__ ids,
                                                          const float* __restrict__ shares, const T* __restrict__ h, T* __restrict__ y, int rows,
                                                          int cols, int ff, int experts, int identity, int top, const int* __restrict__ valid) {
  __shared__ float red[4][PER];
  const int row = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c0 = blockIdx.x * PER;
  if (row >= bound_or(valid, rows)) return;
  float sum[PER];
#pragma unroll
  for (int p = 0; p < PER; ++p) sum[p] = 0.f;
  for (int k = wave; k < top; k += 4) {
    const int pair = row * top + k, e = expert_of(ids[pair], experts, identity);
    const float share = shares[pair];
    if (e < 0) {
      if (lane == 0)
#pragma unroll
        for (int p = 0; p < PER; ++p) sum[p] = fmaf(share, load_one(h + (size_t)row * cols + min(c0 + p, cols - 1)), sum[p]);
      continue;
    }
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
      Run<T, VEC> x, b[PER];
#pragma unroll
      for (int p = 0; p < PER; ++p) b[p].load(dr[p] + f);
      x.load(ar + f);
#pragma unroll
      for (int p = 0; p < PER; ++p) part[p] = add_product(b[p], x, part[p]);
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
                                                           int* __restrict__ place, int* __restrict__ rows_of, int rows, int experts, int identity,
                                                           int top, int most, const int* __restrict__ valid) {
  __shared__ int held[ROUTER_MAX], first[ROUTER_MAX], scan[2][ROUTER_MAX];
  const int t = threadIdx.x, pairs = bound_or(valid, rows) * top;
  held[t] = 0;
  for (int i = t; i < most * 128; i += 1024) rows_of[i] = 0;   // a tile's places past its expert's pairs
  __syncthreads();
  for (int p = t; p < pairs; p += 1024) {
    const int e = expert_of(ids[p], experts, identity);
    if (e >= 0) atomicAdd(&held[e], 1);
  }
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
    const int e = expert_of(ids[p], experts, identity);
    place[p] = -1;
    if (e < 0) continue;
    const int to = min(atomicAdd(&first[e], 1), most * 128 - 1);
    place[p] = to;
    rows_of[to] = p / top;
  }
}

// y[row] = sum over its pairs of share * what the pair's expert left.
__global__ __launch_bounds__(256) void expert_gather_kernel(const bf16_t* __restrict__ outs, const int* __restrict__ place,
                                                            const float* __restrict__ shares, const bf16_t* __restrict__ h, bf16_t* __restrict__ y,
                                                            int rows, int cols, int top, const int* __restrict__ valid) {
  const int row = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 8;
  if (row >= bound_or(valid, rows) || c >= cols) return;
  float sum[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) sum[j] = 0.f;
#pragma unroll 4
  for (int k = 0; k < top; ++k) {
    float f[8];
    const int from = place[row * top + k];
    load_vec<8>((from < 0 ? h + (size_t)row * cols : outs + (size_t)from * cols) + c, f);
    const float share = shares[row * top + k];
#pragma unroll
    for (int j = 0; j < 8; ++j) sum[j] = fmaf(share, f[j], sum[j]);
  }
  store_vec<8>(y + (size_t)row * cols + c, sum);
}

// One row: stream[c] += out_c . made + what its experts make of column c: a block a column, its row of `out` and its experts' rows of
// down as one run of 16-byte pieces.
constexpr int TAIL_EXPERTS = 64;
template <int CH>
__global__ __launch_bounds__(256) void expert_tail_kernel(const bf16_t* __restrict__ out, const bf16_t* __restrict__ made, int inner,
                                                          const bf16_t* __restrict__ down, const bf16_t* __restrict__ acts,
                                                          const int* __restrict__ ids, const float* __restrict__ shares,
                                                          const bf16_t* __restrict__ h, float* __restrict__ stream, int cols, int ff, int experts,
                                                          int identity, int top) {
  __shared__ float red[2][4];
  const int c = blockIdx.x, t = threadIdx.x, lane = t & 63, wave = t >> 6, first = inner / 8, each = ff / 8, pieces = first + top * each;
  const float held = stream[c], own = bf16_to_f32(h[c]);
  const float share_own = lane < top ? shares[lane] : 0.f;
  const int id_own = lane < top ? expert_of(ids[lane], experts, identity) : 0;
  uint4 w[CH], x[CH];
  float by[CH];
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int p = min(t + 256 * i, pieces - 1), k = p < first ? 0 : (p - first) / each, e = __shfl(id_own, k, 64);
    const int at = p < first ? p : (p - first) - k * each;
    const float share = __shfl(share_own, k, 64);
    by[i] = p < first ? 1.f : share;
    if (t + 256 * i >= pieces || (p >= first && e < 0)) by[i] = 0.f;
    w[i] = load_stream(reinterpret_cast<const uint4*>(p < first ? out + (size_t)c * inner : down + ((size_t)max(e, 0) * cols + c) * ff) + at);
    x[i] = reinterpret_cast<const uint4*>(p < first ? made : acts + (size_t)k * ff)[at];
  }
  float mixed = 0.f, routed = 0.f;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const uint4 a[1] = {w[i]}, b[1] = {x[i]};
    const float part = by[i] == 0.f ? 0.f : dot_row<1>(a, b);   // (an identity's activated row is nobody's)
    if (t + 256 * i < first) mixed += part;
    else routed = fmaf(by[i], part, routed);
  }
  if (wave == 0 && lane < top && id_own < 0) routed = fmaf(share_own, own, routed);
  mixed = wave_sum(mixed);
  routed = wave_sum(routed);
  if (lane == 0) {
    red[0][wave] = mixed;
    red[1][wave] = routed;
  }
  __syncthreads();
  if (t == 0)
    stream[c] = held + (round_bf16(red[0][0] + red[0][1] + red[0][2] + red[0][3]) + round_bf16(red[1][0] + red[1][1] + red[1][2] + red[1][3]));
}

// Rows from which a portion's pairs are grouped.
static bool grouped_pays(int rows, int cols, int ff, int is_float) { return !is_float && rows >= 64 && cols % 64 == 0 && ff % 64 == 0; }

}  // namespace iron

using namespace iron;

extern "C" int iron_router(const void* h, const uint16_t* w, const uint16_t* bias, const uint16_t* correction, int scored, int* ids, float* shares,
                           int rows, int cols, int experts, int top, int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(h && w && ids && shares && (scored || correction == nullptr), "router: null operand, or corrections of no scores");
  IRON_REQUIRE(rows > 0 && cols > 0 && experts > 0 && experts <= ROUTER_MAX, "router: rows (%d), cols (%d) positive, experts (%d) from 1 to %d",
               rows, cols, experts, ROUTER_MAX);
  IRON_REQUIRE(top > 0 && top <= experts && top <= 64, "router: top (%d) from 1 to the experts (%d), 64 at most", top, experts);
  const bool vec = cols % 8 == 0 && (((uintptr_t)h | (uintptr_t)w) & 15) == 0;
  // Few rows: a wave an expert, so that a row's weights are all on their way at once.
#define IRON_ROUTER(T, VEC)                                                                                                                \
  {                                                                                                                                        \
    if (rows < 256)                                                                                                                        \
      hipLaunchKernelGGL((router_kernel<T, VEC, 16>), dim3(rows), dim3(1024), 0, (hipStream_t)stream, (const T*)h, w, bias, correction, scored, ids, shares,   \
                         rows, cols, experts, top, valid);                                                                                 \
    else                                                                                                                                   \
      hipLaunchKernelGGL((router_kernel<T, VEC, 4>), dim3(rows), dim3(256), 0, (hipStream_t)stream, (const T*)h, w, bias, correction, scored, ids, shares,     \
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
                            void* y, void* workspace, int rows, int cols, int ff, int experts, int identity, int top, int activation, int is_float,
                            const int* valid, void* stream) {
  IRON_REQUIRE(h && gate && up && down && ids && shares && y && workspace, "experts: null operand");
  IRON_REQUIRE(rows > 0 && cols > 0 && ff > 0 && experts > 0 && identity >= 0 && top > 0 && top <= experts + identity,
               "experts: sizes must be positive, top (%d) of %d experts and %d identities", top, experts, identity);
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
    hipLaunchKernelGGL(expert_plan_kernel, dim3(1), dim3(1024), 0, s, ids, count, which, place, rows_of, rows, experts, identity, top, p.most, valid);
    if (int e = launch_grouped_pair((const bf16_t*)h, gate, up, acts, ff, cols, g, rows_of, activation, s)) return e;
    if (int e = launch_grouped(acts, down, outs, cols, ff, g, s)) return e;
    hipLaunchKernelGGL(expert_gather_kernel, dim3((cols + 2047) / 2048, rows), dim3(256), 0, s, outs, place, shares, (const bf16_t*)h, (bf16_t*)y, rows, cols, top, valid);
    IRON_LAUNCH_CHECK();
  }
  IRON_REQUIRE(rows <= 65535 && (long)rows * top <= (1 << 30), "experts: %d rows of %d experts exceed the grid's y extent", rows, top);
  const int pairs_y = rows * top < 65535 ? rows * top : 65535;
  const bool vec = cols % 8 == 0 && ff % 8 == 0 &&
                   (((uintptr_t)h | (uintptr_t)gate | (uintptr_t)up | (uintptr_t)down | (uintptr_t)workspace | (uintptr_t)y) & 15) == 0;
#define IRON_PAIRS(T, VEC)                                                                                                                    \
  {                                                                                                                                           \
    if (rows > 1 && rows * top <= SHARED_PAIRS && experts <= 65535)                                                                           \
      hipLaunchKernelGGL((expert_shared_kernel<T, VEC>), dim3((ff + 3) / 4, experts), dim3(256), 0, s, (const T*)h, gate, up, ids,            \
                         (T*)workspace, rows, cols, ff, experts, identity, top, activation, valid);                                                     \
    else                                                                                                                                      \
      hipLaunchKernelGGL((expert_pairs_kernel<T, VEC>), dim3((ff + 3) / 4, pairs_y), dim3(256), 0, s, (const T*)h, gate, up, ids,          \
                         (T*)workspace, rows, cols, ff, experts, identity, top, activation, valid);                                                     \
    hipLaunchKernelGGL((expert_sums_kernel<T, VEC, 2>), dim3((cols + 1) / 2, rows), dim3(256), 0, s, (const T*)workspace, down, ids, shares, \
                       (const T*)h, (T*)y, rows, cols, ff, experts, identity, top, valid);                                                                           \
  }
  if (is_float) { if (vec) IRON_PAIRS(float, 8) else IRON_PAIRS(float, 1) }
  else { if (vec) IRON_PAIRS(bf16_t, 8) else IRON_PAIRS(bf16_t, 1) }
#undef IRON_PAIRS
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_experts_tail_bf16(const uint16_t* h, const uint16_t* gate, const uint16_t* up, const uint16_t* down, const int* ids, const float* shares,
                                      const uint16_t* out, const uint16_t* made, float* stream_row, void* workspace, int cols, int ff, int inner,
                                      int experts, int identity, int top, int activation, void* stream) {
  IRON_REQUIRE(h && gate && up && down && ids && shares && out && made && stream_row && workspace, "experts_tail: null operand");
  IRON_REQUIRE(cols > 0 && ff > 0 && inner > 0 && experts > 0 && identity >= 0 && top > 0 && top <= experts + identity && top <= TAIL_EXPERTS,
               "experts_tail: sizes must be positive, top (%d) of %d experts and %d identities, at most %d", top, experts, identity, TAIL_EXPERTS);
  IRON_REQUIRE(activation >= 1 && activation <= 3, "experts_tail: activation (%d) is 1 (SiLU), 2 (GELU, tanh form) or 3 (ReLU)", activation);
  IRON_REQUIRE(cols % 8 == 0 && ff % 8 == 0 && inner % 8 == 0 &&
                   (((uintptr_t)h | (uintptr_t)gate | (uintptr_t)up | (uintptr_t)down | (uintptr_t)out | (uintptr_t)made | (uintptr_t)workspace) & 15) == 0,
               "experts_tail: rows (%d, %d, %d) of whole 16-byte pieces, 16-byte aligned", cols, ff, inner);
  const int pieces = inner / 8 + top * (ff / 8);
  IRON_REQUIRE(pieces <= 16 * 256, "experts_tail: a column's weights (%d) exceed %d pieces", pieces, 16 * 256);
  hipStream_t s = (hipStream_t)stream;
  bf16_t* acts = (bf16_t*)workspace;
  hipLaunchKernelGGL((expert_pairs_kernel<bf16_t, 8>), dim3((ff + 3) / 4, top), dim3(256), 0, s, h, gate, up, ids, acts, 1, cols, ff, experts, identity, top,
                     activation, nullptr);
#define IRON_TAIL(CH) \
  hipLaunchKernelGGL((expert_tail_kernel<CH>), dim3(cols), dim3(256), 0, s, out, made, inner, down, acts, ids, shares, h, stream_row, cols, ff, experts, identity, top)
  switch ((pieces + 255) / 256) {
    case 1: case 2: IRON_TAIL(2); break;
    case 3: IRON_TAIL(3); break;
    case 4: IRON_TAIL(4); break;
    case 5: IRON_TAIL(5); break;
    case 6: IRON_TAIL(6); break;
    case 7: case 8: IRON_TAIL(8); break;
    case 9: case 10: IRON_TAIL(10); break;
    case 11: case 12: IRON_TAIL(12); break;
    default: IRON_TAIL(16);
  }
#undef IRON_TAIL
  IRON_LAUNCH_CHECK();
}
