// The matrix memory of xLSTM (mLSTM) over a batch of spans: per head S <- keep S + write k v^T and n <- keep n + write k,
// with log gates i and f and everything relative to the largest exponent so far, m: m' = max(f + m, i), keep =
// exp(f + m - m'), write = exp(i - m'); m is 0 ahead of a sequence.  The readings S^T q, n . q and m leave as they are;
// memory_gate makes a head's row of them.
//
// A call's rows are a packed projection [q | k | v | .. | i | f]; n is S's column behind v's last (its v is 1), so a state
// is (dim, vdim + 1) floats a slot and head.  m is kept twice, by a position's parity: the blocks of a launch read the one
// and one of them leaves the other.  A span that starts at position 0 reads no state.
//
// Float32 throughout.  A block holds 16 columns of a head's state: a wave 4 columns, 16 lanes a column, NI consecutive rows
// of it a lane.
#include "../../include/iron_hip.h"
#include "matrix_memory.h"

namespace iron {

struct MemoryShape {
  int rows, stride, slots;
  int heads, dim, vdim;
  int i_at, f_at;                        // columns of the gates in a row; q, k and v lead it
  float cap;
};
struct MemoryIn {
  const bf16_t *i_bias, *f_bias;
  float* state;                          // [slots][heads][dim][vdim + 1]
  float* tops;                           // [slots][2][heads]
  const int* spans;
  float* o;                              // [rows][heads * vdim | heads n . q | heads m]
};

constexpr int MEM_TOKENS = 16, MEM_COLUMNS = 16;

template <int NI>
__device__ __forceinline__ void lds_run(const float* __restrict__ p, float (&f)[NI]) {
  if constexpr (NI % 4 == 0) {
#pragma unroll
    for (int e = 0; e < NI; e += 4) {
      const float4 v = *reinterpret_cast<const float4*>(p + e);
      f[e] = v.x; f[e + 1] = v.y; f[e + 2] = v.z; f[e + 3] = v.w;
    }
  } else {
#pragma unroll
    for (int e = 0; e < NI; ++e) f[e] = p[e];
  }
}

template <typename T, int NI>
__global__ __launch_bounds__(256) void matrix_memory_kernel(const T* __restrict__ x, MemoryIn in, MemoryShape a) {
  constexpr int WIDE = 16 * NI;
  __shared__ __align__(16) float qs[MEM_TOKENS][WIDE], ks[MEM_TOKENS][WIDE];
  __shared__ float vs[MEM_TOKENS][MEM_COLUMNS], os[MEM_TOKENS][MEM_COLUMNS + 1], li[MEM_TOKENS], lf[MEM_TOKENS], tops[MEM_TOKENS];
  const int head = blockIdx.y, slot = blockIdx.z;
  const Span s = span_of(in.spans, slot, a.rows);
  if (s.rows == 0) return;
  const int t = threadIdx.x, ig = t & 15, tok = t >> 4;          // staging: 16 threads a token
  const int col = blockIdx.x * MEM_COLUMNS + (t >> 4);           // scanning: 16 lanes a column
  const int vcol = blockIdx.x * MEM_COLUMNS + ig, cols = a.vdim + 1, qk = a.heads * a.dim;
  const int width = a.heads * a.vdim + 2 * a.heads;
  const float scale = 1.0f / sqrtf((float)a.dim);
  float* sp = in.state + ((size_t)slot * a.heads + head) * a.dim * cols;
  float* mp = in.tops + (size_t)slot * 2 * a.heads + head;
  float S[NI];
#pragma unroll
  for (int e = 0; e < NI; ++e) {
    const int i = ig * NI + e;
    S[e] = (s.start > 0 && i < a.dim && col < cols) ? sp[(size_t)i * cols + col] : 0.f;
  }
  float m = s.start > 0 ? mp[((s.start - 1) & 1) * a.heads] : 0.f;
  for (int base = 0; base < s.rows; base += MEM_TOKENS) {
    const bool live = base + tok < s.rows;
    const T* row = x + (size_t)(s.row0 + min(base + tok, s.rows - 1)) * a.stride;
#pragma unroll
    for (int e = 0; e < NI; ++e) {
      const int i = ig * NI + e;
      const bool inside = live && i < a.dim;
      qs[tok][i] = inside ? load_one(row + head * a.dim + i) * scale : 0.f;
      ks[tok][i] = inside ? load_one(row + qk + head * a.dim + i) : 0.f;
    }
    vs[tok][ig] = live && vcol < a.vdim ? load_one(row + 2 * qk + head * a.vdim + vcol) : (vcol == a.vdim ? 1.f : 0.f);
    if (ig == 0) li[tok] = capped(load_one(row + a.i_at + head) + bf16_to_f32(in.i_bias[head]), a.cap);
    if (ig == 1) lf[tok] = log_sigmoid(capped(load_one(row + a.f_at + head) + bf16_to_f32(in.f_bias[head]), a.cap));
    __syncthreads();
    const int n = min(MEM_TOKENS, s.rows - base);
    for (int p = 0; p < n; ++p) {
      float q[NI], k[NI];
      lds_run<NI>(&qs[p][ig * NI], q);
      lds_run<NI>(&ks[p][ig * NI], k);
      const float i = li[p], f = lf[p], top = fmaxf(f + m, i), keep = expf(f + m - top), write = expf(i - top) * vs[p][t >> 4];
      m = top;
      float acc = 0.f;
#pragma unroll
      for (int e = 0; e < NI; ++e) {
        S[e] = fmaf(keep, S[e], write * k[e]);
        acc = fmaf(q[e], S[e], acc);
      }
      acc = group16_sum(acc);
      if (ig == 0) os[p][t >> 4] = acc;
      if (t == 0) tops[p] = m;
    }
    __syncthreads();
    if (live && vcol < cols) {
      float* to = in.o + (size_t)(s.row0 + base + tok) * width;
      if (vcol < a.vdim) to[head * a.vdim + vcol] = os[tok][ig];
      else {
        to[a.heads * a.vdim + head] = os[tok][ig];
        to[a.heads * a.vdim + a.heads + head] = tops[tok];
      }
    }
  }
#pragma unroll
  for (int e = 0; e < NI; ++e) {
    const int i = ig * NI + e;
    if (i < a.dim && col < cols) sp[(size_t)i * cols + col] = S[e];
  }
  if (t == 0 && blockIdx.x == 0) mp[((s.start + s.rows - 1) & 1) * a.heads] = m;
}

// ------------------------------------------------------------- a head's row
// o = S^T q / (max(|n . q|, exp(-m)) + floor), over its root mean square a head, times gain and sigmoid(gate): a wave a
// row and head.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void memory_gate_kernel(const float* __restrict__ o, const T* __restrict__ gate,
                                                          const bf16_t* __restrict__ gain, T* __restrict__ y, int rows, int heads,
                                                          int dim, int gate_stride, int gate_at, float floor, float eps,
                                                          const int* __restrict__ valid) {
  const int unit = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int row = unit / heads, head = unit - row * heads;
  if (row >= bound_or(valid, rows)) return;
  const float* from = o + (size_t)row * (heads * dim + 2 * heads);
  const float by = 1.0f / (fmaxf(fabsf(from[heads * dim + head]), expf(-from[heads * dim + heads + head])) + floor);
  from += head * dim;
  const T* g = gate + (size_t)row * gate_stride + gate_at + head * dim;
  T* to = y + (size_t)row * heads * dim + head * dim;
  float sum = 0.f;
  for (int c = lane * VEC; c < dim; c += 64 * VEC) {
    float f[VEC];
    load_vec<VEC>(from + c, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j) sum = fmaf(f[j] * by, f[j] * by, sum);
  }
  const float inv = by / sqrtf(wave_sum(sum) / (float)dim + eps);
  for (int c = lane * VEC; c < dim; c += 64 * VEC) {
    float f[VEC], z[VEC], w[VEC];
    load_vec<VEC>(from + c, f);
    load_vec<VEC>(g + c, z);
    load_vec<VEC>(gain + head * dim + c, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] = f[j] * inv * w[j] / (1.0f + expf(-z[j]));
    store_vec<VEC>(to + c, f);
  }
}

}  // namespace iron

using namespace iron;

extern "C" int iron_matrix_memory(const void* x, const uint16_t* i_bias, const uint16_t* f_bias, float* state, float* tops, const int* spans,
                                  float* o, int slots, int rows, int stride, int heads, int dim, int vdim, int i_at, int f_at, float cap,
                                  int is_float, void* stream) {
  IRON_REQUIRE(x && i_bias && f_bias && state && tops && spans && o, "matrix_memory: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0, "matrix_memory: spans must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0 && heads > 0 && heads <= 65535, "matrix_memory: slots (%d), rows (%d), heads (%d) must be positive",
               slots, rows, heads);
  IRON_REQUIRE(dim > 0 && dim <= 512 && vdim > 0, "matrix_memory: dim (%d) from 1 to 512, vdim (%d) positive", dim, vdim);
  const int packed = heads * (2 * dim + vdim);
  IRON_REQUIRE(i_at >= packed && f_at >= packed && i_at + heads <= stride && f_at + heads <= stride,
               "matrix_memory: the gates (%d, %d) lie behind q, k, v (%d) in a row of %d", i_at, f_at, packed, stride);
  IRON_REQUIRE(cap > 0.f, "matrix_memory: a cap (%g) above 0", (double)cap);
  const MemoryIn in{i_bias, f_bias, state, tops, spans, o};
  const MemoryShape a{rows, stride, slots, heads, dim, vdim, i_at, f_at, cap};
  const dim3 grid((vdim + 1 + MEM_COLUMNS - 1) / MEM_COLUMNS, heads, slots);
  hipStream_t s = (hipStream_t)stream;
#define IRON_MEMORY(NI)                                                                                                        \
  {                                                                                                                            \
    if (is_float) hipLaunchKernelGGL((matrix_memory_kernel<float, NI>), grid, dim3(256), 0, s, (const float*)x, in, a);       \
    else hipLaunchKernelGGL((matrix_memory_kernel<bf16_t, NI>), grid, dim3(256), 0, s, (const bf16_t*)x, in, a);              \
  }
  if (dim <= 16) IRON_MEMORY(1)
  else if (dim <= 32) IRON_MEMORY(2)
  else if (dim <= 64) IRON_MEMORY(4)
  else if (dim <= 128) IRON_MEMORY(8)
  else if (dim <= 256) IRON_MEMORY(16)
  else IRON_MEMORY(32)
#undef IRON_MEMORY
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_memory_gate(const float* o, const void* gate, const uint16_t* gain, void* y, int rows, int heads, int dim, int gate_stride,
                                int gate_at, float floor, float eps, int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(o && gate && gain && y, "memory_gate: null operand");
  IRON_REQUIRE(rows > 0 && heads > 0 && dim > 0, "memory_gate: rows (%d), heads (%d), dim (%d) must be positive", rows, heads, dim);
  IRON_REQUIRE(gate_at >= 0 && gate_at + heads * dim <= gate_stride, "memory_gate: %d columns from %d of a row of %d", heads * dim, gate_at,
               gate_stride);
  const bool vec = dim % 8 == 0 && gate_stride % 8 == 0 && gate_at % 8 == 0 && (heads * dim + 2 * heads) % 4 == 0 &&
                   (((uintptr_t)o | (uintptr_t)gate | (uintptr_t)gain | (uintptr_t)y) & 15) == 0;
  const dim3 grid((unsigned)(((long)rows * heads + 3) / 4));
#define IRON_GATE(T, VEC)                                                                                                                \
  hipLaunchKernelGGL((memory_gate_kernel<T, VEC>), grid, dim3(256), 0, (hipStream_t)stream, o, (const T*)gate, gain, (T*)y, rows, heads, \
                     dim, gate_stride, gate_at, floor, eps, valid)
  if (is_float) { if (vec) IRON_GATE(float, 8); else IRON_GATE(float, 1); }
  else { if (vec) IRON_GATE(bf16_t, 8); else IRON_GATE(bf16_t, 1); }
#undef IRON_GATE
  IRON_LAUNCH_CHECK();
}
