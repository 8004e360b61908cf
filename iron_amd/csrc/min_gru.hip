// minGRU over `width` channels, each a state of its own that a gate z moves towards a candidate c:
//
//   S_t = (1 - z) S_(t-1) + z c,   z = sigmoid(zx + zb),   c = u + 1/2 where u = ux + ub >= 0, else sigmoid(u)
//   y_t = S_t silu(gx)
//
// zx, ux and gx are columns 0, width and 2 width of a packed projection's row.  Everything in float32.
//
// The step from one state to the next is affine, S -> a S + b, and so is any run of steps.  Over a prompt's portion
// a block takes GRU_CHUNK tokens of 64 or 128 channels, GRU_TOKENS a wave: the waves fold their tokens to an (a, b)
// each, and those to one a chunk.  A first launch does this for every chunk; in a second a block starts from the
// state the chunks before its own leave, a wave from the one the waves before it leave, and walks.  A portion's
// first state is put ahead of its chunks, since the block of its last chunk may replace it: a slot has two states,
// position p's in row p % 2, so that a decode step's blocks leave the one they all read.
#include "../../include/iron_hip.h"
#include "rows.h"

namespace iron {

constexpr int GRU_WAVES = 8, GRU_TOKENS = 16, GRU_CHUNK = GRU_WAVES * GRU_TOKENS;

// Two neighbouring elements, or one.
template <int VEC, typename T>
__device__ __forceinline__ void load_few(const T* __restrict__ p, float (&f)[VEC]) {
  if constexpr (VEC == 1) {
    f[0] = load_one(p);
  } else if constexpr (sizeof(T) == 2) {
    const uint32_t w = *reinterpret_cast<const uint32_t*>(p);
    f[0] = bf16_lo(w);
    f[1] = bf16_hi(w);
  } else {
    const float2 w = *reinterpret_cast<const float2*>(p);
    f[0] = w.x;
    f[1] = w.y;
  }
}
template <int VEC, typename T>
__device__ __forceinline__ void store_few(T* __restrict__ p, const float (&f)[VEC]) {
  if constexpr (VEC == 1) store_one(p, f[0]);
  else if constexpr (sizeof(T) == 2) *reinterpret_cast<uint32_t*>(p) = pack_bf16(f[0], f[1]);
  else *reinterpret_cast<float2*>(p) = make_float2(f[0], f[1]);
}
// The logistic function: by the hardware's exponential and reciprocal (an ulp or two) where rows are bf16.
template <typename T>
__device__ __forceinline__ float logistic(float z) {
  if constexpr (sizeof(T) == 2) return __builtin_amdgcn_rcpf(1.0f + __expf(-z));
  else return 1.0f / (1.0f + expf(-z));
}
// One token's step: the state's factor a, and b.
template <typename T>
__device__ __forceinline__ void gru_step(float zx, float ux, float& a, float& b) {
  const float z = logistic<T>(zx), c = ux >= 0.f ? ux + 0.5f : logistic<T>(ux);
  a = 1.0f - z;
  b = z * c;
}

struct GruShape {
  int slots, rows, stride, width;
};

// Workspace: a (a, b) pair a chunk and channel, each span's chunks behind one more that holds its first state.
__device__ __forceinline__ float2* gru_chunk(float2* work, const int* spans, const GruShape& g, int slot, int chunk) {
  return work + (size_t)(first_chunk(spans, g.slots, slot, g.rows, GRU_CHUNK) * 2 + chunk) * g.width;
}

// A wave's tokens of the columns `at ..` of the projection (its last again past the span's end).
template <typename T, int VEC>
__device__ __forceinline__ void gru_load(const T* __restrict__ x, const GruShape& g, const Span& s, int t0, int at, float (&f)[GRU_TOKENS][VEC]) {
#pragma unroll
  for (int i = 0; i < GRU_TOKENS; ++i) load_few<VEC>(x + (size_t)(s.row0 + min(t0 + i, s.rows - 1)) * g.stride + at, f[i]);
}

// WALK false: every chunk's (a, b) into the workspace, but the last's, which nobody starts from.
template <typename T, int VEC, bool WALK>
__global__ __launch_bounds__(GRU_WAVES * 64) void min_gru_chunks_kernel(const T* __restrict__ x, const bf16_t* __restrict__ zb,
                                                                        const bf16_t* __restrict__ xb, float* __restrict__ state,
                                                                        const int* __restrict__ spans, float2* __restrict__ work,
                                                                        T* __restrict__ y, GruShape g) {
  __shared__ float2 folded[GRU_WAVES][64 * VEC];
  const int slot = blockIdx.z, chunk = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const Span s = span_of(spans, slot, g.rows);
  const int first = chunk * GRU_CHUNK, t0 = first + wave * GRU_TOKENS;
  if (first >= s.rows) return;
  const bool last = first + GRU_CHUNK >= s.rows;
  const int c = (blockIdx.x * 64 + lane) * VEC, at = min(c, g.width - VEC);   // (a lane past the width: the last channels, not stored)
  const bool in = c < g.width;
  float2* chunks = gru_chunk(work, spans, g, slot, 0) + at;
  if (!WALK && chunk == 0 && wave == 0 && in)
#pragma unroll
    for (int j = 0; j < VEC; ++j) chunks[j] = make_float2(0.f, s.start > 0 ? state[(size_t)(2 * slot + ((s.start - 1) & 1)) * g.width + at + j] : 0.f);
  if (!WALK && last) return;
  float z[GRU_TOKENS][VEC], u[GRU_TOKENS][VEC], o[GRU_TOKENS][VEC], zbias[VEC], xbias[VEC];
  gru_load<T, VEC>(x, g, s, t0, at, z);
  gru_load<T, VEC>(x, g, s, t0, at + g.width, u);
  if (WALK) gru_load<T, VEC>(x, g, s, t0, at + 2 * g.width, o);
  load_few<VEC>(zb + at, zbias);
  load_few<VEC>(xb + at, xbias);
  float a[VEC], b[VEC], S[VEC];
#pragma unroll
  for (int j = 0; j < VEC; ++j) a[j] = 1.f, b[j] = 0.f;
#pragma unroll
  for (int i = 0; i < GRU_TOKENS; ++i)
#pragma unroll
    for (int j = 0; j < VEC; ++j) {   // the step's own (a, b) where its two inputs were
      float p, q;
      gru_step<T>(z[i][j] + zbias[j], u[i][j] + xbias[j], p, q);
      z[i][j] = p;
      u[i][j] = q;
      a[j] *= p;
      b[j] = fmaf(p, b[j], q);
    }
#pragma unroll
  for (int j = 0; j < VEC; ++j) folded[wave][lane * VEC + j] = make_float2(a[j], b[j]);
  if (WALK) {
#pragma unroll
    for (int j = 0; j < VEC; ++j) S[j] = chunks[j].y;
#pragma unroll 16
    for (int k = 1; k <= chunk; ++k)
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        const float2 ab = chunks[(size_t)k * g.width + j];
        S[j] = fmaf(ab.x, S[j], ab.y);
      }
  }
  __syncthreads();
  if (!WALK) {
    if (wave > 0 || !in) return;
    for (int w = 1; w < GRU_WAVES; ++w)
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        const float2 ab = folded[w][lane * VEC + j];
        a[j] *= ab.x;
        b[j] = fmaf(ab.x, b[j], ab.y);
      }
#pragma unroll
    for (int j = 0; j < VEC; ++j) chunks[(size_t)(chunk + 1) * g.width + j] = make_float2(a[j], b[j]);
    return;
  }
  for (int w = 0; w < wave; ++w)
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const float2 ab = folded[w][lane * VEC + j];
      S[j] = fmaf(ab.x, S[j], ab.y);
    }
  T* out = y + (size_t)(s.row0 + t0) * g.width + c;
#pragma unroll
  for (int i = 0; i < GRU_TOKENS; ++i) {
    const bool live = t0 + i < s.rows;
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      S[j] = live ? fmaf(z[i][j], S[j], u[i][j]) : S[j];
      o[i][j] = S[j] * (o[i][j] * logistic<T>(o[i][j]));
    }
    if (live && in) store_few<VEC>(out + (size_t)i * g.width, o[i]);
  }
  if (in && t0 < s.rows && t0 + GRU_TOKENS >= s.rows)   // the wave of the span's last row
#pragma unroll
    for (int j = 0; j < VEC; ++j) state[(size_t)(2 * slot + ((s.start + s.rows - 1) & 1)) * g.width + c + j] = S[j];
}

// A span's rows one after the other.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void min_gru_rows_kernel(const T* __restrict__ x, const bf16_t* __restrict__ zb, const bf16_t* __restrict__ xb,
                                                           float* __restrict__ state, const int* __restrict__ spans, T* __restrict__ y, GruShape g) {
  const int slot = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * VEC;
  const Span s = span_of(spans, slot, g.rows);
  if (s.rows == 0 || c >= g.width) return;
  float zbias[VEC], xbias[VEC], S[VEC];
  load_few<VEC>(zb + c, zbias);
  load_few<VEC>(xb + c, xbias);
#pragma unroll
  for (int j = 0; j < VEC; ++j) S[j] = s.start > 0 ? state[(size_t)(2 * slot + ((s.start - 1) & 1)) * g.width + c + j] : 0.f;
  const T* row = x + (size_t)s.row0 * g.stride + c;
  T* out = y + (size_t)s.row0 * g.width + c;
  for (int t = 0; t < s.rows; ++t, row += g.stride, out += g.width) {
    float z[VEC], u[VEC], o[VEC];
    load_few<VEC>(row, z);
    load_few<VEC>(row + g.width, u);
    load_few<VEC>(row + 2 * g.width, o);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      float p, q;
      gru_step<T>(z[j] + zbias[j], u[j] + xbias[j], p, q);
      S[j] = fmaf(p, S[j], q);
      o[j] = S[j] * (o[j] * logistic<T>(o[j]));
    }
    store_few<VEC>(out, o);
  }
#pragma unroll
  for (int j = 0; j < VEC; ++j) state[(size_t)(2 * slot + ((s.start + s.rows - 1) & 1)) * g.width + c + j] = S[j];
}

template <typename T>
static int launch_min_gru(const T* x, const bf16_t* zb, const bf16_t* xb, float* state, const int* spans, T* y, float2* work,
                          const GruShape& g, hipStream_t s) {
  const bool pairs = g.width % 2 == 0 && g.stride % 2 == 0 &&
                     ((((uintptr_t)x | (uintptr_t)y) & (2 * sizeof(T) - 1)) | (((uintptr_t)zb | (uintptr_t)xb) & 3)) == 0;
  const int vec = pairs ? 2 : 1;
  const dim3 chunks((g.width + 64 * vec - 1) / (64 * vec), (g.rows + GRU_CHUNK - 1) / GRU_CHUNK, g.slots);
  const dim3 rows((g.width + 256 * vec - 1) / (256 * vec), g.slots);
#define IRON_GRU(VEC)                                                                                                                \
  if (work != nullptr) {                                                                                                             \
    hipLaunchKernelGGL((min_gru_chunks_kernel<T, VEC, false>), chunks, dim3(GRU_WAVES * 64), 0, s, x, zb, xb, state, spans, work, y, g); \
    hipLaunchKernelGGL((min_gru_chunks_kernel<T, VEC, true>), chunks, dim3(GRU_WAVES * 64), 0, s, x, zb, xb, state, spans, work, y, g);  \
  } else {                                                                                                                           \
    hipLaunchKernelGGL((min_gru_rows_kernel<T, VEC>), rows, dim3(256), 0, s, x, zb, xb, state, spans, y, g);                         \
  }
  if (pairs) { IRON_GRU(2) }
  else { IRON_GRU(1) }
#undef IRON_GRU
  IRON_LAUNCH_CHECK();
}

}  // namespace iron

using namespace iron;

extern "C" int64_t iron_min_gru_workspace_bytes(int slots, int rows, int width) {
  return slots > 0 && rows > 0 && width > 0 ? (int64_t)chunks_of(rows, slots, GRU_CHUNK) * 2 * width * (int64_t)sizeof(float2) : 0;
}

extern "C" int iron_min_gru(const void* x, const uint16_t* z_bias, const uint16_t* x_bias, float* state, const int* spans, void* y,
                            void* workspace, int slots, int rows, int stride, int width, int is_float, void* stream) {
  IRON_REQUIRE(x && z_bias && x_bias && state && spans && y, "min_gru: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0 && ((uintptr_t)workspace & 15) == 0, "min_gru: spans and workspace must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0 && rows <= GRU_CHUNK * 65535L, "min_gru: slots (%d) and rows (%d) must be positive",
               slots, rows);
  IRON_REQUIRE(width > 0 && 3L * width <= stride, "min_gru: a row of %d holds no three projections of %d", stride, width);
  const GruShape g{slots, rows, stride, width};
  hipStream_t s = (hipStream_t)stream;
  if (is_float)
    return launch_min_gru<float>((const float*)x, z_bias, x_bias, state, spans, (float*)y, (float2*)workspace, g, s);
  return launch_min_gru<bf16_t>((const bf16_t*)x, z_bias, x_bias, state, spans, (bf16_t*)y, (float2*)workspace, g, s);
}
