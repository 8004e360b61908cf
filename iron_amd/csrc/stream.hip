// A decoder's residual stream held in float32: rows gathered from a bf16 table into it, a row or its RMS
// norm out of it, a block's normed or gated output added to it, a weighted sum of what it was after every layer in its
// place, plain sums into it with a norm by groups behind them, and the head's scale and soft cap.  One rounding, to the activation type, where a row leaves the stream;
// bandwidth bound, a block a row.
#include "../../include/iron_hip.h"
#include "rows.h"

namespace iron {

template <int VEC>
__global__ __launch_bounds__(256) void stream_embed_kernel(const bf16_t* __restrict__ table, const int* __restrict__ ids,
                                                           float* __restrict__ x, float* __restrict__ also, int rows,
                                                           int table_rows, int cols, float scale, const int* __restrict__ valid) {
  const int row = blockIdx.x;
  if (row >= bound_or(valid, rows)) return;
  const int id = ids[row];
  if (id < 0 || id >= table_rows) return;
  for (int c = threadIdx.x * VEC; c < cols; c += 256 * VEC) {
    float f[VEC];
    load_vec<VEC>(table + (size_t)id * cols + c, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] *= scale;
    store_vec<VEC>(x + (size_t)row * cols + c, f);
    if (also != nullptr) store_vec<VEC>(also + (size_t)row * cols + c, f);
  }
}

__device__ __forceinline__ float row_total(float v, float* part) {
  v = wave_sum(v);
  __syncthreads();   // the last total's readers are done
  if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
  __syncthreads();
  return part[0] + part[1] + part[2] + part[3];
}

// What joins the stream: nothing, a block's row normed (rmsnorm(y + yb) * (unit + wb)), or a block's row gated
// ((y + yb) * sigmoid(gate + gb), the gate columns `at` .. of rows of `stride`).
enum { ADD_NONE = 0, ADD_NORMED = 1, ADD_GATED = 2 };
struct StreamGate {
  const void* gate;          // rows of the activation type
  const bf16_t *bias, *y_bias;   // gb, yb (yb may be null)
  int stride, at;
};
// What leaves it: nothing, its norm (rmsnorm(x) * (unit + w)), or the row itself.
enum { OUT_NONE = 0, OUT_NORM = 1, OUT_CAST = 2 };
// What it was: plane j of `planes` is the stream behind layer j, `plane` floats each; the row as it stands becomes
// plane `index`, and the sum over j <= index of weights[j] times plane j takes its place.
struct StreamDepth {
  float* planes;
  const bf16_t* weights;
  size_t plane;
  int index;
};

// x += what ADD says, in place; then (DEPTH) the weighted sum; then what OUT says.
// A thread holds its first CH pieces of the row between the passes and re-reads the rest.
template <typename T, int VEC, int CH, int ADD, int OUT, bool DEPTH>
__global__ __launch_bounds__(256) void stream_rows_kernel(float* __restrict__ x, const T* __restrict__ y,
                                                          const bf16_t* __restrict__ wb, const bf16_t* __restrict__ w,
                                                          T* __restrict__ h, int rows, int cols, float eps, float unit,
                                                          const int* __restrict__ valid, StreamGate g, StreamDepth d) {
  __shared__ float part[4];
  const int row = blockIdx.x, first = threadIdx.x * VEC;
  constexpr int STEP = 256 * VEC;
  constexpr bool NORM = OUT == OUT_NORM;
  float held[CH][VEC], gain[CH][VEC];
  if (NORM) {
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (first + i * STEP < cols) load_vec<VEC>(w + first + i * STEP, gain[i]);
  }
  if (row >= bound_or(valid, rows)) return;
  float* xr = x + (size_t)row * cols;
#pragma unroll
  for (int i = 0; i < CH; ++i)
    if (first + i * STEP < cols) load_vec<VEC>(xr + first + i * STEP, held[i]);

  if (ADD == ADD_GATED) {
    const T* yr = y + (size_t)row * cols;
    const T* gr = reinterpret_cast<const T*>(g.gate) + (size_t)row * g.stride + g.at;
    auto gated = [&](int c, float (&f)[VEC]) {
      float z[VEC], b[VEC], yb[VEC];
      load_vec<VEC>(yr + c, f);
      load_vec<VEC>(gr + c, z);
      load_vec<VEC>(g.bias + c, b);
      if (g.y_bias != nullptr) {
        load_vec<VEC>(g.y_bias + c, yb);
#pragma unroll
        for (int j = 0; j < VEC; ++j) f[j] += yb[j];
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] *= 1.0f / (1.0f + expf(-(z[j] + b[j])));
    };
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (first + i * STEP < cols) {
        float f[VEC];
        gated(first + i * STEP, f);
#pragma unroll
        for (int j = 0; j < VEC; ++j) held[i][j] += f[j];
        if (!DEPTH) store_vec<VEC>(xr + first + i * STEP, held[i]);
      }
    for (int c = first + CH * STEP; c < cols; c += STEP) {
      float f[VEC], s[VEC];
      gated(c, f);
      load_vec<VEC>(xr + c, s);
#pragma unroll
      for (int j = 0; j < VEC; ++j) s[j] += f[j];
      store_vec<VEC>(xr + c, s);
    }
  }
  if (ADD == ADD_NORMED) {
    const T* yr = y + (size_t)row * cols;
    auto biased = [&](int c, float (&f)[VEC]) {
      load_vec<VEC>(yr + c, f);
      if (g.y_bias != nullptr) {
        float yb[VEC];
        load_vec<VEC>(g.y_bias + c, yb);
#pragma unroll
        for (int j = 0; j < VEC; ++j) f[j] += yb[j];
      }
    };
    float out[CH][VEC], back[CH][VEC];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (first + i * STEP < cols) {
        biased(first + i * STEP, out[i]);
        load_vec<VEC>(wb + first + i * STEP, back[i]);
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss = fmaf(out[i][j], out[i][j], ss);
      }
    for (int c = first + CH * STEP; c < cols; c += STEP) {
      float f[VEC];
      biased(c, f);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss = fmaf(f[j], f[j], ss);
    }
    const float inv = 1.0f / sqrtf(row_total(ss, part) / (float)cols + eps);
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (first + i * STEP < cols) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) held[i][j] += out[i][j] * inv * (unit + back[i][j]);
        if (!DEPTH) store_vec<VEC>(xr + first + i * STEP, held[i]);
      }
    for (int c = first + CH * STEP; c < cols; c += STEP) {
      float f[VEC], b[VEC], s[VEC];
      biased(c, f);
      load_vec<VEC>(wb + c, b);
      load_vec<VEC>(xr + c, s);
#pragma unroll
      for (int j = 0; j < VEC; ++j) s[j] += f[j] * inv * (unit + b[j]);
      store_vec<VEC>(xr + c, s);
    }
  }
  if (DEPTH) {
    auto averaged = [&](int c, float (&s)[VEC]) {
      float* at = d.planes + (size_t)row * cols + c;
      store_vec<VEC>(at + d.index * d.plane, s);
      const float own = bf16_to_f32(d.weights[d.index]);
#pragma unroll
      for (int j = 0; j < VEC; ++j) s[j] *= own;
      int n = 0;
      for (; n + 4 <= d.index; n += 4) {   // four planes' loads in flight
        float f[4][VEC];
#pragma unroll
        for (int q = 0; q < 4; ++q) load_vec<VEC>(at + (n + q) * d.plane, f[q]);
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const float by = bf16_to_f32(d.weights[n + q]);
#pragma unroll
          for (int j = 0; j < VEC; ++j) s[j] = fmaf(by, f[q][j], s[j]);
        }
      }
      for (; n < d.index; ++n) {
        float f[VEC];
        load_vec<VEC>(at + n * d.plane, f);
        const float by = bf16_to_f32(d.weights[n]);
#pragma unroll
        for (int j = 0; j < VEC; ++j) s[j] = fmaf(by, f[j], s[j]);
      }
    };
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (first + i * STEP < cols) {
        averaged(first + i * STEP, held[i]);
        store_vec<VEC>(xr + first + i * STEP, held[i]);
      }
    for (int c = first + CH * STEP; c < cols; c += STEP) {
      float s[VEC];
      load_vec<VEC>(xr + c, s);
      averaged(c, s);
      store_vec<VEC>(xr + c, s);
    }
  }
  if (OUT == OUT_CAST) {
    T* hr = h + (size_t)row * cols;
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (first + i * STEP < cols) store_vec<VEC>(hr + first + i * STEP, held[i]);
    for (int c = first + CH * STEP; c < cols; c += STEP) {
      float f[VEC];
      load_vec<VEC>(xr + c, f);
      store_vec<VEC>(hr + c, f);
    }
  }
  if (NORM) {
    T* hr = h + (size_t)row * cols;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (first + i * STEP < cols) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss = fmaf(held[i][j], held[i][j], ss);
      }
    for (int c = first + CH * STEP; c < cols; c += STEP) {   // this thread's own stores, if it made any
      float f[VEC];
      load_vec<VEC>(xr + c, f);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss = fmaf(f[j], f[j], ss);
    }
    const float inv = 1.0f / sqrtf(row_total(ss, part) / (float)cols + eps);
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (first + i * STEP < cols) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) held[i][j] = held[i][j] * inv * (unit + gain[i][j]);
        store_vec<VEC>(hr + first + i * STEP, held[i]);
      }
    for (int c = first + CH * STEP; c < cols; c += STEP) {
      float f[VEC], gn[VEC];
      load_vec<VEC>(xr + c, f);
      load_vec<VEC>(w + c, gn);
#pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] = f[j] * inv * (unit + gn[j]);
      store_vec<VEC>(hr + c, f);
    }
  }
}

// x += y + y2 (each may be missing), in place; then h = the row, each of its `groups` equal parts over its own root mean
// square, times the gains.  A wave takes whole parts, and holds its first CH pieces of one between the passes.
template <typename T, int VEC, int CH>
__global__ __launch_bounds__(256) void stream_groups_kernel(float* __restrict__ x, const T* __restrict__ y, const T* __restrict__ y2,
                                                            const bf16_t* __restrict__ w, T* __restrict__ h, int rows, int cols, int groups,
                                                            float eps, float unit, const int* __restrict__ valid) {
  const long item = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int row = (int)(item / groups), first = (threadIdx.x & 63) * VEC, part = cols / groups;
  if (row >= bound_or(valid, rows)) return;
  const size_t at = (size_t)row * cols + (item - (long)row * groups) * part;
  constexpr int STEP = 64 * VEC;
  auto load = [&](int c, float (&f)[VEC]) {   // what the stream's element becomes
    load_vec<VEC>(x + at + c, f);
    float a[VEC], b[VEC];
    if (y != nullptr) {
      load_vec<VEC>(y + at + c, a);
      if (y2 != nullptr) load_vec<VEC>(y2 + at + c, b);
#pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] += y2 != nullptr ? a[j] + b[j] : a[j];
    }
  };
  float held[CH][VEC], ss = 0.f;
#pragma unroll
  for (int i = 0; i < CH; ++i)
    if (first + i * STEP < part) load(first + i * STEP, held[i]);
#pragma unroll
  for (int i = 0; i < CH; ++i)
    if (first + i * STEP < part) {
      if (y != nullptr) store_vec<VEC>(x + at + first + i * STEP, held[i]);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss = fmaf(held[i][j], held[i][j], ss);
    }
  for (int c = first + CH * STEP; c < part; c += STEP) {
    float f[VEC];
    load(c, f);
    if (y != nullptr) store_vec<VEC>(x + at + c, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss = fmaf(f[j], f[j], ss);
  }
  if (h == nullptr) return;
  const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)part + eps);
  const bf16_t* gain = w + (at - (size_t)row * cols);
#pragma unroll
  for (int i = 0; i < CH; ++i)
    if (first + i * STEP < part) {
      float g[VEC];
      load_vec<VEC>(gain + first + i * STEP, g);
#pragma unroll
      for (int j = 0; j < VEC; ++j) held[i][j] = held[i][j] * inv * (unit + g[j]);
      store_vec<VEC>(h + at + first + i * STEP, held[i]);
    }
  for (int c = first + CH * STEP; c < part; c += STEP) {   // this thread's own stores, if it made any
    float f[VEC], g[VEC];
    load_vec<VEC>(x + at + c, f);
    load_vec<VEC>(gain + c, g);
#pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] = f[j] * inv * (unit + g[j]);
    store_vec<VEC>(h + at + c, f);
  }
}

// Of rows [.. gate | up ..]: act(gate) * up into columns of rows of another length.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void gated_columns_kernel(const T* __restrict__ x, T* __restrict__ y, int rows, int cols, int stride, int gate_at,
                                                            int width, int at, int kind, float limit, const int* __restrict__ valid) {
  const int pieces = cols / VEC;
  const long item = (long)blockIdx.x * 256 + threadIdx.x;
  const int row = (int)(item / pieces), c = (int)(item - (long)row * pieces) * VEC;
  if (row >= bound_or(valid, rows)) return;
  const T* g = x + (size_t)row * stride + gate_at + c;
  float f[VEC], u[VEC];
  load_vec<VEC>(g, f);
  load_vec<VEC>(g + cols, u);
#pragma unroll
  for (int j = 0; j < VEC; ++j) f[j] = gated_value(kind, limit, f[j], u[j]);
  store_vec<VEC>(y + (size_t)row * width + at + c, f);
}

// The last row of every span, gathered: out[slot] = x[row0 + rows - 1] (an idle slot's row is left).
__global__ __launch_bounds__(256) void span_tails_kernel(const float* __restrict__ x, const int* __restrict__ spans,
                                                         float* __restrict__ out, int rows, int cols) {
  const Span s = span_of(spans, blockIdx.x, rows);
  if (s.rows == 0) return;
  const float* src = x + (size_t)(s.row0 + s.rows - 1) * cols;
  for (int c = threadIdx.x; c < cols; c += 256) out[(size_t)blockIdx.x * cols + c] = src[c];
}

// scale * x, then cap * tanh(x / cap): in float32, and rounded to bf16 for the draw (rows of `stride`,
// whole 16-byte pieces).  cap 0: no cap.
template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(const T* __restrict__ x, float* __restrict__ y,
                                                      bf16_t* __restrict__ rounded, int cols, int stride, float cap, float scale) {
  const size_t row = blockIdx.y;
  for (int i = blockIdx.x * 256 + threadIdx.x; i < cols; i += gridDim.x * 256) {
    float v = load_one(x + row * cols + i) * scale;
    if (cap > 0.f) v = cap * tanhf(v / cap);
    y[row * cols + i] = v;
    rounded[row * stride + i] = f32_to_bf16(v);
  }
}

// relu / silu / gelu (tanh form) of the gate, times up, in float32.
__global__ __launch_bounds__(256) void act_mul_f32_kernel(const float* __restrict__ gate, const float* __restrict__ up,
                                                          float* __restrict__ y, long n, int kind,
                                                          const int* __restrict__ valid, int cols) {
  if (valid != nullptr) n = min(n, (long)max(*valid, 0) * cols);
  for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < n; i += (long)gridDim.x * 256) {
    const float g = gate[i];
    const float a = kind == 3 ? fmaxf(g, 0.f) : (kind == 1 ? g / (1.f + expf(-g)) : gelu_tanh_f32(g));
    y[i] = a * up[i];
  }
}

// silu / gelu (tanh form) / relu, rounded once.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void activation_kernel(const T* __restrict__ x, T* __restrict__ y, long n, int kind,
                                                         const int* __restrict__ valid, int cols) {
  if (valid != nullptr) n = min(n, (long)max(*valid, 0) * cols);
  for (long i = ((long)blockIdx.x * 256 + threadIdx.x) * VEC; i < n; i += (long)gridDim.x * 256 * VEC) {
    float f[VEC];
    load_vec<VEC>(x + i, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] = kind == 3 ? fmaxf(f[j], 0.f) : (kind == 1 ? f[j] / (1.f + expf(-f[j])) : gelu_tanh_f32(f[j]));
    store_vec<VEC>(y + i, f);
  }
}

// y = x W^T over float32 sums, one thread a 4 x 4 patch of a 64 x 64 tile, K through LDS: any sizes.
// The 32-bit model's projections (T = float), and a bf16 row whose length is no whole 16-byte piece.
template <typename T>
__global__ __launch_bounds__(256) void linear_any_kernel(const T* __restrict__ x, const bf16_t* __restrict__ w,
                                                         T* __restrict__ y, int rows, int n, int k,
                                                         const int* __restrict__ valid) {
  constexpr int BK = 16;
  __shared__ float xs[BK][65], ws[BK][65];
  const int live = bound_or(valid, rows);
  const int r0 = blockIdx.y * 64, c0 = blockIdx.x * 64;
  if (r0 >= live) return;
  const int tr = threadIdx.x >> 4, tc = threadIdx.x & 15;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < k; k0 += BK) {
    for (int i = threadIdx.x; i < 64 * BK; i += 256) {
      const int r = i / BK, kk = i % BK;
      const bool in_k = k0 + kk < k;
      xs[kk][r] = (in_k && r0 + r < live) ? load_one(x + (size_t)(r0 + r) * k + k0 + kk) : 0.f;
      ws[kk][r] = (in_k && c0 + r < n) ? bf16_to_f32(w[(size_t)(c0 + r) * k + k0 + kk]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < BK; ++kk) {
      float a[4], b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) { a[i] = xs[kk][tr + 16 * i]; b[i] = ws[kk][tc + 16 * i]; }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a[i], b[j], acc[i][j]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int r = r0 + tr + 16 * i, c = c0 + tc + 16 * j;
      if (r < live && c < n) store_one(y + (size_t)r * n + c, acc[i][j]);
    }
}

template <typename T, int ADD, int OUT, bool DEPTH = false>
static int launch_stream_rows(float* x, const T* y, const bf16_t* wb, const bf16_t* w, T* h, int rows, int cols, float eps, float unit,
                              const int* valid, hipStream_t s, const StreamGate& g = StreamGate{nullptr, nullptr, nullptr, 8, 8},
                              const StreamDepth& d = StreamDepth{nullptr, nullptr, 0, 0}) {
  const bool vec = cols % 8 == 0 && g.stride % 8 == 0 && g.at % 8 == 0 && d.plane % 4 == 0 &&
                   (((uintptr_t)x | (uintptr_t)y | (uintptr_t)wb | (uintptr_t)w | (uintptr_t)h | (uintptr_t)g.gate | (uintptr_t)g.bias |
                     (uintptr_t)g.y_bias | (uintptr_t)d.planes) & 15) == 0;
#define IRON_ROWS(VEC, CH) \
  hipLaunchKernelGGL((stream_rows_kernel<T, VEC, CH, ADD, OUT, DEPTH>), dim3(rows), dim3(256), 0, s, x, y, wb, w, h, rows, cols, eps, unit, valid, g, d)
  if (vec && cols <= 2048) IRON_ROWS(8, 1);
  else if (vec) IRON_ROWS(8, 2);
  else IRON_ROWS(1, 4);
#undef IRON_ROWS
  IRON_LAUNCH_CHECK();
}

static unsigned few_blocks(long n) {
  const long b = (n + 255) / 256;
  return (unsigned)(b > 4096 ? 4096 : b);
}

}  // namespace iron

using namespace iron;

extern "C" int iron_stream_embed(const uint16_t* table, const int* ids, float* x, float* also, int rows, int table_rows, int cols,
                                 float scale, const int* valid, void* stream) {
  IRON_REQUIRE(table && ids && x, "stream_embed: null operand");
  IRON_REQUIRE(rows > 0 && table_rows > 0 && cols > 0, "stream_embed: rows (%d), table_rows (%d), cols (%d) must be positive",
               rows, table_rows, cols);
  if (cols % 8 == 0 && (((uintptr_t)table | (uintptr_t)x | (uintptr_t)also) & 15) == 0)
    hipLaunchKernelGGL((stream_embed_kernel<8>), dim3(rows), dim3(256), 0, (hipStream_t)stream, table, ids, x, also, rows, table_rows, cols, scale, valid);
  else
    hipLaunchKernelGGL((stream_embed_kernel<1>), dim3(rows), dim3(256), 0, (hipStream_t)stream, table, ids, x, also, rows, table_rows, cols, scale, valid);
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_stream_rows(float* x, const void* y, const uint16_t* y_bias, const uint16_t* back_gain, const uint16_t* gain, void* h,
                                int rows, int cols, float eps, float unit, int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(x && (h || y), "stream_rows: null operand");
  IRON_REQUIRE((y == nullptr) == (back_gain == nullptr) && (h == nullptr) == (gain == nullptr),
               "stream_rows: a gain for the row that is added, and one for the norm that is taken");
  IRON_REQUIRE(rows > 0 && cols > 0, "stream_rows: rows (%d) and cols (%d) must be positive", rows, cols);
  hipStream_t s = (hipStream_t)stream;
  const StreamGate g{nullptr, nullptr, y_bias, 8, 8};
#define IRON_STREAM_ROWS(T)                                                                                                             \
  if (y && h) return launch_stream_rows<T, ADD_NORMED, OUT_NORM>(x, (const T*)y, back_gain, gain, (T*)h, rows, cols, eps, unit, valid, s, g); \
  if (y) return launch_stream_rows<T, ADD_NORMED, OUT_NONE>(x, (const T*)y, back_gain, gain, (T*)h, rows, cols, eps, unit, valid, s, g);     \
  return launch_stream_rows<T, ADD_NONE, OUT_NORM>(x, (const T*)y, back_gain, gain, (T*)h, rows, cols, eps, unit, valid, s, g);
  if (is_float) { IRON_STREAM_ROWS(float) }
  IRON_STREAM_ROWS(bf16_t)
#undef IRON_STREAM_ROWS
}

extern "C" int iron_stream_depth_rows(float* x, const void* y, const uint16_t* y_bias, const uint16_t* back_gain, float* planes,
                                      const uint16_t* weights, int plane_rows, int index, void* h, int rows, int cols, float eps, float unit,
                                      int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(x && (h || planes), "stream_depth_rows: null operand");
  IRON_REQUIRE((y == nullptr) == (back_gain == nullptr) && (planes == nullptr) == (weights == nullptr),
               "stream_depth_rows: a gain for the row that is added, and weights for the planes");
  IRON_REQUIRE(rows > 0 && cols > 0, "stream_depth_rows: rows (%d) and cols (%d) must be positive", rows, cols);
  IRON_REQUIRE(planes == nullptr || (index >= 0 && plane_rows >= rows), "stream_depth_rows: plane %d of %d rows for %d", index, plane_rows, rows);
  hipStream_t s = (hipStream_t)stream;
  const StreamGate g{nullptr, nullptr, y_bias, 8, 8};
  const StreamDepth d{planes, weights, (size_t)plane_rows * cols, index};
#define IRON_DEPTH(T, ADD, OUT, DEPTH) \
  return launch_stream_rows<T, ADD, OUT, DEPTH>(x, (const T*)y, back_gain, nullptr, (T*)h, rows, cols, eps, unit, valid, s, g, d)
#define IRON_DEPTHS(T)                                        \
  if (y && planes && h) IRON_DEPTH(T, ADD_NORMED, OUT_CAST, true); \
  if (y && planes) IRON_DEPTH(T, ADD_NORMED, OUT_NONE, true);      \
  if (y) IRON_DEPTH(T, ADD_NORMED, OUT_CAST, false);               \
  if (planes && h) IRON_DEPTH(T, ADD_NONE, OUT_CAST, true);        \
  if (planes) IRON_DEPTH(T, ADD_NONE, OUT_NONE, true);             \
  IRON_DEPTH(T, ADD_NONE, OUT_CAST, false);
  if (is_float) { IRON_DEPTHS(float) }
  IRON_DEPTHS(bf16_t)
#undef IRON_DEPTHS
#undef IRON_DEPTH
}

extern "C" int iron_stream_gated_rows(float* x, const void* y, const uint16_t* y_bias, const void* gate, const uint16_t* gate_bias,
                                      int gate_stride, int gate_at, const uint16_t* gain, void* h, int rows, int cols, float eps,
                                      int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(x && y && gate && gate_bias, "stream_gated_rows: null operand");
  IRON_REQUIRE((h == nullptr) == (gain == nullptr), "stream_gated_rows: a gain for the norm that is taken");
  IRON_REQUIRE(rows > 0 && cols > 0, "stream_gated_rows: rows (%d) and cols (%d) must be positive", rows, cols);
  IRON_REQUIRE(gate_at >= 0 && gate_at + cols <= gate_stride, "stream_gated_rows: columns %d .. + %d of a gate's row of %d", gate_at, cols,
               gate_stride);
  hipStream_t s = (hipStream_t)stream;
  const StreamGate g{gate, gate_bias, y_bias, gate_stride, gate_at};
#define IRON_STREAM_GATED(T)                                                                                                    \
  if (h) return launch_stream_rows<T, ADD_GATED, OUT_NORM>(x, (const T*)y, nullptr, gain, (T*)h, rows, cols, eps, 0.f, valid, s, g); \
  return launch_stream_rows<T, ADD_GATED, OUT_NONE>(x, (const T*)y, nullptr, gain, (T*)h, rows, cols, eps, 0.f, valid, s, g);
  if (is_float) { IRON_STREAM_GATED(float) }
  IRON_STREAM_GATED(bf16_t)
#undef IRON_STREAM_GATED
}

extern "C" int iron_stream_groups(float* x, const void* y, const void* y2, const uint16_t* gain, void* h, int rows, int cols, int groups, float eps,
                                  float unit, int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(x && (h || y), "stream_groups: null operand");
  IRON_REQUIRE((y != nullptr || y2 == nullptr) && (h == nullptr) == (gain == nullptr), "stream_groups: a second row behind a first, gains for a norm");
  IRON_REQUIRE(rows > 0 && cols > 0 && groups > 0 && cols % groups == 0, "stream_groups: rows (%d) positive, cols (%d) in equal groups (%d)", rows, cols, groups);
  const int part = cols / groups;
  const long blocks = ((long)rows * groups + 3) / 4;
  IRON_REQUIRE(blocks < (1L << 31), "stream_groups: %d rows of %d groups exceed the grid", rows, groups);
  hipStream_t s = (hipStream_t)stream;
  const bool vec = part % 8 == 0 && (((uintptr_t)x | (uintptr_t)y | (uintptr_t)y2 | (uintptr_t)gain | (uintptr_t)h) & 15) == 0;
#define IRON_GROUPS(T, VEC, CH) \
  hipLaunchKernelGGL((stream_groups_kernel<T, VEC, CH>), dim3((unsigned)blocks), dim3(256), 0, s, x, (const T*)y, (const T*)y2, gain, (T*)h, rows, cols, groups, eps, unit, valid)
#define IRON_GROUPSS(T)                            \
  {                                                \
    if (vec && part <= 512) IRON_GROUPS(T, 8, 1);  \
    else if (vec) IRON_GROUPS(T, 8, 4);            \
    else IRON_GROUPS(T, 1, 4);                     \
  }
  if (is_float) IRON_GROUPSS(float)
  else IRON_GROUPSS(bf16_t)
#undef IRON_GROUPSS
#undef IRON_GROUPS
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_gated_columns(const void* x, void* y, int rows, int cols, int stride, int gate_at, int width, int at, int kind, float limit,
                                  int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(x && y, "gated_columns: null operand");
  IRON_REQUIRE(rows > 0 && cols > 0, "gated_columns: rows (%d) and cols (%d) must be positive", rows, cols);
  IRON_REQUIRE(gate_at >= 0 && gate_at + 2 * cols <= stride && at >= 0 && at + cols <= width,
               "gated_columns: twice %d columns from %d of a row of %d, into those from %d of %d", cols, gate_at, stride, at, width);
  IRON_REQUIRE(kind >= 0 && kind <= 3 && (kind != 0 || limit > 0.f),
               "gated_columns: kind (%d) is 0 (a limit above 0), 1 (SiLU), 2 (GELU, tanh form) or 3 (ReLU)", kind);
  const bool vec = cols % 8 == 0 && stride % 8 == 0 && gate_at % 8 == 0 && width % 8 == 0 && at % 8 == 0 && (((uintptr_t)x | (uintptr_t)y) & 15) == 0;
  const long blocks = ((long)rows * (vec ? cols / 8 : cols) + 255) / 256;
  IRON_REQUIRE(blocks < (1L << 31), "gated_columns: %d rows of %d exceed the grid", rows, cols);
#define IRON_COLUMNS(T, VEC)                                                                                                               \
  hipLaunchKernelGGL((gated_columns_kernel<T, VEC>), dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream, (const T*)x, (T*)y, rows, cols, \
                     stride, gate_at, width, at, kind, limit, valid)
  if (is_float) { if (vec) IRON_COLUMNS(float, 8); else IRON_COLUMNS(float, 1); }
  else { if (vec) IRON_COLUMNS(bf16_t, 8); else IRON_COLUMNS(bf16_t, 1); }
#undef IRON_COLUMNS
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_span_tails(const float* x, const int* spans, float* out, int slots, int rows, int cols, void* stream) {
  IRON_REQUIRE(x && spans && out, "span_tails: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0, "span_tails: spans must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && rows > 0 && cols > 0, "span_tails: slots (%d), rows (%d), cols (%d) must be positive", slots, rows, cols);
  hipLaunchKernelGGL(span_tails_kernel, dim3(slots), dim3(256), 0, (hipStream_t)stream, x, spans, out, rows, cols);
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_softcap(const void* x, float* y, uint16_t* rounded, int rows, int cols, int rounded_stride, float cap,
                            float scale, int is_float, void* stream) {
  IRON_REQUIRE(x && y && rounded, "softcap: null operand");
  IRON_REQUIRE(rows > 0 && rows <= 65535 && cols > 0 && rounded_stride >= cols && cap >= 0.f,
               "softcap: rows (%d) and cols (%d) must be positive, a rounded row (%d) no shorter, cap (%g) not negative", rows,
               cols, rounded_stride, (double)cap);
  const dim3 grid(few_blocks(cols), rows);
  if (is_float)
    hipLaunchKernelGGL((softcap_kernel<float>), grid, dim3(256), 0, (hipStream_t)stream, (const float*)x, y, rounded, cols, rounded_stride, cap, scale);
  else
    hipLaunchKernelGGL((softcap_kernel<bf16_t>), grid, dim3(256), 0, (hipStream_t)stream, (const bf16_t*)x, y, rounded, cols, rounded_stride, cap, scale);
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_act_mul_f32(const float* gate, const float* up, float* y, int rows, int cols, int activation,
                                const int* valid, void* stream) {
  IRON_REQUIRE(gate && up && y, "act_mul_f32: null operand");
  IRON_REQUIRE(rows > 0 && cols > 0, "act_mul_f32: rows (%d) and cols (%d) must be positive", rows, cols);
  IRON_REQUIRE(activation >= 1 && activation <= 3, "act_mul_f32: activation (%d) is 1 (SiLU), 2 (GELU, tanh form) or 3 (ReLU)", activation);
  const long n = (long)rows * cols;
  hipLaunchKernelGGL(act_mul_f32_kernel, dim3(few_blocks(n)), dim3(256), 0, (hipStream_t)stream, gate, up, y, n, activation, valid, cols);
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_activation(const void* x, void* y, int rows, int cols, int activation, int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(x && y, "activation: null operand");
  IRON_REQUIRE(rows > 0 && cols > 0, "activation: rows (%d) and cols (%d) must be positive", rows, cols);
  IRON_REQUIRE(activation >= 1 && activation <= 3, "activation: kind (%d) is 1 (SiLU), 2 (GELU, tanh form) or 3 (ReLU)", activation);
  const long n = (long)rows * cols;
  const bool vec = cols % 8 == 0 && (((uintptr_t)x | (uintptr_t)y) & 15) == 0;
  const dim3 grid(few_blocks(vec ? n / 8 : n));
#define IRON_ACTIVATION(T, VEC) \
  hipLaunchKernelGGL((activation_kernel<T, VEC>), grid, dim3(256), 0, (hipStream_t)stream, (const T*)x, (T*)y, n, activation, valid, cols)
  if (is_float) { if (vec) IRON_ACTIVATION(float, 8); else IRON_ACTIVATION(float, 1); }
  else { if (vec) IRON_ACTIVATION(bf16_t, 8); else IRON_ACTIVATION(bf16_t, 1); }
#undef IRON_ACTIVATION
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_linear_any(const void* x, const uint16_t* w, void* y, int rows, int n, int k, int is_float,
                               const int* valid, void* stream) {
  IRON_REQUIRE(x && w && y, "linear_any: null operand");
  IRON_REQUIRE(rows > 0 && n > 0 && k > 0, "linear_any: rows (%d), n (%d), k (%d) must be positive", rows, n, k);
  IRON_REQUIRE((rows + 63) / 64 <= 65535, "linear_any: rows (%d) exceed the grid's y extent", rows);
  const dim3 grid((n + 63) / 64, (rows + 63) / 64);
  if (is_float)
    hipLaunchKernelGGL((linear_any_kernel<float>), grid, dim3(256), 0, (hipStream_t)stream, (const float*)x, w, (float*)y, rows, n, k, valid);
  else
    hipLaunchKernelGGL((linear_any_kernel<bf16_t>), grid, dim3(256), 0, (hipStream_t)stream, (const bf16_t*)x, w, (bf16_t*)y, rows, n, k, valid);
  IRON_LAUNCH_CHECK();
}
