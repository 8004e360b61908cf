// One row of a decoder around a float32 stream: a product with what makes its input ahead of it and what takes its
// output behind it, in one launch.
//
//   input:   a bf16 row; the stream's row (whole or in groups), or a bf16 row, RMS-normed; a gated recurrence's step; an
//            activation over the normed powers of a row
//   output:  a bf16 row; or, through a sigmoid gate or as it is, the stream
//
// Every block makes the whole input for its own few rows of the weight (L2 serves it) while those are on their way
// from memory.  What a launch replaces, no other block of it reads: a recurrence has two states, by a position's
// parity, and the stream's row is not an input where it is the output.  Each value is rounded where the separate
// steps round it.
#include "../../include/iron_hip.h"
#include "latent.h"
#include "row_products.h"
#include "rows.h"

namespace iron {

enum { IN_ROW = 0, IN_STREAM_NORM = 1, IN_ROW_NORM = 2, IN_GRU = 3, IN_POLY = 4, IN_STREAM_GROUPS = 5 };
// OUT_LATENT: a row, and the last block a position's latent.  OUT_LOGITS: a row, and a router's logits in float behind it.
enum { OUT_ROW = 0, OUT_GATED = 1, OUT_LATENT = 2, OUT_ADD = 3, OUT_LOGITS = 4 };
constexpr int MOST_GROUPS = 256;

struct StreamIn {
  const void* x;              // float (the stream) or bf16
  const bf16_t* gain;         // a norm's gains; IN_POLY: the four coefficients
  const bf16_t *b0, *b1;      // IN_GRU: the two biases; IN_POLY: its bias
  float* state;               // IN_GRU
  const int* spans;           // IN_GRU, OUT_LATENT
  float eps;
  float unit;                 // added to a norm's gains
  int groups;                 // IN_STREAM_GROUPS
  bf16_t* made;               // ... where the first block leaves the input it made, for later launches (may be NULL)
};
struct StreamOut {
  bf16_t* y;
  float* stream;
  const bf16_t *y_bias, *gate, *gate_bias;   // OUT_ADD: y_bias is a second row that joins the stream
  const bf16_t* router;       // OUT_LOGITS: `logits` more rows of a weight, and where their products go
  float* z;
  int logits;
  // OUT_LATENT
  const bf16_t *row, *c_gain;
  const float* angles;
  bf16_t *latents, *shared_keys;
  LatentShape a;
  int q_rank;
};

__device__ __forceinline__ float4 load_bounded_floats(__amdgpu_buffer_rsrc_t run, int offset) {
  return __builtin_bit_cast(float4, load_bounded(run, offset));
}

// This thread's CH pieces of the product's input: asked for, and then made.
template <int CH, int IN>
struct Made {
  static constexpr bool STREAM = IN == IN_STREAM_NORM || IN == IN_STREAM_GROUPS;
  static constexpr int ROWS = IN == IN_GRU ? 5 : (IN == IN_ROW ? 1 : 2), FLOATS = STREAM || IN == IN_GRU ? 2 : 1;
  uint4 v[ROWS][CH];
  float4 f[FLOATS][CH];
  int4 span;

  __device__ __forceinline__ void issue(const StreamIn& in, int K) {
    const bf16_t* x = reinterpret_cast<const bf16_t*>(in.x);
    const bf16_t* from[5] = {x, nullptr, nullptr, nullptr, nullptr};
    if (STREAM) from[0] = in.gain;
    if (IN == IN_ROW_NORM) from[1] = in.gain;
    if (IN == IN_POLY) from[1] = in.b0;
    if (IN == IN_GRU) {
      from[1] = x + K;
      from[2] = x + 2 * K;
      from[3] = in.b0;
      from[4] = in.b1;
    }
    constexpr int N = STREAM ? 1 : ROWS;
    if (STREAM) {
      const __amdgpu_buffer_rsrc_t run = bounded_bytes(in.x, 4 * K);
#pragma unroll
      for (int i = 0; i < CH; ++i)
#pragma unroll
        for (int h = 0; h < 2; ++h) f[h][i] = load_bounded_floats(run, 32 * ((int)threadIdx.x + 256 * i) + 16 * h);
    }
#pragma unroll
    for (int n = 0; n < N; ++n) {
      const __amdgpu_buffer_rsrc_t run = bounded_bytes(from[n], 2 * K);
#pragma unroll
      for (int i = 0; i < CH; ++i) v[n][i] = load_bounded(run, 16 * ((int)threadIdx.x + 256 * i));
    }
    if (IN == IN_GRU) {
      span = *reinterpret_cast<const int4*>(in.spans);
      const __amdgpu_buffer_rsrc_t run = bounded_bytes(in.state + ((span.z - 1) & 1) * K, 4 * K);
#pragma unroll
      for (int i = 0; i < CH; ++i)
#pragma unroll
        for (int h = 0; h < 2; ++h) f[h][i] = load_bounded_floats(run, 32 * ((int)threadIdx.x + 256 * i) + 16 * h);
    }
  }

  // sums, inverses (IN_STREAM_GROUPS): LDS, a float a 16-byte piece of the row and one a group.
  __device__ __forceinline__ void finish(const StreamIn& in, int K, float (*part)[4], uint4 (&out)[CH], float* sums = nullptr,
                                         float* inverses = nullptr) {
    if (IN == IN_ROW) {
#pragma unroll
      for (int i = 0; i < CH; ++i) out[i] = v[0][i];
      return;
    }
    if (IN == IN_STREAM_GROUPS) {
      float x[CH][8];
      const int pieces = K / 8 / in.groups, lane = threadIdx.x & 63;
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        const float4 a = f[0][i], b = f[FLOATS - 1][i];
        x[i][0] = a.x; x[i][1] = a.y; x[i][2] = a.z; x[i][3] = a.w;
        x[i][4] = b.x; x[i][5] = b.y; x[i][6] = b.z; x[i][7] = b.w;
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < 8; ++j) sum = fmaf(x[i][j], x[i][j], sum);
        sums[threadIdx.x + 256 * i] = sum;
      }
      block_barrier_lds();
      for (int g = threadIdx.x >> 6; g < in.groups; g += 4) {   // a wave a group
        float sum = 0.f;
        for (int c = lane; c < pieces; c += 64) sum += sums[g * pieces + c];
        sum = wave_sum(sum);
        if (lane == 0) inverses[g] = 1.0f / sqrtf(sum / (float)(pieces * 8) + in.eps);
      }
      block_barrier_lds();
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        float g[8];
        const int c = threadIdx.x + 256 * i;
        const float inv = inverses[min(c / pieces, in.groups - 1)];
        unpack8(v[0][i], g);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[i][j] = x[i][j] * inv * (in.unit + g[j]);
        out[i] = pack8(x[i]);
        if (blockIdx.x == 0 && in.made != nullptr && c < (K >> 3)) reinterpret_cast<uint4*>(in.made)[c] = out[i];
      }
      return;
    }
    if (IN == IN_STREAM_NORM || IN == IN_ROW_NORM) {
      float x[CH][8], sum = 0.f;
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        if (IN == IN_ROW_NORM) {
          unpack8(v[0][i], x[i]);
        } else {
          const float4 a = f[0][i], b = f[FLOATS - 1][i];
          x[i][0] = a.x; x[i][1] = a.y; x[i][2] = a.z; x[i][3] = a.w;
          x[i][4] = b.x; x[i][5] = b.y; x[i][6] = b.z; x[i][7] = b.w;
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) sum = fmaf(x[i][j], x[i][j], sum);
      }
      const float inv = 1.0f / sqrtf(block_sum(sum, part[0]) / (float)K + in.eps);
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        float g[8];
        unpack8(v[IN == IN_ROW_NORM ? ROWS - 1 : 0][i], g);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[i][j] = x[i][j] * inv * (in.unit + g[j]);
        out[i] = pack8(x[i]);
      }
      return;
    }
    if (IN == IN_GRU) {
      const bool older = span.z > 0;
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        float z[8], u[8], g[8], zb[8], ub[8];
        unpack8(v[0][i], z);
        unpack8(v[ROWS > 1 ? 1 : 0][i], u);
        unpack8(v[ROWS > 2 ? 2 : 0][i], g);
        unpack8(v[ROWS > 3 ? 3 : 0][i], zb);
        unpack8(v[ROWS > 4 ? 4 : 0][i], ub);
        const float4 a = f[0][i], b = f[FLOATS - 1][i];
        float S[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float share = __builtin_amdgcn_rcpf(1.0f + __expf(-(z[j] + zb[j]))), n = u[j] + ub[j];
          const float c = n >= 0.f ? n + 0.5f : __builtin_amdgcn_rcpf(1.0f + __expf(-n));
          S[j] = fmaf(1.0f - share, older ? S[j] : 0.f, share * c);
          g[j] = S[j] * (g[j] * __builtin_amdgcn_rcpf(1.0f + __expf(-g[j])));
        }
        out[i] = pack8(g);
        const int c = (int)threadIdx.x + 256 * i;
        if (blockIdx.x == 0 && span.y > 0 && c < (K >> 3)) {
          float4* to = reinterpret_cast<float4*>(in.state + (span.z & 1) * K) + 2 * c;
          to[0] = make_float4(S[0], S[1], S[2], S[3]);
          to[1] = make_float4(S[4], S[5], S[6], S[7]);
        }
      }
      return;
    }
    // IN_POLY
    const float ca = bf16_to_f32(in.gain[0]), cb = bf16_to_f32(in.gain[1]), cc = bf16_to_f32(in.gain[2]), ce = bf16_to_f32(in.gain[3]);
    float x[CH][8], s1 = 0.f, s2 = 0.f, s3 = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      float b[8];
      unpack8(v[0][i], x[i]);
      unpack8(v[ROWS - 1][i], b);   // (past the row's end both are zeros)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        x[i][j] += b[j];
        const float p = x[i][j] * x[i][j], q = p * x[i][j];
        s1 += p;
        s2 = fmaf(p, p, s2);
        s3 = fmaf(q, q, s3);
      }
    }
    s1 = wave_sum(s1);
    s2 = wave_sum(s2);
    s3 = wave_sum(s3);
    if ((threadIdx.x & 63) == 0) {
      const int w = threadIdx.x >> 6;
      part[0][w] = s1;
      part[1][w] = s2;
      part[2][w] = s3;
    }
    __syncthreads();
    auto over = [&](int k, float by) { return by / sqrtf((part[k][0] + part[k][1] + part[k][2] + part[k][3]) / (float)K + in.eps); };
    const float f1 = over(0, ca), f2 = over(1, cb), f3 = over(2, cc);
#pragma unroll
    for (int i = 0; i < CH; ++i) {
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] = fmaf(x[i][j], fmaf(x[i][j], fmaf(x[i][j], f3, f2), f1), ce);
      out[i] = pack8(x[i]);
    }
  }
};

template <int RPW, int CH, int IN, int OUT>
__global__ __launch_bounds__(256) void stream_product_kernel(const bf16_t* __restrict__ W, StreamIn in, StreamOut out, int M, int K) {
  __shared__ float part[3][4], sums[4][RPW];
  __shared__ float piece_sums[IN == IN_STREAM_GROUPS ? CH * 256 : 1], inverses[IN == IN_STREAM_GROUPS ? MOST_GROUPS : 1];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, row0 = blockIdx.x * RPW;
  if (OUT == OUT_LATENT && row0 >= M) {   // the one block behind the product's
    const int4 span = *reinterpret_cast<const int4*>(in.spans);
    if (span.y > 0)
      latent_row<bf16_t, 2, false>(out.row + out.q_rank, LatentRow{nullptr, out.c_gain, out.angles, out.q_rank, in.eps}, out.a, 0, span.z, nullptr, out.latents,
                            out.shared_keys, part);
    return;
  }
  Made<CH, IN> made;
  made.issue(in, K);
  uint4 w[RPW][CH];
#pragma unroll
  for (int r = 0; r < RPW; ++r) {
    const int row = row0 + r;
    const bf16_t* from = OUT == OUT_LOGITS && row >= M ? out.router + (size_t)min(row - M, out.logits - 1) * K : W + (size_t)min(row, M - 1) * K;
    load_row<CH>(from, K, w[r]);
  }
  // What the output's threads need at the end, asked for by all of them ahead of the wait.
  float held = 0.f;
  bf16_t yb = 0, gate = 0, gb = 0;
  if (OUT == OUT_ADD) {
    const int row = min(row0 + min((int)threadIdx.x, RPW - 1), M - 1);
    held = out.stream[row];
    if (out.y_bias != nullptr) yb = out.y_bias[row];
  }
  if (OUT == OUT_GATED) {
    const int row = min(row0 + min((int)threadIdx.x, RPW - 1), M - 1);
    held = out.stream[row];
    gate = out.gate[row];
    gb = out.gate_bias[row];
    if (out.y_bias != nullptr) yb = out.y_bias[row];
  }
  uint4 x[CH];
  made.finish(in, K, part, x, piece_sums, inverses);
#pragma unroll
  for (int r = 0; r < RPW; ++r) {
    const float a = wave_sum(dot_row<CH>(w[r], x));
    if (lane == 0) sums[wave][r] = a;
  }
  __syncthreads();
  const int r = threadIdx.x, row = row0 + r;
  if (r >= RPW || row >= (OUT == OUT_LOGITS ? M + out.logits : M)) return;
  const float whole = sums[0][r] + sums[1][r] + sums[2][r] + sums[3][r], v = round_bf16(whole);
  if (OUT == OUT_LOGITS && row >= M) {
    out.z[row - M] = whole;
    return;
  }
  if (OUT == OUT_ADD) {
    out.stream[row] = held + (out.y_bias != nullptr ? v + bf16_to_f32(yb) : v);
    return;
  }
  if (OUT == OUT_GATED) out.stream[row] = held + (v + bf16_to_f32(yb)) * (1.0f / (1.0f + expf(-(bf16_to_f32(gate) + bf16_to_f32(gb)))));
  else out.y[row] = f32_to_bf16(v);
}

template <int IN, int OUT>
static int launch_stream_product(const bf16_t* W, const StreamIn& in, const StreamOut& out, int M, int K, hipStream_t s) {
  const int ch = K <= 2048 ? 1 : (K <= 4096 ? 2 : (K <= 8192 ? 4 : 8));
#define IRON_PRODUCT(RPW, CH)                                                                                                     \
  {                                                                                                                               \
    const int rows = OUT == OUT_LOGITS ? M + out.logits : M, blocks = (rows + RPW - 1) / RPW + (OUT == OUT_LATENT ? 1 : 0);                                                         \
    hipLaunchKernelGGL((stream_product_kernel<RPW, CH, IN, OUT>), dim3(blocks), dim3(256), 0, s, W, in, out, M, K);               \
    IRON_LAUNCH_CHECK();                                                                                                          \
  }
  // Rows a block takes (measured): more where the input is long in the making and the matrix is tall.
  constexpr bool NORM = IN == IN_STREAM_NORM || IN == IN_STREAM_GROUPS, MADE = NORM || IN == IN_GRU;
  if (ch == 1 && NORM && M >= 8192) IRON_PRODUCT(8, 1)
  if (ch == 1 && IN == IN_GRU) IRON_PRODUCT(4, 1)
  if (ch == 1 && M > 2048) IRON_PRODUCT(2, 1)
  if (ch == 1) IRON_PRODUCT(1, 1)
  if (ch == 2 && MADE) IRON_PRODUCT(4, 2)
  if (ch == 2) IRON_PRODUCT(2, 2)
  if (ch == 4) IRON_PRODUCT(4, 4)
  if constexpr (OUT == OUT_ADD) {
    if (K > 8 * 2048) IRON_PRODUCT(1, 16)
  }
  IRON_PRODUCT(2, 8)
#undef IRON_PRODUCT
}

}  // namespace iron

using namespace iron;

extern "C" int iron_stream_product_bf16(int input, const void* x, const uint16_t* gain, const uint16_t* b0, const uint16_t* b1, float* state,
                                        const int* spans, float eps, float unit, const uint16_t* W, int M, int K, uint16_t* y, float* stream_row,
                                        const uint16_t* y_bias, const uint16_t* gate, const uint16_t* gate_bias, void* stream) {
  IRON_REQUIRE(input >= IN_ROW && input <= IN_POLY, "stream_product: input (%d) is 0 to 4", input);
  IRON_REQUIRE(x && W && ((y != nullptr) != (stream_row != nullptr)), "stream_product: null operand, or not one output");
  IRON_REQUIRE(M > 0 && K > 0 && K % 8 == 0 && K <= 8 * 2048, "stream_product: M (%d) positive, K (%d) a multiple of 8 up to %d", M, K, 8 * 2048);
  IRON_REQUIRE(input == IN_ROW || input == IN_GRU || gain, "stream_product: a norm's gains, or the powers' coefficients");
  IRON_REQUIRE(input != IN_GRU || (b0 && b1 && state && spans), "stream_product: a recurrence's biases, state and spans");
  IRON_REQUIRE(input != IN_POLY || b0, "stream_product: the activation's bias");
  IRON_REQUIRE(stream_row == nullptr || (gate && gate_bias), "stream_product: a gate and its bias");
  IRON_REQUIRE(stream_row == nullptr || input != IN_STREAM_NORM, "stream_product: the stream is an input or the output");
  IRON_REQUIRE((((uintptr_t)x | (uintptr_t)W | (uintptr_t)b0 | (uintptr_t)b1 | (uintptr_t)state | (uintptr_t)spans |
                 (input == IN_POLY ? 0 : (uintptr_t)gain)) & 15) == 0, "stream_product: operands must be 16-byte aligned");
  const StreamIn in{x, gain, b0, b1, state, spans, eps, unit, 1, nullptr};
  StreamOut out{};
  out.y = y;
  out.stream = stream_row;
  out.y_bias = y_bias;
  out.gate = gate;
  out.gate_bias = gate_bias;
  hipStream_t s = (hipStream_t)stream;
  if (y != nullptr) {
    if (input == IN_STREAM_NORM) return launch_stream_product<IN_STREAM_NORM, OUT_ROW>(W, in, out, M, K, s);
    if (input == IN_ROW_NORM) return launch_stream_product<IN_ROW_NORM, OUT_ROW>(W, in, out, M, K, s);
    if (input == IN_ROW) return launch_stream_product<IN_ROW, OUT_ROW>(W, in, out, M, K, s);
    IRON_REQUIRE(false, "stream_product: input %d is served into a stream only", input);
  }
  if (input == IN_GRU) return launch_stream_product<IN_GRU, OUT_GATED>(W, in, out, M, K, s);
  if (input == IN_POLY) return launch_stream_product<IN_POLY, OUT_GATED>(W, in, out, M, K, s);
  if (input == IN_ROW) return launch_stream_product<IN_ROW, OUT_GATED>(W, in, out, M, K, s);
  IRON_REQUIRE(false, "stream_product: input %d is served into a row only", input);
}

extern "C" int iron_norm_product_bf16(const float* x, const uint16_t* gain, int groups, float eps, float unit, const uint16_t* W, int M, int K,
                                      uint16_t* y, uint16_t* h, const uint16_t* router, int logits, float* z, void* stream) {
  IRON_REQUIRE(x && gain && W && y && (router == nullptr || z), "norm_product: null operand");
  IRON_REQUIRE(M > 0 && K > 0 && K % 8 == 0 && K <= 8 * 2048, "norm_product: M (%d) positive, K (%d) a multiple of 8 up to %d", M, K, 8 * 2048);
  IRON_REQUIRE(groups > 0 && groups <= MOST_GROUPS && K % (8 * groups) == 0, "norm_product: K (%d) in equal groups (%d, up to %d) of whole 16-byte pieces", K,
               groups, MOST_GROUPS);
  IRON_REQUIRE(router == nullptr || logits > 0, "norm_product: logits (%d) must be positive", logits);
  IRON_REQUIRE((((uintptr_t)x | (uintptr_t)gain | (uintptr_t)W | (uintptr_t)h | (uintptr_t)router) & 15) == 0, "norm_product: operands must be 16-byte aligned");
  const StreamIn in{x, gain, nullptr, nullptr, nullptr, nullptr, eps, unit, groups, h};
  StreamOut out{};
  out.y = y;
  out.router = router;
  out.z = z;
  out.logits = logits;
  if (router != nullptr) return launch_stream_product<IN_STREAM_GROUPS, OUT_LOGITS>(W, in, out, M, K, (hipStream_t)stream);
  return launch_stream_product<IN_STREAM_GROUPS, OUT_ROW>(W, in, out, M, K, (hipStream_t)stream);
}

extern "C" int iron_product_sum_bf16(const uint16_t* x, const uint16_t* W, int M, int K, const uint16_t* also, float* stream_row, void* stream) {
  IRON_REQUIRE(x && W && stream_row, "product_sum: null operand");
  IRON_REQUIRE(M > 0 && K > 0 && K % 8 == 0 && K <= 16 * 2048, "product_sum: M (%d) positive, K (%d) a multiple of 8 up to %d", M, K, 16 * 2048);
  IRON_REQUIRE((((uintptr_t)x | (uintptr_t)W) & 15) == 0, "product_sum: operands must be 16-byte aligned");
  const StreamIn in{x, nullptr, nullptr, nullptr, nullptr, nullptr, 0.f, 0.f, 1, nullptr};
  StreamOut out{};
  out.stream = stream_row;
  out.y_bias = also;
  return launch_stream_product<IN_ROW, OUT_ADD>(W, in, out, M, K, (hipStream_t)stream);
}

extern "C" int iron_latent_query_bf16(const uint16_t* x, const uint16_t* q_gain, const uint16_t* c_gain, const float* angles, const int* spans,
                                      const uint16_t* W, uint16_t* q, uint16_t* latents, uint16_t* shared_keys, int M, int stride, int q_rank,
                                      int rank, int rot, int turned, int angle_rows, int ring, float eps, void* stream) {
  IRON_REQUIRE(x && q_gain && c_gain && spans && W && q && latents && (rot == 0 || shared_keys), "latent_query: null operand");
  const LatentShape a{1, 1, 1, 1, rot, 1, rank, turned, angle_rows, 1, ring, 0, 1.f};
  IRON_REQUIRE(M > 0 && q_rank > 0 && q_rank <= 8 * 2048 && rank > 0 && ring > 0 && q_rank + rank + rot <= stride,
               "latent_query: M (%d) positive, a row of %d holding latents of %d and %d + %d", M, stride, q_rank, rank, rot);
  IRON_REQUIRE(latent_row_wide(a, stride, q_rank) && rank + rot <= 2 * 2048, "latent_query: latents (%d, %d + %d, %d turned) of whole 16-byte pieces",
               q_rank, rank, rot, turned);
  IRON_REQUIRE(turned <= rot && (turned == 0 || (angles && angle_rows > 0)), "latent_query: %d of %d columns turn, by a table of %d rows", turned, rot, angle_rows);
  IRON_REQUIRE((((uintptr_t)x | (uintptr_t)q_gain | (uintptr_t)c_gain | (uintptr_t)spans | (uintptr_t)W | (uintptr_t)latents | (uintptr_t)shared_keys) & 15) == 0,
               "latent_query: operands must be 16-byte aligned");
  const StreamIn in{x, q_gain, nullptr, nullptr, nullptr, spans, eps, 0.f, 1, nullptr};
  StreamOut out{};
  out.y = q;
  out.row = x;
  out.c_gain = c_gain;
  out.angles = angles;
  out.latents = latents;
  out.shared_keys = shared_keys;
  out.a = a;
  out.q_rank = q_rank;
  return launch_stream_product<IN_ROW_NORM, OUT_LATENT>(W, in, out, M, q_rank, (hipStream_t)stream);
}
