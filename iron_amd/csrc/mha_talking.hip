// Attention within chunks whose heads' weights are mixed behind the softmax, over a batch of spans: position i sees
// the j <= i of its own chunk of `chunk` positions (counted from the sequence's start); per head an ordinary softmax
// over the scores, then weight_h <- sum_g talk[h, g] weight_g, and head h applies its mixed weights to the values of
// its own key/value head.
//
// turned_heads makes the rows it reads of a packed projection [q heads | k heads | v heads]: biases, RMS norm and
// rotation of q and k a head, the scores' scale in q, and values blended with an earlier layer's.
//
// The history is a ring of `ring` rows a slot (position p in row p % ring), with ring = chunk: at a position only its
// chunk's own rows are seen, and those are the ring's first.  A span's own keys and values are read from its rows, so the
// ring is written after they have been attended.
//
//   rows kernel:    a block a query row with all its heads, twice over the keys (either type)
#include "../../include/iron_hip.h"
#include "window.h"

namespace iron {

// --------------------------------------------------------------- the rows
struct TurnShape {
  int rows, stride, slots;
  int heads, kv_heads, dim, vdim;
  int turned, angle_rows;                // leading columns of a head that turn, in neighbouring pairs; the table's rows
  float scale, eps;
};
struct TurnIn {
  const bf16_t *bias, *q_gain, *k_gain, *temp;
  const float* angles;                   // [angle_rows][turned]: cos and sin side by side
  const bf16_t* share;                   // the other values' share, one number, and their rows
  const void* first;
  int first_stride, first_at;
};

// LANES lanes a head, 8 consecutive columns each (VEC), or a wave a head, column by column.
template <typename T, int LANES, bool VEC>
__global__ __launch_bounds__(256) void turned_heads_kernel(const T* __restrict__ x, T* __restrict__ y, const int* __restrict__ spans,
                                                           TurnIn in, TurnShape a, const int* __restrict__ valid) {
  const int row = blockIdx.x;
  if (row >= bound_or(valid, a.rows)) return;
  const int slot = slot_of_row(spans, a.slots, a.rows, row);
  if (slot < 0) return;
  const Span s = span_of(spans, slot, a.rows);
  const int pos = min(s.start + row - s.row0, a.angle_rows - 1);
  const float* turn = in.angles + (size_t)pos * a.turned;
  const int lane = threadIdx.x % LANES, qk = a.heads + a.kv_heads, units = qk + a.kv_heads;
  const float share = in.first != nullptr ? bf16_to_f32(*in.share) : 0.f;
  for (int u = threadIdx.x / LANES; u < units; u += 256 / LANES) {
    const bool value = u >= qk, query = u < a.heads;
    const int at = value ? qk * a.dim + (u - qk) * a.vdim : u * a.dim, n = value ? a.vdim : a.dim;
    const T* xr = x + (size_t)row * a.stride + at;
    T* yr = y + (size_t)row * a.stride + at;
    const T* fr = reinterpret_cast<const T*>(in.first) + (size_t)row * in.first_stride + in.first_at + (u - qk) * a.vdim;
    if constexpr (VEC) {
      const int c = lane * 8;
      float f[8], b[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] = 0.f;
      if (c < n) {
        load_vec<8>(xr + c, f);
        load_vec<8>(in.bias + at + c, b);
#pragma unroll
        for (int j = 0; j < 8; ++j) f[j] += b[j];
      }
      if (value) {
        if (c < n) {
          if (in.first != nullptr) {
            load_vec<8>(fr + c, b);
#pragma unroll
            for (int j = 0; j < 8; ++j) f[j] = (1.f - share) * f[j] + share * b[j];
          }
          store_vec<8>(yr + c, f);
        }
        continue;
      }
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) sum = fmaf(f[j], f[j], sum);
#pragma unroll
      for (int m = 1; m < LANES; m <<= 1) sum += __shfl_xor(sum, m, 64);
      if (c >= n) continue;
      const float inv = 1.0f / sqrtf(sum / (float)n + a.eps), by = query ? a.scale * bf16_to_f32(in.temp[u]) : 1.f;
      load_vec<8>((query ? in.q_gain : in.k_gain) + c, b);
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] = f[j] * inv * b[j];
#pragma unroll
      for (int j = 0; j < 8; j += 2)
        if (c + j < a.turned) {
          const float2 t = *reinterpret_cast<const float2*>(turn + c + j);
          const float p = f[j], q = f[j + 1];
          f[j] = p * t.x - q * t.y;
          f[j + 1] = q * t.x + p * t.y;
        }
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] *= by;
      store_vec<8>(yr + c, f);
    } else {
      if (value) {
        for (int c = lane; c < n; c += LANES) {
          float v = load_one(xr + c) + bf16_to_f32(in.bias[at + c]);
          if (in.first != nullptr) v = (1.f - share) * v + share * load_one(fr + c);
          store_one(yr + c, v);
        }
        continue;
      }
      float sum = 0.f;
      for (int c = lane; c < n; c += LANES) {
        const float v = load_one(xr + c) + bf16_to_f32(in.bias[at + c]);
        sum = fmaf(v, v, sum);
      }
      sum = wave_sum(sum);
      const float inv = 1.0f / sqrtf(sum / (float)n + a.eps), by = query ? a.scale * bf16_to_f32(in.temp[u]) : 1.f;
      const bf16_t* gain = query ? in.q_gain : in.k_gain;
      auto normed = [&](int c) { return (load_one(xr + c) + bf16_to_f32(in.bias[at + c])) * inv * bf16_to_f32(gain[c]); };
      for (int c = lane; c < n; c += LANES) {
        float v = normed(c);
        if (c < a.turned) {
          const float other = normed(c ^ 1), cs = turn[c & ~1], sn = turn[c | 1];
          v = (c & 1) ? v * cs + other * sn : v * cs - other * sn;
        }
        store_one(yr + c, v * by);
      }
    }
  }
}

// ------------------------------------------------------------ row by row
struct TalkShape {
  PackedHeads p;
  int chunk, out_stride;
};
constexpr int TALK_KEYS = 64;   // keys at a time

__host__ __device__ inline int talk_row_words(int heads, int dim, int vdim) {
  return heads * dim + heads * vdim + 2 * heads * TALK_KEYS + 2 * heads;
}

template <typename T, int VEC, bool STORE>
__global__ __launch_bounds__(256) void talking_rows_kernel(const T* __restrict__ x, T* __restrict__ keys, T* __restrict__ values,
                                                           const bf16_t* __restrict__ talk, const int* __restrict__ spans,
                                                           T* __restrict__ out, TalkShape a) {
  extern __shared__ __align__(16) float lds[];
  const int slot = blockIdx.y, i = blockIdx.x;
  const Span s = span_of(spans, slot, a.p.rows);
  if (i >= s.rows || (STORE && i > 0)) return;
  const int H = a.p.heads, G = a.p.kv_heads, D = a.p.dim, V = a.p.vdim, each = H / G, nk = G * D, nv = G * V;
  float* qs = lds;                        // [H][D]
  float* acc = qs + H * D;                // [H][V]
  float* ps = acc + H * V;                // [H][TALK_KEYS]
  float* mixed = ps + H * TALK_KEYS;      // [H][TALK_KEYS]
  float* ms = mixed + H * TALK_KEYS;      // [H] the largest score, [H] one over the sum
  float* ls = ms + H;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
  const int pos = s.start + i, lo = pos / a.chunk * a.chunk, count = pos - lo + 1;
  const T* row = x + (size_t)(s.row0 + i) * a.p.stride;
  auto key_at = [&](int p) {
    return p >= s.start ? x + (size_t)(s.row0 + p - s.start) * a.p.stride + H * D : keys + ((size_t)slot * a.p.ring + p % a.p.ring) * nk;
  };
  auto value_at = [&](int p) {
    return p >= s.start ? x + (size_t)(s.row0 + p - s.start) * a.p.stride + H * D + nk : values + ((size_t)slot * a.p.ring + p % a.p.ring) * nv;
  };
  for (int c = t; c < H * D; c += 256) qs[c] = load_one(row + c);
  for (int c = t; c < H * V; c += 256) acc[c] = 0.f;
  for (int h = t; h < H; h += 256) {
    ms[h] = -INFINITY;
    ls[h] = 0.f;
  }
  if (STORE) {
    T* kd = keys + ((size_t)slot * a.p.ring + pos % a.p.ring) * nk;
    T* vd = values + ((size_t)slot * a.p.ring + pos % a.p.ring) * nv;
    for (int c = t; c < nk; c += 256) kd[c] = row[H * D + c];
    for (int c = t; c < nv; c += 256) vd[c] = row[H * D + nk + c];
  }
  __syncthreads();
  auto score = [&](int h, int k0) {
    if (k0 + lane >= count) return -INFINITY;
    const T* kr = key_at(lo + k0 + lane) + h / each * D;
    float dot = 0.f;
    for (int c = 0; c < D; c += VEC) {
      float f[VEC];
      load_vec<VEC>(kr + c, f);
#pragma unroll
      for (int j = 0; j < VEC; ++j) dot = fmaf(f[j], qs[h * D + c + j], dot);
    }
    return dot;
  };
  for (int k0 = 0; k0 < count; k0 += TALK_KEYS)
    for (int h = wave; h < H; h += 4) {   // a head's statistics are its wave's own
      const float v = score(h, k0), top = fmaxf(ms[h], wave_max(v));
      const float l = ls[h] * expf(ms[h] - top) + wave_sum(expf(v - top));
      __builtin_amdgcn_wave_barrier();
      if (lane == 0) {
        ms[h] = top;
        ls[h] = l;
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
    }
  for (int k0 = 0; k0 < count; k0 += TALK_KEYS) {
    for (int h = wave; h < H; h += 4) ps[h * TALK_KEYS + lane] = expf(score(h, k0) - ms[h]) / ls[h];
    __syncthreads();   // (also behind the last tile's readers of `mixed`)
    for (int h = wave; h < H; h += 4) {
      float sum = 0.f;
      for (int g = 0; g < H; ++g) sum = fmaf(bf16_to_f32(talk[h * H + g]), ps[g * TALK_KEYS + lane], sum);
      mixed[h * TALK_KEYS + lane] = sum;
    }
    __syncthreads();
    const int n = min(TALK_KEYS, count - k0);
    for (int o = t; o < H * V; o += 256) {
      const int h = o / V, c = h / each * V + o - h * V;
      float sum = acc[o];
      for (int j = 0; j < n; ++j) sum = fmaf(mixed[h * TALK_KEYS + j], load_one(value_at(lo + k0 + j) + c), sum);
      acc[o] = sum;
    }
  }
  for (int o = t; o < H * V; o += 256) store_one(out + (size_t)(s.row0 + i) * a.out_stride + o, acc[o]);   // (its own)
}

}  // namespace iron

using namespace iron;

extern "C" int iron_turned_heads(const void* x, void* y, const uint16_t* bias, const uint16_t* q_gain, const uint16_t* k_gain,
                                 const uint16_t* temp, const float* angles, const uint16_t* share, const void* first, int first_stride,
                                 int first_at, const int* spans, int slots, int rows, int stride, int heads, int kv_heads, int dim, int vdim,
                                 int turned, int angle_rows, float scale, float eps, int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(x && y && bias && q_gain && k_gain && temp && spans && (turned == 0 || angles), "turned_heads: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0 && ((uintptr_t)angles & 7) == 0, "turned_heads: spans must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && rows > 0 && heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0, "turned_heads: sizes must be positive");
  IRON_REQUIRE(turned >= 0 && turned % 2 == 0 && turned <= dim && angle_rows > 0, "turned_heads: %d of %d columns turn, in pairs", turned, dim);
  IRON_REQUIRE(stride >= heads * dim + kv_heads * (dim + vdim), "turned_heads: a row of %d holds no q, k and v of %d heads", stride, heads);
  IRON_REQUIRE(first == nullptr || (share && first_at >= 0 && first_at + kv_heads * vdim <= first_stride),
               "turned_heads: %d values from column %d of a row of %d", kv_heads * vdim, first_at, first_stride);
  const TurnIn in{bias, q_gain, k_gain, temp, angles, share, first, first_stride, first_at};
  const TurnShape a{rows, stride, slots, heads, kv_heads, dim, vdim, turned, angle_rows, scale, eps};
  const int wide = dim > vdim ? dim : vdim;
  const bool vec = dim % 8 == 0 && vdim % 8 == 0 && stride % 8 == 0 && first_stride % 8 == 0 && first_at % 8 == 0 && wide <= 512 &&
                   (((uintptr_t)x | (uintptr_t)y | (uintptr_t)bias | (uintptr_t)q_gain | (uintptr_t)k_gain | (uintptr_t)first) & 15) == 0;
#define IRON_TURN(T, LANES, VEC) \
  hipLaunchKernelGGL((turned_heads_kernel<T, LANES, VEC>), dim3(rows), dim3(256), 0, (hipStream_t)stream, (const T*)x, (T*)y, spans, in, a, valid)
#define IRON_TURNS(T)                              \
  {                                                \
    if (!vec) IRON_TURN(T, 64, false);             \
    else if (wide <= 64) IRON_TURN(T, 8, true);    \
    else if (wide <= 128) IRON_TURN(T, 16, true);  \
    else if (wide <= 256) IRON_TURN(T, 32, true);  \
    else IRON_TURN(T, 64, true);                   \
  }
  if (is_float) IRON_TURNS(float)
  else IRON_TURNS(bf16_t)
#undef IRON_TURNS
#undef IRON_TURN
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_mha_talking(const void* x, void* keys, void* values, const uint16_t* talk, const int* spans, void* out, int slots, int rows,
                                int stride, int heads, int kv_heads, int dim, int vdim, int chunk, int ring, int single, int is_float,
                                void* stream) {
  IRON_REQUIRE(x && keys && values && talk && spans && out, "mha_talking: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0, "mha_talking: spans must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0, "mha_talking: slots (%d) and rows (%d) must be positive", slots, rows);
  IRON_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0, "mha_talking: kv_heads (%d) must divide heads (%d)",
               kv_heads, heads);
  IRON_REQUIRE(chunk > 0 && ring == chunk, "mha_talking: a ring (%d) of a chunk's (%d) rows", ring, chunk);
  IRON_REQUIRE(stride >= heads * dim + kv_heads * (dim + vdim), "mha_talking: a row of %d holds no q, k and v of %d heads", stride, heads);
  const TalkShape a{{rows, stride, heads, kv_heads, dim, vdim, ring}, chunk, heads * vdim};
  hipStream_t s = (hipStream_t)stream;
  const bool aligned = stride % 8 == 0 && dim % 8 == 0 && vdim % 8 == 0 && (((uintptr_t)x | (uintptr_t)keys | (uintptr_t)values) & 15) == 0;
  const size_t lds = (size_t)talk_row_words(heads, dim, vdim) * 4;
  IRON_REQUIRE(lds <= 160 * 1024, "mha_talking: %d heads of %d + %d need %zu bytes of LDS", heads, dim, vdim, lds);
#define IRON_TALK_ROWS(T, VEC, STORE, ROWS)                                                                                              \
  {                                                                                                                                      \
    static LdsOptIn opt;                                                                                                                 \
    const hipError_t e = opt.ensure(reinterpret_cast<const void*>(&talking_rows_kernel<T, VEC, STORE>), 160 * 1024);                     \
    if (e != hipSuccess) { set_error("%s", hipGetErrorString(e)); return (int)e; }                                                       \
    hipLaunchKernelGGL((talking_rows_kernel<T, VEC, STORE>), dim3(ROWS, slots), dim3(256), lds, s, (const T*)x, (T*)keys, (T*)values,   \
                       talk, spans, (T*)out, a);                                                                                         \
  }
  if (single) {   // the caller's spans have one row at most, which goes into the ring here
    if (is_float) { if (aligned) IRON_TALK_ROWS(float, 8, true, 1) else IRON_TALK_ROWS(float, 1, true, 1) }
    else { if (aligned) IRON_TALK_ROWS(bf16_t, 8, true, 1) else IRON_TALK_ROWS(bf16_t, 1, true, 1) }
    IRON_LAUNCH_CHECK();
  }
  if (is_float) { if (aligned) IRON_TALK_ROWS(float, 8, false, rows) else IRON_TALK_ROWS(float, 1, false, rows) }
  else { if (aligned) IRON_TALK_ROWS(bf16_t, 8, false, rows) else IRON_TALK_ROWS(bf16_t, 1, false, rows) }
#undef IRON_TALK_ROWS
  if (is_float) launch_ring_store<float>(x, keys, values, spans, a.p, slots, s);
  else launch_ring_store<bf16_t>(x, keys, values, spans, a.p, slots, s);
  IRON_LAUNCH_CHECK();
}
