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
//   step kernels:   one row a slot: all scores first, then a block some columns of a key/value head's values
//   prompt kernels: bf16 MFMAs; the rows' softmax statistics a head first, then 16 queries with all their heads a block
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

template <typename T, int VEC>
__global__ __launch_bounds__(256) void talking_rows_kernel(const T* __restrict__ x, const T* __restrict__ keys, const T* __restrict__ values,
                                                           const bf16_t* __restrict__ talk, const int* __restrict__ spans,
                                                           T* __restrict__ out, TalkShape a) {
  extern __shared__ __align__(16) float lds[];
  const int slot = blockIdx.y, i = blockIdx.x;
  const Span s = span_of(spans, slot, a.p.rows);
  if (i >= s.rows) return;
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

// ---------------------------------------------------------------- a step
// One row a slot, three launches.  talking_scores: a wave 64 keys of one key head: the scores of its query heads, left in memory,
// their largest and the sum of exponentials under it; the row's own key and value go into the ring.  talking_mix: the heads'
// weights from all scores, mixed.  talking_values: times the values.
struct StepWork {   // floats a slot: scores [heads][chunk], (largest, sum) [heads][pieces of 64 keys], mixed weights [heads][chunk]
  int pieces;
  size_t stats, mixed, words;
  __host__ __device__ StepWork(int heads, int chunk)
      : pieces((chunk + 63) / 64), stats(((size_t)heads * chunk + 1) & ~(size_t)1), mixed(stats + (size_t)heads * 2 * pieces),
        words((mixed + (size_t)heads * chunk + 1) & ~(size_t)1) {}
};
template <typename T>
__device__ __forceinline__ float weight_exp(float x) {
  if constexpr (sizeof(T) == 2) return __expf(x);
  else return expf(x);
}

template <typename T, int VEC>
__global__ __launch_bounds__(64) void talking_scores_kernel(const T* __restrict__ x, T* __restrict__ keys, T* __restrict__ values,
                                                            const int* __restrict__ spans, float* __restrict__ work, TalkShape a) {
  extern __shared__ __align__(16) float qs[];   // [each][dim]
  const int g = blockIdx.y, slot = blockIdx.z, k0 = blockIdx.x * 64, lane = threadIdx.x;
  const Span s = span_of(spans, slot, a.p.rows);
  const int pos = s.start, lo = pos / a.chunk * a.chunk, count = pos - lo + 1;
  if (s.rows == 0 || k0 >= count) return;
  const int H = a.p.heads, G = a.p.kv_heads, D = a.p.dim, V = a.p.vdim, each = H / G;
  const T* row = x + (size_t)s.row0 * a.p.stride;
  const T* own = row + H * D + g * D;
  T* ring = keys + (size_t)slot * a.p.ring * G * D + g * D;
  const int j = k0 + lane, p = lo + min(j, count - 1);
  const T* kr = p == pos ? own : ring + (size_t)(p - lo) * G * D;
  constexpr int FIRST = 8;   // pieces of the key asked for ahead of the queries
  float kf[FIRST][VEC];
#pragma unroll
  for (int u = 0; u < FIRST; ++u) load_vec<VEC>(kr + min(u * VEC, D - VEC), kf[u]);
  for (int c = lane; c < each * D; c += 64) qs[c] = load_one(row + g * each * D + c);
  if (k0 == 0) {
    const T* v = row + (H + G) * D + g * V;
    T* vd = values + ((size_t)slot * a.p.ring + pos % a.p.ring) * G * V + g * V;
    for (int c = lane; c < D; c += 64) ring[(size_t)(pos % a.p.ring) * G * D + c] = own[c];
    for (int c = lane; c < V; c += 64) vd[c] = v[c];
  }
  __syncthreads();
  const StepWork w(H, a.chunk);
  float* mine = work + slot * w.words;
  for (int e0 = 0; e0 < each; e0 += 4) {
    float dot[4] = {0.f, 0.f, 0.f, 0.f};
    auto add = [&](int c, const float (&f)[VEC]) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float* q = qs + min(e0 + e, each - 1) * D + c;
#pragma unroll
        for (int n = 0; n < VEC; ++n) dot[e] = fmaf(f[n], q[n], dot[e]);
      }
    };
#pragma unroll
    for (int u = 0; u < FIRST; ++u)
      if (u * VEC < D) add(u * VEC, kf[u]);
#pragma unroll 8
    for (int c = FIRST * VEC; c < D; c += VEC) {
      float f[VEC];
      load_vec<VEC>(kr + c, f);
      add(c, f);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (e0 + e >= each) continue;
      const int h = g * each + e0 + e;
      const float v = j < count ? dot[e] : -INFINITY, top = wave_max(v), sum = wave_sum(weight_exp<T>(v - top));
      if (j < count) mine[(size_t)h * a.chunk + j] = v;
      if (lane == 0) {
        float* st = mine + w.stats + ((size_t)h * w.pieces + blockIdx.x) * 2;
        st[0] = top;
        st[1] = sum;
      }
    }
  }
}

// The weights of 64 keys for HEADS heads a wave: a key a lane.
template <typename T, int HEADS>
__global__ __launch_bounds__(64) void talking_mix_kernel(const bf16_t* __restrict__ talk, const int* __restrict__ spans, float* __restrict__ work,
                                                         TalkShape a) {
  extern __shared__ __align__(16) float by[];   // [H][HEADS]: what the wave's heads take of a head, over its sum; [H]: its largest score
  const int slot = blockIdx.z, h0 = blockIdx.y * HEADS, k0 = blockIdx.x * 64, lane = threadIdx.x, H = a.p.heads;
  const Span s = span_of(spans, slot, a.p.rows);
  const int count = s.start - s.start / a.chunk * a.chunk + 1, live = (count + 63) / 64;
  if (s.rows == 0 || k0 >= count) return;
  const StepWork w(H, a.chunk);
  float* mine = work + slot * w.words;
  const int j = min(k0 + lane, count - 1);
  constexpr int AT_ONCE = 32;   // scores asked for together, the first ahead of the statistics
  float raw[AT_ONCE];
  auto fetch = [&](int first) {
#pragma unroll
    for (int u = 0; u < AT_ONCE; ++u) raw[u] = mine[(size_t)min(first + u, H - 1) * a.chunk + j];
  };
  fetch(0);
  for (int h = lane; h < H; h += 64) {
    const float2* st = reinterpret_cast<const float2*>(mine + w.stats) + (size_t)h * w.pieces;
    float m = -INFINITY, l = 0.f;
#pragma unroll 8
    for (int i = 0; i < live; ++i) {
      const float2 v = st[i];
      const float higher = fmaxf(m, v.x);
      l = l * expf(m - higher) + v.y * expf(v.x - higher);   // (each piece has a key: its largest is finite)
      m = higher;
    }
    by[H * HEADS + h] = m;
#pragma unroll
    for (int e = 0; e < HEADS; ++e) by[h * HEADS + e] = bf16_to_f32(talk[(size_t)min(h0 + e, H - 1) * H + h]) / l;
  }
  __syncthreads();
  float mixed[HEADS];
#pragma unroll
  for (int e = 0; e < HEADS; ++e) mixed[e] = 0.f;
  for (int first = 0; first < H; first += AT_ONCE) {
    if (first > 0) fetch(first);
#pragma unroll
    for (int u = 0; u < AT_ONCE; ++u) {
      if (first + u >= H) continue;
      const float weight = weight_exp<T>(raw[u] - by[H * HEADS + first + u]);
#pragma unroll
      for (int e = 0; e < HEADS; ++e) mixed[e] = fmaf(by[(first + u) * HEADS + e], weight, mixed[e]);
    }
  }
#pragma unroll
  for (int e = 0; e < HEADS; ++e)
    if (h0 + e < H && k0 + lane < count) mine[w.mixed + (size_t)(h0 + e) * a.chunk + j] = mixed[e];
}

// VEC columns of a value head for HEADS of its query heads a block, a thread a key.
template <typename T, int VEC, int HEADS>
__global__ __launch_bounds__(1024) void talking_values_kernel(const T* __restrict__ x, const T* __restrict__ values, const int* __restrict__ spans,
                                                              const float* __restrict__ work, T* __restrict__ out, TalkShape a) {
  __shared__ float red[16][HEADS * VEC];
  const int slot = blockIdx.z, t = threadIdx.x, lane = t & 63, wave = t >> 6, waves = blockDim.x >> 6;
  const Span s = span_of(spans, slot, a.p.rows);
  if (s.rows == 0) return;
  const int H = a.p.heads, G = a.p.kv_heads, D = a.p.dim, V = a.p.vdim, each = H / G, sets = (each + HEADS - 1) / HEADS;
  const int g = blockIdx.y / sets, e0 = blockIdx.y % sets * HEADS, n = min(HEADS, each - e0), c = blockIdx.x * VEC;
  const int pos = s.start, lo = pos / a.chunk * a.chunk, count = pos - lo + 1;
  const StepWork w(H, a.chunk);
  const float* mixed = work + slot * w.words + w.mixed;
  const T* own = x + (size_t)s.row0 * a.p.stride + (H + G) * D + g * V + c;
  const T* ring = values + (size_t)slot * a.p.ring * G * V + g * V + c;
  float acc[HEADS][VEC];
#pragma unroll
  for (int e = 0; e < HEADS; ++e)
#pragma unroll
    for (int k = 0; k < VEC; ++k) acc[e][k] = 0.f;
  for (int j = t; j < count; j += blockDim.x) {
    float f[VEC], by[HEADS];
    load_vec<VEC>(lo + j == pos ? own : ring + (size_t)j * G * V, f);
#pragma unroll
    for (int e = 0; e < HEADS; ++e) by[e] = mixed[(size_t)(g * each + min(e0 + e, each - 1)) * a.chunk + j];
#pragma unroll
    for (int e = 0; e < HEADS; ++e)
#pragma unroll
      for (int k = 0; k < VEC; ++k) acc[e][k] = fmaf(by[e], f[k], acc[e][k]);
  }
#pragma unroll
  for (int e = 0; e < HEADS; ++e)
    if (e < n) {
#pragma unroll
      for (int k = 0; k < VEC; ++k) {
        const float sum = wave_sum(acc[e][k]);
        if (lane == 0) red[wave][e * VEC + k] = sum;
      }
    }
  __syncthreads();
  if (t < n * VEC) {
    float sum = 0.f;
    for (int i = 0; i < waves; ++i) sum += red[i][t];
    store_one(out + (size_t)s.row0 * a.out_stride + (g * each + e0 + t / VEC) * V + c + t % VEC, sum);
  }
}

// -------------------------------------------------------------- a prompt
// Two launches.  talking_stats: a block 64 queries of one head, flash attention without values: the logarithm (base 2) of
// each row's softmax denominator.  With it a weight is one exponential, and what a key adds needs no rescaling: talking_prompt,
// a block 16 queries with all heads, walks the keys KT at a time.  A wave makes the weights of eight heads against 16 keys
// (keys down the MFMA's rows, queries across), which lie in LDS a pair (query, key) at a time, heads side by side: one MFMA
// operand of the heads' mixing, whose result goes back to LDS a head at a time, keys side by side: one operand of the
// product with the values (transposed in LDS).  Two barriers a tile; keys and values of the next are on their way meanwhile.
// A row's keys are dealt to blocks PART at a time; where that makes more than one, float32 sums are left and a last launch adds
// them.
struct PromptWork {   // floats: each row's statistics, then the parts' sums [part][row][heads * vdim]
  int least, parts;   // the fewest keys of a part, and how many parts that makes of a row's at most
  size_t sums, words;
  __host__ __device__ PromptWork(int rows, int heads, int vdim, int chunk) {
    least = ((chunk + 7) / 8 + 127) / 128 * 128;   // (whole tiles of any size)
    parts = (chunk + 15 + least - 1) / least;      // of sixteen rows that begin at a chunk's last
    sums = ((size_t)rows * heads + 3) & ~(size_t)3;
    words = sums + (parts > 1 ? (size_t)parts * rows * heads * vdim : 0);
  }
  // Where there are blocks enough, longer parts: a block takes as long to begin as for half a dozen tiles of keys.
  __device__ int part(const Span& s, int slots) const { return max(least, s.rows >= 1024 ? 512 : (s.rows * slots >= 1024 ? 256 : 128)); }
};
constexpr float LOG2E = 1.4426950408889634f;
constexpr int STAT_KEYS = 64;

// The row of key or value `p`, of the chunk that starts at `from` or later: positions ahead of the span are that chunk's, in the
// ring's rows from its first on.  (Rows and their lengths are below 2^24.)
__device__ __forceinline__ const bf16_t* row_of(const bf16_t* __restrict__ own, const bf16_t* __restrict__ held, int p, int start, int stride,
                                                int width, int from) {
  const bool mine = p >= start;
  const unsigned at = __umul24(mine ? p - start : p - from, mine ? stride : width);
  return (mine ? own : held) + at;
}

template <int KD>
__global__ __launch_bounds__(256) void talking_stats_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ keys,
                                                            const int* __restrict__ spans, float* __restrict__ stats, int slots,
                                                            TalkShape a) {
  constexpr int DP = KD * 32, KP = STAT_KEYS * DP / 8 / 256;
  __shared__ __align__(16) bf16_t kt[2][STAT_KEYS][DP + 8];
  const int head = blockIdx.x;
  int slot, q0;
  if (!tile_of(spans, slots, a.p.rows, 64, blockIdx.y, slot, q0)) return;
  const Span s = span_of(spans, slot, a.p.rows);
  const int H = a.p.heads, D = a.p.dim, G = a.p.kv_heads, g = head / (H / G);
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, l16 = lane & 15, quad = lane >> 4;
  const int first = s.start + q0, last = s.start + min(q0 + 64, s.rows) - 1, from = first / a.chunk * a.chunk;
  const bf16_t* own = x + (size_t)s.row0 * a.p.stride + H * D + g * D;
  const bf16_t* held = keys + (size_t)slot * a.p.ring * G * D + g * D;
  const int i = min(q0 + wave * 16 + l16, s.rows - 1), pos = s.start + i, lo = pos / a.chunk * a.chunk;
  bf16x8 qf[KD];
#pragma unroll
  for (int d = 0; d < KD; ++d) {
    const int c = d * 32 + quad * 8;
    uint4 v = make_uint4(0, 0, 0, 0);
    if (c < D) v = *reinterpret_cast<const uint4*>(x + (size_t)(s.row0 + i) * a.p.stride + head * D + c);
    qf[d] = __builtin_bit_cast(bf16x8, v);
  }
  u32x4 kn[KP];
  auto fetch = [&](int base) {
#pragma unroll
    for (int e = 0; e < KP; ++e) {
      const int u = t + 256 * e, c = min((u % (DP / 8)) * 8, D - 8);   // (columns past a head's: q is zero there)
      kn[e] = *reinterpret_cast<const u32x4*>(row_of(own, held, min(base + u / (DP / 8), last), s.start, a.p.stride, G * D, from) + c);
    }
  };
  fetch(from);
  float m = -1e30f, l = 0.f;
  int turn = 0;
  for (int base = from; base <= last; base += STAT_KEYS, turn ^= 1) {
#pragma unroll
    for (int e = 0; e < KP; ++e) {
      const int u = t + 256 * e;
      *reinterpret_cast<u32x4*>(&kt[turn][u / (DP / 8)][(u % (DP / 8)) * 8]) = kn[e];
    }
    block_barrier_lds();
    fetch(min(base + STAT_KEYS, last));
    f32x4 sc[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      sc[k] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int d = 0; d < KD; ++d)
        sc[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(&kt[turn][k * 16 + l16][d * 32 + quad * 8]), qf[d], sc[k], 0, 0, 0);
    }
    float top = -INFINITY;
    const bool whole = base + STAT_KEYS - 1 <= first && base >= last / a.chunk * a.chunk;   // every row sees every key
#pragma unroll
    for (int k = 0; k < 4; ++k)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int p = base + k * 16 + quad * 4 + r;
        const float v = sc[k][r] * LOG2E;
        sc[k][r] = whole || (p <= pos && p >= lo) ? v : -INFINITY;
        top = fmaxf(top, sc[k][r]);
      }
    if (__builtin_amdgcn_ballot_w64(top > m + 8.f) != 0) {
      top = fmaxf(top, __shfl_xor(top, 16, 64));
      top = fmaxf(top, __shfl_xor(top, 32, 64));
      top = fmaxf(m, top);
      l *= __builtin_amdgcn_exp2f(m - top);
      m = top;
    }
#pragma unroll
    for (int k = 0; k < 4; ++k)
#pragma unroll
      for (int r = 0; r < 4; ++r) l += __builtin_amdgcn_exp2f(sc[k][r] - m);
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (quad == 0 && q0 + wave * 16 + l16 < s.rows) stats[(size_t)(s.row0 + i) * H + head] = m + log2f(l);
}

// NG groups of eight heads (H <= 8 NG), KD pieces of 32 key columns, VT tiles of 16 value columns a head; EACH query heads in a
// row share a key head.
template <int NG, int KD, int VT>
struct Talking {
  static constexpr int KT = 128 / NG, HP = 8 * NG, HN = (HP + 15) / 16;
  static constexpr int PAIR = KT * HP + 8;            // a query's weights: [key][head]
  static constexpr int MIX = HP * (KT + 8) + 8;       // a query's mixed weights: [head][key]
  static size_t lds(int kv_width) { return ((size_t)16 * PAIR + (size_t)16 * MIX + (size_t)kv_width * (KT + 8)) * 2; }
};

template <int NG, int KD, int VT, int EACH>
__global__ __launch_bounds__(512) void talking_prompt_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ keys,
                                                             const bf16_t* __restrict__ values, const bf16_t* __restrict__ talk,
                                                             const int* __restrict__ spans, float* __restrict__ stats,
                                                             bf16_t* __restrict__ out, int slots, TalkShape a) {
  using S = Talking<NG, KD, VT>;
  // A wave's weights: HU heads against KU * 16 keys, its queries in registers throughout.  A set of heads shares its key head.
  constexpr int KT = S::KT, HP = S::HP, HU = KD <= 2 ? 8 : 4, KU = 8 / HU, SETS = HU / EACH;
  constexpr bool AHEAD = SETS * KU * KD <= 8 && NG * VT <= 16;   // a tile's keys are fetched under the tile before
  extern __shared__ __align__(16) bf16_t shared[];
  bf16_t* pair = shared;
  bf16_t* mix = pair + 16 * S::PAIR;
  bf16_t* vt = mix + 16 * S::MIX;                     // [G * V][KT + 8]
  int slot, q0;
  if (!tile_of(spans, slots, a.p.rows, 16, (int)gridDim.x - 1 - (int)blockIdx.x, slot, q0)) return;
  const Span s = span_of(spans, slot, a.p.rows);
  const int H = a.p.heads, G = a.p.kv_heads, D = a.p.dim, V = a.p.vdim, each = H / G, nk = G * D, nv = G * V;
  const int t = threadIdx.x, lane = t & 63, wave = __builtin_amdgcn_readfirstlane(t >> 6), l16 = lane & 15, quad = lane >> 4;
  const int first = s.start + q0, end = s.start + min(q0 + 16, s.rows) - 1, from = first / a.chunk * a.chunk;
  const PromptWork work(a.p.rows, H, V, a.chunk);
  const int part = work.part(s, slots), begin = from + (int)blockIdx.y * part, last = min(end, begin + part - 1);
  if (begin > end) return;
  const bf16_t* own_k = x + (size_t)s.row0 * a.p.stride + H * D;
  const bf16_t* own_v = own_k + nk;
  const bf16_t* held_k = keys + (size_t)slot * a.p.ring * nk;
  const bf16_t* held_v = values + (size_t)slot * a.p.ring * nv;
  const int i = min(q0 + l16, s.rows - 1), pos = s.start + i, lo = pos / a.chunk * a.chunk, end_lo = end / a.chunk * a.chunk;
  const bf16_t* q_row = x + (size_t)(s.row0 + i) * a.p.stride;

  const int h0 = wave % (HP / HU) * HU, k0 = wave / (HP / HU) * KU * 16;   // the wave's first head, and its keys' first place in a tile
  bf16x8 qf[HU][KD];
  float lse[HU];
#pragma unroll
  for (int e = 0; e < HU; ++e) {
    lse[e] = stats[(size_t)(s.row0 + i) * H + min(h0 + e, H - 1)];   // (no branch around a load: they go out together)
#pragma unroll
    for (int d = 0; d < KD; ++d) {
      const int c = d * 32 + quad * 8;
      u32x4 v = *reinterpret_cast<const u32x4*>(q_row + min(h0 + e, H - 1) * D + min(c, D - 8));
      if (c >= D) v = u32x4{0, 0, 0, 0};
      qf[e][d] = __builtin_bit_cast(bf16x8, v);
    }
  }
#pragma unroll
  for (int e = 0; e < HU; ++e) lse[e] = h0 + e < H ? lse[e] : INFINITY;   // a head that is none: no weight
  // The heads' mixing as the second operand: head l16 (+ 16 n) of the result down its columns.
  bf16x8 tf[S::HN];
#pragma unroll
  for (int n = 0; n < S::HN; ++n) {
    bf16_t w[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int h = n * 16 + l16, g = quad * 8 + j;
      w[j] = talk[min(h, H - 1) * H + min(g, H - 1)];
    }
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (n * 16 + l16 >= H || quad * 8 + j >= H) w[j] = 0;
    tf[n] = __builtin_bit_cast(bf16x8, make_uint4(w[0] | (uint32_t)w[1] << 16, w[2] | (uint32_t)w[3] << 16, w[4] | (uint32_t)w[5] << 16, w[6] | (uint32_t)w[7] << 16));
  }
  f32x4 acc[NG][VT];
#pragma unroll
  for (int e = 0; e < NG; ++e)
#pragma unroll
    for (int v = 0; v < VT; ++v) acc[e][v] = f32x4{0.f, 0.f, 0.f, 0.f};

  bf16x8 kf[AHEAD ? SETS : 1][KU][KD];
  u32x4 vn[4];   // the thread's first piece of a tile's values, on its way
  const int v_pieces = (KT / 4) * (nv / 8);   // a column group's keys over neighbouring lanes, for the turned stores' banks
  auto fetch_keys = [&](int base, int set, bf16x8 (&to)[KU][KD]) {
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      const bf16_t* at = row_of(own_k, held_k, min(base + k0 + u * 16 + l16, last), s.start, a.p.stride, nk, from) + min(h0 + set * EACH, H - 1) / each * D;
#pragma unroll
      for (int d = 0; d < KD; ++d) to[u][d] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(at + min(d * 32 + quad * 8, D - 8)));
    }
  };
  auto fetch_ahead = [&](int base) {
    if constexpr (AHEAD) {
#pragma unroll
      for (int set = 0; set < SETS; ++set) fetch_keys(base, set, kf[set]);
    }
  };
  auto fetch_values = [&](int base, int piece, u32x4 (&v)[4]) {   // four keys of eight columns
    const int k4 = piece % (KT / 4) * 4, c = piece / (KT / 4) * 8;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      v[j] = *reinterpret_cast<const u32x4*>(row_of(own_v, held_v, min(base + k4 + j, last), s.start, a.p.stride, nv, from) + c);
  };
  auto lay_values = [&](int piece, const u32x4 (&v)[4]) {   // turned: a column's four keys side by side
    const int k4 = piece % (KT / 4) * 4, c = piece / (KT / 4) * 8;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      *reinterpret_cast<uint2*>(vt + (c + 2 * j) * (KT + 8) + k4) =
          make_uint2((v[0][j] & 0xffffu) | (v[1][j] << 16), (v[2][j] & 0xffffu) | (v[3][j] << 16));
      *reinterpret_cast<uint2*>(vt + (c + 2 * j + 1) * (KT + 8) + k4) =
          make_uint2((v[0][j] >> 16) | (v[1][j] & 0xffff0000u), (v[2][j] >> 16) | (v[3][j] & 0xffff0000u));
    }
  };
  fetch_ahead(begin);
  if (t < v_pieces) fetch_values(begin, t, vn);
  for (int base = begin; base <= last; base += KT) {
    // ---- weights
    f32x4 sc[HU][KU];
#pragma unroll
    for (int e = 0; e < HU; ++e) {
      if constexpr (!AHEAD) {
        if (e % EACH == 0) fetch_keys(base, e / EACH, kf[0]);
      }
#pragma unroll
      for (int u = 0; u < KU; ++u) {
        sc[e][u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int d = 0; d < KD; ++d) sc[e][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[AHEAD ? e / EACH : 0][u][d], qf[e][d], sc[e][u], 0, 0, 0);
      }
    }
    const bool whole = base + KT - 1 <= first && base >= end_lo;   // every query sees every key
#pragma unroll
    for (int u = 0; u < KU; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = k0 + u * 16 + quad * 4 + r, p = base + j;
        const bool seen = whole || (p <= pos && p >= lo);
        uint32_t w[HU / 2];
#pragma unroll
        for (int e = 0; e < HU; e += 2) {
          const uint32_t two = pack_bf16(__builtin_amdgcn_exp2f(fmaf(sc[e][u][r], LOG2E, -lse[e])), __builtin_amdgcn_exp2f(fmaf(sc[e + 1][u][r], LOG2E, -lse[e + 1])));
          w[e / 2] = seen ? two : 0;
        }
        bf16_t* to = pair + l16 * S::PAIR + j * HP + h0;
        if constexpr (HU == 8) *reinterpret_cast<u32x4*>(to) = u32x4{w[0], w[1], w[2], w[3]};
        else *reinterpret_cast<uint2*>(to) = make_uint2(w[0], w[1]);
      }
    block_barrier_lds();   // the weights are there, and the last tile's products are done
    fetch_ahead(min(base + KT, last));
    // ---- values, turned, and the next ones on their way
    if (t < v_pieces) lay_values(t, vn);
    for (int piece = t + 512; piece < v_pieces; piece += 512) {
      u32x4 v[4];
      fetch_values(base, piece, v);
      lay_values(piece, v);
    }
    if (t < v_pieces) fetch_values(min(base + KT, last), t, vn);
    // ---- the heads mixed: 16 keys of one query at a time
#pragma unroll
    for (int n8 = 0; n8 < KT / 8; ++n8) {   // KT / 16 pieces of each of 16 queries
      const int u = n8 * 8 + wave, qi = u / (KT / 16), j0 = u % (KT / 16) * 16;
      uint4 v = *reinterpret_cast<const uint4*>(pair + qi * S::PAIR + (j0 + l16) * HP + (quad * 8 < HP ? quad * 8 : 0));
      if (quad * 8 >= HP) v = make_uint4(0, 0, 0, 0);
#pragma unroll
      for (int n = 0; n < S::HN; ++n) {
        const f32x4 zero = f32x4{0.f, 0.f, 0.f, 0.f};
        const f32x4 m = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, v), tf[n], zero, 0, 0, 0);
        if (n * 16 + l16 < HP)
          *reinterpret_cast<uint2*>(mix + qi * S::MIX + (n * 16 + l16) * (KT + 8) + j0 + quad * 4) = make_uint2(pack_bf16(m[0], m[1]), pack_bf16(m[2], m[3]));
      }
    }
    block_barrier_lds();
    // ---- times the values: NG heads a wave
    auto weights = [&](int h, int k) { return *reinterpret_cast<const bf16x8*>(mix + l16 * S::MIX + h * (KT + 8) + k + quad * 8); };
    auto value = [&](int at, int v, int k) {
      return *reinterpret_cast<const bf16x8*>(vt + min(at + v * 16 + l16, nv - 1) * (KT + 8) + k + quad * 8);
    };
    if constexpr (EACH == 4) {   // the wave's heads share their values
      if (wave * NG < H) {
        const int at = wave * NG / each * V;
#pragma unroll
        for (int k = 0; k < KT; k += 32) {
          bf16x8 pf[NG];
#pragma unroll
          for (int e = 0; e < NG; ++e) pf[e] = weights(min(wave * NG + e, H - 1), k);
#pragma unroll
          for (int v = 0; v < VT; ++v) {
            if (v * 16 >= V) continue;
            const bf16x8 vf = value(at, v, k);
#pragma unroll
            for (int e = 0; e < NG; ++e) acc[e][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[e], acc[e][v], 0, 0, 0);
          }
        }
      }
    } else {
#pragma unroll
      for (int e = 0; e < NG; ++e) {
        const int h = wave * NG + e;
        if (h >= H) continue;
#pragma unroll
        for (int k = 0; k < KT; k += 32) {
          const bf16x8 pf = weights(h, k);
#pragma unroll
          for (int v = 0; v < VT; ++v)
            if (v * 16 < V) acc[e][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(value(h / each * V, v, k), pf, acc[e][v], 0, 0, 0);
        }
      }
    }
  }
  if (q0 + l16 >= s.rows) return;
#pragma unroll
  for (int e = 0; e < NG; ++e) {
    const int h = wave * NG + e;
    if (h >= H) continue;
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      const int c = v * 16 + quad * 4;
      if (c >= V) continue;
      if (end - from < part)
        *reinterpret_cast<uint2*>(out + (size_t)(s.row0 + i) * a.out_stride + h * V + c) =
            make_uint2(pack_bf16(acc[e][v][0], acc[e][v][1]), pack_bf16(acc[e][v][2], acc[e][v][3]));
      else
        *reinterpret_cast<float4*>(stats + work.sums + ((size_t)blockIdx.y * a.p.rows + s.row0 + i) * H * V + h * V + c) =
            make_float4(acc[e][v][0], acc[e][v][1], acc[e][v][2], acc[e][v][3]);
    }
  }
}

// A row whose keys went to several blocks: their sums, added in the parts' order.
__global__ __launch_bounds__(256) void talking_sums_kernel(const float* __restrict__ stats, const int* __restrict__ spans, bf16_t* __restrict__ out,
                                                           int slots, TalkShape a) {
  const int row = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 4, slot = slot_of_row(spans, slots, a.p.rows, row);
  if (slot < 0) return;
  const Span s = span_of(spans, slot, a.p.rows);
  const int wide = a.p.heads * a.p.vdim, q0 = (row - s.row0) / 16 * 16;
  const int from = (s.start + q0) / a.chunk * a.chunk, end = s.start + min(q0 + 16, s.rows) - 1;
  const PromptWork work(a.p.rows, a.p.heads, a.p.vdim, a.chunk);
  const int parts = (end - from) / work.part(s, slots) + 1;
  if (parts < 2 || c >= wide) return;
  const float* at = stats + work.sums + (size_t)row * wide + c;
  float4 sum = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 4
  for (int p = 0; p < parts; ++p) {
    const float4 v = *reinterpret_cast<const float4*>(at + (size_t)p * a.p.rows * wide);
    sum.x += v.x;
    sum.y += v.y;
    sum.z += v.z;
    sum.w += v.w;
  }
  *reinterpret_cast<uint2*>(out + (size_t)row * a.out_stride + c) = make_uint2(pack_bf16(sum.x, sum.y), pack_bf16(sum.z, sum.w));
}

template <int NG, int KD, int VT, int EACH>
static int launch_talking_prompt(const bf16_t* x, const bf16_t* keys, const bf16_t* values, const bf16_t* talk, const int* spans,
                                 float* stats, bf16_t* out, const TalkShape& a, int slots, hipStream_t s) {
  const size_t lds = Talking<NG, KD, VT>::lds(a.p.kv_heads * a.p.vdim);
  const int parts = PromptWork(a.p.rows, a.p.heads, a.p.vdim, a.chunk).parts;
  static LdsOptIn opt;
  const hipError_t e = opt.ensure(reinterpret_cast<const void*>(&talking_prompt_kernel<NG, KD, VT, EACH>), 160 * 1024);
  if (e != hipSuccess) { set_error("%s", hipGetErrorString(e)); return (int)e; }
  hipLaunchKernelGGL((talking_prompt_kernel<NG, KD, VT, EACH>), dim3((a.p.rows + 15) / 16 + slots - 1, parts), dim3(512), lds, s, x, keys, values, talk,
                     spans, stats, out, slots, a);
  if (parts > 1) hipLaunchKernelGGL(talking_sums_kernel, dim3((a.out_stride + 1023) / 1024, a.p.rows), dim3(256), 0, s, stats, spans, out, slots, a);
  IRON_LAUNCH_CHECK();
}
// The groups of heads a prompt's kernel takes these sizes in, 0 where it takes them not at all.
static int talking_groups(int heads, int kv_heads, int dim, int vdim, int is_float) {
  if (is_float || heads > 32 || dim % 8 || vdim % 8 || dim > 128 || vdim > 128) return 0;
  for (int ng = heads <= 8 ? 1 : (heads <= 16 ? 2 : 4); ng <= 4; ng *= 2) {
    const size_t kt = 128 / ng, lds = 32 * (kt * 8 * ng + 8) + 32 * (8 * ng * (kt + 8) + 8) + 2 * (size_t)kv_heads * vdim * (kt + 8);
    if (lds <= 160 * 1024) return ng;
  }
  return 0;
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

extern "C" int64_t iron_mha_talking_workspace_bytes(int slots, int rows, int heads, int vdim, int chunk, int single) {
  return 4 * (int64_t)(single ? slots * StepWork(heads, chunk).words : PromptWork(rows, heads, vdim, chunk).words);
}


extern "C" int iron_mha_talking(const void* x, void* keys, void* values, const uint16_t* talk, const int* spans, void* out, void* workspace,
                                int slots, int rows, int stride, int heads, int kv_heads, int dim, int vdim, int chunk, int ring, int single, int is_float,
                                void* stream) {
  IRON_REQUIRE(x && keys && values && talk && spans && out && workspace, "mha_talking: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0, "mha_talking: spans must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0, "mha_talking: slots (%d) and rows (%d) must be positive", slots, rows);
  IRON_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0, "mha_talking: kv_heads (%d) must divide heads (%d)",
               kv_heads, heads);
  IRON_REQUIRE(chunk > 0 && ring == chunk, "mha_talking: a ring (%d) of a chunk's (%d) rows", ring, chunk);
  IRON_REQUIRE(stride >= heads * dim + kv_heads * (dim + vdim), "mha_talking: a row of %d holds no q, k and v of %d heads", stride, heads);
  const TalkShape a{{rows, stride, heads, kv_heads, dim, vdim, ring}, chunk, heads * vdim};
  hipStream_t s = (hipStream_t)stream;
  const bool aligned = stride % 8 == 0 && dim % 8 == 0 && vdim % 8 == 0 && (((uintptr_t)x | (uintptr_t)keys | (uintptr_t)values) & 15) == 0;
  IRON_REQUIRE(((uintptr_t)workspace & 15) == 0, "mha_talking: the workspace must be 16-byte aligned");
  if (single) {   // the caller's spans have one row at most
    const int each = heads / kv_heads, at_once = each == 1 ? 1 : (each <= 4 ? 4 : 8), sets = (each + at_once - 1) / at_once, threads = chunk >= 1024 ? 1024 : (chunk + 63) / 64 * 64;
    const size_t q_bytes = (size_t)each * dim * 4;
    IRON_REQUIRE(kv_heads * sets <= 65535 && q_bytes <= 64 * 1024 && heads <= 1024, "mha_talking: %d heads of %d (%d key heads) in a step",
                 heads, dim, kv_heads);
    float* work = (float*)workspace;
    constexpr int MIXED = 8;
#define IRON_TALK_VALUES(T, VEC, HEADS)                                                                                                     \
  hipLaunchKernelGGL((talking_values_kernel<T, VEC, HEADS>), dim3(vdim / VEC, kv_heads * sets, slots), dim3(threads), 0, s, (const T*)x,    \
                     (const T*)values, spans, work, (T*)out, a)
#define IRON_TALK_STEP(T, VEC)                                                                                                                \
  {                                                                                                                                           \
    hipLaunchKernelGGL((talking_scores_kernel<T, VEC>), dim3((chunk + 63) / 64, kv_heads, slots), dim3(64), q_bytes, s, (const T*)x, (T*)keys, \
                       (T*)values, spans, work, a);                                                                                           \
    hipLaunchKernelGGL((talking_mix_kernel<T, MIXED>), dim3((chunk + 63) / 64, (heads + MIXED - 1) / MIXED, slots), dim3(64),                 \
                       (size_t)heads * (MIXED + 1) * 4, s, talk, spans, work, a);                                                             \
    if (at_once == 1) IRON_TALK_VALUES(T, VEC, 1);                                                                                            \
    else if (at_once == 4) IRON_TALK_VALUES(T, VEC, 4);                                                                                       \
    else IRON_TALK_VALUES(T, VEC, 8);                                                                                                         \
  }
    if (is_float) { if (aligned) IRON_TALK_STEP(float, 8) else IRON_TALK_STEP(float, 1) }
    else { if (aligned) IRON_TALK_STEP(bf16_t, 8) else IRON_TALK_STEP(bf16_t, 1) }
#undef IRON_TALK_VALUES
#undef IRON_TALK_STEP
    IRON_LAUNCH_CHECK();
  }
  const size_t lds = (size_t)talk_row_words(heads, dim, vdim) * 4;
  const int groups = aligned && ((uintptr_t)out & 7) == 0 ? talking_groups(heads, kv_heads, dim, vdim, is_float) : 0;
  if (groups > 0) {
    IRON_REQUIRE(rows <= 65535 && stride < (1 << 24) && (long)rows * stride < (1L << 31) && (long)chunk * kv_heads * (dim > vdim ? dim : vdim) < (1L << 31) && chunk < (1 << 24),
                 "mha_talking: %d rows of %d, chunks of %d: a row's place takes 32 bits", rows, stride, chunk);
    const bf16_t *xb = (const bf16_t*)x, *kb = (const bf16_t*)keys, *vb = (const bf16_t*)values;
    float* stats = (float*)workspace;
    const dim3 grid(heads, (rows + 63) / 64 + slots - 1);
    if (dim <= 64) hipLaunchKernelGGL((talking_stats_kernel<2>), grid, dim3(256), 0, s, xb, kb, spans, stats, slots, a);
    else hipLaunchKernelGGL((talking_stats_kernel<4>), grid, dim3(256), 0, s, xb, kb, spans, stats, slots, a);
    const bool fours = heads / kv_heads % 4 == 0;
    int e;
#define IRON_TALK(NG, KD, VT)                                                                                                \
  e = fours ? launch_talking_prompt<NG, KD, VT, 4>(xb, kb, vb, talk, spans, stats, (bf16_t*)out, a, slots, s)                \
            : launch_talking_prompt<NG, KD, VT, 1>(xb, kb, vb, talk, spans, stats, (bf16_t*)out, a, slots, s)
#define IRON_TALKS(NG)                                       \
  {                                                          \
    if (dim <= 64 && vdim <= 64) IRON_TALK(NG, 2, 4);        \
    else if (dim <= 64) IRON_TALK(NG, 2, 8);                 \
    else if (vdim <= 64) IRON_TALK(NG, 4, 4);                \
    else IRON_TALK(NG, 4, 8);                                \
  }
    if (groups == 1) IRON_TALKS(1)
    else if (groups == 2) IRON_TALKS(2)
    else IRON_TALKS(4)
#undef IRON_TALKS
#undef IRON_TALK
    if (e != IRON_OK) return e;
    launch_ring_store<bf16_t>(x, keys, values, spans, a.p, slots, s);
    IRON_LAUNCH_CHECK();
  }
  IRON_REQUIRE(lds <= 160 * 1024, "mha_talking: %d heads of %d + %d need %zu bytes of LDS", heads, dim, vdim, lds);
#define IRON_TALK_ROWS(T, VEC)                                                                                                          \
  {                                                                                                                                     \
    static LdsOptIn opt;                                                                                                                \
    const hipError_t e = opt.ensure(reinterpret_cast<const void*>(&talking_rows_kernel<T, VEC>), 160 * 1024);                           \
    if (e != hipSuccess) { set_error("%s", hipGetErrorString(e)); return (int)e; }                                                      \
    hipLaunchKernelGGL((talking_rows_kernel<T, VEC>), dim3(rows, slots), dim3(256), lds, s, (const T*)x, (const T*)keys,                \
                       (const T*)values, talk, spans, (T*)out, a);                                                                      \
  }
  if (is_float) { if (aligned) IRON_TALK_ROWS(float, 8) else IRON_TALK_ROWS(float, 1) }
  else { if (aligned) IRON_TALK_ROWS(bf16_t, 8) else IRON_TALK_ROWS(bf16_t, 1) }
#undef IRON_TALK_ROWS
  if (is_float) launch_ring_store<float>(x, keys, values, spans, a.p, slots, s);
  else launch_ring_store<bf16_t>(x, keys, values, spans, a.p, slots, s);
  IRON_LAUNCH_CHECK();
}
