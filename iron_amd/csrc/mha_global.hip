// Causal attention over whole sequences, a batch of spans: scores through a soft cap (cap tanh(score / cap)) where the design has
// one, softmax, with one more in its denominator where the design has that sink, keys and values of different widths, grouped
// query heads.
//
// cached_heads makes a packed projection's rows [q heads | k heads | v heads] ready: q and k normed a head and turned by position,
// v over its root mean square; q out, a position's key and value into its row of the slot's cache, a key head's rows one after
// the other.  A call's own rows are in the cache before they are attended.
//
//   rows kernel:    a block a query row and head, waves splitting the keys (any sizes, either type)
//   prefill kernel: bf16 MFMA flash attention, 64 or 128 queries a block
//   step kernels:   one row a slot: the keys dealt to blocks, up to 16 query heads of a key head the columns of an MFMA; a launch
//                   that adds the blocks' sums
//
// Scores behind a cap are bounded.  Where their exponentials cannot leave a float's range either way (SCORES_FIXED) they are taken
// as they are: no largest score is looked for and nothing is rescaled.
#include "../../include/iron_hip.h"
#include "router.h"
#include "window.h"

namespace iron {

constexpr float GLOBAL_LOG2E = 1.4426950408889634f;
constexpr float FIXED_BOUND = 60.f;   // of a score in powers of two: 2^60 times a context's keys is far inside a float
enum { SCORES_PLAIN = 0, SCORES_CAPPED = 1, SCORES_FIXED = 2 };

// --------------------------------------------------------------- the rows
struct CacheShape {
  int rows, stride, slots, heads, kv_heads, dim, vdim, context;
  int turned, angle_rows, value_norm;
  float eps;
};
struct CacheIn {
  const bf16_t *q_gain, *k_gain;
  const float* angles;                   // [angle_rows][turned]: cos and sin side by side
};

// LANES lanes a head, 8 consecutive columns each (VEC), or a wave a head, column by column.  A row's heads from unit `first` on,
// every `step`-th set of as many as the block takes at once.
template <typename T, int LANES, bool VEC>
__device__ __forceinline__ void cached_row(const T* __restrict__ x, T* __restrict__ q, T* __restrict__ keys, T* __restrict__ values, const CacheIn& in,
                                           const CacheShape& a, const Span& s, int slot, int row, int first, int step) {
  const int pos = s.start + row - s.row0, half = a.turned / 2;
  if (pos >= a.context) return;
  const float* turn = in.angles + (size_t)min(pos, a.angle_rows - 1) * a.turned;
  const int lane = threadIdx.x % LANES, qk = a.heads + a.kv_heads, units = qk + a.kv_heads;
  for (int u = first + threadIdx.x / LANES; u < units; u += step) {
    const bool value = u >= qk, query = u < a.heads;
    const int at = value ? qk * a.dim + (u - qk) * a.vdim : u * a.dim, n = value ? a.vdim : a.dim;
    const T* xr = x + (size_t)row * a.stride + at;
    T* to = query ? q + ((size_t)row * a.heads + u) * a.dim
                  : (value ? values + (((size_t)slot * a.kv_heads + u - qk) * a.context + pos) * a.vdim
                           : keys + (((size_t)slot * a.kv_heads + u - a.heads) * a.context + pos) * a.dim);
    const bf16_t* gain = query ? in.q_gain : in.k_gain;
    const bool normed = !value || a.value_norm;
    constexpr int MINE = VEC ? 8 : 1;
    float sum = 0.f, f[MINE];
    const int c0 = lane * MINE;
    if constexpr (VEC) {
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] = 0.f;
      if (c0 < n) load_vec<8>(xr + c0, f);
#pragma unroll
      for (int j = 0; j < 8; ++j) sum = fmaf(f[j], f[j], sum);
#pragma unroll
      for (int m = 1; m < LANES; m <<= 1) sum += __shfl_xor(sum, m, 64);
    } else {
      for (int c = lane; c < n; c += LANES) {
        const float v = load_one(xr + c);
        sum = fmaf(v, v, sum);
      }
      sum = wave_sum(sum);
    }
    const float inv = normed ? 1.0f / sqrtf(sum / (float)n + a.eps) : 1.f;
    // what column c becomes, v its projection
    auto made = [&](int c, float v) {
      v *= inv;
      if (value) return v;
      v *= bf16_to_f32(gain[c]);
      if (c >= a.turned) return v;
      const int i = c < half ? c : c - half, other = c < half ? c + half : i;
      const float o = load_one(xr + other) * inv * bf16_to_f32(gain[other]), cs = turn[2 * i], sn = turn[2 * i + 1];
      return c < half ? v * cs - o * sn : v * cs + o * sn;
    };
    if constexpr (VEC) {
      if (c0 >= n) continue;
      if (value || c0 >= a.turned || half % 8 != 0) {
#pragma unroll
        for (int j = 0; j < 8; ++j) f[j] = made(c0 + j, f[j]);
      } else {   // the eight partners side by side
        const bool first = c0 < half;
        const int i = first ? c0 : c0 - half, other = first ? c0 + half : i;
        float o[8], g[8], og[8], t[16];
        load_vec<8>(xr + other, o);
        load_vec<8>(gain + c0, g);
        load_vec<8>(gain + other, og);
#pragma unroll
        for (int j = 0; j < 8; ++j) reinterpret_cast<float2*>(t)[j] = reinterpret_cast<const float2*>(turn + 2 * i)[j];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float v = f[j] * inv * g[j], w = o[j] * inv * og[j];
          f[j] = first ? v * t[2 * j] - w * t[2 * j + 1] : v * t[2 * j] + w * t[2 * j + 1];
        }
      }
      store_vec<8>(to + c0, f);
    } else {
      for (int c = lane; c < n; c += LANES) store_one(to + c, made(c, load_one(xr + c)));
    }
  }
}

template <typename T, int LANES, bool VEC>
__global__ __launch_bounds__(256) void cached_heads_kernel(const T* __restrict__ x, T* __restrict__ q, T* __restrict__ keys,
                                                           T* __restrict__ values, const int* __restrict__ spans, CacheIn in, CacheShape a,
                                                           const int* __restrict__ valid) {
  const int row = blockIdx.x;
  if (row >= bound_or(valid, a.rows)) return;
  const int slot = slot_of_row(spans, a.slots, a.rows, row);
  if (slot < 0) return;
  cached_row<T, LANES, VEC>(x, q, keys, values, in, a, span_of(spans, slot, a.rows), slot, row, blockIdx.y * (256 / LANES), gridDim.y * (256 / LANES));
}

// One row a slot, bf16: its heads dealt to the first blocks, beside them a feed-forward's gated columns of the row, and a router's
// choice for slot 0.
struct StepColumns {
  bf16_t* out;                            // the rows the columns go to
  int out_stride, cols, gate_at, gated_at, kind;
  float limit;
};
template <int LANES>
__global__ __launch_bounds__(256) void decode_heads_kernel(const bf16_t* __restrict__ x, bf16_t* __restrict__ q, bf16_t* __restrict__ keys,
                                                           bf16_t* __restrict__ values, const int* __restrict__ spans, CacheIn in, CacheShape a,
                                                           StepColumns g, RouterChoice choice) {
  constexpr int AT_ONCE = 256 / LANES;
  __shared__ float lds[2][ROUTER_MAX];
  const int slot = blockIdx.y, head_blocks = (a.heads + 2 * a.kv_heads + AT_ONCE - 1) / AT_ONCE, block = blockIdx.x;
  const Span s = span_of(spans, slot, a.rows);
  if (choice.z != nullptr && block == (int)gridDim.x - 1) {   // (whether the slot has a row or not, as the router by itself)
    choose_row(choice, lds[0], lds[1]);
    return;
  }
  if (s.rows == 0) return;
  if (block < head_blocks) {
    cached_row<bf16_t, LANES, true>(x, q, keys, values, in, a, s, slot, s.row0, block * AT_ONCE, 1 << 30);
    return;
  }
  const int c = (block - head_blocks) * 256 + threadIdx.x;
  const bf16_t* row = x + (size_t)s.row0 * a.stride + g.gate_at;
  if (c < g.cols)
    g.out[(size_t)s.row0 * g.out_stride + g.gated_at + c] = f32_to_bf16(gated_value(g.kind, g.limit, bf16_to_f32(row[c]), bf16_to_f32(row[g.cols + c])));
}

// ------------------------------------------------------------ row by row
struct GlobalShape {
  int slots, rows, heads, kv_heads, dim, vdim, context;
  int out_stride, out_at, sink;
  float scale, cap;
};

// NW waves to a query row and head.  A wave takes 64 keys at a time: a key a lane for the scores, then columns over the lanes.
constexpr int GLOBAL_COLUMNS = 4;   // columns a lane holds: vdim up to 256
template <typename T, int VEC, int NW>
__global__ __launch_bounds__(NW * 64) void global_rows_kernel(const T* __restrict__ q, const T* __restrict__ keys, const T* __restrict__ values,
                                                              const int* __restrict__ spans, T* __restrict__ out, GlobalShape a) {
  __shared__ float qs[256], ps[NW][64], ms[NW], ls[NW], red[NW][256];
  const int head = blockIdx.x, i = blockIdx.y, slot = blockIdx.z;
  const Span s = span_of(spans, slot, a.rows);
  if (i >= s.rows) return;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, g = head / (a.heads / a.kv_heads);
  const int count = min(s.start + i + 1, a.context);
  const T* kr = keys + ((size_t)slot * a.kv_heads + g) * a.context * a.dim;
  const T* vr = values + ((size_t)slot * a.kv_heads + g) * a.context * a.vdim;
  for (int c = t; c < a.dim; c += NW * 64) qs[c] = load_one(q + ((size_t)(s.row0 + i) * a.heads + head) * a.dim + c) * a.scale;
  __syncthreads();
  float acc[GLOBAL_COLUMNS], m = a.sink ? 0.f : -INFINITY, l = a.sink && t == 0 ? 1.f : 0.f;
#pragma unroll
  for (int e = 0; e < GLOBAL_COLUMNS; ++e) acc[e] = 0.f;
  for (int k0 = wave * 64; k0 < count; k0 += NW * 64) {
    float score = -INFINITY;
    if (k0 + lane < count) {
      const T* at = kr + (size_t)(k0 + lane) * a.dim;
      float dot = 0.f;
#pragma unroll 4
      for (int c = 0; c < a.dim; c += VEC) {
        float f[VEC];
        load_vec<VEC>(at + c, f);
#pragma unroll
        for (int j = 0; j < VEC; ++j) dot = fmaf(f[j], qs[c + j], dot);
      }
      score = a.cap > 0.f ? a.cap * tanhf(dot / a.cap) : dot;
    }
    const float top = fmaxf(m, wave_max(score));   // finite: this piece has a key
    const float fade = expf(m - top), p = expf(score - top);
    m = top;
    l = l * fade + p;
    ps[wave][lane] = p;
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int e = 0; e < GLOBAL_COLUMNS; ++e) acc[e] *= fade;
    const int n = min(64, count - k0);
    for (int j = 0; j < n; ++j) {
      const T* at = vr + (size_t)(k0 + j) * a.vdim;
      const float w = ps[wave][j];
#pragma unroll
      for (int e = 0; e < GLOBAL_COLUMNS; ++e)
        if (lane + 64 * e < a.vdim) acc[e] = fmaf(w, load_one(at + lane + 64 * e), acc[e]);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  l = wave_sum(l);
  if (lane == 0) {
    ms[wave] = m;
    ls[wave] = l;
  }
#pragma unroll
  for (int e = 0; e < GLOBAL_COLUMNS; ++e)
    if (lane + 64 * e < a.vdim) red[wave][lane + 64 * e] = acc[e];
  __syncthreads();
  float top = ms[0], total = 0.f;   // (the first wave has a key)
#pragma unroll
  for (int w = 1; w < NW; ++w) top = fmaxf(top, ms[w]);
#pragma unroll
  for (int w = 0; w < NW; ++w) total += ls[w] * expf(ms[w] - top);   // a wave without a key: 0
  for (int c = t; c < a.vdim; c += NW * 64) {
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) sum = fmaf(red[w][c], expf(ms[w] - top), sum);
    store_one(out + (size_t)(s.row0 + i) * a.out_stride + a.out_at + head * a.vdim + c, sum / total);
  }
}

// -------------------------------------------------------------- on the MFMAs
// Scores are computed transposed (keys down the MFMA's rows, queries across its columns): a lane holds one query's scores, so the
// row statistics are a lane's own, and the weights are the second product's B operand as they stand.

// A score in powers of two behind its cap: C tanh(s / cap) with C = cap log2(e), by way of 1 - 2 / (1 + exp(2 s / cap)).
struct Capping {
  float by, c2, c;   // 2 scale log2(e) / cap, -2 C, C
  __device__ __forceinline__ explicit Capping(const GlobalShape& a)
      : by(a.cap > 0.f ? 2.f * a.scale * GLOBAL_LOG2E / a.cap : 0.f), c2(-2.f * a.cap * GLOBAL_LOG2E), c(a.cap * GLOBAL_LOG2E) {}
  __device__ __forceinline__ float operator()(float dot) const {
    return fmaf(c2, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(dot * by)), c);
  }
};

constexpr int GLOBAL_KEYS = 64;   // keys a tile
template <int DKP, int DVP>
struct GlobalShared {
  __align__(16) bf16_t k[GLOBAL_KEYS][DKP + 8];
  __align__(16) bf16_t vt[DVP][GLOBAL_KEYS + 8];
};

// A block takes QT * 64 queries of one head, QT * 16 a wave, and walks the keys 64 at a time.
template <int DKP, int DVP, int QT, int MODE>
__global__ __launch_bounds__(256, DKP + DVP <= 256 ? 2 : 1) void global_prefill_kernel(const bf16_t* __restrict__ q, const bf16_t* __restrict__ keys,
                                                                                       const bf16_t* __restrict__ values,
                                                                                       const int* __restrict__ spans, bf16_t* __restrict__ out,
                                                                                       GlobalShape a) {
  constexpr bool FIXED = MODE == SCORES_FIXED;
  constexpr int BQ = QT * 64, KD = DKP / 32, VD = DVP / 16;
  constexpr int BUFFERS = DKP + DVP <= 256 ? 2 : 1;
  constexpr int KP = GLOBAL_KEYS * DKP / 8 / 256;      // 16-byte pieces of a key tile a thread stages
  constexpr int VP = (GLOBAL_KEYS / 4) * (DVP / 8);    // four-key pieces of a value tile
  constexpr int VT = (VP + 255) / 256;
  __shared__ GlobalShared<DKP, DVP> tiles_lds[BUFFERS];
  int slot, q0;
  if (!tile_of(spans, a.slots, a.rows, BQ, (int)gridDim.y - 1 - (int)blockIdx.y, slot, q0)) return;   // the longest first
  const Span s = span_of(spans, slot, a.rows);
  // Where the heads divide by the XCDs, those of a group on one XCD, whose L2 then reads their keys and values once.
  const int x8 = blockIdx.x, head = a.heads % 8 == 0 ? (x8 & 7) * (a.heads >> 3) + (x8 >> 3) : x8;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, lo16 = lane & 15, quad = lane >> 4, g = head / (a.heads / a.kv_heads);
  const int end = min(s.start + s.rows, a.context);                                // first position without a key
  const int first_pos = s.start + q0, last_pos = min(first_pos + BQ, end) - 1;     // the block's queries
  const int tiles = last_pos / GLOBAL_KEYS + 1;

  bf16x8 qf[QT][KD];
#pragma unroll
  for (int u = 0; u < QT; ++u) {
    const int i = q0 + wave * QT * 16 + u * 16 + lo16;
#pragma unroll
    for (int d = 0; d < KD; ++d) {
      const int c = d * 32 + quad * 8;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (i < s.rows && c < a.dim) v = *reinterpret_cast<const uint4*>(q + ((size_t)(s.row0 + i) * a.heads + head) * a.dim + c);
      qf[u][d] = __builtin_bit_cast(bf16x8, v);
    }
  }
  f32x4 acc[QT][VD];
  float m[QT], l[QT];
#pragma unroll
  for (int u = 0; u < QT; ++u) {
    m[u] = a.sink || FIXED ? 0.f : -1e30f;
    l[u] = a.sink && quad == 0 ? 1.f : 0.f;   // (a query's sum is over its four lanes)
#pragma unroll
    for (int d = 0; d < VD; ++d) acc[u][d] = f32x4{0.f, 0.f, 0.f, 0.f};
  }

  // The next tile on its way from memory, by 32-bit offsets into bounded buffers: rows past the last key, which may hold anything,
  // read as zeros.  Columns past a head's width read its last ones: q is zero there, and those of v are not stored.
  const __amdgpu_buffer_rsrc_t kb = bounded_bytes(keys + ((size_t)slot * a.kv_heads + g) * a.context * a.dim, end * a.dim * 2);
  const __amdgpu_buffer_rsrc_t vb = bounded_bytes(values + ((size_t)slot * a.kv_heads + g) * a.context * a.vdim, end * a.vdim * 2);
  auto v_row = [&](int e) { return (e >> 2) & 15; };                      // a piece's keys, in fours
  auto v_col = [&](int e) { return ((e >> 6) * 4 + (e & 3)) * 8; };       // ... and its columns
  u32x4 kn[KP], vn[VT][4];
  int k_at[KP], v_at[VT];
#pragma unroll
  for (int i = 0; i < KP; ++i) {
    const int e = t + 256 * i;
    k_at[i] = (e / (DKP / 8) * a.dim + min((e % (DKP / 8)) * 8, a.dim - 8)) * 2;
  }
#pragma unroll
  for (int i = 0; i < VT; ++i) {
    const int e = t + 256 * i;
    v_at[i] = (v_row(e) * 4 * a.vdim + min(v_col(e), a.vdim - 8)) * 2;
  }
  auto fetch = [&](int base) {
    const int ko = base * a.dim * 2, vo = base * a.vdim * 2;
#pragma unroll
    for (int i = 0; i < KP; ++i) kn[i] = __builtin_amdgcn_raw_buffer_load_b128(kb, k_at[i], ko, 0);
#pragma unroll
    for (int i = 0; i < VT; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) vn[i][j] = __builtin_amdgcn_raw_buffer_load_b128(vb, v_at[i], vo + j * a.vdim * 2, 0);
  };
  fetch(0);
  const Capping capped(a);
  const float scale = a.scale * GLOBAL_LOG2E;
  for (int n = 0; n < tiles; ++n) {
    const int base = n * GLOBAL_KEYS;
    GlobalShared<DKP, DVP>& sh = tiles_lds[BUFFERS == 2 ? n & 1 : 0];   // two: its last readers are behind the barrier between
    if (BUFFERS == 1 && n > 0) block_barrier_lds();
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int e = t + 256 * i;
      *reinterpret_cast<u32x4*>(&sh.k[e / (DKP / 8)][(e % (DKP / 8)) * 8]) = kn[i];
    }
#pragma unroll
    for (int i = 0; i < VT; ++i) {
      const int e = t + 256 * i, r4 = v_row(e), c = v_col(e);
      if (e < VP) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {   // two columns at a time: four keys each, 8 bytes
          const uint32_t w0 = vn[i][0][j], w1 = vn[i][1][j], w2 = vn[i][2][j], w3 = vn[i][3][j];
          *reinterpret_cast<uint2*>(&sh.vt[c + 2 * j][r4 * 4]) = make_uint2((w0 & 0xffffu) | (w1 << 16), (w2 & 0xffffu) | (w3 << 16));
          *reinterpret_cast<uint2*>(&sh.vt[c + 2 * j + 1][r4 * 4]) =
              make_uint2((w0 >> 16) | (w1 & 0xffff0000u), (w2 >> 16) | (w3 & 0xffff0000u));
        }
      }
    }
    block_barrier_lds();
    if (n + 1 < tiles) fetch(base + GLOBAL_KEYS);

    f32x4 sc[QT][4];
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
      bf16x8 kf[KD];
#pragma unroll
      for (int d = 0; d < KD; ++d) kf[d] = *reinterpret_cast<const bf16x8*>(&sh.k[kt * 16 + lo16][d * 32 + quad * 8]);
#pragma unroll
      for (int u = 0; u < QT; ++u) {
        sc[u][kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int d = 0; d < KD; ++d) sc[u][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[d], qf[u][d], sc[u][kt], 0, 0, 0);
      }
    }
    const bool edge = base + GLOBAL_KEYS - 1 > first_pos;   // some query does not see every key
    bf16x8 pf[QT][2];
#pragma unroll
    for (int u = 0; u < QT; ++u) {
      if constexpr (MODE != SCORES_PLAIN) {
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int r = 0; r < 4; ++r) sc[u][kt][r] = capped(sc[u][kt][r]);
      } else {
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) sc[u][kt] *= scale;
      }
      if (edge) {
        const int ahead = first_pos + wave * QT * 16 + u * 16 + lo16 - base - quad * 4;   // i - j of the lane's first key
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int r = 0; r < 4; ++r) sc[u][kt][r] = ahead >= kt * 16 + r ? sc[u][kt][r] : -INFINITY;
      }
      if constexpr (!FIXED) {
        float top = -INFINITY;
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) top = fmaxf(top, fmaxf(fmaxf(sc[u][kt][0], sc[u][kt][1]), fmaxf(sc[u][kt][2], sc[u][kt][3])));
        // The reference the exponents are taken from moves only where a score would exceed it by more than 2^8: it cancels in the
        // quotient, and the products need no rescaling between.
        if (__builtin_amdgcn_ballot_w64(top > m[u] + 8.f) != 0) {
          top = fmaxf(top, __shfl_xor(top, 16, 64));
          top = fmaxf(top, __shfl_xor(top, 32, 64));
          top = fmaxf(m[u], top);
          const float fade = __builtin_amdgcn_exp2f(m[u] - top);
          m[u] = top;
          l[u] *= fade;
#pragma unroll
          for (int d = 0; d < VD; ++d)
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[u][d][r] *= fade;
        }
      }
      float sum = 0.f;
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          sc[u][kt][r] = __builtin_amdgcn_exp2f(FIXED ? sc[u][kt][r] : sc[u][kt][r] - m[u]);
          sum += sc[u][kt][r];
        }
      l[u] += sum;
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const uint4 v = make_uint4(pack_bf16(sc[u][2 * h][0], sc[u][2 * h][1]), pack_bf16(sc[u][2 * h][2], sc[u][2 * h][3]),
                                   pack_bf16(sc[u][2 * h + 1][0], sc[u][2 * h + 1][1]), pack_bf16(sc[u][2 * h + 1][2], sc[u][2 * h + 1][3]));
        pf[u][h] = __builtin_bit_cast(bf16x8, v);
      }
    }
#pragma unroll
    for (int d = 0; d < VD; ++d)
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const uint2 lo = *reinterpret_cast<const uint2*>(&sh.vt[d * 16 + lo16][h * 32 + quad * 4]);
        const uint2 hi = *reinterpret_cast<const uint2*>(&sh.vt[d * 16 + lo16][h * 32 + 16 + quad * 4]);
        const bf16x8 vf = __builtin_bit_cast(bf16x8, make_uint4(lo.x, lo.y, hi.x, hi.y));
#pragma unroll
        for (int u = 0; u < QT; ++u) acc[u][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[u][h], acc[u][d], 0, 0, 0);
      }
  }
#pragma unroll
  for (int u = 0; u < QT; ++u) {
    float sum = l[u];
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    const int i = q0 + wave * QT * 16 + u * 16 + lo16;
    if (i >= s.rows) continue;
    const float inv = 1.0f / sum;
    bf16_t* to = out + (size_t)(s.row0 + i) * a.out_stride + a.out_at + head * a.vdim;
#pragma unroll
    for (int d = 0; d < VD; ++d) {
      const int c = d * 16 + quad * 4;
      if (c < a.vdim)
        *reinterpret_cast<uint2*>(to + c) = make_uint2(pack_bf16(acc[u][d][0] * inv, acc[u][d][1] * inv),
                                                       pack_bf16(acc[u][d][2] * inv, acc[u][d][3] * inv));
    }
  }
}

// -------------------------------------------------------------- a decode step
// One row a slot.  A block takes a run of the keys for up to 16 query heads of one key head, a wave 32 keys of it at a time.
constexpr int STEP_TILE = 32, STEP_BLOCK = 4 * STEP_TILE, STEP_HEADS = 16;
struct StepShape {
  int each, sets, splits;   // query heads a key head, blocks they take, runs there can be
  __host__ __device__ StepShape(int slots, int heads, int kv_heads, int context) {
    each = heads / kv_heads;
    sets = (each + STEP_HEADS - 1) / STEP_HEADS;
    const int most = (context + STEP_BLOCK - 1) / STEP_BLOCK, room = 1024 / (kv_heads * sets * slots);
    splits = room < 1 ? 1 : (room < most ? room : most);
  }
  __device__ int run(int count) const {   // keys of a run, where a sequence has `count`
    const int tiles = (count + STEP_BLOCK - 1) / STEP_BLOCK;
    return (tiles + splits - 1) / splits * STEP_BLOCK;
  }
};
// floats: the sums [slot][head][split][vdim], then (largest score in powers of two, sum of exponentials under it) [slot][head][split]
struct GlobalWork {
  size_t stats, words;
  __host__ __device__ GlobalWork(int slots, int heads, int vdim, int splits)
      : stats((size_t)slots * heads * splits * vdim), words(stats + (size_t)slots * heads * splits * 2) {}
};

template <int DKP, int DVP, int MODE>
__global__ __launch_bounds__(256) void global_step_kernel(const bf16_t* __restrict__ q, const bf16_t* __restrict__ keys,
                                                          const bf16_t* __restrict__ values, const int* __restrict__ spans,
                                                          float* __restrict__ work, GlobalShape a) {
  constexpr bool FIXED = MODE == SCORES_FIXED;
  constexpr int KD = DKP / 32, VD = DVP / 16, VT = DVP / 64, PITCH = STEP_TILE + 8;
  // Each wave's values, turned; then the waves' sums, [wave][head][column].
  constexpr int VALUES = 4 * DVP * PITCH * 2, SUMS = 4 * STEP_HEADS * (DVP + 4) * 4;
  __shared__ __align__(16) char lds[VALUES > SUMS ? VALUES : SUMS];
  __shared__ float ms[4][STEP_HEADS], ls[4][STEP_HEADS];
  const StepShape step(a.slots, a.heads, a.kv_heads, a.context);
  const int slot = blockIdx.z, g = blockIdx.y / step.sets, h0 = blockIdx.y % step.sets * STEP_HEADS;
  const Span s = span_of(spans, slot, a.rows);
  const int count = min(s.start + 1, a.context), run = step.run(count), begin = (int)blockIdx.x * run, end = min(count, begin + run);
  if (s.rows == 0 || begin >= count) return;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, l16 = lane & 15, quad = lane >> 4;
  const bf16_t* kr = keys + ((size_t)slot * a.kv_heads + g) * a.context * a.dim;
  const bf16_t* vr = values + ((size_t)slot * a.kv_heads + g) * a.context * a.vdim;
  bf16_t* vt = reinterpret_cast<bf16_t*>(lds) + wave * DVP * PITCH;
  auto v_row = [&](int e) { return ((e >> 2) & 7) * 4; };
  auto v_col = [&](int e) { return ((e >> 5) * 4 + (e & 3)) * 8; };
  bf16x8 kf[2][KD], qf[KD];
  u32x4 vn[VT][4];
  auto fetch = [&](int base) {   // rows past the run's last are that one again: masked
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int d = 0; d < KD; ++d)
        kf[kt][d] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(kr + (size_t)min(base + kt * 16 + l16, end - 1) * a.dim + min(d * 32 + quad * 8, a.dim - 8)));
#pragma unroll
    for (int i = 0; i < VT; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j)
        vn[i][j] = *reinterpret_cast<const u32x4*>(vr + (size_t)min(base + v_row(lane + 64 * i) + j, end - 1) * a.vdim + min(v_col(lane + 64 * i), a.vdim - 8));
  };
  fetch(begin + wave * STEP_TILE);
  const bool live = h0 + l16 < step.each;
#pragma unroll
  for (int d = 0; d < KD; ++d) {
    const int c = d * 32 + quad * 8;
    u32x4 v = *reinterpret_cast<const u32x4*>(q + ((size_t)s.row0 * a.heads + g * step.each + min(h0 + l16, step.each - 1)) * a.dim + min(c, a.dim - 8));
    if (!live || c >= a.dim) v = u32x4{0, 0, 0, 0};
    qf[d] = __builtin_bit_cast(bf16x8, v);
  }
  f32x4 acc[VD];
#pragma unroll
  for (int d = 0; d < VD; ++d) acc[d] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = FIXED ? 0.f : -1e30f, l = 0.f;
  const Capping capped(a);
  const float scale = a.scale * GLOBAL_LOG2E;
  for (int base = begin + wave * STEP_TILE; base < end; base += STEP_BLOCK) {
    f32x4 sc[2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
      sc[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int d = 0; d < KD; ++d) sc[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[kt][d], qf[d], sc[kt], 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < VT; ++i) {
      const int r = v_row(lane + 64 * i), c = v_col(lane + 64 * i);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const uint32_t w0 = vn[i][0][j], w1 = vn[i][1][j], w2 = vn[i][2][j], w3 = vn[i][3][j];
        *reinterpret_cast<uint2*>(vt + (c + 2 * j) * PITCH + r) = make_uint2((w0 & 0xffffu) | (w1 << 16), (w2 & 0xffffu) | (w3 << 16));
        *reinterpret_cast<uint2*>(vt + (c + 2 * j + 1) * PITCH + r) = make_uint2((w0 >> 16) | (w1 & 0xffff0000u), (w2 >> 16) | (w3 & 0xffff0000u));
      }
    }
    if (base + STEP_BLOCK < end) fetch(base + STEP_BLOCK);
    float top = -INFINITY;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float v = MODE != SCORES_PLAIN ? capped(sc[kt][r]) : sc[kt][r] * scale;
        sc[kt][r] = base + kt * 16 + quad * 4 + r < end ? v : -INFINITY;
        top = fmaxf(top, sc[kt][r]);
      }
    if constexpr (!FIXED) {
      top = fmaxf(top, __shfl_xor(top, 16, 64));
      top = fmaxf(top, __shfl_xor(top, 32, 64));
      top = fmaxf(m, top);
      const float fade = __builtin_amdgcn_exp2f(m - top);
      m = top;
      l *= fade;
#pragma unroll
      for (int d = 0; d < VD; ++d)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[d][r] *= fade;
    }
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        sc[kt][r] = __builtin_amdgcn_exp2f(FIXED ? sc[kt][r] : sc[kt][r] - m);
        l += sc[kt][r];
      }
    const bf16x8 pf = __builtin_bit_cast(bf16x8, make_uint4(pack_bf16(sc[0][0], sc[0][1]), pack_bf16(sc[0][2], sc[0][3]),
                                                            pack_bf16(sc[1][0], sc[1][1]), pack_bf16(sc[1][2], sc[1][3])));
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");   // the wave's own values
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int d = 0; d < VD; ++d) {
      const uint2 lo = *reinterpret_cast<const uint2*>(vt + (d * 16 + l16) * PITCH + quad * 4);
      const uint2 hi = *reinterpret_cast<const uint2*>(vt + (d * 16 + l16) * PITCH + 16 + quad * 4);
      acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, make_uint4(lo.x, lo.y, hi.x, hi.y)), pf, acc[d], 0, 0, 0);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (quad == 0) {
    ms[wave][l16] = m;
    ls[wave][l16] = l;
  }
  __syncthreads();   // also: every wave is done with its values
  float* sums = reinterpret_cast<float*>(lds);
#pragma unroll
  for (int d = 0; d < VD; ++d)
    *reinterpret_cast<float4*>(sums + (wave * STEP_HEADS + l16) * (DVP + 4) + d * 16 + quad * 4) = make_float4(acc[d][0], acc[d][1], acc[d][2], acc[d][3]);
  __syncthreads();
  const GlobalWork w(a.slots, a.heads, a.vdim, step.splits);
  const int mine = min(STEP_HEADS, step.each - h0);
  for (int e = t; e < mine * a.vdim; e += 256) {
    const int h = e / a.vdim, c = e - h * a.vdim;
    float top = ms[0][h], sum = 0.f;
#pragma unroll
    for (int v = 1; v < 4; ++v) top = fmaxf(top, ms[v][h]);
#pragma unroll
    for (int v = 0; v < 4; ++v) sum = fmaf(sums[(v * STEP_HEADS + h) * (DVP + 4) + c], FIXED ? 1.f : __builtin_amdgcn_exp2f(ms[v][h] - top), sum);
    const size_t at = ((size_t)slot * a.heads + g * step.each + h0 + h) * step.splits + blockIdx.x;
    work[at * a.vdim + c] = sum;
    if (c == 0) {
      float total = 0.f;
#pragma unroll
      for (int v = 0; v < 4; ++v) total = fmaf(ls[v][h], FIXED ? 1.f : __builtin_amdgcn_exp2f(ms[v][h] - top), total);
      reinterpret_cast<float2*>(work + w.stats)[at] = make_float2(top, total);
    }
  }
}

// The runs' sums of one head added: four columns a thread, runs over the rest of the block.
__global__ __launch_bounds__(256) void global_merge_kernel(const float* __restrict__ work, const int* __restrict__ spans, bf16_t* __restrict__ out,
                                                           GlobalShape a) {
  __shared__ __align__(16) float part[1024];
  __shared__ float by[1024], totals[4];
  const int head = blockIdx.x, slot = blockIdx.y, t = threadIdx.x;
  const Span s = span_of(spans, slot, a.rows);
  if (s.rows == 0) return;
  const StepShape step(a.slots, a.heads, a.kv_heads, a.context);
  const GlobalWork w(a.slots, a.heads, a.vdim, step.splits);
  const int count = min(s.start + 1, a.context), run = step.run(count), runs = (count + run - 1) / run;
  const size_t at = ((size_t)slot * a.heads + head) * step.splits;
  const float2* st = reinterpret_cast<const float2*>(work + w.stats) + at;
  const int pieces = a.vdim / 4, groups = 256 / pieces, c = t % pieces * 4, first = t / pieces;
  float4 ahead = make_float4(0.f, 0.f, 0.f, 0.f);   // the thread's first run, on its way
  if (first < groups && first < runs) ahead = *reinterpret_cast<const float4*>(work + (at + first) * a.vdim + c);
  float top = a.sink ? 0.f : -INFINITY;
  for (int i = t; i < runs; i += 256) top = fmaxf(top, st[i].x);
  top = wave_max(top);
  if ((t & 63) == 0) totals[t >> 6] = top;
  __syncthreads();
  top = fmaxf(fmaxf(totals[0], totals[1]), fmaxf(totals[2], totals[3]));
  float total = a.sink && t == 0 ? __builtin_amdgcn_exp2f(-top) : 0.f;
  for (int i = t; i < runs; i += 256) {
    const float fade = __builtin_amdgcn_exp2f(st[i].x - top);
    by[i] = fade;
    total = fmaf(st[i].y, fade, total);
  }
  total = wave_sum(total);
  __syncthreads();
  if ((t & 63) == 0) totals[t >> 6] = total;
  __syncthreads();
  total = totals[0] + totals[1] + totals[2] + totals[3];
  float4 sum = make_float4(0.f, 0.f, 0.f, 0.f);
  if (first < groups)
    for (int i = first; i < runs; i += groups) {
      const float4 v = i == first ? ahead : *reinterpret_cast<const float4*>(work + (at + i) * a.vdim + c);
      sum.x = fmaf(v.x, by[i], sum.x);
      sum.y = fmaf(v.y, by[i], sum.y);
      sum.z = fmaf(v.z, by[i], sum.z);
      sum.w = fmaf(v.w, by[i], sum.w);
    }
  if (first < groups) *reinterpret_cast<float4*>(part + first * a.vdim + c) = sum;
  __syncthreads();
  if (t >= a.vdim) return;
  float v = 0.f;
  for (int i = 0; i < groups; ++i) v += part[i * a.vdim + t];
  out[(size_t)s.row0 * a.out_stride + a.out_at + head * a.vdim + t] = f32_to_bf16(v / total);
}

template <int DKP, int MODE>
static void launch_global_step(const bf16_t* q, const bf16_t* keys, const bf16_t* values, const int* spans, float* work, const GlobalShape& a,
                               hipStream_t s) {
  const StepShape step(a.slots, a.heads, a.kv_heads, a.context);
  const dim3 grid(step.splits, a.kv_heads * step.sets, a.slots);
#define IRON_GLOBAL_STEP(DVP) hipLaunchKernelGGL((global_step_kernel<DKP, DVP, MODE>), grid, dim3(256), 0, s, q, keys, values, spans, work, a)
  if (a.vdim <= 64) IRON_GLOBAL_STEP(64);
  else if (a.vdim <= 128) IRON_GLOBAL_STEP(128);
  else IRON_GLOBAL_STEP(256);
#undef IRON_GLOBAL_STEP
}

template <int DKP, int MODE>
static void launch_global_prefill(const bf16_t* q, const bf16_t* keys, const bf16_t* values, const int* spans, bf16_t* out, const GlobalShape& a,
                                  hipStream_t s) {
  // 128 queries a block where narrow heads leave it the registers and that still gives the chip its blocks.
  const bool wide = (long)a.rows / 128 * a.heads >= 512;
#define IRON_GLOBAL(DVP, QT)                                                                                                                    \
  hipLaunchKernelGGL((global_prefill_kernel<DKP, DVP, QT, MODE>), dim3(a.heads, (a.rows + 64 * QT - 1) / (64 * QT) + a.slots - 1), dim3(256), 0, s, \
                     q, keys, values, spans, out, a)
#define IRON_GLOBALS(DVP)                                                     \
  {                                                                           \
    if (DKP + DVP <= 256 && wide) IRON_GLOBAL(DVP, (DKP + DVP <= 256 ? 2 : 1)); \
    else IRON_GLOBAL(DVP, 1);                                                 \
  }
  if (a.vdim <= 64) IRON_GLOBALS(64)
  else if (a.vdim <= 128) IRON_GLOBALS(128)
  else IRON_GLOBALS(256)
#undef IRON_GLOBALS
#undef IRON_GLOBAL
}

}  // namespace iron

using namespace iron;

extern "C" int iron_cached_heads(const void* x, void* q, void* keys, void* values, const uint16_t* q_gain, const uint16_t* k_gain,
                                 const float* angles, const int* spans, int slots, int rows, int stride, int heads, int kv_heads, int dim,
                                 int vdim, int context, int turned, int angle_rows, int value_norm, float eps, int is_float, const int* valid,
                                 void* stream) {
  IRON_REQUIRE(x && q && keys && values && q_gain && k_gain && spans && (turned == 0 || angles), "cached_heads: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0 && ((uintptr_t)angles & 7) == 0, "cached_heads: spans must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && rows > 0 && heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0 && context > 0, "cached_heads: sizes must be positive");
  IRON_REQUIRE(turned >= 0 && turned % 2 == 0 && turned <= dim && angle_rows > 0, "cached_heads: %d of %d columns turn, in pairs", turned, dim);
  IRON_REQUIRE(stride >= heads * dim + kv_heads * (dim + vdim), "cached_heads: a row of %d holds no q, k and v of %d heads", stride, heads);
  const CacheIn in{q_gain, k_gain, angles};
  const CacheShape a{rows, stride, slots, heads, kv_heads, dim, vdim, context, turned, angle_rows, value_norm, eps};
  const int wide = dim > vdim ? dim : vdim;
  const bool vec = dim % 8 == 0 && vdim % 8 == 0 && stride % 8 == 0 && wide <= 512 &&
                   (((uintptr_t)x | (uintptr_t)q | (uintptr_t)keys | (uintptr_t)values | (uintptr_t)q_gain | (uintptr_t)k_gain) & 15) == 0;
#define IRON_HEADS(T, LANES, VEC)                                                                                                          \
  hipLaunchKernelGGL((cached_heads_kernel<T, LANES, VEC>), dim3(rows, rows < 256 ? (heads + 2 * kv_heads + 256 / LANES - 1) / (256 / LANES) : 1), dim3(256), 0, (hipStream_t)stream, (const T*)x, (T*)q, (T*)keys, \
                     (T*)values, spans, in, a, valid)
#define IRON_HEADSS(T)                              \
  {                                                 \
    if (!vec) IRON_HEADS(T, 64, false);             \
    else if (wide <= 64) IRON_HEADS(T, 8, true);    \
    else if (wide <= 128) IRON_HEADS(T, 16, true);  \
    else if (wide <= 256) IRON_HEADS(T, 32, true);  \
    else IRON_HEADS(T, 64, true);                   \
  }
  if (is_float) IRON_HEADSS(float)
  else IRON_HEADSS(bf16_t)
#undef IRON_HEADSS
#undef IRON_HEADS
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_decode_heads_global_bf16(const uint16_t* x, uint16_t* q, uint16_t* keys, uint16_t* values, const uint16_t* q_gain,
                                             const uint16_t* k_gain, const float* angles, const int* spans, int slots, int rows, int stride,
                                             int heads, int kv_heads, int dim, int vdim, int context, int turned, int angle_rows, int value_norm,
                                             float eps, uint16_t* out, int out_stride, int cols, int gate_at, int gated_at, int kind, float limit,
                                             const float* z, const uint16_t* correction, int logits, int top, int* ids, float* shares,
                                             void* stream) {
  IRON_REQUIRE(x && q && keys && values && q_gain && k_gain && spans && (turned == 0 || angles), "decode_heads_global: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0 && ((uintptr_t)angles & 7) == 0, "decode_heads_global: spans must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0 && heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0 && context > 0,
               "decode_heads_global: sizes must be positive");
  IRON_REQUIRE(turned >= 0 && turned % 2 == 0 && turned <= dim && angle_rows > 0, "decode_heads_global: %d of %d columns turn, in pairs", turned, dim);
  IRON_REQUIRE(stride >= heads * dim + kv_heads * (dim + vdim), "decode_heads_global: a row of %d holds no q, k and v of %d heads", stride, heads);
  const int wide = dim > vdim ? dim : vdim;
  IRON_REQUIRE(dim % 8 == 0 && vdim % 8 == 0 && stride % 8 == 0 && wide <= 256 &&
                   (((uintptr_t)x | (uintptr_t)q | (uintptr_t)keys | (uintptr_t)values | (uintptr_t)q_gain | (uintptr_t)k_gain) & 15) == 0,
               "decode_heads_global: heads of whole 16-byte pieces up to 256 columns");
  IRON_REQUIRE(cols >= 0 && (cols == 0 || (out && gate_at >= 0 && gate_at + 2 * cols <= stride && gated_at >= 0 && gated_at + cols <= out_stride)),
               "decode_heads_global: twice %d gated columns from %d, into those from %d", cols, gate_at, gated_at);
  IRON_REQUIRE(kind >= 0 && kind <= 3, "decode_heads_global: kind (%d) is 0 to 3", kind);
  IRON_ROUTER_CHOICE_REQUIRE("decode_heads_global");
  const CacheIn in{q_gain, k_gain, angles};
  const CacheShape a{rows, stride, slots, heads, kv_heads, dim, vdim, context, turned, angle_rows, value_norm, eps};
  const StepColumns g{out, out_stride, cols, gate_at, gated_at, kind, limit};
  const RouterChoice choice{z, correction, logits, top, ids, shares};
#define IRON_STEP_HEADS(LANES)                                                                                                                    \
  hipLaunchKernelGGL((decode_heads_kernel<LANES>),                                                                                                \
                     dim3((heads + 2 * kv_heads + 256 / LANES - 1) / (256 / LANES) + (cols + 255) / 256 + (z != nullptr), slots), dim3(256), 0,    \
                     (hipStream_t)stream, x, q, keys, values, spans, in, a, g, choice)
  if (wide <= 64) IRON_STEP_HEADS(8);
  else if (wide <= 128) IRON_STEP_HEADS(16);
  else IRON_STEP_HEADS(32);
#undef IRON_STEP_HEADS
  IRON_LAUNCH_CHECK();
}

extern "C" int64_t iron_mha_global_workspace_bytes(int slots, int heads, int kv_heads, int vdim, int context, int single) {
  if (!single) return 0;
  return 4 * (int64_t)GlobalWork(slots, heads, vdim, StepShape(slots, heads, kv_heads, context).splits).words;
}

extern "C" int iron_mha_global(const void* q, const void* keys, const void* values, const int* spans, void* y, void* workspace, int slots,
                               int rows, int heads, int kv_heads, int dim, int vdim, int context, float scale, float cap, int sink,
                               int out_stride, int out_at, int single, int is_float, void* stream) {
  IRON_REQUIRE(q && keys && values && spans && y && (workspace || !single), "mha_global: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0 && ((uintptr_t)workspace & 15) == 0, "mha_global: spans and workspace must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0 && rows <= 65535, "mha_global: slots (%d) and rows (%d) from 1 to 65535", slots, rows);
  IRON_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "mha_global: kv_heads (%d) must divide heads (%d)", kv_heads, heads);
  IRON_REQUIRE(dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256, "mha_global: dim (%d) and vdim (%d) from 1 to 256", dim, vdim);
  IRON_REQUIRE(context > 0 && (long)context * (dim > vdim ? dim : vdim) < (1L << 30), "mha_global: a head's cache (%d rows) is addressed with 32-bit offsets", context);
  IRON_REQUIRE(cap >= 0.f && out_at >= 0 && out_at + heads * vdim <= out_stride, "mha_global: a cap (%g) not negative, %d columns from %d of an output row of %d",
               (double)cap, heads * vdim, out_at, out_stride);
  const GlobalShape a{slots, rows, heads, kv_heads, dim, vdim, context, out_stride, out_at, sink, scale, cap};
  hipStream_t s = (hipStream_t)stream;
  const bool aligned = dim % 8 == 0 && vdim % 8 == 0 && (((uintptr_t)q | (uintptr_t)keys | (uintptr_t)values) & 15) == 0;
  const int mode = cap <= 0.f ? SCORES_PLAIN : (cap * GLOBAL_LOG2E <= FIXED_BOUND ? SCORES_FIXED : SCORES_CAPPED);
  const bf16_t *qb = (const bf16_t*)q, *kb = (const bf16_t*)keys, *vb = (const bf16_t*)values;
#define IRON_BY_MODE(LAUNCH, WIDTH, ...)                              \
  {                                                                    \
    if (mode == SCORES_FIXED) LAUNCH<WIDTH, SCORES_FIXED>(__VA_ARGS__); \
    else if (mode == SCORES_CAPPED) LAUNCH<WIDTH, SCORES_CAPPED>(__VA_ARGS__); \
    else LAUNCH<WIDTH, SCORES_PLAIN>(__VA_ARGS__);                     \
  }
#define IRON_BY_WIDTH(LAUNCH, ...)                        \
  {                                                       \
    if (dim <= 64) IRON_BY_MODE(LAUNCH, 64, __VA_ARGS__)  \
    else if (dim <= 128) IRON_BY_MODE(LAUNCH, 128, __VA_ARGS__) \
    else IRON_BY_MODE(LAUNCH, 256, __VA_ARGS__)           \
  }
  if (single && !is_float && aligned) {   // the caller's spans have one row at most
    const StepShape step(slots, heads, kv_heads, context);
    IRON_REQUIRE(kv_heads * step.sets <= 65535 && step.splits <= 1024, "mha_global: %d key heads, %d runs of keys", kv_heads, step.splits);
    float* work = (float*)workspace;
    IRON_BY_WIDTH(launch_global_step, qb, kb, vb, spans, work, a, s)
    hipLaunchKernelGGL(global_merge_kernel, dim3(heads, slots), dim3(256), 0, s, work, spans, (bf16_t*)y, a);
    IRON_LAUNCH_CHECK();
  }
  if (!single && !is_float && aligned && out_stride % 4 == 0 && out_at % 4 == 0 && ((uintptr_t)y & 7) == 0) {
    IRON_BY_WIDTH(launch_global_prefill, qb, kb, vb, spans, (bf16_t*)y, a, s)
    IRON_LAUNCH_CHECK();
  }
#undef IRON_BY_WIDTH
#undef IRON_BY_MODE
#define IRON_GLOBAL_ROWS(T, VEC, NW)                                                                                                      \
  hipLaunchKernelGGL((global_rows_kernel<T, VEC, NW>), dim3(heads, single ? 1 : rows, slots), dim3(NW * 64), 0, s, (const T*)q, (const T*)keys, \
                     (const T*)values, spans, (T*)y, a)
#define IRON_GLOBAL_ROWSS(T)                                                                         \
  {                                                                                                  \
    if (single) { if (aligned) IRON_GLOBAL_ROWS(T, 8, 16); else IRON_GLOBAL_ROWS(T, 1, 16); }        \
    else { if (aligned) IRON_GLOBAL_ROWS(T, 8, 4); else IRON_GLOBAL_ROWS(T, 1, 4); }                 \
  }
  if (is_float) IRON_GLOBAL_ROWSS(float)
  else IRON_GLOBAL_ROWSS(bf16_t)
#undef IRON_GLOBAL_ROWSS
#undef IRON_GLOBAL_ROWS
  IRON_LAUNCH_CHECK();
}
