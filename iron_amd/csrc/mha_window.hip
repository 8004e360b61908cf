// Sliding-window attention with a learned bias by distance, over a batch of spans: score = q . k scale
// + bias[head][i - j] for 0 <= i - j < window, ordinary softmax, keys and values of different widths,
// grouped query heads.  A call's rows are the packed projection [q heads | k heads | v heads].
//
// The history is a ring of `ring` >= window rows a slot (position p in row p % ring).  A span's own keys
// and values are read from the projection's rows, so the ring is written after they have been attended,
// and needs no room for a prompt's portion.
//
//   rows kernel:    a block a query row and head, waves splitting the keys (decode; either type)
//   prefill kernel: bf16 MFMA flash attention, 64 or 128 queries a block
#include "../../include/iron_hip.h"
#include "window.h"

namespace iron {

struct WindowShape {
  int rows, stride;                      // the projection's rows, and their length
  int heads, kv_heads, dim, vdim;
  int window, ring;
  int out_stride, out_at;                // the output's rows, and the first of the heads' columns there
  float scale, out_scale;
};

constexpr float LOG2E = 1.4426950408889634f;

// --------------------------------------------------------------- row by row
// NW waves to a query row and head.  A wave takes 64 keys at a time: a key a lane for the scores, then
// VEC columns a lane (as many keys at once as rows of vdim fit a wave) for the weighted sum.
// STORE: the span is one row, and the first head of each group leaves its key and value in the ring.
template <typename T, int VEC, int NW, bool STORE>
__global__ __launch_bounds__(NW * 64) void window_rows_kernel(const T* __restrict__ x, T* __restrict__ keys, T* __restrict__ values,
                                                              const float* __restrict__ bias, const int* __restrict__ spans,
                                                              T* __restrict__ out, WindowShape a) {
  constexpr int EACH = VEC == 8 ? 1 : 4;              // column pieces a lane holds: vdim up to 512 or 256
  __shared__ float qs[256], ps[NW][64], ms[NW], ls[NW];
  extern __shared__ float red[];                      // [NW][groups][vdim]
  const int head = blockIdx.x, slot = blockIdx.y, i = blockIdx.z;
  const Span s = span_of(spans, slot, a.rows);
  if (i >= s.rows || (STORE && i > 0)) return;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
  const int g = head / (a.heads / a.kv_heads), nk = a.kv_heads * a.dim, nv = a.kv_heads * a.vdim;
  const int pos = s.start + i, lo = max(0, pos - a.window + 1), count = pos - lo + 1;
  const T* row = x + (size_t)(s.row0 + i) * a.stride;
  const T* own_k = x + a.heads * a.dim + g * a.dim;   // + a row of the call: that row's key for this group
  const T* own_v = x + a.heads * a.dim + nk + g * a.vdim;
  const T* ring_k = keys + (size_t)slot * a.ring * nk + g * a.dim;
  const T* ring_v = values + (size_t)slot * a.ring * nv + g * a.vdim;
  for (int c = t; c < a.dim; c += NW * 64) qs[c] = load_one(row + head * a.dim + c) * a.scale;
  if (STORE && head % (a.heads / a.kv_heads) == 0) {
    T* kd = keys + ((size_t)slot * a.ring + pos % a.ring) * nk + g * a.dim;
    T* vd = values + ((size_t)slot * a.ring + pos % a.ring) * nv + g * a.vdim;
    const T* kr = own_k + (size_t)(s.row0 + i) * a.stride;
    const T* vr = own_v + (size_t)(s.row0 + i) * a.stride;
    for (int c = t; c < a.dim; c += NW * 64) kd[c] = kr[c];
    for (int c = t; c < a.vdim; c += NW * 64) vd[c] = vr[c];
  }
  __syncthreads();

  const int pieces = VEC == 8 ? a.vdim / 8 : min(a.vdim, 64);   // lanes a value row takes
  const int groups = 64 / pieces, mine = lane / pieces, piece = lane - mine * pieces;
  float acc[EACH][VEC], m = -INFINITY, l = 0.f;
#pragma unroll
  for (int e = 0; e < EACH; ++e)
#pragma unroll
    for (int j = 0; j < VEC; ++j) acc[e][j] = 0.f;
  auto key_at = [&](int p) {
    return p >= s.start ? own_k + (size_t)(s.row0 + p - s.start) * a.stride : ring_k + (size_t)(p % a.ring) * nk;
  };
  auto value_at = [&](int p) {
    return p >= s.start ? own_v + (size_t)(s.row0 + p - s.start) * a.stride : ring_v + (size_t)(p % a.ring) * nv;
  };
  for (int k0 = wave * 64; k0 < count; k0 += NW * 64) {
    float score = -INFINITY;
    if (k0 + lane < count) {
      const int p = lo + k0 + lane;
      const T* kr = key_at(p);
      float dot = 0.f;
#pragma unroll 4
      for (int c = 0; c < a.dim; c += VEC) {
        float f[VEC];
        load_vec<VEC>(kr + c, f);
#pragma unroll
        for (int j = 0; j < VEC; ++j) dot = fmaf(f[j], qs[c + j], dot);
      }
      score = dot + bias[(size_t)head * a.window + (pos - p)];
    }
    const float top = fmaxf(m, wave_max(score));   // finite: this piece has a key
    const float fade = expf(m - top);
    const float p = expf(score - top);
    m = top;
    l = l * fade + p;
    ps[wave][lane] = p;
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int e = 0; e < EACH; ++e)
#pragma unroll
      for (int j = 0; j < VEC; ++j) acc[e][j] *= fade;
    const int n = min(64, count - k0);
    if (mine < groups)
#pragma unroll 4
      for (int q = mine; q < n; q += groups) {
        const T* vr = value_at(lo + k0 + q);
        const float w = ps[wave][q];
#pragma unroll
        for (int e = 0; e < EACH; ++e) {
          const int c = (piece + e * 64) * VEC;
          if (c >= a.vdim) continue;
          float f[VEC];
          load_vec<VEC>(vr + c, f);
#pragma unroll
          for (int j = 0; j < VEC; ++j) acc[e][j] = fmaf(w, f[j], acc[e][j]);
        }
      }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  l = wave_sum(l);
  if (lane == 0) {
    ms[wave] = m;
    ls[wave] = l;
  }
  if (mine < groups)
#pragma unroll
    for (int e = 0; e < EACH; ++e) {
      const int c = (piece + e * 64) * VEC;
      if (c < a.vdim)
#pragma unroll
        for (int j = 0; j < VEC; ++j) red[(size_t)(wave * groups + mine) * a.vdim + c + j] = acc[e][j];
    }
  __syncthreads();
  float top = ms[0];
#pragma unroll
  for (int w = 1; w < NW; ++w) top = fmaxf(top, ms[w]);
  float total = 0.f;
#pragma unroll
  for (int w = 0; w < NW; ++w) total += ls[w] * expf(ms[w] - top);   // a wave without a key: 0
  for (int c = t; c < a.vdim; c += NW * 64) {
    float sum = 0.f;
    for (int w = 0; w < NW; ++w) {
      float part = 0.f;
      for (int r = 0; r < groups; ++r) part += red[(size_t)(w * groups + r) * a.vdim + c];
      sum = fmaf(part, expf(ms[w] - top), sum);
    }
    store_one(out + (size_t)(s.row0 + i) * a.out_stride + a.out_at + head * a.vdim + c, sum / total * a.out_scale);
  }
}

// ------------------------------------------------------------------- prefill
// A block takes QT * 64 queries of one head, QT * 16 a wave, and walks the window 64 keys at a time.
// Scores are computed transposed (keys down the MFMA's rows, queries across its columns): a lane holds
// one query's scores, so the row statistics are a lane's own, and the weights are the second product's
// B operand as they stand (its sum over keys taken in the order the lanes hold them).  The bias, the
// window and the causal edge are one table of the distances a tile can meet, -inf where it is masked.
constexpr int WIN_KEYS = 64;

template <int DKP, int DVP>
struct WindowShared {
  __align__(16) bf16_t k[WIN_KEYS][DKP + 8];
  __align__(16) bf16_t vt[DVP][WIN_KEYS + 8];
  float by_distance[192 + 64];
};

template <int DKP, int DVP, int QT>
__device__ __forceinline__ void window_prefill_body(const bf16_t* __restrict__ x, const bf16_t* __restrict__ keys,
                                                    const bf16_t* __restrict__ values, const float* __restrict__ bias,
                                                    bf16_t* __restrict__ out, const WindowShape& a, const Span& s, int slot,
                                                    int head, int tile, WindowShared<DKP, DVP>* pair) {
  constexpr int BQ = QT * 64, KD = DKP / 32, VD = DVP / 16;
  constexpr int KP = WIN_KEYS * DKP / 8 / 256;         // 16-byte pieces of a key tile a thread stages
  constexpr int VP = (WIN_KEYS / 4) * (DVP / 8);       // four-key pieces of a value tile
  constexpr int VT = (VP + 255) / 256;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, lo16 = lane & 15, quad = lane >> 4;
  const int g = head / (a.heads / a.kv_heads), nk = a.kv_heads * a.dim, nv = a.kv_heads * a.vdim;
  const int q0 = tile * BQ;
  const int end = s.start + s.rows;                                          // first position without a key
  const int first_pos = s.start + q0, last_pos = min(first_pos + BQ, end) - 1;   // the block's queries
  const bf16_t* own_k = x + a.heads * a.dim + g * a.dim;
  const bf16_t* own_v = x + a.heads * a.dim + nk + g * a.vdim;
  const bf16_t* ring_k = keys + (size_t)slot * a.ring * nk + g * a.dim;
  const bf16_t* ring_v = values + (size_t)slot * a.ring * nv + g * a.vdim;
  // Tiles of the span's own keys start at its start, tiles of the ring's end there (the first may begin
  // before the window, or before position 0): no tile has keys of both.
  const int from = max(0, first_pos - a.window + 1);
  const int old_tiles = from < s.start ? (s.start - from + WIN_KEYS - 1) / WIN_KEYS : 0;
  const int first_base = from < s.start ? s.start - old_tiles * WIN_KEYS : from;
  const int tiles = (last_pos - first_base) / WIN_KEYS + 1;

  bf16x8 qf[QT][KD];
#pragma unroll
  for (int q = 0; q < QT; ++q) {
    const int i = q0 + wave * QT * 16 + q * 16 + lo16;
#pragma unroll
    for (int d = 0; d < KD; ++d) {
      const int c = d * 32 + quad * 8;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (i < s.rows && c < a.dim) v = *reinterpret_cast<const uint4*>(x + (size_t)(s.row0 + i) * a.stride + head * a.dim + c);
      qf[q][d] = __builtin_bit_cast(bf16x8, v);
    }
  }
  f32x4 acc[QT][VD];
  float m[QT], l[QT];
#pragma unroll
  for (int q = 0; q < QT; ++q) {
    m[q] = -1e30f;
    l[q] = 0.f;
#pragma unroll
    for (int d = 0; d < VD; ++d) acc[q][d] = f32x4{0.f, 0.f, 0.f, 0.f};
  }

  u32x4 kn[KP], vn[VT][4];
  float bn = 0.f;
  // The next tile on its way from memory: keys at positions base .. base + 63, by 32-bit offsets into bounded
  // buffers: a row past the span's last, which may hold anything, reads as zeros.  A thread's offsets into a tile of the call's own rows are the same for every tile.
  // Columns past a head's width read its last ones: q is zero there, and those of v are not stored.
  const __amdgpu_buffer_rsrc_t own_kb = bounded_bytes(own_k + (size_t)s.row0 * a.stride, (int)(((long)s.rows * a.stride - (own_k - x)) * 2));
  const __amdgpu_buffer_rsrc_t own_vb = bounded_bytes(own_v + (size_t)s.row0 * a.stride, (int)(((long)s.rows * a.stride - (own_v - x)) * 2));
  const __amdgpu_buffer_rsrc_t old_kb = bounded_bytes(ring_k, (a.ring * nk - g * a.dim) * 2);
  const __amdgpu_buffer_rsrc_t old_vb = bounded_bytes(ring_v, (a.ring * nv - g * a.vdim) * 2);
  int k_col[KP], v_col[VT], k_own[KP], v_own[VT], k_mod[KP], v_mod[VT][4];
#pragma unroll
  for (int i = 0; i < KP; ++i) {
    const int e = t + 256 * i, row = e / (DKP / 8);
    k_mod[i] = row % a.ring;
    k_col[i] = 2 * min((e % (DKP / 8)) * 8, a.dim - 8);
    k_own[i] = row * a.stride * 2 + k_col[i];
  }
#pragma unroll
  for (int i = 0; i < VT; ++i) {
    const int e = t + 256 * i, row = (e / (DVP / 8) * 4) % WIN_KEYS;
#pragma unroll
    for (int j = 0; j < 4; ++j) v_mod[i][j] = (row + j) % a.ring;
    v_col[i] = 2 * min((e % (DVP / 8)) * 8, a.vdim - 8);
    v_own[i] = row * a.stride * 2 + v_col[i];
  }
  auto fetch = [&](int base) {
    if (base >= s.start) {
      const int at = (base - s.start) * a.stride * 2;
#pragma unroll
      for (int i = 0; i < KP; ++i) kn[i] = __builtin_amdgcn_raw_buffer_load_b128(own_kb, k_own[i], at, 0);
#pragma unroll
      for (int i = 0; i < VT; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) vn[i][j] = __builtin_amdgcn_raw_buffer_load_b128(own_vb, v_own[i], at + j * a.stride * 2, 0);
    } else {
      const int wrap = ((base % a.ring) + a.ring) % a.ring;
      auto place = [&](int r) { return wrap + r - (a.ring & -(int)(wrap + r >= a.ring)); };   // r < ring
#pragma unroll
      for (int i = 0; i < KP; ++i) kn[i] = __builtin_amdgcn_raw_buffer_load_b128(old_kb, place(k_mod[i]) * nk * 2 + k_col[i], 0, 0);
#pragma unroll
      for (int i = 0; i < VT; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          vn[i][j] = __builtin_amdgcn_raw_buffer_load_b128(old_vb, place(v_mod[i][j]) * nv * 2 + v_col[i], 0, 0);
    }
    // entry t: the distance first_pos - base + BQ - 1 - t (masked where it is used)
    bn = bias[(size_t)head * a.window + max(0, min(first_pos - base + BQ - 1 - t, a.window - 1))];
  };
  fetch(first_base);
  const float scale = a.scale * LOG2E;
  for (int n = 0; n < tiles; ++n) {
    const int base = first_base + n * WIN_KEYS;
    WindowShared<DKP, DVP>& sh = pair[n & 1];   // its last readers are behind the barrier of the tile between
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      const int e = t + 256 * i;
      *reinterpret_cast<u32x4*>(&sh.k[e / (DKP / 8)][(e % (DKP / 8)) * 8]) = kn[i];
    }
#pragma unroll
    for (int i = 0; i < VT; ++i) {
      const int e = t + 256 * i, r4 = e / (DVP / 8), c = (e % (DVP / 8)) * 8;
      if (e < VP) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {   // two columns at a time: four keys each, 8 bytes
          const uint32_t w0 = vn[i][0][j], w1 = vn[i][1][j], w2 = vn[i][2][j], w3 = vn[i][3][j];
          const uint2 even = make_uint2((w0 & 0xffffu) | (w1 << 16), (w2 & 0xffffu) | (w3 << 16));
          const uint2 odd = make_uint2((w0 >> 16) | (w1 & 0xffff0000u), (w2 >> 16) | (w3 & 0xffff0000u));
          *reinterpret_cast<uint2*>(&sh.vt[c + 2 * j][r4 * 4]) = even;
          *reinterpret_cast<uint2*>(&sh.vt[c + 2 * j + 1][r4 * 4]) = odd;
        }
      }
    }
    const int dist = first_pos - base + BQ - 1 - t;
    sh.by_distance[t] = (dist >= 0 && dist < a.window) ? bn * LOG2E : -INFINITY;
    __syncthreads();
    if (n + 1 < tiles) fetch(base + WIN_KEYS);

    f32x4 sc[QT][4];
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
      bf16x8 kf[KD];
#pragma unroll
      for (int d = 0; d < KD; ++d) kf[d] = *reinterpret_cast<const bf16x8*>(&sh.k[kt * 16 + lo16][d * 32 + quad * 8]);
#pragma unroll
      for (int q = 0; q < QT; ++q) {
        sc[q][kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int d = 0; d < KD; ++d) sc[q][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[d], qf[q][d], sc[q][kt], 0, 0, 0);
      }
    }
    bf16x8 pf[QT][2];
#pragma unroll
    for (int q = 0; q < QT; ++q) {
      const float* by = sh.by_distance + BQ - 1 - ((wave * QT + q) * 16 + lo16) + quad * 4;   // key r of tile kt: + 16 kt + r
      float top = -INFINITY;
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) sc[q][kt][r] = fmaf(sc[q][kt][r], scale, by[kt * 16 + r]);
      if (base < 0) {   // keys ahead of the sequence
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (base + kt * 16 + quad * 4 + r < 0) sc[q][kt][r] = -INFINITY;
      }
#pragma unroll
      for (int kt = 0; kt < 4; ++kt) top = fmaxf(top, fmaxf(fmaxf(sc[q][kt][0], sc[q][kt][1]), fmaxf(sc[q][kt][2], sc[q][kt][3])));
      // The reference the exponents are taken from moves only where a score would exceed it by more than 2^8:
      // it cancels in the quotient, and the products need no rescaling between.
      if (__builtin_amdgcn_ballot_w64(top > m[q] + 8.f) != 0) {
        top = fmaxf(top, __shfl_xor(top, 16, 64));
        top = fmaxf(top, __shfl_xor(top, 32, 64));
        top = fmaxf(m[q], top);
        const float fade = __builtin_amdgcn_exp2f(m[q] - top);
        m[q] = top;
        l[q] *= fade;
#pragma unroll
        for (int d = 0; d < VD; ++d)
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[q][d][r] *= fade;
      }
      float sum = 0.f;
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          sc[q][kt][r] = __builtin_amdgcn_exp2f(sc[q][kt][r] - m[q]);
          sum += sc[q][kt][r];
        }
      l[q] += sum;
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const uint4 v = make_uint4(pack_bf16(sc[q][2 * h][0], sc[q][2 * h][1]), pack_bf16(sc[q][2 * h][2], sc[q][2 * h][3]),
                                   pack_bf16(sc[q][2 * h + 1][0], sc[q][2 * h + 1][1]), pack_bf16(sc[q][2 * h + 1][2], sc[q][2 * h + 1][3]));
        pf[q][h] = __builtin_bit_cast(bf16x8, v);
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
        for (int q = 0; q < QT; ++q) acc[q][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[q][h], acc[q][d], 0, 0, 0);
      }
  }
#pragma unroll
  for (int q = 0; q < QT; ++q) {
    float sum = l[q];
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    const int i = q0 + wave * QT * 16 + q * 16 + lo16;
    if (i >= s.rows) continue;
    const float inv = a.out_scale / sum;
    bf16_t* to = out + (size_t)(s.row0 + i) * a.out_stride + a.out_at + head * a.vdim;
#pragma unroll
    for (int d = 0; d < VD; ++d) {
      const int c = d * 16 + quad * 4;
      if (c < a.vdim)
        *reinterpret_cast<uint2*>(to + c) = make_uint2(pack_bf16(acc[q][d][0] * inv, acc[q][d][1] * inv),
                                                       pack_bf16(acc[q][d][2] * inv, acc[q][d][3] * inv));
    }
  }
}

// The spans' lengths are known on the device only: a block takes 128 queries where that still gives the
// chip a block a CU, 64 otherwise (the grid is sized for 64; the blocks left over return).
template <int DKP, int DVP>
__global__ __launch_bounds__(256) void window_prefill_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ keys,
                                                             const bf16_t* __restrict__ values, const float* __restrict__ bias,
                                                             const int* __restrict__ spans, bf16_t* __restrict__ out, WindowShape a) {
  __shared__ WindowShared<DKP, DVP> sh[2];
  const Span s = span_of(spans, blockIdx.z, a.rows);
  // Heads fastest, so that the blocks with work are a run of the grid (a pattern of idle blocks within it
  // would leave the same compute units idle each time round), and, where they divide by the XCDs, the
  // heads of a group on one XCD, whose L2 then reads their keys and values once.
  const int tile = blockIdx.y, x8 = blockIdx.x;
  const int head = a.heads % 8 == 0 ? (x8 & 7) * (a.heads >> 3) + (x8 >> 3) : x8;
  constexpr bool CAN_WIDE = DVP <= 128 && DKP <= 128;   // registers
  if (CAN_WIDE && (long)((s.rows + 127) / 128) * a.heads >= 256) {
    if (tile * 128 < s.rows)
      window_prefill_body<DKP, DVP, CAN_WIDE ? 2 : 1>(x, keys, values, bias, out, a, s, blockIdx.z, head, tile, sh);
  } else if (tile * 64 < s.rows) {
    window_prefill_body<DKP, DVP, 1>(x, keys, values, bias, out, a, s, blockIdx.z, head, tile, sh);
  }
}

template <int DKP>
static int launch_window_prefill(int dvp, const bf16_t* x, const bf16_t* keys, const bf16_t* values, const float* bias,
                                 const int* spans, bf16_t* out, const WindowShape& a, int slots, hipStream_t s) {
  const dim3 grid(a.heads, (a.rows + 63) / 64, slots);
#define IRON_WINDOW(DVP) \
  hipLaunchKernelGGL((window_prefill_kernel<DKP, DVP>), grid, dim3(256), 0, s, x, keys, values, bias, spans, out, a)
  if (dvp <= 32) IRON_WINDOW(32);
  else if (dvp <= 64) IRON_WINDOW(64);
  else if (dvp <= 128) IRON_WINDOW(128);
  else IRON_WINDOW(256);
#undef IRON_WINDOW
  IRON_LAUNCH_CHECK();
}

}  // namespace iron

using namespace iron;

extern "C" int iron_mha_window(const void* x, void* keys, void* values, const float* bias, const int* spans, void* out,
                               int slots, int rows, int stride, int heads, int kv_heads, int dim, int vdim, int window, int ring,
                               float scale, int out_stride, int out_at, float out_scale, int single, int is_float, void* stream) {
  IRON_REQUIRE(x && keys && values && bias && spans && out, "mha_window: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0, "mha_window: spans must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0, "mha_window: slots (%d) and rows (%d) must be positive", slots, rows);
  IRON_REQUIRE(heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0, "mha_window: kv_heads (%d) must divide heads (%d)",
               kv_heads, heads);
  IRON_REQUIRE(dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256, "mha_window: dim (%d) and vdim (%d) from 1 to 256", dim, vdim);
  IRON_REQUIRE(window > 0 && ring >= window, "mha_window: a window (%d) of at least 1 within the ring (%d)", window, ring);
  IRON_REQUIRE(stride >= heads * dim + kv_heads * (dim + vdim), "mha_window: a row of %d holds no q, k and v of %d heads", stride, heads);
  IRON_REQUIRE(out_at >= 0 && out_at + heads * vdim <= out_stride, "mha_window: %d columns from %d of an output row of %d",
               heads * vdim, out_at, out_stride);
  IRON_REQUIRE((long)rows * stride < (1L << 30) && (long)ring * kv_heads * (dim > vdim ? dim : vdim) < (1L << 30),
               "mha_window: the batch's rows and a slot's ring are addressed with 32-bit offsets");
  const WindowShape a{rows, stride, heads, kv_heads, dim, vdim, window, ring, out_stride, out_at, scale, out_scale};
  hipStream_t s = (hipStream_t)stream;
  const bool aligned = stride % 8 == 0 && dim % 8 == 0 && vdim % 8 == 0 && (((uintptr_t)x | (uintptr_t)keys | (uintptr_t)values) & 15) == 0;
  const bool out_aligned = out_stride % 4 == 0 && out_at % 4 == 0 && ((uintptr_t)out & 7) == 0;
#define IRON_WINDOW_ROWS(T, VEC, NW, STORE, ROWS)                                                                          \
  {                                                                                                                        \
    const int pieces = VEC == 8 ? vdim / 8 : (vdim < 64 ? vdim : 64);                                                      \
    const size_t lds = (size_t)NW * (64 / pieces) * vdim * 4;                                                              \
    hipLaunchKernelGGL((window_rows_kernel<T, VEC, NW, STORE>), dim3(heads, slots, ROWS), dim3(NW * 64), lds, s, (const T*)x, \
                       (T*)keys, (T*)values, bias, spans, (T*)out, a);                                                     \
  }
  if (single) {   // the caller's spans have one row at most, which goes into the ring here
    if (is_float) { if (aligned) IRON_WINDOW_ROWS(float, 8, 16, true, 1) else IRON_WINDOW_ROWS(float, 1, 16, true, 1) }
    else { if (aligned) IRON_WINDOW_ROWS(bf16_t, 8, 16, true, 1) else IRON_WINDOW_ROWS(bf16_t, 1, 16, true, 1) }
    IRON_LAUNCH_CHECK();
  }
  IRON_REQUIRE(rows <= 65535, "mha_window: rows (%d) exceed the grid's z extent", rows);
  if (!is_float && aligned && out_aligned) {
    const bf16_t *xb = (const bf16_t*)x, *kb = (const bf16_t*)keys, *vb = (const bf16_t*)values;
    int e;
    if (dim <= 32) e = launch_window_prefill<32>(vdim, xb, kb, vb, bias, spans, (bf16_t*)out, a, slots, s);
    else if (dim <= 64) e = launch_window_prefill<64>(vdim, xb, kb, vb, bias, spans, (bf16_t*)out, a, slots, s);
    else if (dim <= 128) e = launch_window_prefill<128>(vdim, xb, kb, vb, bias, spans, (bf16_t*)out, a, slots, s);
    else e = launch_window_prefill<256>(vdim, xb, kb, vb, bias, spans, (bf16_t*)out, a, slots, s);
    if (e != IRON_OK) return e;
  } else if (is_float) {
    if (aligned) IRON_WINDOW_ROWS(float, 8, 2, false, rows) else IRON_WINDOW_ROWS(float, 1, 2, false, rows)
  } else {
    IRON_WINDOW_ROWS(bf16_t, 1, 2, false, rows)
  }
#undef IRON_WINDOW_ROWS
  // Attended: the span's last rows go into the ring.
  const PackedHeads packed{rows, stride, heads, kv_heads, dim, vdim, ring};
  if (is_float) launch_ring_store<float>(x, keys, values, spans, packed, slots, s);
  else launch_ring_store<bf16_t>(x, keys, values, spans, packed, slots, s);
  IRON_LAUNCH_CHECK();
}
