// Latent attention over a batch of spans: what a position leaves behind is one short row -- a normed latent
// of `rank` columns, and where the design has one, a key part of `rot` columns turned by its position that
// all heads share.  Per head h, with U_h (dim, rank) and V_h (vdim, rank) rows of one weight `up`:
//
//   score_ij = (q_i . U_h c_j + turned(qr_i) . r_j) * scale,   0 <= i - j < window
//   y_i      = sum_j p_ij V_h c_j,   p the softmax over the visible j, with exp(sink_h) in its denominator if given
//
// A prompt's portion expands the keys it attends once into keys and values of every head (a product of the
// gathered latents and `up`) and runs flash attention over them.  A decode step works in the latent's space:
// q_h U_h meets the latents themselves (read once for 16 heads), and V_h is applied to the weighted sum.
//
// Caches are rings: position p's rows in row p % ring of its slot.  A call's own rows are stored before they
// are attended, so a ring holds at least the window and a portion.
#include "../../include/iron_hip.h"
#include "latent.h"

namespace iron {

constexpr float LATENT_LOG2E = 1.4426950408889634f;

// The key rows a slot's span attends: positions first .. first + count - 1, expanded in rows row0 ..
struct KeyRun {
  int row0, first, count;
};
__device__ __forceinline__ int keys_of(const Span& s, int window) { return s.rows > 0 ? min(s.start, window - 1) + s.rows : 0; }
__device__ __forceinline__ KeyRun key_run(const int* __restrict__ spans, int slot, const LatentShape& a) {
  KeyRun k{0, 0, 0};
  for (int i = 0; i < slot; ++i) k.row0 += keys_of(span_of(spans, i, a.rows), a.window);
  const Span s = span_of(spans, slot, a.rows);
  k.row0 = min(k.row0, a.cap);
  k.count = min(keys_of(s, a.window), a.cap - k.row0);
  k.first = s.start - min(s.start, a.window - 1);
  return k;
}

template <typename T>
__device__ __forceinline__ float latent_exp2(float x) {
  if constexpr (sizeof(T) == 2) return __builtin_amdgcn_exp2f(x);
  else return exp2f(x);
}

// ------------------------------------------------------------------ the rows
// A row of the packed projection, [query latent | key latent | shared key part | ..]: both latents over their
// root mean square, the key part turned; the query's out, the rest into the caches.
template <typename T>
__global__ __launch_bounds__(256) void latent_rows_kernel(const T* __restrict__ x, const bf16_t* __restrict__ q_gain,
                                                          const bf16_t* __restrict__ c_gain, const float* __restrict__ angles,
                                                          const int* __restrict__ spans, T* __restrict__ q_out,
                                                          T* __restrict__ latents, T* __restrict__ shared_keys, LatentShape a,
                                                          int stride, int q_rank, float eps) {
  __shared__ float part[2][4];
  const int row = blockIdx.x, t = threadIdx.x;
  int slot = -1;
  Span s{0, 0, 0};
  for (int i = 0; i < a.slots; ++i) {
    const Span o = span_of(spans, i, a.rows);
    if (row >= o.row0 && row < o.row0 + o.rows) {
      slot = i;
      s = o;
    }
  }
  if (slot < 0) return;
  const int pos = s.start + row - s.row0, at = pos % a.ring;
  const T* xr = x + (size_t)row * stride;
  const T* cr = xr + q_rank;
  float qs = 0.f, cs = 0.f;
  for (int c = t; c < q_rank; c += 256) {
    const float v = load_one(xr + c);
    qs = fmaf(v, v, qs);
  }
  for (int c = t; c < a.rank; c += 256) {
    const float v = load_one(cr + c);
    cs = fmaf(v, v, cs);
  }
  qs = wave_sum(qs);
  cs = wave_sum(cs);
  if ((t & 63) == 0) {
    part[0][t >> 6] = qs;
    part[1][t >> 6] = cs;
  }
  __syncthreads();
  const float qi = 1.0f / sqrtf((part[0][0] + part[0][1] + part[0][2] + part[0][3]) / (float)q_rank + eps);
  const float ci = 1.0f / sqrtf((part[1][0] + part[1][1] + part[1][2] + part[1][3]) / (float)a.rank + eps);
  for (int c = t; c < q_rank; c += 256) store_one(q_out + (size_t)row * q_rank + c, load_one(xr + c) * qi * bf16_to_f32(q_gain[c]));
  T* cd = latents + ((size_t)slot * a.ring + at) * a.rank;
  for (int c = t; c < a.rank; c += 256) store_one(cd + c, load_one(cr + c) * ci * bf16_to_f32(c_gain[c]));
  if (a.rot == 0) return;
  const T* rr = cr + a.rank;
  T* rd = shared_keys + ((size_t)slot * a.ring + at) * a.rot;
  const float* turn = angles + (size_t)min(pos, a.angle_rows - 1) * a.turned;
  for (int c = t; c < a.rot; c += 256) {
    float v = load_one(rr + c);
    if (c < a.turned) {
      const float cosine = turn[c & ~1], sine = turn[c | 1], other = load_one(rr + (c ^ 1));
      v = (c & 1) ? v * cosine + other * sine : v * cosine - other * sine;
    }
    store_one(rd + c, v);
  }
}

// The same in 16-byte pieces.
template <typename T, int CH>
__global__ __launch_bounds__(256) void latent_rows_wide_kernel(const T* __restrict__ x, LatentRow g, const int* __restrict__ spans,
                                                               T* __restrict__ q_out, T* __restrict__ latents,
                                                               T* __restrict__ shared_keys, LatentShape a, int stride) {
  __shared__ float part[2][4];
  const int row = blockIdx.x;
  for (int slot = 0; slot < a.slots; ++slot) {
    const Span s = span_of(spans, slot, a.rows);
    if (row >= s.row0 && row < s.row0 + s.rows) {
      latent_row<T, CH, true>(x + (size_t)row * stride, g, a, slot, s.start + row - s.row0, q_out + (size_t)row * g.q_rank, latents, shared_keys, part);
      return;
    }
  }
}
// --------------------------------------------------------------- expansion
// The latents a portion attends, slot after slot, with their shared key parts, and behind the last a tile's rows of
// zeros, so that a tile may be read whole wherever it starts; and how many rows that is.
constexpr int LATENT_KEYS = 64;   // keys a tile
constexpr int GATHER_ROWS = 16;
__host__ __device__ inline long expanded_rows(long cap) { return (cap + LATENT_KEYS + 255) / 256 * 256; }   // (whole tiles of the product)
template <typename T, int VEC>
__device__ __forceinline__ void copy_or_zero(const T* from, T* to, int n, int lane) {
  for (int c = lane * VEC; c < n; c += 64 * VEC) {
    float f[VEC];
    if (from != nullptr) {
      load_vec<VEC>(from + c, f);
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] = 0.f;
    }
    store_vec<VEC>(to + c, f);
  }
}
template <typename T, int VEC>
__global__ __launch_bounds__(256) void latent_gather_kernel(const T* __restrict__ latents, const T* __restrict__ shared_keys,
                                                            const int* __restrict__ spans, T* __restrict__ out, T* __restrict__ shared_out,
                                                            int* __restrict__ count, LatentShape a) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, first_row = blockIdx.x * GATHER_ROWS;
  int total = 0;
  for (int slot = 0; slot < a.slots; ++slot) {
    const Span s = span_of(spans, slot, a.rows);
    const int n = keys_of(s, a.window), first = s.start - min(s.start, a.window - 1);
    const int lo = max(first_row, total), hi = min(min(first_row + GATHER_ROWS, total + n), a.cap);
    for (int r = lo + wave; r < hi; r += 4) {
      const size_t at = (size_t)slot * a.ring + (first + r - total) % a.ring;
      copy_or_zero<T, VEC>(latents + at * a.rank, out + (size_t)r * a.rank, a.rank, lane);
      copy_or_zero<T, VEC>(shared_keys + at * a.rot, shared_out + (size_t)r * a.rot, a.rot, lane);
    }
    total += n;
  }
  total = min(total, a.cap);
  for (int r = max(first_row, total) + wave; r < min(first_row + GATHER_ROWS, total + LATENT_KEYS); r += 4) {
    copy_or_zero<T, VEC>(nullptr, out + (size_t)r * a.rank, a.rank, lane);
    copy_or_zero<T, VEC>(nullptr, shared_out + (size_t)r * a.rot, a.rot, lane);
  }
  if (blockIdx.x == 0 && threadIdx.x == 0) *count = total + LATENT_KEYS;
}

// ------------------------------------------------------- a portion, row by row
// Any sizes, either type: a wave a query row and head, 64 keys at a time, a key a lane for the scores and
// columns over the lanes for the weighted sum.
constexpr int ROWS_COLUMNS = 16;   // columns a lane may hold: vdim up to 1024
template <typename T>
__global__ __launch_bounds__(64) void latent_rows_attention_kernel(const T* __restrict__ q, const T* __restrict__ kv,
                                                                   const T* __restrict__ shared_keys, const float* __restrict__ angles,
                                                                   const bf16_t* __restrict__ sink, const int* __restrict__ spans,
                                                                   T* __restrict__ y, LatentShape a) {
  extern __shared__ float lds[];   // the query, then the weights
  float* qs = lds;
  float* ps = lds + a.dim + a.rot;
  const int head = blockIdx.x, i = blockIdx.y, slot = blockIdx.z, lane = threadIdx.x;
  const Span s = span_of(spans, slot, a.rows);
  if (i >= s.rows) return;
  const KeyRun k = key_run(spans, slot, a);
  const int pos = s.start + i, lo = max(0, pos - a.window + 1), hi = min(pos + 1, k.first + k.count), wide = a.dim + a.rot;
  const T* qr = q + ((size_t)(s.row0 + i) * a.heads + head) * wide;
  const float* turn = angles + (size_t)min(pos, a.angle_rows - 1) * a.turned;
  for (int c = lane; c < wide; c += 64) {
    float v = load_one(qr + c);
    const int r = c - a.dim;
    if (r >= 0 && r < a.turned) {
      const float cosine = turn[r & ~1], sine = turn[r | 1], other = load_one(qr + a.dim + (r ^ 1));
      v = (r & 1) ? v * cosine + other * sine : v * cosine - other * sine;
    }
    qs[c] = v;
  }
  __syncthreads();
  const size_t width = (size_t)a.heads * (a.dim + a.vdim);
  const T* keys = kv + (size_t)head * a.dim;
  const T* values = kv + (size_t)a.heads * a.dim + (size_t)head * a.vdim;
  float acc[ROWS_COLUMNS], m = sink != nullptr ? bf16_to_f32(sink[head]) : -INFINITY, l = sink != nullptr && lane == 0 ? 1.f : 0.f;
#pragma unroll
  for (int e = 0; e < ROWS_COLUMNS; ++e) acc[e] = 0.f;
  for (int p0 = lo; p0 < hi; p0 += 64) {
    float score = -INFINITY;
    if (p0 + lane < hi) {
      const int p = p0 + lane;
      const T* kr = keys + (size_t)(k.row0 + p - k.first) * width;
      const T* rr = shared_keys + (size_t)(k.row0 + p - k.first) * a.rot;
      float dot = 0.f;
      for (int c = 0; c < a.dim; ++c) dot = fmaf(load_one(kr + c), qs[c], dot);
      for (int c = 0; c < a.rot; ++c) dot = fmaf(load_one(rr + c), qs[a.dim + c], dot);
      score = dot * a.scale;
    }
    const float top = fmaxf(m, wave_max(score));
    const float fade = expf(m - top), w = expf(score - top);
    m = top;
    l = l * fade + w;
    ps[lane] = w;
    __syncthreads();
    const int n = min(64, hi - p0);
#pragma unroll
    for (int e = 0; e < ROWS_COLUMNS; ++e) acc[e] *= fade;
    for (int j = 0; j < n; ++j) {
      const T* vr = values + (size_t)(k.row0 + p0 + j - k.first) * width;
      const float w1 = ps[j];
#pragma unroll
      for (int e = 0; e < ROWS_COLUMNS; ++e)
        if (lane + 64 * e < a.vdim) acc[e] = fmaf(w1, load_one(vr + lane + 64 * e), acc[e]);
    }
    __syncthreads();
  }
  l = wave_sum(l);
#pragma unroll
  for (int e = 0; e < ROWS_COLUMNS; ++e)
    if (lane + 64 * e < a.vdim) store_one(y + ((size_t)(s.row0 + i) * a.heads + head) * a.vdim + lane + 64 * e, acc[e] / l);
}

// ------------------------------------------------------ a portion on the MFMAs
// A block takes QT * 64 queries of one head, QT * 16 a wave, and walks the keys 64 at a time.  Scores are
// computed transposed (keys down the MFMA's rows, queries across its columns): a lane holds one query's
// scores, so the row statistics are a lane's own, and the weights are the second product's B operand as they
// stand.  A sink is where a query's statistics start: a maximum, and one term of the sum.
template <int DKP, int DVP>
struct LatentShared {
  __align__(16) bf16_t k[LATENT_KEYS][DKP + 8];
  __align__(16) bf16_t vt[DVP][LATENT_KEYS + 8];
};

template <int DKP, int DVP, int QT, int BUFFERS>
__device__ __forceinline__ void latent_prefill_body(const bf16_t* __restrict__ q, const bf16_t* __restrict__ kv,
                                                    const bf16_t* __restrict__ shared_keys, const float* __restrict__ angles,
                                                    const bf16_t* __restrict__ sink, bf16_t* __restrict__ y, const LatentShape& a,
                                                    const Span& s, const KeyRun& run, int head, int tile,
                                                    LatentShared<DKP, DVP>* tiles_lds) {
  constexpr int BQ = QT * 64, KD = DKP / 32, VD = DVP / 16;
  constexpr int KP = LATENT_KEYS * DKP / 8 / 256;      // 16-byte pieces of a key tile a thread stages
  constexpr int VP = (LATENT_KEYS / 4) * (DVP / 8);    // four-key pieces of a value tile
  constexpr int VT = (VP + 255) / 256;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, lo16 = lane & 15, quad = lane >> 4;
  const int wide = a.dim + a.rot, width = a.heads * (a.dim + a.vdim), q0 = tile * BQ;
  const int end = run.first + run.count;                                         // first position without a key
  const int first_pos = s.start + q0, last_pos = min(first_pos + BQ, end) - 1;   // the block's queries
  const int from = max(0, first_pos - a.window + 1);
  const int tiles = (last_pos - from) / LATENT_KEYS + 1;

  bf16x8 qf[QT][KD];
#pragma unroll
  for (int n = 0; n < QT; ++n) {
    const int i = q0 + wave * QT * 16 + n * 16 + lo16;
    const float* turn = angles + (size_t)min(s.start + i, a.angle_rows - 1) * a.turned;
#pragma unroll
    for (int d = 0; d < KD; ++d) {
      const int c = d * 32 + quad * 8;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (i < s.rows && c < wide) {
        v = *reinterpret_cast<const uint4*>(q + ((size_t)(s.row0 + i) * a.heads + head) * wide + c);
        const int r = c - a.dim;
        if (r >= 0 && r < a.turned) {   // (turned is a multiple of 8 here)
          float f[8];
          unpack8(v, f);
          const float4 lo = *reinterpret_cast<const float4*>(turn + r), hi = *reinterpret_cast<const float4*>(turn + r + 4);
          const float cosine[4] = {lo.x, lo.z, hi.x, hi.z}, sine[4] = {lo.y, lo.w, hi.y, hi.w};
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const float u = f[2 * j], w = f[2 * j + 1];
            f[2 * j] = u * cosine[j] - w * sine[j];
            f[2 * j + 1] = w * cosine[j] + u * sine[j];
          }
          v = pack8(f);
        }
      }
      qf[n][d] = __builtin_bit_cast(bf16x8, v);
    }
  }
  const bool sunk = sink != nullptr;
  const float sink2 = sunk ? bf16_to_f32(sink[head]) * LATENT_LOG2E : -1e30f;
  f32x4 acc[QT][VD];
  float m[QT], l[QT];
#pragma unroll
  for (int n = 0; n < QT; ++n) {
    m[n] = sink2;
    l[n] = sunk && quad == 0 ? 1.f : 0.f;   // (a query's sum is over its four lanes)
#pragma unroll
    for (int d = 0; d < VD; ++d) acc[n][d] = f32x4{0.f, 0.f, 0.f, 0.f};
  }

  // The next tile on its way from memory: a pointer a piece, moved on by a tile, and no load behind a branch.  A key's
  // pieces past its head's width read other columns, against zeros of q.  A value piece is four keys of eight columns;
  // a wave takes four such pieces side by side, so that its rows are read in 64-byte runs and written to LDS without
  // conflicts.
  u32x4 kn[KP], vn[VT][4];
  const bf16_t *k_at[KP], *v_at[VT];
  int k_step[KP];
  const size_t row0 = (size_t)(run.row0 + from - run.first);
#pragma unroll
  for (int i = 0; i < KP; ++i) {
    const int e = t + 256 * i, c = (e % (DKP / 8)) * 8, row = e / (DKP / 8);
    const bool part = c >= a.dim && c < wide;
    k_step[i] = part ? a.rot : width;
    k_at[i] = part ? shared_keys + (row0 + row) * a.rot + c - a.dim : kv + (row0 + row) * width + head * a.dim + (c < a.dim ? c : 0);
    k_step[i] *= LATENT_KEYS;
  }
  auto v_row = [&](int e) { return (e >> 2) & 15; };                      // a piece's keys, in fours
  auto v_col = [&](int e) { return ((e >> 6) * 4 + (e & 3)) * 8; };       // ... and its columns
#pragma unroll
  for (int i = 0; i < VT; ++i) {
    const int e = t + 256 * i;
    v_at[i] = kv + (row0 + v_row(e) * 4) * width + a.heads * a.dim + head * a.vdim + min(v_col(e), a.vdim - 8);
  }
  auto fetch = [&]() {
#pragma unroll
    for (int i = 0; i < KP; ++i) {
      kn[i] = *reinterpret_cast<const u32x4*>(k_at[i]);
      k_at[i] += k_step[i];
    }
#pragma unroll
    for (int i = 0; i < VT; ++i) {
#pragma unroll
      for (int j = 0; j < 4; ++j) vn[i][j] = *reinterpret_cast<const u32x4*>(v_at[i] + (size_t)j * width);
      v_at[i] += (size_t)LATENT_KEYS * width;
    }
  };
  fetch();
  const float scale = a.scale * LATENT_LOG2E;
  for (int n = 0; n < tiles; ++n) {
    const int base = from + n * LATENT_KEYS;
    LatentShared<DKP, DVP>& sh = tiles_lds[BUFFERS == 2 ? n & 1 : 0];   // two: its last readers are behind the barrier between
    if (BUFFERS == 1 && n > 0) __syncthreads();
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
    __syncthreads();
    if (n + 1 < tiles) fetch();

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
    // A tile all of whose keys all of the block's queries see needs no mask.  (One branch around selects: a branch
    // a score, right behind the products, has read scores of a tile that was not done.)
    const bool edge = base + LATENT_KEYS - 1 > first_pos || first_pos + BQ - 1 - base >= a.window;
    bf16x8 pf[QT][2];
#pragma unroll
    for (int u = 0; u < QT; ++u) {
#pragma unroll
      for (int kt = 0; kt < 4; ++kt) sc[u][kt] *= scale;
      if (edge) {
        const int ahead = first_pos + wave * QT * 16 + u * 16 + lo16 - base - quad * 4;   // i - j of the lane's first key
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int r = 0; r < 4; ++r) sc[u][kt][r] = (unsigned)(ahead - kt * 16 - r) < (unsigned)a.window ? sc[u][kt][r] : -INFINITY;
      }
      float top = -INFINITY;
#pragma unroll
      for (int kt = 0; kt < 4; ++kt) top = fmaxf(top, fmaxf(fmaxf(sc[u][kt][0], sc[u][kt][1]), fmaxf(sc[u][kt][2], sc[u][kt][3])));
      // The reference the exponents are taken from moves only where a score would exceed it by more than 2^8:
      // it cancels in the quotient, and the products need no rescaling between.
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
      float sum = 0.f;
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          sc[u][kt][r] = __builtin_amdgcn_exp2f(sc[u][kt][r] - m[u]);
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
    bf16_t* to = y + ((size_t)(s.row0 + i) * a.heads + head) * a.vdim;
#pragma unroll
    for (int d = 0; d < VD; ++d) {
      const int c = d * 16 + quad * 4;
      if (c < a.vdim)
        *reinterpret_cast<uint2*>(to + c) = make_uint2(pack_bf16(acc[u][d][0] * inv, acc[u][d][1] * inv),
                                                       pack_bf16(acc[u][d][2] * inv, acc[u][d][3] * inv));
    }
  }
}

// The spans' lengths are known on the device only: a block takes 128 queries where narrow heads leave it the
// registers and that still gives the chip a block a CU, 64 otherwise (the grid is sized for 64; the blocks left
// over return).  The tiles with the most keys go first and those with the fewest last but in rising order, so that
// two blocks that share a CU have about the same number of keys together, whichever CU it is.
template <int DKP, int DVP>
__global__ __launch_bounds__(256, DKP + DVP <= 384 ? 2 : 1) void latent_prefill_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ kv, const bf16_t* __restrict__ shared_keys, const float* __restrict__ angles,
    const bf16_t* __restrict__ sink, const int* __restrict__ spans, bf16_t* __restrict__ y, LatentShape a) {
  constexpr int BUFFERS = DKP + DVP <= 192 ? 2 : 1;   // LDS: several blocks a CU
  constexpr bool CAN_WIDE = DKP + DVP <= 192;
  __shared__ LatentShared<DKP, DVP> sh[BUFFERS];
  const Span s = span_of(spans, blockIdx.z, a.rows);
  const int head = blockIdx.x, y_at = blockIdx.y;
  const bool wide = CAN_WIDE && (long)((s.rows + 127) / 128) * a.heads >= 256;
  const int count = wide ? (s.rows + 127) / 128 : (s.rows + 63) / 64;
  if (y_at >= count) return;
  const int half = (count + 1) / 2, tile = y_at < half ? count - 1 - y_at : y_at - half;
  const KeyRun run = key_run(spans, blockIdx.z, a);
  if (run.count < s.rows) return;   // no room was made for these keys
  if (wide) latent_prefill_body<DKP, DVP, CAN_WIDE ? 2 : 1, BUFFERS>(q, kv, shared_keys, angles, sink, y, a, s, run, head, tile, sh);
  else latent_prefill_body<DKP, DVP, 1, BUFFERS>(q, kv, shared_keys, angles, sink, y, a, s, run, head, tile, sh);
}

template <int DKP>
static void launch_latent_prefill(const bf16_t* q, const bf16_t* kv, const bf16_t* shared_keys, const float* angles, const bf16_t* sink,
                                  const int* spans, bf16_t* y, const LatentShape& a, hipStream_t s) {
  const dim3 grid(a.heads, (a.rows + 63) / 64, a.slots);
#define IRON_LATENT(DVP) \
  hipLaunchKernelGGL((latent_prefill_kernel<DKP, DVP>), grid, dim3(256), 0, s, q, kv, shared_keys, angles, sink, spans, y, a)
  if (a.vdim <= 32) IRON_LATENT(32);
  else if (a.vdim <= 64) IRON_LATENT(64);
  else if (a.vdim <= 128) IRON_LATENT(128);
  else IRON_LATENT(256);
#undef IRON_LATENT
}

// -------------------------------------------------------------- a decode step
// The keys of a slot's one row, dealt to `splits` blocks in runs of whole 64-key tiles.
constexpr int STEP_KEYS = 64;
struct StepKeys {
  int first, count, per, live;   // first position, keys; keys a split, splits that have any
};
__device__ __forceinline__ StepKeys step_keys(const Span& s, const LatentShape& a, int splits) {
  StepKeys k;
  k.count = min(s.start + 1, a.window);
  k.first = s.start + 1 - k.count;
  const int tiles = (k.count + STEP_KEYS - 1) / STEP_KEYS, each = (tiles + splits - 1) / splits;
  k.per = each * STEP_KEYS;
  k.live = (tiles + each - 1) / each;
  return k;
}

// A head's query in the latents' space, q_h U_h, and its turned columns behind it.
template <typename T, typename OUT, int VEC>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const T* __restrict__ q, const bf16_t* __restrict__ up,
                                                            const float* __restrict__ angles, const int* __restrict__ spans,
                                                            OUT* __restrict__ out, LatentShape a) {
  constexpr int COLUMNS = 16 * VEC;
  extern __shared__ float lds[];            // the query's unturned columns, then 16 partial sums a column
  float* red = lds + ((a.dim + 3) & ~3);
  const int head = blockIdx.x, slot = blockIdx.y, t = threadIdx.x, wide = a.dim + a.rot;
  const Span s = span_of(spans, slot, a.rows);
  if (s.rows == 0) return;
  const T* qr = q + ((size_t)s.row0 * a.heads + head) * wide;
  OUT* to = out + ((size_t)slot * a.heads + head) * (a.rank + a.rot);
  for (int c = t; c < a.dim; c += 256) lds[c] = load_one(qr + c);
  if (blockIdx.z == 0) {
    const float* turn = angles + (size_t)min(s.start, a.angle_rows - 1) * a.turned;
    for (int c = t; c < a.rot; c += 256) {
      float v = load_one(qr + a.dim + c);
      if (c < a.turned) {
        const float cosine = turn[c & ~1], sine = turn[c | 1], other = load_one(qr + a.dim + (c ^ 1));
        v = (c & 1) ? v * cosine + other * sine : v * cosine - other * sine;
      }
      store_one(to + a.rank + c, v);
    }
  }
  __syncthreads();
  const int col = blockIdx.z * COLUMNS + (t & 15) * VEC, group = t >> 4;
  float acc[VEC];
#pragma unroll
  for (int j = 0; j < VEC; ++j) acc[j] = 0.f;
  if (col < a.rank) {
    const bf16_t* w = up + (size_t)head * a.dim * a.rank + col;
#pragma unroll 4
    for (int d = group; d < a.dim; d += 16) {
      float f[VEC];
      load_vec<VEC>(w + (size_t)d * a.rank, f);
#pragma unroll
      for (int j = 0; j < VEC; ++j) acc[j] = fmaf(lds[d], f[j], acc[j]);
    }
  }
#pragma unroll
  for (int j = 0; j < VEC; ++j) red[group * COLUMNS + (t & 15) * VEC + j] = acc[j];
  __syncthreads();
  if (t < COLUMNS && blockIdx.z * COLUMNS + t < a.rank) {
    float sum = 0.f;
#pragma unroll
    for (int g = 0; g < 16; ++g) sum += red[g * COLUMNS + t];
    store_one(to + blockIdx.z * COLUMNS + t, sum);
  }
}

// A split's weighted sum of latents a head, (rank), before division, and its maximum (in powers of two) and sum.
struct StepParts {
  float *sums, *stats;   // (slots, splits, heads, rank) and (.., 2)
};

// Any sizes: a head and split a block, a key a wave.
template <typename T>
__global__ __launch_bounds__(256) void latent_step_kernel(const float* __restrict__ q, const T* __restrict__ latents,
                                                          const T* __restrict__ shared_keys, const int* __restrict__ spans,
                                                          StepParts to, LatentShape a, int splits) {
  extern __shared__ float lds[];   // the query, then each wave's sums
  __shared__ float ms[4], ls[4];
  const int head = blockIdx.x, split = blockIdx.y, slot = blockIdx.z, t = threadIdx.x, lane = t & 63, wave = t >> 6;
  const Span s = span_of(spans, slot, a.rows);
  if (s.rows == 0) return;
  const StepKeys k = step_keys(s, a, splits);
  if (split >= k.live) return;
  const int wide = a.rank + a.rot;
  float* acc = lds + wide + wave * a.rank;
  for (int c = t; c < wide; c += 256) lds[c] = q[((size_t)slot * a.heads + head) * wide + c] * (a.scale * LATENT_LOG2E);
  for (int c = lane; c < a.rank; c += 64) acc[c] = 0.f;
  __syncthreads();
  float m = -1e30f, l = 0.f;
  const int hi = min(k.count, (split + 1) * k.per);
  for (int j = split * k.per + wave; j < hi; j += 4) {
    const size_t at = (size_t)slot * a.ring + (k.first + j) % a.ring;
    const T *c = latents + at * a.rank, *r = shared_keys + at * a.rot;
    float dot = 0.f;
    for (int e = lane; e < a.rank; e += 64) dot = fmaf(load_one(c + e), lds[e], dot);
    for (int e = lane; e < a.rot; e += 64) dot = fmaf(load_one(r + e), lds[a.rank + e], dot);
    dot = wave_sum(dot);
    const float top = fmaxf(m, dot), fade = latent_exp2<T>(m - top), w = latent_exp2<T>(dot - top);
    m = top;
    l = fmaf(l, fade, w);
    for (int e = lane; e < a.rank; e += 64) acc[e] = fmaf(w, load_one(c + e), acc[e] * fade);
  }
  if (lane == 0) {
    ms[wave] = m;
    ls[wave] = l;
  }
  __syncthreads();
  const float top = fmaxf(fmaxf(ms[0], ms[1]), fmaxf(ms[2], ms[3]));
  float f[4], total = 0.f;
#pragma unroll
  for (int w = 0; w < 4; ++w) {   // (a wave without a key: its sums are zeros)
    f[w] = latent_exp2<T>(ms[w] - top);
    total = fmaf(ls[w], f[w], total);
  }
  const size_t part = ((size_t)slot * splits + split) * a.heads + head;
  for (int c = t; c < a.rank; c += 256) {
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) sum = fmaf(lds[wide + w * a.rank + c], f[w], sum);
    to.sums[part * a.rank + c] = sum;
  }
  if (t == 0) {
    to.stats[2 * part] = top;
    to.stats[2 * part + 1] = total;
  }
}

// bf16, rank and rot multiples of 8: sixteen heads a block on the MFMAs, two teams of four waves with 32 keys at a
// time each.  A team's keys lie in LDS as [latent, padded to 64s | shared part, padded to 32s]; its waves deal the
// columns of the scores' product, add their parts up in LDS, and deal the columns of the weighted sum.  Heads are
// an MFMA's columns throughout.  NG: groups of 64 latent columns a wave sums.
constexpr int TEAM_KEYS = 32, TEAM_PARTS = 4 * 2 * 64 * 16;   // keys, and bytes of scores in parts
template <int NG>
__global__ __launch_bounds__(512) void latent_step_mfma_kernel(const bf16_t* __restrict__ q, const bf16_t* __restrict__ latents,
                                                               const bf16_t* __restrict__ shared_keys, const int* __restrict__ spans,
                                                               StepParts to, LatentShape a, int splits, unsigned each_inverse) {
  constexpr int PIECES = 5 * NG;              // 16-byte pieces of a tile a thread stages
  constexpr int STEPS = (10 * NG + 3) / 4;    // 32-column steps of the scores' product a wave takes
  extern __shared__ __align__(16) unsigned char dyn[];
  const int head0 = blockIdx.x * 16, split = blockIdx.y, slot = blockIdx.z;
  const int team = threadIdx.x >> 8, t = threadIdx.x & 255, lane = t & 63, wave = t >> 6, lo16 = lane & 15, quad = lane >> 4;
  const Span s = span_of(spans, slot, a.rows);
  if (s.rows == 0) return;
  const StepKeys k = step_keys(s, a, splits);
  if (split >= k.live) return;
  const int rank_pad = (a.rank + 63) & ~63, rot_pad = (a.rot + 31) & ~31, pitch = rank_pad + rot_pad + 8, wide = a.rank + a.rot;
  unsigned char* mine = dyn + team * (TEAM_PARTS + TEAM_KEYS * pitch * 2);
  f32x4* parts = reinterpret_cast<f32x4*>(mine);                  // [wave][key tile][lane]
  bf16_t* tile = reinterpret_cast<bf16_t*>(mine + TEAM_PARTS);    // [32][pitch]

  const int hi = min(k.count, (split + 1) * k.per), each = wide / 8;
  int p_row[PIECES], p_col[PIECES];
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    const int e = t + 256 * i;
    const int row = (int)__umulhi((unsigned)e, each_inverse);   // e / each
    p_row[i] = e < TEAM_KEYS * each ? row : -1;
    p_col[i] = (e - row * each) * 8;
  }
  u32x4 held[PIECES];
  const int wrap = k.first % a.ring;
  auto fetch = [&](int base) {
#pragma unroll
    for (int i = 0; i < PIECES; ++i)
      if (p_row[i] >= 0) {
        const int in_ring = wrap + min(base + p_row[i], hi - 1);   // past the last: the last again
        const size_t at = (size_t)slot * a.ring + (in_ring < a.ring ? in_ring : in_ring - a.ring);
        const bf16_t* from = p_col[i] < a.rank ? latents + at * a.rank + p_col[i] : shared_keys + at * a.rot + p_col[i] - a.rank;
        held[i] = *reinterpret_cast<const u32x4*>(from);
      }
  };
  int base = split * k.per + team * TEAM_KEYS;
  fetch(base);
  bf16x8 qf[STEPS];
  const int steps = (rank_pad + rot_pad) / 32;
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int c = (wave + 4 * i) * 32 + quad * 8, from = c < rank_pad ? (c < a.rank ? c : -1) : (c - rank_pad < a.rot ? a.rank + c - rank_pad : -1);
    uint4 v = make_uint4(0, 0, 0, 0);
    if (from >= 0) v = *reinterpret_cast<const uint4*>(q + ((size_t)slot * a.heads + min(head0 + lo16, a.heads - 1)) * wide + from);
    qf[i] = __builtin_bit_cast(bf16x8, v);
  }
  // The padding's zeros, which no tile replaces.
  const int pad_pieces = (pitch - 8 - wide) / 8;
  for (int e = t; e < TEAM_KEYS * pad_pieces; e += 256) {
    const int row = e / pad_pieces, i = (e - row * pad_pieces) * 8, gap = rank_pad - a.rank;
    *reinterpret_cast<uint4*>(tile + row * pitch + (i < gap ? a.rank + i : rank_pad + a.rot + i - gap)) = make_uint4(0, 0, 0, 0);
  }
  f32x4 acc[NG][4];
#pragma unroll
  for (int g = 0; g < NG; ++g)
#pragma unroll
    for (int e = 0; e < 4; ++e) acc[g][e] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -1e30f, l = 0.f;
  const float scale = a.scale * LATENT_LOG2E;
  for (; base - team * TEAM_KEYS < hi; base += STEP_KEYS) {   // (a team past the last key: weights of zero)
    __syncthreads();   // the last tile's readers are done
#pragma unroll
    for (int i = 0; i < PIECES; ++i)
      if (p_row[i] >= 0)
        *reinterpret_cast<u32x4*>(tile + p_row[i] * pitch + (p_col[i] < a.rank ? p_col[i] : rank_pad + p_col[i] - a.rank)) = held[i];
    __syncthreads();
    if (base - team * TEAM_KEYS + STEP_KEYS < hi) fetch(base + STEP_KEYS);
    f32x4 sc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int i = 0; i < STEPS; ++i) {
      if (wave + 4 * i >= steps) break;
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(tile + (kt * 16 + lo16) * pitch + (wave + 4 * i) * 32 + quad * 8);
        sc[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[i], sc[kt], 0, 0, 0);
      }
    }
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) parts[(wave * 2 + kt) * 64 + lane] = sc[kt];
    __syncthreads();
    float top = m;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
      sc[kt] = parts[kt * 64 + lane];
#pragma unroll
      for (int w = 1; w < 4; ++w) sc[kt] += parts[(w * 2 + kt) * 64 + lane];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        sc[kt][r] = base + kt * 16 + quad * 4 + r < hi ? sc[kt][r] * scale : -INFINITY;
        top = fmaxf(top, sc[kt][r]);
      }
    }
    top = fmaxf(top, __shfl_xor(top, 16, 64));
    top = fmaxf(top, __shfl_xor(top, 32, 64));
    const float fade = __builtin_amdgcn_exp2f(m - top);
    m = top;
    l *= fade;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        sc[kt][r] = __builtin_amdgcn_exp2f(sc[kt][r] - top);
        l += sc[kt][r];
      }
    const bf16x8 pf = __builtin_bit_cast(bf16x8, make_uint4(pack_bf16(sc[0][0], sc[0][1]), pack_bf16(sc[0][2], sc[0][3]),
                                                            pack_bf16(sc[1][0], sc[1][1]), pack_bf16(sc[1][2], sc[1][3])));
    // Lane (quad, lo16) of a group reads columns lo16 * 4 .. + 3 of its eight keys: register e of four products' A
    // operands, whose rows are then columns 4 row + e.
#pragma unroll
    for (int g = 0; g < NG; ++g) {
      if ((wave + 4 * g) * 64 >= rank_pad) break;
      uint2 w[8];
#pragma unroll
      for (int j = 0; j < 8; ++j)
        w[j] = *reinterpret_cast<const uint2*>(tile + ((j >> 2) * 16 + quad * 4 + (j & 3)) * pitch + (wave + 4 * g) * 64 + lo16 * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        uint32_t f[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const uint32_t x0 = e < 2 ? w[2 * j].x : w[2 * j].y, x1 = e < 2 ? w[2 * j + 1].x : w[2 * j + 1].y;
          f[j] = e & 1 ? (x0 >> 16) | (x1 & 0xffff0000u) : (x0 & 0xffffu) | (x1 << 16);
        }
        f32x4& o = acc[g][e];
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] *= fade;
        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, make_uint4(f[0], f[1], f[2], f[3])), pf, o, 0, 0, 0);
      }
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  // The second team's sums join the first's, through the LDS its keys lay in.
  __syncthreads();
  const int other_pitch = rank_pad + 4;   // (sixteen heads side by side over all banks)
  float* other = reinterpret_cast<float*>(dyn + 2 * TEAM_PARTS + TEAM_KEYS * pitch * 2);   // [16][other_pitch]
  float* other_stats = reinterpret_cast<float*>(dyn + TEAM_PARTS + TEAM_KEYS * pitch * 2);
  if (team == 1) {
#pragma unroll
    for (int g = 0; g < NG; ++g)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = (wave + 4 * g) * 64 + (quad * 4 + r) * 4;
        if (c < rank_pad) *reinterpret_cast<float4*>(other + lo16 * other_pitch + c) = make_float4(acc[g][0][r], acc[g][1][r], acc[g][2][r], acc[g][3][r]);
      }
    if (wave == 0 && quad == 0) {
      other_stats[2 * lo16] = m;
      other_stats[2 * lo16 + 1] = l;
    }
  }
  __syncthreads();
  const int head = head0 + lo16;
  if (team == 1 || head >= a.heads) return;
  const float om = other_stats[2 * lo16], top = fmaxf(m, om), f0 = __builtin_amdgcn_exp2f(m - top), f1 = __builtin_amdgcn_exp2f(om - top);
  const size_t part = ((size_t)slot * splits + split) * a.heads + head;
#pragma unroll
  for (int g = 0; g < NG; ++g)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int c = (wave + 4 * g) * 64 + (quad * 4 + r) * 4;
      if (c < a.rank) {
        const float4 o = *reinterpret_cast<const float4*>(other + lo16 * other_pitch + c);
        *reinterpret_cast<float4*>(to.sums + part * a.rank + c) =
            make_float4(fmaf(acc[g][0][r], f0, o.x * f1), fmaf(acc[g][1][r], f0, o.y * f1), fmaf(acc[g][2][r], f0, o.z * f1), fmaf(acc[g][3][r], f0, o.w * f1));
      }
    }
  if (wave == 0 && quad == 0) {
    to.stats[2 * part] = top;
    to.stats[2 * part + 1] = fmaf(l, f0, other_stats[2 * lo16 + 1] * f1);
  }
}

// The splits' sums become a head's latent, and V_h makes its values of it: a wave VALUE_ROWS value columns, whose
// weights (CH 16-byte pieces a lane; 0: any rank, read where they are needed) are on their way from the start.
constexpr int VALUE_ROWS = 8, VALUE_AHEAD = 16;   // ... and the splits whose sums are asked for together
template <typename T, int CH>
__global__ __launch_bounds__(256) void latent_values_kernel(StepParts from, const bf16_t* __restrict__ up, const bf16_t* __restrict__ sink,
                                                            const int* __restrict__ spans, T* __restrict__ y, LatentShape a, int splits) {
  constexpr int HELD = CH > 0 ? CH : 1;
  extern __shared__ __align__(16) float lds[];   // the latent, then a weight a split
  const int head = blockIdx.x, slot = blockIdx.z, t = threadIdx.x, lane = t & 63, wave = t >> 6;
  const int v0 = (blockIdx.y * 4 + wave) * VALUE_ROWS;
  const bf16_t* rows = up + ((size_t)a.heads * a.dim + (size_t)head * a.vdim) * a.rank;
  uint4 w[VALUE_ROWS][HELD];
  if (CH > 0) {
#pragma unroll
    for (int r = 0; r < VALUE_ROWS; ++r) {
      const __amdgpu_buffer_rsrc_t run = bounded_bytes(rows + (size_t)min(v0 + r, a.vdim - 1) * a.rank, a.rank * 2);
#pragma unroll
      for (int i = 0; i < CH; ++i) w[r][i] = load_bounded(run, 16 * (lane + 64 * i));
    }
  }
  const Span s = span_of(spans, slot, a.rows);
  if (s.rows == 0) return;
  const StepKeys k = step_keys(s, a, splits);
  float* latent = lds;
  float* shares = lds + ((a.rank + 511) & ~511);
  const size_t part = (size_t)slot * splits * a.heads + head;
  const float sunk = sink != nullptr ? bf16_to_f32(sink[head]) * LATENT_LOG2E : -1e30f;
  float top = sunk, total = 0.f;
  for (int i = lane; i < k.live; i += 64) top = fmaxf(top, from.stats[2 * (part + (size_t)i * a.heads)]);
  top = wave_max(top);
  const int padded = (k.live + VALUE_AHEAD - 1) & ~(VALUE_AHEAD - 1);   // (past the last: no share of the last)
  for (int i = lane; i < padded; i += 64) {
    const size_t at = 2 * (part + (size_t)min(i, k.live - 1) * a.heads);
    const float share = i < k.live ? latent_exp2<T>(from.stats[at] - top) : 0.f;
    if (wave == 0) shares[i] = share;
    total = fmaf(share, from.stats[at + 1], total);
  }
  total = wave_sum(total) + (sink != nullptr ? latent_exp2<T>(sunk - top) : 0.f);
  __syncthreads();
  const float inv = 1.0f / total;
  for (int c = t; c < ((a.rank + 511) & ~511); c += 256) {
    float sum = 0.f;
    const int col = min(c, a.rank - 1);
    for (int i = 0; i < padded; i += VALUE_AHEAD) {
      float v[VALUE_AHEAD];
#pragma unroll
      for (int j = 0; j < VALUE_AHEAD; ++j) v[j] = from.sums[(part + (size_t)min(i + j, k.live - 1) * a.heads) * a.rank + col];
#pragma unroll
      for (int j = 0; j < VALUE_AHEAD; ++j) sum = fmaf(v[j], shares[i + j], sum);
    }
    latent[c] = c < a.rank ? sum * inv : 0.f;
  }
  __syncthreads();
#pragma unroll
  for (int r = 0; r < VALUE_ROWS; ++r) {
    if (v0 + r >= a.vdim) break;
    float sum = 0.f;
    if (CH > 0) {
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        float f[8];
        unpack8(w[r][i], f);
        const float4 lo = *reinterpret_cast<const float4*>(latent + (lane + 64 * i) * 8), hi = *reinterpret_cast<const float4*>(latent + (lane + 64 * i) * 8 + 4);
        sum = fmaf(f[0], lo.x, sum); sum = fmaf(f[1], lo.y, sum); sum = fmaf(f[2], lo.z, sum); sum = fmaf(f[3], lo.w, sum);
        sum = fmaf(f[4], hi.x, sum); sum = fmaf(f[5], hi.y, sum); sum = fmaf(f[6], hi.z, sum); sum = fmaf(f[7], hi.w, sum);
      }
    } else {
      for (int c = lane; c < a.rank; c += 64) sum = fmaf(bf16_to_f32(rows[(size_t)(v0 + r) * a.rank + c]), latent[c], sum);
    }
    sum = wave_sum(sum);
    if (lane == 0) store_one(y + ((size_t)s.row0 * a.heads + head) * a.vdim + v0 + r, sum);
  }
}

// ------------------------------------------------------------------ host side
static bool latent_aligned(const LatentShape& a) { return a.rank % 8 == 0 && a.rot % 8 == 0; }
// LDS of the MFMA step, or 0 where its sizes are not served.
static size_t step_mfma_lds(const LatentShape& a) {
  const int ng = a.rank <= 256 ? 1 : (a.rank <= 512 ? 2 : 4);
  if (!latent_aligned(a) || a.rank > 1024 || a.rot > 64 * ng) return 0;
  const size_t bytes = 2 * (TEAM_PARTS + (size_t)TEAM_KEYS * (((a.rank + 63) & ~63) + ((a.rot + 31) & ~31) + 8) * 2);
  return bytes <= 163840 ? bytes : 0;
}
static int step_splits(const LatentShape& a) {
  const int most = a.window < a.ring ? a.window : a.ring, tiles = (most + STEP_KEYS - 1) / STEP_KEYS;
  int splits = 512 / (a.slots * ((a.heads + 15) / 16));
  splits = splits < 8 ? 8 : (splits > 64 ? 64 : splits);
  return tiles < splits ? tiles : splits;
}
static size_t rounded16(size_t n) { return (n + 15) & ~(size_t)15; }

static int check_latent(const char* what, const LatentShape& a, const void* spans, const void* shared_keys, const void* angles) {
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0, "%s: spans must be 16-byte aligned", what);
  IRON_REQUIRE(a.slots > 0 && a.slots <= 65535 && a.rows > 0, "%s: slots (%d) and rows (%d) must be positive", what, a.slots, a.rows);
  IRON_REQUIRE(a.heads > 0 && a.heads <= 65535 && a.dim > 0 && a.vdim > 0 && a.rank > 0 && a.rot >= 0, "%s: heads (%d) of %d + %d and %d, rank %d",
               what, a.heads, a.dim, a.rot, a.vdim, a.rank);
  IRON_REQUIRE(a.dim + a.rot <= 4096 && a.rank + a.rot <= 4096 && a.vdim <= 1024, "%s: keys (%d + %d) and latents (%d) up to 4096, values (%d) up to 1024",
               what, a.dim, a.rot, a.rank, a.vdim);
  IRON_REQUIRE(a.turned >= 0 && a.turned <= a.rot && a.turned % 2 == 0 && (a.rot == 0 || shared_keys) && (a.turned == 0 || (angles && a.angle_rows > 0)),
               "%s: %d of %d shared columns turn, by a table of %d rows", what, a.turned, a.rot, a.angle_rows);
  IRON_REQUIRE(a.window > 0 && a.ring > 0, "%s: a window (%d) and a ring (%d) of at least 1", what, a.window, a.ring);
  return IRON_OK;
}

}  // namespace iron

using namespace iron;

extern "C" int iron_latent_rows(const void* x, const uint16_t* q_gain, const uint16_t* c_gain, const float* angles, const int* spans,
                                void* q_out, void* latents, void* shared_keys, int slots, int rows, int stride, int q_rank, int rank,
                                int rot, int turned, int angle_rows, int ring, float eps, int is_float, void* stream) {
  IRON_REQUIRE(x && q_gain && c_gain && spans && q_out && latents, "latent_rows: null operand");
  const LatentShape a{slots, rows, 1, 1, rot, 1, rank, turned, angle_rows, 1, ring, 0, 1.f};
  if (const int e = check_latent("latent_rows", a, spans, shared_keys, angles)) return e;
  IRON_REQUIRE(q_rank > 0 && q_rank + rank + rot <= stride, "latent_rows: a row of %d holds no latents of %d and %d + %d", stride, q_rank, rank, rot);
  const LatentRow g{q_gain, c_gain, angles, q_rank, eps};
  const bool wide = latent_row_wide(a, stride, q_rank) && (((uintptr_t)x | (uintptr_t)q_gain | (uintptr_t)c_gain | (uintptr_t)q_out | (uintptr_t)latents |
                                                            (uintptr_t)shared_keys) & 15) == 0;
#define IRON_LATENT_ROWS(T, CH)                                                                                                   \
  hipLaunchKernelGGL((latent_rows_wide_kernel<T, CH>), dim3(rows), dim3(256), 0, (hipStream_t)stream, (const T*)x, g, spans, (T*)q_out, \
                     (T*)latents, (T*)shared_keys, a, stride)
  const bool two = q_rank + rank + rot <= 2 * 2048;
  if (wide && is_float) { if (two) IRON_LATENT_ROWS(float, 2); else IRON_LATENT_ROWS(float, 4); }
  else if (wide) { if (two) IRON_LATENT_ROWS(bf16_t, 2); else IRON_LATENT_ROWS(bf16_t, 4); }
#undef IRON_LATENT_ROWS
  else if (is_float)
    hipLaunchKernelGGL((latent_rows_kernel<float>), dim3(rows), dim3(256), 0, (hipStream_t)stream, (const float*)x, q_gain, c_gain, angles, spans,
                       (float*)q_out, (float*)latents, (float*)shared_keys, a, stride, q_rank, eps);
  else
    hipLaunchKernelGGL((latent_rows_kernel<bf16_t>), dim3(rows), dim3(256), 0, (hipStream_t)stream, (const bf16_t*)x, q_gain, c_gain, angles, spans,
                       (bf16_t*)q_out, (bf16_t*)latents, (bf16_t*)shared_keys, a, stride, q_rank, eps);
  IRON_LAUNCH_CHECK();
}

extern "C" int64_t iron_mha_latent_workspace_bytes(int slots, int rows, int heads, int dim, int rot, int vdim, int rank, int window, int ring,
                                                   int cap, int single, int is_float) {
  const LatentShape a{slots, rows, heads, dim, rot, vdim, rank, 0, 0, window, ring, cap, 1.f};
  if (slots <= 0 || heads <= 0 || rank <= 0 || window <= 0 || ring <= 0) return 0;
  const size_t each = is_float ? 4 : 2;
  if (!single) {
    const size_t n = (size_t)expanded_rows(cap);
    return (int64_t)(16 + rounded16(n * rank * each) + rounded16(n * rot * each) + n * heads * (dim + vdim) * each);
  }
  return (int64_t)(rounded16((size_t)slots * heads * (rank + rot) * 4) + rounded16((size_t)slots * step_splits(a) * heads * rank * 4) +
                   (size_t)slots * step_splits(a) * heads * 8);
}

extern "C" int iron_mha_latent(const void* q, const void* latents, const void* shared_keys, const uint16_t* up, const uint16_t* sink,
                               const float* angles, const int* spans, void* y, void* workspace, int slots, int rows, int heads, int dim,
                               int rot, int vdim, int rank, int turned, int angle_rows, int window, int ring, int cap, float scale, int single,
                               int is_float, void* stream) {
  IRON_REQUIRE(q && latents && up && spans && y && workspace, "mha_latent: null operand");
  const LatentShape a{slots, rows, heads, dim, rot, vdim, rank, turned, angle_rows, window, ring, cap, scale};
  if (const int e = check_latent("mha_latent", a, spans, shared_keys, angles)) return e;
  IRON_REQUIRE((((uintptr_t)q | (uintptr_t)latents | (uintptr_t)shared_keys | (uintptr_t)up | (uintptr_t)y | (uintptr_t)workspace |
                 (uintptr_t)angles) & 15) == 0, "mha_latent: operands must be 16-byte aligned");
  hipStream_t s = (hipStream_t)stream;
  unsigned char* work = (unsigned char*)workspace;
  const int width = heads * (dim + vdim);
  if (single) {   // the caller's spans have one row at most
    const int splits = step_splits(a);
    const size_t mfma_lds = is_float ? 0 : step_mfma_lds(a);
    void* absorbed = work;
    StepParts parts;
    parts.sums = (float*)(work + rounded16((size_t)slots * heads * (rank + rot) * 4));
    parts.stats = (float*)((unsigned char*)parts.sums + rounded16((size_t)slots * splits * heads * rank * 4));
    const bool vec = rank % 8 == 0;
    const dim3 ag(heads, slots, vec ? (rank + 127) / 128 : (rank + 15) / 16);
    const size_t alds = (size_t)(((dim + 3) & ~3) + 16 * (vec ? 128 : 16)) * 4;
#define IRON_ABSORB(T, OUT)                                                                                                              \
  {                                                                                                                                      \
    if (vec) hipLaunchKernelGGL((latent_absorb_kernel<T, OUT, 8>), ag, dim3(256), alds, s, (const T*)q, up, angles, spans, (OUT*)absorbed, a); \
    else hipLaunchKernelGGL((latent_absorb_kernel<T, OUT, 1>), ag, dim3(256), alds, s, (const T*)q, up, angles, spans, (OUT*)absorbed, a);     \
  }
    if (is_float) IRON_ABSORB(float, float)
    else if (mfma_lds) IRON_ABSORB(bf16_t, bf16_t)
    else IRON_ABSORB(bf16_t, float)
#undef IRON_ABSORB
    if (mfma_lds) {
      const dim3 grid((heads + 15) / 16, splits, slots);
#define IRON_STEP(NG)                                                                                                        \
  static LdsOptIn opted##NG;                                                                                                 \
  if (const hipError_t e = opted##NG.ensure((const void*)latent_step_mfma_kernel<NG>, 163840)) {                             \
    set_error("mha_latent: %s", hipGetErrorString(e));                                                                       \
    return (int)e;                                                                                                           \
  }                                                                                                                          \
  hipLaunchKernelGGL((latent_step_mfma_kernel<NG>), grid, dim3(512), mfma_lds, s, (const bf16_t*)absorbed, (const bf16_t*)latents, \
                     (const bf16_t*)shared_keys, spans, parts, a, splits, (unsigned)((1ull << 32) / (unsigned)((rank + rot) / 8) + 1))
      if (rank <= 256) { IRON_STEP(1); }
      else if (rank <= 512) { IRON_STEP(2); }
      else { IRON_STEP(4); }
#undef IRON_STEP
    } else {
      const dim3 grid(heads, splits, slots);
      const size_t lds = (size_t)(rank + rot + 4 * rank) * 4;
      IRON_REQUIRE(lds <= 65536 - 64, "mha_latent: a latent of %d columns does not fit a block's LDS", rank);
      if (is_float)
        hipLaunchKernelGGL((latent_step_kernel<float>), grid, dim3(256), lds, s, (const float*)absorbed, (const float*)latents,
                           (const float*)shared_keys, spans, parts, a, splits);
      else
        hipLaunchKernelGGL((latent_step_kernel<bf16_t>), grid, dim3(256), lds, s, (const float*)absorbed, (const bf16_t*)latents,
                           (const bf16_t*)shared_keys, spans, parts, a, splits);
    }
    const dim3 vg(heads, (vdim + 4 * VALUE_ROWS - 1) / (4 * VALUE_ROWS), slots);
    const size_t vlds = (size_t)(splits + VALUE_AHEAD + ((rank + 511) & ~511)) * 4;
#define IRON_VALUES_CH(T, CH) hipLaunchKernelGGL((latent_values_kernel<T, CH>), vg, dim3(256), vlds, s, parts, up, sink, spans, (T*)y, a, splits)
#define IRON_VALUES(T)                                  \
  {                                                     \
    if (vec && rank <= 512) IRON_VALUES_CH(T, 1);       \
    else if (vec && rank <= 1024) IRON_VALUES_CH(T, 2); \
    else IRON_VALUES_CH(T, 0);                          \
  }
    if (is_float) IRON_VALUES(float)
    else IRON_VALUES(bf16_t)
#undef IRON_VALUES
#undef IRON_VALUES_CH
    IRON_LAUNCH_CHECK();
  }

  IRON_REQUIRE(cap > 0 && rows <= 65535, "mha_latent: room for keys (%d), and rows (%d) within the grid's extent", cap, rows);
  IRON_REQUIRE((long)LATENT_KEYS * width < (1L << 31) && expanded_rows(cap) < (1L << 31), "mha_latent: a tile's rows are addressed with 32-bit offsets");
  const size_t n = (size_t)expanded_rows(cap), each = is_float ? 4 : 2;
  int* count = (int*)work;
  void* gathered = work + 16;
  void* shared = work + 16 + rounded16(n * rank * each);
  void* kv = work + 16 + rounded16(n * rank * each) + rounded16(n * rot * each);
  const dim3 gg((cap + LATENT_KEYS + GATHER_ROWS - 1) / GATHER_ROWS);
  const bool vec = rank % 8 == 0;
#define IRON_GATHER(T)                                                                                                                      \
  {                                                                                                                                         \
    if (vec && rot % 8 == 0)                                                                                                                \
      hipLaunchKernelGGL((latent_gather_kernel<T, 8>), gg, dim3(256), 0, s, (const T*)latents, (const T*)shared_keys, spans, (T*)gathered, (T*)shared, count, a); \
    else                                                                                                                                    \
      hipLaunchKernelGGL((latent_gather_kernel<T, 1>), gg, dim3(256), 0, s, (const T*)latents, (const T*)shared_keys, spans, (T*)gathered, (T*)shared, count, a); \
  }
  if (is_float) IRON_GATHER(float)
  else IRON_GATHER(bf16_t)
#undef IRON_GATHER
  const int e = is_float || !vec ? iron_linear_any(gathered, up, kv, (int)n, width, rank, is_float, count, stream)
                                 : iron_gemm_bf16((const uint16_t*)gathered, up, (uint16_t*)kv, (int)n, width, rank, 1, 0, count, nullptr, stream);
  if (e != IRON_OK) return e;
  const bool tiles = !is_float && dim % 8 == 0 && rot % 8 == 0 && turned % 8 == 0 && vdim % 8 == 0 && dim + rot <= 256 && vdim <= 256;
  if (tiles) {
    const bf16_t *qb = (const bf16_t*)q, *kvb = (const bf16_t*)kv, *rb = (const bf16_t*)shared;
    if (dim + rot <= 32) launch_latent_prefill<32>(qb, kvb, rb, angles, sink, spans, (bf16_t*)y, a, s);
    else if (dim + rot <= 64) launch_latent_prefill<64>(qb, kvb, rb, angles, sink, spans, (bf16_t*)y, a, s);
    else if (dim + rot <= 128) launch_latent_prefill<128>(qb, kvb, rb, angles, sink, spans, (bf16_t*)y, a, s);
    else if (dim + rot <= 192) launch_latent_prefill<192>(qb, kvb, rb, angles, sink, spans, (bf16_t*)y, a, s);
    else launch_latent_prefill<256>(qb, kvb, rb, angles, sink, spans, (bf16_t*)y, a, s);
  } else {
    const dim3 grid(heads, rows, slots);
    const size_t lds = (size_t)(dim + rot + 64) * 4;
    if (is_float)
      hipLaunchKernelGGL((latent_rows_attention_kernel<float>), grid, dim3(64), lds, s, (const float*)q, (const float*)kv, (const float*)shared,
                         angles, sink, spans, (float*)y, a);
    else
      hipLaunchKernelGGL((latent_rows_attention_kernel<bf16_t>), grid, dim3(64), lds, s, (const bf16_t*)q, (const bf16_t*)kv, (const bf16_t*)shared,
                         angles, sink, spans, (bf16_t*)y, a);
  }
  IRON_LAUNCH_CHECK();
}
