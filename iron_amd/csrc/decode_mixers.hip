// One token a slot through a stateful mixer, in one launch where a prompt's portion takes several:
//
//   decode_parallel: low-rank decay, time-mixing step, head norm and gate (a block a head)
//                    beside sliding-window attention with its distance bias (a block a query head)
//   decode_delta:    short convolution, unit q and k, gated delta rule, head norm and gate
//   decode_hgrn2:    forget gate, fading memory, head norm (a block a head) beside a feed-forward's gated columns and a router's
//                    choice
//
// bf16 rows, float32 inside.  A block is 16 waves.  A head's state (dim rows of `wide` columns, wide a power
// of two from 16 to 256) is read once, four columns a thread, and kept in registers until it is replaced;
// what the step's arithmetic needs of the state's sums is a sum down its rows: across a wave's rows by
// shuffles, across the waves through LDS.  Blocks of one slot read states that none of them replaces:
// rings with a row to spare (see the prompt kernels, whose layouts these are).
#include "../../include/iron_hip.h"
#include "hgrn2.h"
#include "router.h"

namespace iron {

constexpr int DM_WAVES = 16, DM_THREADS = DM_WAVES * 64;

__device__ __forceinline__ float silu_exact(float z) { return z / (1.0f + expf(-z)); }

// The sum over the block of every thread's v (all threads get it); `part` DM_WAVES floats nobody else uses.
__device__ __forceinline__ float dm_block_sum(float v, float* part) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
  __syncthreads();
  float sum = 0.f;
#pragma unroll
  for (int w = 0; w < DM_WAVES; ++w) sum += part[w];
  return sum;
}

// A head's state over the block's threads: thread t holds columns 4 (t % quads) .. + 3 of rows t / quads,
// t / quads + stride, ...
struct StateTiles {
  int quads, col, row, stride;
  __device__ __forceinline__ explicit StateTiles(int wide) {
    quads = wide >> 2;
    col = ((int)threadIdx.x & (quads - 1)) * 4;
    row = (int)threadIdx.x / quads;
    stride = DM_THREADS / quads;
  }
  // Sums over the rows a wave holds; afterwards lanes 0 .. quads - 1 of the wave have them.
  __device__ __forceinline__ void fold(float4& v) const {
    for (int mask = quads; mask < 64; mask <<= 1) {
      v.x += __shfl_xor(v.x, mask, 64);
      v.y += __shfl_xor(v.y, mask, 64);
      v.z += __shfl_xor(v.z, mask, 64);
      v.w += __shfl_xor(v.w, mask, 64);
    }
  }
};

struct HeadOut {            // where a head's gated row goes
  const bf16_t* gate;       // the batch row's gate, this head's columns
  const bf16_t* gain;
  bf16_t* to;
  float eps, scale;
};
// o (wide floats in LDS, whole) -> o / rms * gain * silu(gate) * scale, by the block's first threads.
__device__ __forceinline__ void finish_head(const float* o, int wide, const HeadOut& h, float* part) {
  const int t = threadIdx.x;
  const float v = t < wide ? o[t] : 0.f;
  const float z = t < wide ? bf16_to_f32(h.gate[t]) : 0.f, g = t < wide ? bf16_to_f32(h.gain[t]) : 0.f;
  const float inv = 1.0f / sqrtf(dm_block_sum(v * v, part) / (float)wide + h.eps);
  if (t < wide) h.to[t] = f32_to_bf16(v * inv * g * silu_exact(z) * h.scale);
}

// ---------------------------------------------------------------- time mixing
struct TimeMixStep {
  const bf16_t *r, *k, *v, *g, *z;        // (slots, heads * dim) each, z (slots, rank)
  const bf16_t *w2, *w0, *u, *norm;
  float* state;                           // (slots, heads, dim, dim)
  bf16_t* out;                            // (slots, out_stride), from out_at
  int heads, dim, rank, out_stride, out_at;
  float eps, scale;
};
struct TimeMixShared {
  float r[256], k[256], w[256], v[256], o[256], z[512];
  float sums[DM_WAVES][256];
  float part[2][DM_WAVES];
};

template <int NR>
__device__ __forceinline__ void time_mix_step(const TimeMixStep& a, const Span& s, int slot, int head, TimeMixShared& sh) {
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, dim = a.dim;
  const StateTiles tile(dim);
  float* sp = a.state + ((size_t)slot * a.heads + head) * dim * dim;
  float4 S[NR];
#pragma unroll
  for (int n = 0; n < NR; ++n) {
    const int i = tile.row + n * tile.stride;
    S[n] = (s.start > 0 && i < dim) ? *reinterpret_cast<const float4*>(sp + (size_t)i * dim + tile.col) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  const size_t row = s.row0, at = row * a.heads * dim + head * dim;
  float bonus = 0.f;
  if (t < dim) {
    const float r = bf16_to_f32(a.r[at + t]), k = bf16_to_f32(a.k[at + t]);
    sh.r[t] = r;
    sh.k[t] = k;
    sh.v[t] = bf16_to_f32(a.v[at + t]);
    bonus = r * k * bf16_to_f32(a.u[head * dim + t]);
  }
  for (int i = t; i < a.rank; i += DM_THREADS) sh.z[i] = tanhf(bf16_to_f32(a.z[row * a.rank + i]));
  // The decays: a channel's row of w2 over as many lanes as it has 16-byte pieces, the first ones asked for
  // ahead of the barrier; or, where its pieces are no power of two, over a wave.
  const int pieces = a.rank >> 3, piece = t & (pieces - 1);
  const bool dealt = a.rank % 8 == 0 && (pieces & (pieces - 1)) == 0 && pieces <= 64;
  uint4 ahead = make_uint4(0, 0, 0, 0);
  if (dealt && t / pieces < dim) ahead = reinterpret_cast<const uint4*>(a.w2 + (size_t)(head * dim + t / pieces) * a.rank)[piece];
  bonus = dm_block_sum(bonus, sh.part[0]);   // its barrier is the one the LDS rows wait for, too
  if (dealt) {
    for (int c = t / pieces; c - t / pieces < dim; c += DM_THREADS / pieces) {
      float f[8], sum = 0.f;
      unpack8(ahead, f);
#pragma unroll
      for (int j = 0; j < 8; ++j) sum = fmaf(f[j], sh.z[piece * 8 + j], sum);
      for (int mask = 1; mask < pieces; mask <<= 1) sum += __shfl_xor(sum, mask, 64);
      if (piece == 0 && c < dim) sh.w[c] = expf(-expf(sum + bf16_to_f32(a.w0[head * dim + c])));
      const int next = c + DM_THREADS / pieces;
      if (next < dim) ahead = reinterpret_cast<const uint4*>(a.w2 + (size_t)(head * dim + next) * a.rank)[piece];
    }
  } else for (int c = wave; c < dim; c += DM_WAVES) {
    const bf16_t* w = a.w2 + (size_t)(head * dim + c) * a.rank;
    float sum = 0.f;
    for (int i = lane; i < a.rank; i += 64) sum = fmaf(bf16_to_f32(w[i]), sh.z[i], sum);
    sum = wave_sum(sum);
    if (lane == 0) sh.w[c] = expf(-expf(sum + bf16_to_f32(a.w0[head * dim + c])));
  }
  __syncthreads();
  const float4 v = *reinterpret_cast<const float4*>(&sh.v[tile.col]);
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
  for (int n = 0; n < NR; ++n) {
    const int i = tile.row + n * tile.stride;
    if (i < dim) {
      const float r = sh.r[i], k = sh.k[i], w = sh.w[i];
      o.x = fmaf(r, S[n].x, o.x); o.y = fmaf(r, S[n].y, o.y); o.z = fmaf(r, S[n].z, o.z); o.w = fmaf(r, S[n].w, o.w);
      S[n].x = fmaf(w, S[n].x, k * v.x); S[n].y = fmaf(w, S[n].y, k * v.y);
      S[n].z = fmaf(w, S[n].z, k * v.z); S[n].w = fmaf(w, S[n].w, k * v.w);
      *reinterpret_cast<float4*>(sp + (size_t)i * dim + tile.col) = S[n];
    }
  }
  tile.fold(o);
  if (lane < tile.quads) *reinterpret_cast<float4*>(&sh.sums[wave][tile.col]) = o;
  __syncthreads();
  if (t < dim) {
    float sum = bonus * sh.v[t];
#pragma unroll
    for (int w = 0; w < DM_WAVES; ++w) sum += sh.sums[w][t];
    sh.o[t] = sum;   // read back by the same thread
  }
  finish_head(sh.o, dim, HeadOut{a.g + at, a.norm + head * dim, a.out + row * a.out_stride + a.out_at + head * dim, a.eps, a.scale}, sh.part[1]);
}

// ------------------------------------------------------------------ attention
struct WindowStep {
  const bf16_t* x;                        // (slots, stride): q heads, k heads, v heads
  bf16_t *keys, *values;                  // (slots, ring, kv_heads, dim / vdim)
  const float* bias;                      // (heads, window)
  bf16_t* out;
  int stride, heads, kv_heads, dim, vdim, window, ring, out_stride, out_at;
  float scale, out_scale;
};
struct WindowShared1 {
  float q[256], p[DM_WAVES][64], m[DM_WAVES], l[DM_WAVES];
  __align__(16) float red[DM_WAVES * 512];              // [wave][keys at once][vdim], at most 512 floats a wave
};

__device__ __forceinline__ void window_step(const WindowStep& a, const Span& s, int slot, int head, WindowShared1& sh) {
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, group = a.heads / a.kv_heads, g = head / group;
  const int nk = a.kv_heads * a.dim, nv = a.kv_heads * a.vdim;
  const int pos = s.start, lo = max(0, pos - a.window + 1), count = pos - lo + 1;
  const bf16_t* row = a.x + (size_t)s.row0 * a.stride;
  const bf16_t* own_k = row + a.heads * a.dim + g * a.dim;
  const bf16_t* own_v = row + a.heads * a.dim + nk + g * a.vdim;
  bf16_t* ring_k = a.keys + (size_t)slot * a.ring * nk + g * a.dim;
  bf16_t* ring_v = a.values + (size_t)slot * a.ring * nv + g * a.vdim;
  for (int c = t; c < a.dim; c += DM_THREADS) sh.q[c] = bf16_to_f32(row[head * a.dim + c]) * a.scale;
  if (head % group == 0) {   // position pos - ring, whose row this replaces, is outside the window
    const int at = pos % a.ring;
    for (int c = t; c < a.dim; c += DM_THREADS) ring_k[(size_t)at * nk + c] = own_k[c];
    for (int c = t; c < a.vdim; c += DM_THREADS) ring_v[(size_t)at * nv + c] = own_v[c];
  }
  __syncthreads();
  const int pieces = a.vdim / 8, keys_at_once = 64 / pieces, mine = lane / pieces, piece = lane - mine * pieces;
  float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, m = -INFINITY, l = 0.f;
  for (int k0 = wave * 64; k0 < count; k0 += DM_THREADS) {
    float score = -INFINITY;
    if (k0 + lane < count) {
      const int p = lo + k0 + lane;
      const bf16_t* kr = p == pos ? own_k : ring_k + (size_t)(p % a.ring) * nk;
      const float by = a.bias[(size_t)head * a.window + (pos - p)];
      float dot = 0.f;
#pragma unroll 8
      for (int c = 0; c < a.dim; c += 8) {
        float f[8];
        unpack8(*reinterpret_cast<const uint4*>(kr + c), f);
#pragma unroll
        for (int j = 0; j < 8; ++j) dot = fmaf(f[j], sh.q[c + j], dot);
      }
      score = dot + by;
    }
    const float top = fmaxf(m, wave_max(score));
    const float fade = __expf(m - top), p = __expf(score - top);
    m = top;
    l = l * fade + p;
    sh.p[wave][lane] = p;
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[j] *= fade;
    const int n = min(64, count - k0);
    if (mine < keys_at_once)
#pragma unroll 8
      for (int q = mine; q < n; q += keys_at_once) {
        const int at = lo + k0 + q;
        const bf16_t* vr = at == pos ? own_v : ring_v + (size_t)(at % a.ring) * nv;
        const float w = sh.p[wave][q];
        float f[8];
        unpack8(*reinterpret_cast<const uint4*>(vr + piece * 8), f);
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[j] = fmaf(w, f[j], acc[j]);
      }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  l = wave_sum(l);
  if (lane == 0) {
    sh.m[wave] = m;
    sh.l[wave] = l;
  }
  if (mine < keys_at_once)
#pragma unroll
    for (int j = 0; j < 8; ++j) sh.red[(wave * keys_at_once + mine) * a.vdim + piece * 8 + j] = acc[j];
  __syncthreads();
  float top = sh.m[0];
#pragma unroll
  for (int w = 1; w < DM_WAVES; ++w) top = fmaxf(top, sh.m[w]);
  if (t < a.vdim) {
    float total = 0.f, sum = 0.f;
    for (int w = 0; w < DM_WAVES; ++w) {
      if (w * 64 >= count) break;   // a wave without a key
      const float fade = __expf(sh.m[w] - top);
      total = fmaf(sh.l[w], fade, total);
      float part = 0.f;
      for (int r = 0; r < keys_at_once; ++r) part += sh.red[(w * keys_at_once + r) * a.vdim + t];
      sum = fmaf(part, fade, sum);
    }
    a.out[(size_t)s.row0 * a.out_stride + a.out_at + head * a.vdim + t] = f32_to_bf16(sum / total * a.out_scale);
  }
}

// The same where keys and values are LANES 16-byte pieces wide: LANES lanes to a key, 64 / LANES keys at a
// time, eight such steps' keys, values and biases asked for together.  A lane's scores are its own keys',
// and it weighs the same keys' values, so nothing is exchanged until the waves meet.
template <int LANES>
__device__ __forceinline__ float lanes_sum(float v) {
  static_assert(LANES == 4 || LANES == 8 || LANES == 16 || LANES == 32, "a power of two of lanes");
  v += IRON_DPP(0.f, v, 0xB1, 0xF);
  v += IRON_DPP(0.f, v, 0x4E, 0xF);
  if (LANES >= 8) v += IRON_DPP(0.f, v, 0x141, 0xF);
  if (LANES >= 16) v += IRON_DPP(0.f, v, 0x140, 0xF);
  if (LANES >= 32) v += __shfl_xor(v, 16, 64);
  return v;
}
template <int LANES>
__device__ __forceinline__ void window_step_lanes(const WindowStep& a, const Span& s, int slot, int head, WindowShared1& sh) {
  constexpr int AT_ONCE = 64 / LANES, STEPS = 8, KEYS = AT_ONCE * STEPS;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, group = a.heads / a.kv_heads, g = head / group;
  const int nk = a.kv_heads * a.dim, part = lane % LANES, mine = lane / LANES;
  const int pos = s.start, lo = max(0, pos - a.window + 1), count = pos - lo + 1, wrap = lo % a.ring;
  const bf16_t* row = a.x + (size_t)s.row0 * a.stride;
  const bf16_t* own_k = row + a.heads * a.dim + g * a.dim;
  const bf16_t* own_v = own_k + nk;
  bf16_t* ring_k = a.keys + (size_t)slot * a.ring * nk + g * a.dim;
  bf16_t* ring_v = a.values + (size_t)slot * a.ring * nk + g * a.dim;
  float q[8];
  unpack8(*reinterpret_cast<const uint4*>(row + head * a.dim + part * 8), q);
#pragma unroll
  for (int j = 0; j < 8; ++j) q[j] *= a.scale;
  if (head % group == 0 && t < 2 * LANES) {   // position pos - ring, whose row this replaces, is outside the window
    const bf16_t* src = t < LANES ? own_k : own_v;
    bf16_t* dst = (t < LANES ? ring_k : ring_v) + (size_t)(pos % a.ring) * nk;
    reinterpret_cast<uint4*>(dst)[part] = reinterpret_cast<const uint4*>(src)[part];
  }
  const long own_k_from = (const char*)own_k - (const char*)ring_k, own_v_from = (const char*)own_v - (const char*)ring_v;
  const float* by = a.bias + (size_t)head * a.window;
  float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, m = -INFINITY, l = 0.f;
  for (int k0 = wave * KEYS; k0 < count; k0 += DM_WAVES * KEYS) {
    u32x4 kv[STEPS], vv[STEPS];
    float score[STEPS];
#pragma unroll
    for (int i = 0; i < STEPS; ++i) {
      const int n = min(k0 + i * AT_ONCE + mine, count - 1);
      const long mask = -(long)(n == count - 1);
      const int at = wrap + n, back = at - a.ring;
      const long old = (long)(back >= 0 ? back : at) * (2 * nk);
      kv[i] = *reinterpret_cast<const u32x4*>((const char*)(ring_k + part * 8) + ((own_k_from & mask) | (old & ~mask)));
      vv[i] = *reinterpret_cast<const u32x4*>((const char*)(ring_v + part * 8) + ((own_v_from & mask) | (old & ~mask)));
      score[i] = by[count - 1 - n];
    }
    float top = m;
#pragma unroll
    for (int i = 0; i < STEPS; ++i) {
      float f[8], dot = 0.f;
      unpack8(make_uint4(kv[i].x, kv[i].y, kv[i].z, kv[i].w), f);
#pragma unroll
      for (int j = 0; j < 8; ++j) dot = fmaf(f[j], q[j], dot);
      score[i] = k0 + i * AT_ONCE + mine < count ? score[i] + lanes_sum<LANES>(dot) : -INFINITY;
      top = fmaxf(top, score[i]);
    }
#pragma unroll
    for (int mask = LANES; mask < 64; mask <<= 1) top = fmaxf(top, __shfl_xor(top, mask, 64));
    const float fade = __expf(m - top);   // top is finite: the piece's first key is one
    m = top;
    l *= fade;
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[j] *= fade;
#pragma unroll
    for (int i = 0; i < STEPS; ++i) {
      float f[8];
      const float p = __expf(score[i] - top);
      l += p;
      unpack8(make_uint4(vv[i].x, vv[i].y, vv[i].z, vv[i].w), f);
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] = fmaf(p, f[j], acc[j]);
    }
  }
#pragma unroll
  for (int mask = LANES; mask < 64; mask <<= 1) {
    l += __shfl_xor(l, mask, 64);
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[j] += __shfl_xor(acc[j], mask, 64);
  }
  if (lane == 0) {
    sh.m[wave] = m;
    sh.l[wave] = l;
  }
  if (mine == 0) {
    float4* to = reinterpret_cast<float4*>(&sh.red[wave * a.dim + part * 8]);
    to[0] = make_float4(acc[0], acc[1], acc[2], acc[3]);
    to[1] = make_float4(acc[4], acc[5], acc[6], acc[7]);
  }
  __syncthreads();
  if (t < a.dim) {
    float top = sh.m[0], total = 0.f, sum = 0.f;
#pragma unroll
    for (int w = 1; w < DM_WAVES; ++w) top = fmaxf(top, sh.m[w]);
#pragma unroll
    for (int w = 0; w < DM_WAVES; ++w) {   // a wave without a key: m is -inf, the rest 0
      const float fade = __expf(sh.m[w] - top);
      total = fmaf(sh.l[w], fade, total);
      sum = fmaf(sh.red[w * a.dim + t], fade, sum);
    }
    a.out[(size_t)s.row0 * a.out_stride + a.out_at + head * a.dim + t] = f32_to_bf16(sum / total * a.out_scale);
  }
}

__device__ __forceinline__ void window_step_any(const WindowStep& a, const Span& s, int slot, int head, WindowShared1& sh) {
  if (a.dim == a.vdim && a.dim == 64) window_step_lanes<8>(a, s, slot, head, sh);
  else if (a.dim == a.vdim && a.dim == 128) window_step_lanes<16>(a, s, slot, head, sh);
  else if (a.dim == a.vdim && a.dim == 32) window_step_lanes<4>(a, s, slot, head, sh);
  else if (a.dim == a.vdim && a.dim == 256) window_step_lanes<32>(a, s, slot, head, sh);
  else window_step(a, s, slot, head, sh);
}

union ParallelShared {
  TimeMixShared mix;
  WindowShared1 win;
};
template <int NR>
__global__ __launch_bounds__(DM_THREADS) void decode_parallel_kernel(TimeMixStep mix, WindowStep win, const int* __restrict__ spans, int rows) {
  __shared__ __align__(16) ParallelShared sh;
  const int slot = blockIdx.y;
  const Span s = span_of(spans, slot, rows);
  if (s.rows == 0) return;
  if ((int)blockIdx.x < win.heads) window_step_any(win, s, slot, blockIdx.x, sh.win);
  else time_mix_step<NR>(mix, s, slot, blockIdx.x - win.heads, sh.mix);
}

// --------------------------------------------------------------- the delta rule
struct DeltaStep {
  const bf16_t* x;                        // (slots, stride): q, k, v, .. gate .., b, a
  const bf16_t *taps_w, *a_log, *dt_bias, *norm;
  bf16_t* inputs;                         // (slots, taps, channels)
  float* state;                           // (slots, heads, dim, vdim)
  bf16_t* out;                            // (slots, heads * vdim)
  int stride, heads, kv_heads, dim, vdim, taps, gate_at, b_at, a_at;
  float eps;
};
struct DeltaShared {
  __align__(16) float q[256], k[256], v[256], u[256];
  float o[256];
  float read[DM_WAVES][256], outs[DM_WAVES][256];
  float part[4][DM_WAVES];
};

template <int NR>
__global__ __launch_bounds__(DM_THREADS) void decode_delta_kernel(DeltaStep a, const int* __restrict__ spans, int rows) {
  __shared__ DeltaShared sh;
  const int slot = blockIdx.y, head = blockIdx.x;
  const Span s = span_of(spans, slot, rows);
  if (s.rows == 0) return;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, dim = a.dim, vdim = a.vdim;
  const int group = a.heads / a.kv_heads, g = head / group, qk = a.kv_heads * dim, channels = 2 * qk + a.heads * vdim;
  const StateTiles tile(vdim);
  float* sp = a.state + ((size_t)slot * a.heads + head) * dim * vdim;
  float4 S[NR];
#pragma unroll
  for (int n = 0; n < NR; ++n) {
    const int i = tile.row + n * tile.stride;
    S[n] = (s.start > 0 && i < dim) ? *reinterpret_cast<const float4*>(sp + (size_t)i * vdim + tile.col) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  const bf16_t* row = a.x + (size_t)s.row0 * a.stride;
  bf16_t* held = a.inputs + (size_t)slot * a.taps * channels;
  // Threads 0 .. dim - 1 make q, the next dim k, the next vdim v (a wave of q's or k's lanes is whole).
  const int padded = (dim + 63) & ~63;
  const int part_of = t < padded ? 0 : (t < 2 * padded ? 1 : 2), j = t - part_of * padded;
  const int len = part_of == 2 ? vdim : dim;
  float f = 0.f;
  if (j < len) {
    const int ch = part_of == 0 ? g * dim + j : (part_of == 1 ? qk + g * dim + j : 2 * qk + head * vdim + j);
    const bf16_t now = row[ch];
    float acc = bf16_to_f32(a.taps_w[(size_t)ch * a.taps + a.taps - 1]) * bf16_to_f32(now);
    for (int i = 1; i < a.taps; ++i)
      if (s.start - i >= 0)
        acc = fmaf(bf16_to_f32(a.taps_w[(size_t)ch * a.taps + a.taps - 1 - i]),
                   bf16_to_f32(held[(size_t)((s.start - i) % a.taps) * channels + ch]), acc);
    f = silu_exact(acc);
    // The step's input: its ring row is no row the step reads.
    if (part_of == 2 || head % group == 0) held[(size_t)(s.start % a.taps) * channels + ch] = now;
  }
  const float mine = f * f;
  const float qq = wave_sum(part_of == 0 ? mine : 0.f), kk = wave_sum(part_of == 1 ? mine : 0.f);
  if (lane == 0) {
    sh.part[0][wave] = qq;
    sh.part[1][wave] = kk;
  }
  if (j < len) (part_of == 0 ? sh.q : part_of == 1 ? sh.k : sh.v)[j] = f;
  // Every thread computes the head's two scalars (behind the convolution's loads).
  const float da = bf16_to_f32(row[a.a_at + head]) + bf16_to_f32(a.dt_bias[head]);
  const float soft = da > 20.f ? da : log1pf(expf(da));
  const float decay = expf(-expf(bf16_to_f32(a.a_log[head])) * soft);
  const float beta = 1.0f / (1.0f + expf(-bf16_to_f32(row[a.b_at + head])));
  __syncthreads();
  float q2 = 0.f, k2 = 0.f;
#pragma unroll
  for (int w = 0; w < DM_WAVES; ++w) {
    q2 += sh.part[0][w];
    k2 += sh.part[1][w];
  }
  const float qs = 1.0f / sqrtf(q2 + 1e-6f) * (1.0f / sqrtf((float)dim)), ks = 1.0f / sqrtf(k2 + 1e-6f);
  float4 read = make_float4(0.f, 0.f, 0.f, 0.f), out = read;
  float kq = 0.f;
#pragma unroll
  for (int n = 0; n < NR; ++n) {
    const int i = tile.row + n * tile.stride;
    if (i < dim) {
      const float q = sh.q[i] * qs, k = sh.k[i] * ks;
      read.x = fmaf(k, S[n].x, read.x); read.y = fmaf(k, S[n].y, read.y); read.z = fmaf(k, S[n].z, read.z); read.w = fmaf(k, S[n].w, read.w);
      out.x = fmaf(q, S[n].x, out.x); out.y = fmaf(q, S[n].y, out.y); out.z = fmaf(q, S[n].z, out.z); out.w = fmaf(q, S[n].w, out.w);
    }
  }
  if (t < dim) kq = sh.q[t] * qs * (sh.k[t] * ks);
  tile.fold(read);
  tile.fold(out);
  if (lane < tile.quads) {
    *reinterpret_cast<float4*>(&sh.read[wave][tile.col]) = read;
    *reinterpret_cast<float4*>(&sh.outs[wave][tile.col]) = out;
  }
  kq = dm_block_sum(kq, sh.part[2]);   // its barrier is the sums', too
  if (t < vdim) {
    float r = 0.f, o = 0.f;
#pragma unroll
    for (int w = 0; w < DM_WAVES; ++w) {
      r += sh.read[w][t];
      o += sh.outs[w][t];
    }
    const float u = beta * fmaf(-decay, r, sh.v[t]);
    sh.u[t] = u;
    sh.o[t] = fmaf(kq, u, decay * o);
  }
  __syncthreads();
  const float4 u = *reinterpret_cast<const float4*>(&sh.u[tile.col]);
#pragma unroll
  for (int n = 0; n < NR; ++n) {
    const int i = tile.row + n * tile.stride;
    if (i < dim) {
      const float k = sh.k[i] * ks;
      S[n].x = fmaf(k, u.x, decay * S[n].x); S[n].y = fmaf(k, u.y, decay * S[n].y);
      S[n].z = fmaf(k, u.z, decay * S[n].z); S[n].w = fmaf(k, u.w, decay * S[n].w);
      *reinterpret_cast<float4*>(sp + (size_t)i * vdim + tile.col) = S[n];
    }
  }
  finish_head(sh.o, vdim, HeadOut{row + a.gate_at + head * vdim, a.norm, a.out + ((size_t)s.row0 * a.heads + head) * vdim, a.eps, 1.f}, sh.part[3]);
}

// ---------------------------------------------------------------------- HGRN2
struct FadeStep {
  const bf16_t* x;                        // (slots, stride): q, f, v
  FadeGates g;
  const bf16_t* norm;                     // (vdim)
  float* state;                           // (slots, heads, dim, vdim)
  bf16_t* out;                            // (slots, out_stride), from out_at
  int stride, heads, dim, vdim, out_stride, out_at;
  float eps;
  int cols, gate_at, gated_at, kind;      // gated columns of the same rows: how many, where from, where to
  float limit;
  RouterChoice choice;                    // of slot 0's logits
};
struct FadeShared {
  float q[256], keep[256], write[256], v[256];
  float sums[DM_WAVES][256];
  float part[DM_WAVES];
};
union FadeOrChoice {
  FadeShared fade;
  float choice[2][ROUTER_MAX];
};

template <int NR>
__global__ __launch_bounds__(DM_THREADS) void decode_hgrn2_kernel(FadeStep a, const int* __restrict__ spans, int rows) {
  __shared__ __align__(16) FadeOrChoice lds;
  FadeShared& sh = lds.fade;
  const int slot = blockIdx.y, head = blockIdx.x, t = threadIdx.x;
  const Span s = span_of(spans, slot, rows);
  if (a.choice.z != nullptr && blockIdx.x == gridDim.x - 1) {   // (whether the slot has a row or not, as the router by itself)
    choose_row(a.choice, lds.choice[0], lds.choice[1]);
    return;
  }
  if (s.rows == 0) return;
  const bf16_t* row = a.x + (size_t)s.row0 * a.stride;
  bf16_t* to = a.out + (size_t)s.row0 * a.out_stride;
  if (head >= a.heads) {
    const int c = (head - a.heads) * DM_THREADS + t;
    if (c < a.cols)
      to[a.gated_at + c] = f32_to_bf16(gated_value(a.kind, a.limit, bf16_to_f32(row[a.gate_at + c]), bf16_to_f32(row[a.gate_at + a.cols + c])));
    return;
  }
  const int lane = t & 63, wave = t >> 6, dim = a.dim, vdim = a.vdim;
  const StateTiles tile(vdim);
  float* sp = a.state + ((size_t)slot * a.heads + head) * dim * vdim;
  float4 S[NR];
#pragma unroll
  for (int n = 0; n < NR; ++n) {
    const int i = tile.row + n * tile.stride;
    S[n] = (s.start > 0 && i < dim) ? *reinterpret_cast<const float4*>(sp + (size_t)i * vdim + tile.col) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  const float gain = t < vdim ? bf16_to_f32(a.norm[t]) : 0.f;
  if (t < dim) {
    const int c = head * dim + t;
    const Fade f = fade_of<bf16_t>(bf16_to_f32(row[a.heads * dim + c]), bf16_to_f32(a.g.bias[c]), bf16_to_f32(a.g.lower[c]));
    sh.q[t] = silu_read<bf16_t>(bf16_to_f32(row[c]));
    sh.keep[t] = f.keep;
    sh.write[t] = f.write;
  } else if (t >= 512 && t < 512 + vdim) {
    sh.v[t - 512] = bf16_to_f32(row[2 * a.heads * dim + head * vdim + t - 512]);
  }
  __syncthreads();
  const float4 v = *reinterpret_cast<const float4*>(&sh.v[tile.col]);
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
  for (int n = 0; n < NR; ++n) {
    const int i = tile.row + n * tile.stride;
    if (i < dim) {
      const float q = sh.q[i], k = sh.write[i], w = sh.keep[i];
      S[n].x = fmaf(w, S[n].x, k * v.x); S[n].y = fmaf(w, S[n].y, k * v.y);
      S[n].z = fmaf(w, S[n].z, k * v.z); S[n].w = fmaf(w, S[n].w, k * v.w);
      o.x = fmaf(q, S[n].x, o.x); o.y = fmaf(q, S[n].y, o.y); o.z = fmaf(q, S[n].z, o.z); o.w = fmaf(q, S[n].w, o.w);
      *reinterpret_cast<float4*>(sp + (size_t)i * vdim + tile.col) = S[n];
    }
  }
  tile.fold(o);
  if (lane < tile.quads) *reinterpret_cast<float4*>(&sh.sums[wave][tile.col]) = o;
  __syncthreads();
  float sum = 0.f;
  if (t < vdim) {
#pragma unroll
    for (int w = 0; w < DM_WAVES; ++w) sum += sh.sums[w][t];
  }
  const float inv = 1.0f / sqrtf(dm_block_sum(sum * sum, sh.part) / (float)vdim + a.eps);
  if (t < vdim) to[a.out_at + head * vdim + t] = f32_to_bf16(sum * inv * gain);
}

static bool whole_columns(int n) { return n >= 16 && n <= 256 && (n & (n - 1)) == 0; }
static int rows_a_thread(int dim, int wide) {   // the power of two that covers dim over the block's rows
  const int stride = DM_THREADS / (wide / 4);
  int nr = 1;
  while (nr * stride < dim) nr *= 2;
  return nr;
}

}  // namespace iron

using namespace iron;

extern "C" int iron_decode_parallel_bf16(const uint16_t* r, const uint16_t* k, const uint16_t* v, const uint16_t* gate,
                                         const uint16_t* z, const uint16_t* w2, const uint16_t* w0, const uint16_t* u,
                                         const uint16_t* norm, float* memory, int mix_heads, int mix_dim, int rank, float eps,
                                         float mix_scale, int mix_at, const uint16_t* x, uint16_t* keys, uint16_t* values,
                                         const float* bias, int stride, int heads, int kv_heads, int dim, int vdim, int window,
                                         int ring, float scale, float out_scale, int win_at, const int* spans, uint16_t* out,
                                         int slots, int rows, int out_stride, void* stream) {
  IRON_REQUIRE(r && k && v && gate && z && w2 && w0 && u && norm && memory && x && keys && values && bias && spans && out,
               "decode_parallel: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0, "decode_parallel: spans must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0, "decode_parallel: slots (%d) and rows (%d) must be positive", slots, rows);
  IRON_REQUIRE(mix_heads > 0 && whole_columns(mix_dim) && rank > 0 && rank <= 512,
               "decode_parallel: mix_dim (%d) is a power of two from 16 to 256, rank (%d) from 1 to 512", mix_dim, rank);
  IRON_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "decode_parallel: kv_heads (%d) must divide heads (%d)", kv_heads, heads);
  IRON_REQUIRE(dim > 0 && dim <= 256 && dim % 8 == 0 && vdim > 0 && vdim <= 256 && vdim % 8 == 0 && stride % 8 == 0,
               "decode_parallel: dim (%d), vdim (%d) up to 256 and the row (%d) are multiples of 8", dim, vdim, stride);
  IRON_REQUIRE(stride >= heads * dim + kv_heads * (dim + vdim), "decode_parallel: a row of %d holds no q, k and v", stride);
  IRON_REQUIRE(window > 0 && ring >= window, "decode_parallel: a window (%d) of at least 1 within the ring (%d)", window, ring);
  IRON_REQUIRE(mix_at >= 0 && mix_at + mix_heads * mix_dim <= out_stride && win_at >= 0 && win_at + heads * vdim <= out_stride,
               "decode_parallel: the heads' columns do not fit an output row of %d", out_stride);
  IRON_REQUIRE((((uintptr_t)x | (uintptr_t)keys | (uintptr_t)values | (uintptr_t)memory) & 15) == 0,
               "decode_parallel: operands must be 16-byte aligned");
  const TimeMixStep mix{r, k, v, gate, z, w2, w0, u, norm, memory, out, mix_heads, mix_dim, rank, out_stride, mix_at, eps, mix_scale};
  const WindowStep win{x, keys, values, bias, out, stride, heads, kv_heads, dim, vdim, window, ring, out_stride, win_at, scale, out_scale};
  const dim3 grid(heads + mix_heads, slots);
#define IRON_PARALLEL(NR)                                                                                                 \
  {                                                                                                                       \
    hipLaunchKernelGGL((decode_parallel_kernel<NR>), grid, dim3(DM_THREADS), 0, (hipStream_t)stream, mix, win, spans, rows); \
    break;                                                                                                                \
  }
  switch (rows_a_thread(mix_dim, mix_dim)) {
    case 1: IRON_PARALLEL(1)
    case 2: IRON_PARALLEL(2)
    case 4: IRON_PARALLEL(4)
    case 8: IRON_PARALLEL(8)
    default: IRON_PARALLEL(16)
  }
#undef IRON_PARALLEL
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_decode_delta_bf16(const uint16_t* x, const uint16_t* taps_w, const uint16_t* a_log, const uint16_t* dt_bias,
                                      const uint16_t* norm, uint16_t* inputs, float* state, const int* spans, uint16_t* out,
                                      int slots, int rows, int stride, int heads, int kv_heads, int dim, int vdim, int taps,
                                      int gate_at, int b_at, int a_at, float eps, void* stream) {
  IRON_REQUIRE(x && taps_w && a_log && dt_bias && norm && inputs && state && spans && out, "decode_delta: null operand");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0 && ((uintptr_t)state & 15) == 0, "decode_delta: spans and state must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0, "decode_delta: slots (%d) and rows (%d) must be positive", slots, rows);
  IRON_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "decode_delta: kv_heads (%d) must divide heads (%d)", kv_heads, heads);
  IRON_REQUIRE(dim > 0 && dim <= 256 && whole_columns(vdim), "decode_delta: dim (%d) up to 256, vdim (%d) a power of two from 16 to 256", dim, vdim);
  IRON_REQUIRE(taps >= 1 && taps <= 17, "decode_delta: taps (%d) from 1 to 17", taps);
  const int channels = 2 * kv_heads * dim + heads * vdim;
  IRON_REQUIRE(gate_at >= channels && gate_at + heads * vdim <= stride && b_at >= channels && b_at + heads <= stride &&
                   a_at >= channels && a_at + heads <= stride,
               "decode_delta: gate (%d), b (%d) and a (%d) lie behind q, k, v (%d) in a row of %d", gate_at, b_at, a_at, channels, stride);
  const DeltaStep a{x, taps_w, a_log, dt_bias, norm, inputs, state, out, stride, heads, kv_heads, dim, vdim, taps, gate_at, b_at, a_at, eps};
  const dim3 grid(heads, slots);
#define IRON_DELTA_STEP(NR)                                                                                          \
  {                                                                                                                  \
    hipLaunchKernelGGL((decode_delta_kernel<NR>), grid, dim3(DM_THREADS), 0, (hipStream_t)stream, a, spans, rows);   \
    break;                                                                                                           \
  }
  switch (rows_a_thread(dim, vdim)) {
    case 1: IRON_DELTA_STEP(1)
    case 2: IRON_DELTA_STEP(2)
    case 4: IRON_DELTA_STEP(4)
    case 8: IRON_DELTA_STEP(8)
    default: IRON_DELTA_STEP(16)
  }
#undef IRON_DELTA_STEP
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_decode_hgrn2_bf16(const uint16_t* x, const uint16_t* f_bias, const uint16_t* lower, const uint16_t* norm, float* state,
                                      const int* spans, uint16_t* out, int slots, int rows, int stride, int heads, int dim, int vdim, int out_stride,
                                      int out_at, float eps, int cols, int gate_at, int gated_at, int kind, float limit, const float* z,
                                      const uint16_t* correction, int logits, int top, int* ids, float* shares, void* stream) {
  IRON_REQUIRE(x && f_bias && lower && norm && state && spans && out, "decode_hgrn2: null operand");
  IRON_ROUTER_CHOICE_REQUIRE("decode_hgrn2");
  IRON_REQUIRE(((uintptr_t)spans & 15) == 0 && ((uintptr_t)state & 15) == 0, "decode_hgrn2: spans and state must be 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0, "decode_hgrn2: slots (%d) and rows (%d) must be positive", slots, rows);
  IRON_REQUIRE(heads > 0 && dim > 0 && dim <= 256 && whole_columns(vdim), "decode_hgrn2: dim (%d) up to 256, vdim (%d) a power of two from 16 to 256", dim, vdim);
  IRON_REQUIRE(stride >= heads * (2 * dim + vdim) && out_at >= 0 && out_at + heads * vdim <= out_stride,
               "decode_hgrn2: rows of %d and %d for %d heads of %d and %d", stride, out_stride, heads, dim, vdim);
  IRON_REQUIRE(cols >= 0 && (cols == 0 || (gate_at >= 0 && gate_at + 2 * cols <= stride && gated_at >= 0 && gated_at + cols <= out_stride)),
               "decode_hgrn2: twice %d gated columns from %d, into those from %d", cols, gate_at, gated_at);
  IRON_REQUIRE(kind >= 0 && kind <= 3, "decode_hgrn2: kind (%d) is 0 to 3", kind);
  const FadeStep a{x, FadeGates{f_bias, lower}, norm, state, out, stride, heads, dim, vdim, out_stride, out_at, eps, cols, gate_at, gated_at, kind, limit,
                   RouterChoice{z, correction, logits, top, ids, shares}};
  const dim3 grid(heads + (cols + DM_THREADS - 1) / DM_THREADS + (z != nullptr), slots);
#define IRON_FADE_STEP(NR)                                                                                           \
  {                                                                                                                  \
    hipLaunchKernelGGL((decode_hgrn2_kernel<NR>), grid, dim3(DM_THREADS), 0, (hipStream_t)stream, a, spans, rows);   \
    break;                                                                                                           \
  }
  switch (rows_a_thread(dim, vdim)) {
    case 1: IRON_FADE_STEP(1)
    case 2: IRON_FADE_STEP(2)
    case 4: IRON_FADE_STEP(4)
    case 8: IRON_FADE_STEP(8)
    default: IRON_FADE_STEP(16)
  }
#undef IRON_FADE_STEP
  IRON_LAUNCH_CHECK();
}
