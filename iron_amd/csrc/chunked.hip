// Time mixing, the delta rule, the matrix memory and HGRN2 over a prompt's portion, sixteen tokens at a time on float32 MFMAs.
//
// Within a chunk of 16 tokens everything that does not touch the state depends on the chunk alone, so a
// first launch computes it for all chunks at once: what earlier tokens of the chunk leave of themselves
// in later ones' outputs (a 16 x 16 matrix), and for the delta rule the inverse that turns the chunk's
// 16 coupled updates into one product.  A second launch walks the chunks in order: a head's state, split
// by columns over blocks and by rows over a block's four waves, is a few products a chunk.
//
// The 16x16x4 MFMA leaves lane (quad, l16) rows quad * 4 .. + 3 of column l16.  Taken as the B operand of
// a following product, register r of such a result is its rows {r, 4 + r, 8 + r, 12 + r}: four products,
// one a register, with the A operand's columns in the same order, need no exchange between lanes.  "Frag"
// below is that A operand: lane (quad, l16) holds [l16][quad * 4 + r] in its r-th float.
//
// Decays enter as exponentials of differences of running sums of logarithms, later minus earlier: never
// above 1, however strong the decay.
#include "../../include/iron_hip.h"
#include "hgrn2.h"
#include "matrix_memory.h"
#include "rows.h"

namespace iron {

constexpr int CHUNK = 16;

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ f32x4 product16(const f32x4& a, const f32x4& b, f32x4 c) {
#pragma unroll
  for (int r = 0; r < 4; ++r) c = mfma4(a[r], b[r], c);
  return c;
}
// exp of a number that is not above 0: the hardware's where rows are bf16, the library's in 32 bits.
template <typename T>
__device__ __forceinline__ float decay_exp(float x) {
  if constexpr (sizeof(T) == 2) return __expf(x);
  else return expf(x);
}
__device__ __forceinline__ float widened(bf16_t v) { return bf16_to_f32(v); }
__device__ __forceinline__ float widened(float v) { return v; }
__device__ __forceinline__ float pick4(const f32x4& v, int i) { return i < 2 ? (i == 0 ? v[0] : v[1]) : (i == 2 ? v[2] : v[3]); }

// ---------------------------------------------------------------- time mixing
// Workspace of a chunk and head: r exp(L before it) frags, k exp(L_end - L) frags transposed (both 16 a
// row tile), exp(L_end), and the 16 x 16 matrix's frag.
__host__ __device__ inline int mix_words(int tiles) { return tiles * (2 * 256 + 16) + 256; }

template <typename T>
__global__ __launch_bounds__(256) void time_mix_chunks_kernel(const T* __restrict__ r, const T* __restrict__ k,
                                                              const float* __restrict__ log_decay, const bf16_t* __restrict__ u,
                                                              const int* __restrict__ spans, float* __restrict__ work, int rows,
                                                              int slots, int heads, int dim) {
  extern __shared__ __align__(16) float lds[];
  const int head = blockIdx.y, slot = blockIdx.z, base = blockIdx.x * CHUNK;
  const Span s = span_of(spans, slot, rows);
  if (base >= s.rows) return;
  const int n = min(CHUNK, s.rows - base), tiles = (dim + 15) / 16, wide = tiles * 16, pitch = wide + 4, t = threadIdx.x;
  float* rs = lds;                       // [16][pitch]
  float* ks = rs + CHUNK * pitch;
  float* ls = ks + CHUNK * pitch;        // [17][pitch]: row i + 1 the sum up to token i
  float* am = ls + (CHUNK + 1) * pitch;  // [16][17]
  const size_t width = (size_t)heads * dim, at = (size_t)(s.row0 + base) * width + head * dim;
  for (int e = t; e < CHUNK * wide; e += 256) {
    const int i = e / wide, c = e - i * wide;
    const bool in = i < n && c < dim;
    rs[i * pitch + c] = in ? load_one(r + at + i * width + c) : 0.f;
    ks[i * pitch + c] = in ? load_one(k + at + i * width + c) : 0.f;
    ls[(i + 1) * pitch + c] = in ? log_decay[at + i * width + c] : 0.f;
  }
  for (int e = t; e < CHUNK * 17; e += 256) am[e] = 0.f;
  __syncthreads();
  for (int c = t; c < wide; c += 256) {
    float v[CHUNK];
#pragma unroll
    for (int i = 0; i < CHUNK; ++i) v[i] = ls[(i + 1) * pitch + c];
    float sum = 0.f;
    ls[c] = 0.f;
#pragma unroll
    for (int i = 0; i < CHUNK; ++i) {
      sum += v[i];
      ls[(i + 1) * pitch + c] = sum;
    }
  }
  __syncthreads();
  float* out = work + ((size_t)(first_chunk(spans, slots, slot, rows, CHUNK) + blockIdx.x) * heads + head) * mix_words(tiles);
  for (int e = t; e < tiles * 64; e += 256) {
    const int tile = e >> 6, lane = e & 63, l16 = lane & 15, quad = lane >> 4;
    float4 a, b;
    {
      const int c = tile * 16 + quad * 4;
      const float4 rv = *reinterpret_cast<const float4*>(rs + l16 * pitch + c), lv = *reinterpret_cast<const float4*>(ls + l16 * pitch + c);
      a = make_float4(rv.x * decay_exp<T>(lv.x), rv.y * decay_exp<T>(lv.y), rv.z * decay_exp<T>(lv.z), rv.w * decay_exp<T>(lv.w));
    }
    {
      const int c = tile * 16 + l16;
      const float end = ls[CHUNK * pitch + c];
      float f[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) f[j] = ks[(quad * 4 + j) * pitch + c] * decay_exp<T>(end - ls[(quad * 4 + j + 1) * pitch + c]);
      b = make_float4(f[0], f[1], f[2], f[3]);
    }
    reinterpret_cast<float4*>(out)[e] = a;
    reinterpret_cast<float4*>(out + tiles * 256)[e] = b;
  }
  for (int c = t; c < wide; c += 256) out[tiles * 512 + c] = decay_exp<T>(ls[CHUNK * pitch + c]);
  // Pairs (i, j), j < i: 64 at a time, four threads a pair.
  for (int p = t >> 2; p < CHUNK * (CHUNK - 1) / 2; p += 64) {
    int i = 1, j = p;
    while (j >= i) j -= i++;
    float sum = 0.f;
    for (int c = (t & 3) * 4; c < wide; c += 16) {
      const float4 rv = *reinterpret_cast<const float4*>(rs + i * pitch + c), kv = *reinterpret_cast<const float4*>(ks + j * pitch + c);
      const float4 a = *reinterpret_cast<const float4*>(ls + i * pitch + c), b = *reinterpret_cast<const float4*>(ls + (j + 1) * pitch + c);
      sum = fmaf(rv.x * kv.x, decay_exp<T>(a.x - b.x), sum);
      sum = fmaf(rv.y * kv.y, decay_exp<T>(a.y - b.y), sum);
      sum = fmaf(rv.z * kv.z, decay_exp<T>(a.z - b.z), sum);
      sum = fmaf(rv.w * kv.w, decay_exp<T>(a.w - b.w), sum);
    }
    sum += IRON_DPP(0.f, sum, 0xB1, 0xF);
    sum += IRON_DPP(0.f, sum, 0x4E, 0xF);
    if ((t & 3) == 0) am[i * 17 + j] = sum;
  }
  {   // the current token's bonus
    const int i = t >> 4;
    float sum = 0.f;
    for (int c = t & 15; c < dim; c += 16) sum = fmaf(rs[i * pitch + c] * bf16_to_f32(u[head * dim + c]), ks[i * pitch + c], sum);
    sum = group16_sum(sum);
    if ((t & 15) == 0) am[i * 17 + i] = sum;
  }
  __syncthreads();
  out[tiles * 528 + t] = am[((t >> 2) & 15) * 17 + (t >> 6) * 4 + (t & 3)];
}

// The walk asks for a chunk's operands DEPTH chunks ahead (a chunk's products take a fraction of a trip to
// memory), into registers of their own: every chunk of the unrolled loop issues the same loads, rows and
// tiles past the end clamped where they are read and zeroed where they are used, so that no branch stands
// between the loads in flight.
template <typename T, int NT>
struct MixOperands {
  float4 r[NT], k[NT], w[NT];
  float a;
  T v[4];   // as loaded: widened where it is used, not where it would be waited for
};

// COUNTED: the state has a column behind v's last, of a v that is 1; its reading goes behind all heads' own.
struct WalkShape {
  int rows, slots, heads, dim, vdim;
  int v_stride, o_stride;                // lengths of the rows v lies in (vdim columns a head) and of the readings' rows
};

template <typename T, int NT, int DEPTH, bool COUNTED = false>
__global__ __launch_bounds__(256) void time_mix_walk_kernel(const T* __restrict__ v, float* __restrict__ state,
                                                            const int* __restrict__ spans, const float* __restrict__ work,
                                                            float* __restrict__ o, WalkShape a) {
  __shared__ float4 os[2][4][64];
  const int head = blockIdx.x, slot = blockIdx.z;   // heads fastest: a head's column blocks share an XCD's L2
  const int rows = a.rows, slots = a.slots, heads = a.heads, dim = a.dim, vdim = a.vdim, cols = COUNTED ? vdim + 1 : vdim;
  const Span s = span_of(spans, slot, rows);
  if (s.rows == 0) return;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, l16 = lane & 15, quad = lane >> 4;
  const int tiles = (dim + 15) / 16, words = mix_words(tiles), col = blockIdx.y * 16 + l16;
  const int count = (s.rows + CHUNK - 1) / CHUNK;
  float* sp = state + ((size_t)slot * heads + head) * dim * cols;
  const float* at = work + ((size_t)first_chunk(spans, slots, slot, rows, CHUNK) * heads + head) * words;
  // The span's rows by 32-bit offsets; a store to an offset outside them is dropped.
  constexpr int E = (int)sizeof(T);
  const __amdgpu_buffer_rsrc_t vb = bounded_bytes(v + (size_t)s.row0 * a.v_stride + head * vdim, (int)(((size_t)(s.rows - 1) * a.v_stride + vdim) * E));
  const __amdgpu_buffer_rsrc_t ob = bounded_bytes(o + (size_t)s.row0 * a.o_stride, (int)((size_t)s.rows * a.o_stride * 4));
  const int v_at = quad * 4 * a.v_stride * E + min(col, vdim - 1) * E, row_v = a.v_stride * E;
  const int o_col = COUNTED && col == vdim ? heads * vdim + head : head * vdim + col;
  const int o_at = col < cols ? ((quad * 4 + wave) * a.o_stride + o_col) * 4 : 0x7fffffff;
  f32x4 S[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int i = (wave * NT + n) * 16 + quad * 4 + j;
      S[n][j] = (s.start > 0 && i < dim && col < cols) ? sp[(size_t)i * cols + col] : 0.f;
    }
  MixOperands<T, NT> ops[DEPTH];
  auto fetch = [&](MixOperands<T, NT>& x, int c) {
    c = min(c, count - 1);
    const float* w = at + (size_t)c * heads * words;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const int tile = min(wave * NT + n, tiles - 1);
      x.r[n] = reinterpret_cast<const float4*>(w)[tile * 64 + lane];
      x.k[n] = reinterpret_cast<const float4*>(w + tiles * 256)[tile * 64 + lane];
      x.w[n] = *reinterpret_cast<const float4*>(w + tiles * 512 + tile * 16 + quad * 4);
    }
    x.a = w[tiles * 528 + lane * 4 + wave];
#pragma unroll
    for (int j = 0; j < 4; ++j) {   // zero past the span's last row
      if constexpr (sizeof(T) == 2) x.v[j] = (T)__builtin_amdgcn_raw_buffer_load_b16(vb, v_at + j * row_v, c * CHUNK * row_v, 0);
      else x.v[j] = __builtin_bit_cast(float, __builtin_amdgcn_raw_buffer_load_b32(vb, v_at + j * row_v, c * CHUNK * row_v, 0));
    }
  };
  // A chunk's sums of the four waves' parts: asked for ahead of the next chunk's products, and used behind them.
  float part[4];
  auto ask = [&](int c) {   // wave w finishes rows quad * 4 + w
#pragma unroll
    for (int w = 0; w < 4; ++w) part[w] = reinterpret_cast<const float*>(&os[c & 1][w][lane])[wave];
  };
  auto finish = [&](int c) {
    const float sum = part[0] + part[1] + part[2] + part[3];
    __builtin_amdgcn_raw_buffer_store_b32(__builtin_bit_cast(unsigned, sum), ob, o_at, c * CHUNK * a.o_stride * 4, 0);
  };
  auto run = [&](const MixOperands<T, NT>& x, int c) {
    if (c > 0) ask(c - 1);
    f32x4 vf, next[NT], out[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int j = 0; j < 4; ++j) vf[j] = COUNTED && col == vdim ? 1.f : widened(x.v[j]);
    float r[NT][4], k[NT][4];
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const bool in = wave * NT + n < tiles;   // S of a tile past the last stays 0
      r[n][0] = x.r[n].x; r[n][1] = x.r[n].y; r[n][2] = x.r[n].z; r[n][3] = x.r[n].w;
      k[n][0] = in ? x.k[n].x : 0.f; k[n][1] = in ? x.k[n].y : 0.f; k[n][2] = in ? x.k[n].z : 0.f; k[n][3] = in ? x.k[n].w : 0.f;
      next[n] = S[n] * f32x4{x.w[n].x, x.w[n].y, x.w[n].z, x.w[n].w};
    }
    out[1] = mfma4(x.a, pick4(vf, wave), out[1]);
    // Chains side by side: a product waits for the one before it in its own chain, not for its neighbours.
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        out[n & 1] = mfma4(r[n][j], S[n][j], out[n & 1]);
        next[n] = mfma4(k[n][j], vf[j], next[n]);
      }
#pragma unroll
    for (int n = 0; n < NT; ++n) S[n] = next[n];
    const f32x4 both = out[0] + out[1];
    if (c > 0) finish(c - 1);
    os[c & 1][wave][lane] = make_float4(both[0], both[1], both[2], both[3]);
    block_barrier_lds();   // (the other buffer's readers are behind it, too)
  };
#pragma unroll
  for (int d = 0; d < DEPTH; ++d) {
    fetch(ops[d], d);
    __builtin_amdgcn_sched_barrier(0);   // the loads go out, and are counted down, in the chunks' order
  }
  int c = 0;
  for (; c + DEPTH <= count; c += DEPTH) {
#pragma unroll
    for (int d = 0; d < DEPTH; ++d) {
      run(ops[d], c + d);
      fetch(ops[d], c + d + DEPTH);
      __builtin_amdgcn_sched_barrier(0);
    }
  }
#pragma unroll
  for (int d = 0; d < DEPTH; ++d)
    if (c + d < count) run(ops[d], c + d);
  ask(count - 1);
  finish(count - 1);
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int i = (wave * NT + n) * 16 + quad * 4 + j;
      if (i < dim && col < cols) sp[(size_t)i * cols + col] = S[n][j];
    }
}

// ---------------------------------------------------------------------- HGRN2
// The same walk, read behind the write: queries enter as q 2^L, L the running sum of the gates' logarithms with the token's own in it,
// keys are what the gates leave, and the 16 x 16 matrix has its diagonal, undecayed.
template <typename T>
__device__ __forceinline__ float decay_exp2(float x) {
  if constexpr (sizeof(T) == 2) return __builtin_amdgcn_exp2f(x);
  else return exp2f(x);
}

// VEC: rows and gains of whole 16-byte pieces, eight columns of a token a thread at a time; else one.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void hgrn2_chunks_kernel(const T* __restrict__ x, FadeGates g, const int* __restrict__ spans,
                                                           float* __restrict__ work, int rows, int slots, int stride, int heads, int dim) {
  extern __shared__ __align__(16) float lds[];
  const int head = blockIdx.y, slot = blockIdx.z, base = blockIdx.x * CHUNK;
  const Span s = span_of(spans, slot, rows);
  if (base >= s.rows) return;
  const int n = min(CHUNK, s.rows - base), tiles = (dim + 15) / 16, wide = tiles * 16, pitch = wide + 4, t = threadIdx.x;
  float* qs = lds;                       // [16][pitch]
  float* ks = qs + CHUNK * pitch;
  float* ls = ks + CHUNK * pitch;        // the sum up to and with token i
  float* am = ls + CHUNK * pitch;        // [16][17]
  const T* row = x + (size_t)(s.row0 + base) * stride + head * dim;
  const int pieces = wide / VEC;
  for (int e = t; e < CHUNK * pieces; e += 256) {
    const int i = e / pieces, c = (e - i * pieces) * VEC;
    float q[VEC], z[VEC], bias[VEC], lower[VEC];
    const bool in = i < n && c < dim;
    if (in) {
      load_vec<VEC>(row + (size_t)i * stride + c, q);
      load_vec<VEC>(row + (size_t)i * stride + heads * dim + c, z);
      load_vec<VEC>(g.bias + head * dim + c, bias);
      load_vec<VEC>(g.lower + head * dim + c, lower);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      if (in) {
        const Fade f = fade_of<T>(z[j], bias[j], lower[j]);
        q[j] = silu_read<T>(q[j]);
        z[j] = f.write;
        bias[j] = log2_fade<T>(f);
      } else {   // past the last token: nothing read or written, nothing fades
        q[j] = z[j] = bias[j] = 0.f;
      }
    }
    store_vec<VEC>(qs + i * pitch + c, q);
    store_vec<VEC>(ks + i * pitch + c, z);
    store_vec<VEC>(ls + i * pitch + c, bias);
  }
  for (int e = t; e < CHUNK * 17; e += 256) am[e] = 0.f;
  __syncthreads();
  for (int c = t; c < wide; c += 256) {
    float v[CHUNK];
#pragma unroll
    for (int i = 0; i < CHUNK; ++i) v[i] = ls[i * pitch + c];
#pragma unroll
    for (int i = 1; i < CHUNK; ++i) {
      v[i] += v[i - 1];
      ls[i * pitch + c] = v[i];
    }
  }
  __syncthreads();
  float* out = work + ((size_t)(first_chunk(spans, slots, slot, rows, CHUNK) + blockIdx.x) * heads + head) * mix_words(tiles);
  const float* end = ls + (CHUNK - 1) * pitch;
  for (int e = t; e < tiles * 64; e += 256) {
    const int tile = e >> 6, lane = e & 63, l16 = lane & 15, quad = lane >> 4, c = tile * 16 + l16;
    const float4 q = *reinterpret_cast<const float4*>(qs + l16 * pitch + tile * 16 + quad * 4), l = *reinterpret_cast<const float4*>(ls + l16 * pitch + tile * 16 + quad * 4);
    float f[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) f[j] = ks[(quad * 4 + j) * pitch + c] * decay_exp2<T>(end[c] - ls[(quad * 4 + j) * pitch + c]);
    reinterpret_cast<float4*>(out)[e] = make_float4(q.x * decay_exp2<T>(l.x), q.y * decay_exp2<T>(l.y), q.z * decay_exp2<T>(l.z), q.w * decay_exp2<T>(l.w));
    reinterpret_cast<float4*>(out + tiles * 256)[e] = make_float4(f[0], f[1], f[2], f[3]);
  }
  for (int c = t; c < wide; c += 256) out[tiles * 512 + c] = decay_exp2<T>(end[c]);
  // Pairs (i, j), j <= i: 64 at a time, four threads a pair.
  for (int p = t >> 2; p < CHUNK * (CHUNK + 1) / 2; p += 64) {
    int i = 0, j = p;
    while (j > i) j -= ++i;
    float sum = 0.f;
#pragma unroll 2
    for (int c = (t & 3) * 4; c < wide; c += 16) {
      const float4 q = *reinterpret_cast<const float4*>(qs + i * pitch + c), k = *reinterpret_cast<const float4*>(ks + j * pitch + c);
      const float4 a = *reinterpret_cast<const float4*>(ls + i * pitch + c), b = *reinterpret_cast<const float4*>(ls + j * pitch + c);
      sum = fmaf(q.x * k.x, decay_exp2<T>(a.x - b.x), sum);
      sum = fmaf(q.y * k.y, decay_exp2<T>(a.y - b.y), sum);
      sum = fmaf(q.z * k.z, decay_exp2<T>(a.z - b.z), sum);
      sum = fmaf(q.w * k.w, decay_exp2<T>(a.w - b.w), sum);
    }
    sum += IRON_DPP(0.f, sum, 0xB1, 0xF);
    sum += IRON_DPP(0.f, sum, 0x4E, 0xF);
    if ((t & 3) == 0) am[i * 17 + j] = sum;
  }
  __syncthreads();
  out[tiles * 528 + t] = am[((t >> 2) & 15) * 17 + (t >> 6) * 4 + (t & 3)];
}

// ----------------------------------------------------------- the matrix memory
// The same walk: with F the chunk's running sum of log forget gates and m0 the largest exponent ahead of it, m_t =
// max(F_t + m0, max over s <= t of F_t - F_s + i_s); queries enter as q exp(F_t + m0 - m_t), keys leave as k exp(F_end - F_s +
// i_s - m_end), the state shrinks by exp(F_end + m0 - m_end), and the 16 x 16 matrix is (q_t . k_s) exp(F_t - F_s + i_s - m_t).
// The m0 of all chunks come first, by a launch that composes the chunks' (F_end, max over s of F_end - F_s + i_s).
constexpr int TOPS_THREADS = 1024;

template <typename T>
__device__ __forceinline__ void log_gates(const T* __restrict__ row, const MemoryGates& g, int head, float& i, float& f) {
  i = capped(load_one(row + g.i_at + head) + bf16_to_f32(g.i_bias[head]), g.cap);
  f = log_sigmoid(capped(load_one(row + g.f_at + head) + bf16_to_f32(g.f_bias[head]), g.cap));
}

template <typename T>
__global__ __launch_bounds__(TOPS_THREADS) void memory_tops_kernel(const T* __restrict__ x, MemoryGates g, float* __restrict__ tops,
                                                                   const int* __restrict__ spans, float* __restrict__ starts, int rows,
                                                                   int slots, int stride, int heads) {
  constexpr int AT_ONCE = TOPS_THREADS / CHUNK;
  __shared__ float sums[2][AT_ONCE], most[2][AT_ONCE];
  const int head = blockIdx.x, slot = blockIdx.y, t = threadIdx.x, l16 = t & 15;
  const Span s = span_of(spans, slot, rows);
  if (s.rows == 0) return;
  float* mp = tops + (size_t)slot * 2 * heads + head;
  float m = s.start > 0 ? mp[((s.start - 1) & 1) * heads] : 0.f;
  const int first = first_chunk(spans, slots, slot, rows, CHUNK), count = (s.rows + CHUNK - 1) / CHUNK;
  for (int base = 0, turn = 0; base < s.rows; base += TOPS_THREADS, turn ^= 1) {
    float i = -INFINITY, f = 0.f;
    if (base + t < s.rows) log_gates(x + (size_t)(s.row0 + base + t) * stride, g, head, i, f);
#pragma unroll
    for (int d = 1; d < CHUNK; d <<= 1) {
      const float before = __shfl_up(f, d, CHUNK);
      if (l16 >= d) f += before;
    }
    const float end = __shfl(f, CHUNK - 1, CHUNK);
    float top = end - f + i;
#pragma unroll
    for (int d = 1; d < CHUNK; d <<= 1) top = fmaxf(top, __shfl_xor(top, d, CHUNK));
    if (l16 == 0) {
      sums[turn][t / CHUNK] = end;
      most[turn][t / CHUNK] = top;
    }
    __syncthreads();   // (two sets: the next turn's writers do not meet this one's readers)
    const int n = min(AT_ONCE, count - base / CHUNK);
#pragma unroll 8
    for (int c = 0; c < n; ++c) {
      if (t == 0) starts[(size_t)(first + base / CHUNK + c) * heads + head] = m;
      m = fmaxf(sums[turn][c] + m, most[turn][c]);
    }
  }
  if (t == 0) mp[((s.start + s.rows - 1) & 1) * heads] = m;
}

template <typename T>
__global__ __launch_bounds__(256) void memory_chunks_kernel(const T* __restrict__ x, MemoryGates g, const int* __restrict__ spans,
                                                            const float* __restrict__ starts, float* __restrict__ work,
                                                            float* __restrict__ o, int rows, int slots, int stride, int heads, int dim,
                                                            int vdim) {
  extern __shared__ __align__(16) float lds[];
  __shared__ float4 qk[4][64];
  __shared__ float gates[2][CHUNK], into[CHUNK], outof[CHUNK], run[CHUNK], top[CHUNK];
  const int head = blockIdx.y, slot = blockIdx.z, base = blockIdx.x * CHUNK;
  const Span s = span_of(spans, slot, rows);
  if (base >= s.rows) return;
  const int n = min(CHUNK, s.rows - base), tiles = (dim + 15) / 16, wide = tiles * 16, pitch = wide + 4, t = threadIdx.x;
  const int lane = t & 63, wave = t >> 6, l16 = lane & 15, quad = lane >> 4, chunk = first_chunk(spans, slots, slot, rows, CHUNK) + blockIdx.x;
  float* qs = lds;                       // [16][pitch]
  float* ks = qs + CHUNK * pitch;
  const T* row = x + (size_t)(s.row0 + base) * stride;
  const float m0 = starts[(size_t)chunk * heads + head], scale = 1.0f / sqrtf((float)dim);
  if (t < CHUNK) {
    float i = -INFINITY, f = 0.f;
    if (t < n) log_gates(row + (size_t)t * stride, g, head, i, f);
    gates[0][t] = i;
    gates[1][t] = f;
  }
  for (int e = t; e < CHUNK * wide; e += 256) {
    const int i = e / wide, c = e - i * wide;
    const bool in = i < n && c < dim;
    const T* at = row + (size_t)i * stride + head * dim + c;
    qs[i * pitch + c] = in ? load_one(at) * scale : 0.f;
    ks[i * pitch + c] = in ? load_one(at + heads * dim) : 0.f;
  }
  __syncthreads();
  if (t == 0) {
    float sum = 0.f, m = m0;
    for (int i = 0; i < CHUNK; ++i) {
      m = fmaxf(gates[1][i] + m, gates[0][i]);   // (of a token past the last: as it was)
      sum += gates[1][i];
      run[i] = sum;
      top[i] = m;
    }
  }
  __syncthreads();
  const float end = run[CHUNK - 1], m_end = top[CHUNK - 1];
  if (t < CHUNK) {
    into[t] = expf(run[t] + m0 - top[t]);
    outof[t] = expf(end - run[t] + gates[0][t] - m_end);   // 0 past the last token
    if (t < n) o[(size_t)(s.row0 + base + t) * (heads * vdim + 2 * heads) + heads * vdim + heads + head] = top[t];
  }
  f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int tile = wave; tile < tiles; tile += 4) {
    const int c = tile * 16 + quad * 4;
    const float4 q = *reinterpret_cast<const float4*>(qs + l16 * pitch + c), k = *reinterpret_cast<const float4*>(ks + l16 * pitch + c);
    acc = product16(f32x4{q.x, q.y, q.z, q.w}, f32x4{k.x, k.y, k.z, k.w}, acc);
  }
  qk[wave][lane] = make_float4(acc[0], acc[1], acc[2], acc[3]);
  __syncthreads();
  float* out = work + ((size_t)chunk * heads + head) * mix_words(tiles);
  for (int e = t; e < tiles * 64; e += 256) {
    const int tile = e >> 6;
    const float by = into[l16];
    const float4 q = *reinterpret_cast<const float4*>(qs + l16 * pitch + tile * 16 + quad * 4);
    float f[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) f[j] = ks[(quad * 4 + j) * pitch + tile * 16 + l16] * outof[quad * 4 + j];
    reinterpret_cast<float4*>(out)[e] = make_float4(q.x * by, q.y * by, q.z * by, q.w * by);
    reinterpret_cast<float4*>(out + tiles * 256)[e] = make_float4(f[0], f[1], f[2], f[3]);
  }
  const float keep = expf(end + m0 - m_end);
  for (int c = t; c < wide; c += 256) out[tiles * 512 + c] = keep;
  {
    const int i = quad * 4 + wave, j = l16;
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) sum += reinterpret_cast<const float*>(&qk[w][lane])[wave];
    // the frag's place of element (i, j): lane (j / 4) * 16 + i, float j % 4
    out[tiles * 528 + ((j >> 2) * 16 + i) * 4 + (j & 3)] = j <= i && j < n ? sum * expf(run[i] - run[j] + gates[0][j] - top[i]) : 0.f;
  }
}

// ------------------------------------------------------------- the delta rule
// With G the running product of decays: u_t = beta_t (v_t - G_t S0^T k_t - sum_{s<t} (G_t/G_s) (k_t.k_s) u_s),
// so U = T (beta V - beta G (K S0)), T the inverse of I + [beta_t (G_t/G_s) (k_t.k_s)]_{s<t};
// o = G (Q S0) + P U, P = [(G_t/G_s) (q_t.k_s)]_{s<=t}; S <- G_end S0 + [(G_end/G_s) k_s] U.
// Workspace of a chunk and head: T's and P's frags, the 16 G, G_end/G and beta.
constexpr int DELTA_WORDS = 256 + 256 + 3 * 16;

template <int NT>
__global__ __launch_bounds__(256) void delta_chunks_kernel(const float* __restrict__ x, const int* __restrict__ spans,
                                                           float* __restrict__ work, int rows, int slots, int heads, int kv_heads,
                                                           int dim, int vdim) {
  __shared__ float4 kk[4][64], qk[4][64];
  __shared__ float m[CHUNK][CHUNK + 1], inv[CHUNK][CHUNK + 1], p[CHUNK][CHUNK + 1], logs[CHUNK], beta[CHUNK];
  const int head = blockIdx.y, slot = blockIdx.z, base = blockIdx.x * CHUNK;
  const Span s = span_of(spans, slot, rows);
  if (base >= s.rows) return;
  const int n = min(CHUNK, s.rows - base), t = threadIdx.x, lane = t & 63, wave = t >> 6, l16 = lane & 15, quad = lane >> 4;
  const int group = head / (heads / kv_heads), qkw = kv_heads * dim, channels = 2 * qkw + heads * vdim, wide = channels + 2 * heads;
  const float* row = x + (size_t)(s.row0 + base) * wide;
  // Both products' operands are a token's row a lane, four of its columns.
  f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f}, b = a;
#pragma unroll
  for (int e = 0; e < NT; ++e) {
    f32x4 q = f32x4{0.f, 0.f, 0.f, 0.f}, k = q;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = (wave * NT + e) * 16 + quad * 4 + j;
      const bool in = l16 < n && c < dim;
      q[j] = in ? row[(size_t)l16 * wide + group * dim + c] : 0.f;
      k[j] = in ? row[(size_t)l16 * wide + qkw + group * dim + c] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      a = mfma4(k[j], k[j], a);
      b = mfma4(q[j], k[j], b);
    }
  }
  kk[wave][lane] = make_float4(a[0], a[1], a[2], a[3]);
  qk[wave][lane] = make_float4(b[0], b[1], b[2], b[3]);
  if (t < CHUNK) {
    float sum = 0.f;
    for (int i = 0; i <= t; ++i) sum += i < n ? row[(size_t)i * wide + channels + head] : 0.f;
    logs[t] = sum;
    beta[t] = t < n ? row[(size_t)t * wide + channels + heads + head] : 0.f;
  }
  __syncthreads();
  {
    const int i = quad * 4 + wave, j = l16;   // this thread's element: a quarter of the result's lanes' registers
    float k2 = 0.f, q2 = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      k2 += reinterpret_cast<const float*>(&kk[w][lane])[wave];
      q2 += reinterpret_cast<const float*>(&qk[w][lane])[wave];
    }
    const float ratio = j <= i ? expf(logs[i] - logs[j]) : 0.f;
    m[i][j] = j < i ? beta[i] * ratio * k2 : 0.f;
    p[i][j] = ratio * q2;
  }
  __syncthreads();
  if (t < CHUNK) {   // a column of the inverse a thread, by substitution
    float c[CHUNK];
#pragma unroll
    for (int i = 0; i < CHUNK; ++i) {
      float sum = i == t ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) sum = fmaf(-m[i][j], c[j], sum);
      c[i] = sum;
      inv[i][t] = sum;
    }
  }
  __syncthreads();
  float* out = work + ((size_t)(first_chunk(spans, slots, slot, rows, CHUNK) + blockIdx.x) * heads + head) * DELTA_WORDS;
  const int fl = t >> 2, fr = t & 3;
  out[t] = inv[fl & 15][(fl >> 4) * 4 + fr];
  out[256 + t] = p[fl & 15][(fl >> 4) * 4 + fr];
  if (t < CHUNK) {
    out[512 + t] = expf(logs[t]);
    out[528 + t] = expf(logs[CHUNK - 1] - logs[t]);
    out[544 + t] = beta[t];
  }
}

template <int NT>
struct DeltaOperands {
  float4 q[NT], k[NT], T, G, left, beta;
  float kt[NT][4], v[4], whole, P;
};

// VEC: q and k rows are whole 16-byte pieces.
template <int NT, int DEPTH, bool VEC>
__global__ __launch_bounds__(256) void delta_walk_kernel(const float* __restrict__ x, float* __restrict__ state,
                                                         const int* __restrict__ spans, const float* __restrict__ work,
                                                         float* __restrict__ o, int rows, int slots, int heads, int kv_heads,
                                                         int dim, int vdim) {
  __shared__ float4 ys[2][4][64], os[2][4][64];
  const int head = blockIdx.x, slot = blockIdx.z;   // heads fastest: a head's column blocks share an XCD's L2
  const Span s = span_of(spans, slot, rows);
  if (s.rows == 0) return;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, l16 = lane & 15, quad = lane >> 4;
  const int group = head / (heads / kv_heads), qkw = kv_heads * dim, channels = 2 * qkw + heads * vdim, wide = channels + 2 * heads;
  const int col = blockIdx.y * 16 + l16, count = (s.rows + CHUNK - 1) / CHUNK;
  float* sp = state + ((size_t)slot * heads + head) * dim * vdim;
  const float* at = work + ((size_t)first_chunk(spans, slots, slot, rows, CHUNK) * heads + head) * DELTA_WORDS;
  const __amdgpu_buffer_rsrc_t xb = bounded_bytes(x + (size_t)s.row0 * wide, (int)((size_t)s.rows * wide * 4));
  const __amdgpu_buffer_rsrc_t ob = bounded_bytes(o + (size_t)s.row0 * heads * vdim, (int)((size_t)s.rows * heads * vdim * 4));
  const int o_at = col < vdim ? ((quad * 4 + wave) * heads * vdim + head * vdim + col) * 4 : 0x7fffffff;
  f32x4 S[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int i = (wave * NT + n) * 16 + quad * 4 + j;
      S[n][j] = (s.start > 0 && i < dim && col < vdim) ? sp[(size_t)i * vdim + col] : 0.f;
    }
  DeltaOperands<NT> ops[DEPTH];
  auto one = [&](int at) { return __builtin_bit_cast(float, __builtin_amdgcn_raw_buffer_load_b32(xb, at, 0, 0)); };
  auto four = [&](int row, int i) {   // columns i .. i + 3 of dim, from byte `row`, held inside them
    if (VEC) return __builtin_bit_cast(float4, __builtin_amdgcn_raw_buffer_load_b128(xb, row + 4 * min(i, dim - 4), 0, 0));
    return make_float4(one(row + 4 * min(i, dim - 1)), one(row + 4 * min(i + 1, dim - 1)), one(row + 4 * min(i + 2, dim - 1)),
                       one(row + 4 * min(i + 3, dim - 1)));
  };
  auto fetch = [&](DeltaOperands<NT>& p, int c) {
    c = min(c, count - 1);
    const float* w = at + (size_t)c * heads * DELTA_WORDS;
    // (past the span's last row that row again: its update is zero, and zero times anything finite stays so)
    const int mine = (min(c * CHUNK + l16, s.rows - 1) * wide + group * dim) * 4;
    int down[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) down[j] = min(c * CHUNK + quad * 4 + j, s.rows - 1) * wide * 4;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const int tile = wave * NT + n;
      p.q[n] = four(mine, tile * 16 + quad * 4);
      p.k[n] = four(mine + 4 * qkw, tile * 16 + quad * 4);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        p.kt[n][j] = one(down[j] + 4 * (qkw + group * dim + min(tile * 16 + l16, dim - 1)));
    }
    p.T = reinterpret_cast<const float4*>(w)[lane];
    p.G = reinterpret_cast<const float4*>(w + 512)[quad];
    p.left = reinterpret_cast<const float4*>(w + 528)[quad];
    p.beta = reinterpret_cast<const float4*>(w + 544)[quad];
    // (by a vector register's index: a scalar load would be waited for with the next LDS read)
    int last = 512 + CHUNK - 1;
    asm volatile("" : "+v"(last));
    p.whole = w[last];
    p.P = w[256 + lane * 4 + wave];
#pragma unroll
    for (int j = 0; j < 4; ++j) p.v[j] = one(down[j] + 4 * (2 * qkw + head * vdim + min(col, vdim - 1)));
  };
  auto finish = [&](int c) {   // chunk c's outputs: wave w adds up and writes rows quad * 4 + w
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) sum += reinterpret_cast<const float*>(&os[c & 1][w][lane])[wave];
    __builtin_amdgcn_raw_buffer_store_b32(__builtin_bit_cast(unsigned, sum), ob, o_at, c * CHUNK * heads * vdim * 4, 0);
  };
  auto run = [&](const DeltaOperands<NT>& p, int c) {
    // A row past the span's last: T's and P's columns for it are zero but for T's diagonal, its beta is zero,
    // so its update is zero; what its q, k and v read as does not matter.
    f32x4 y = f32x4{0.f, 0.f, 0.f, 0.f}, out = y;
#pragma unroll
    for (int n = 0; n < NT; ++n) y = product16(f32x4{p.k[n].x, p.k[n].y, p.k[n].z, p.k[n].w}, S[n], y);   // rows past dim: S is 0
    ys[c & 1][wave][lane] = make_float4(y[0], y[1], y[2], y[3]);
#pragma unroll
    for (int n = 0; n < NT; ++n) out = product16(f32x4{p.q[n].x, p.q[n].y, p.q[n].z, p.q[n].w}, S[n], out);
    const f32x4 G = f32x4{p.G.x, p.G.y, p.G.z, p.G.w}, left = f32x4{p.left.x, p.left.y, p.left.z, p.left.w};
    f32x4 kept[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const float in = (wave * NT + n) * 16 + l16 < dim ? 1.f : 0.f;
      kept[n] = f32x4{p.kt[n][0], p.kt[n][1], p.kt[n][2], p.kt[n][3]} * left * in;
    }
    out *= G;
    block_barrier_lds();
    f32x4 sum = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float4 part = ys[c & 1][w][lane];
      sum += f32x4{part.x, part.y, part.z, part.w};
    }
    const f32x4 X = f32x4{p.beta.x, p.beta.y, p.beta.z, p.beta.w} * (f32x4{p.v[0], p.v[1], p.v[2], p.v[3]} - G * sum);
    const f32x4 U = product16(f32x4{p.T.x, p.T.y, p.T.z, p.T.w}, X, f32x4{0.f, 0.f, 0.f, 0.f});
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      S[n] *= p.whole;
      S[n] = product16(kept[n], U, S[n]);
    }
    out = mfma4(p.P, pick4(U, wave), out);
    os[c & 1][wave][lane] = make_float4(out[0], out[1], out[2], out[3]);
    if (c > 0) finish(c - 1);   // behind this chunk's barrier
  };
#pragma unroll
  for (int d = 0; d < DEPTH; ++d) {
    fetch(ops[d], d);
    __builtin_amdgcn_sched_barrier(0);   // the loads go out, and are counted down, in the chunks' order
  }
  int c = 0;
  for (; c + DEPTH <= count; c += DEPTH) {
#pragma unroll
    for (int d = 0; d < DEPTH; ++d) {
      run(ops[d], c + d);
      fetch(ops[d], c + d + DEPTH);
      __builtin_amdgcn_sched_barrier(0);
    }
  }
#pragma unroll
  for (int d = 0; d < DEPTH; ++d)
    if (c + d < count) run(ops[d], c + d);
  __syncthreads();
  finish(count - 1);
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int i = (wave * NT + n) * 16 + quad * 4 + j;
      if (i < dim && col < vdim) sp[(size_t)i * vdim + col] = S[n][j];
    }
}

}  // namespace iron

using namespace iron;

extern "C" int64_t iron_time_mix_workspace_bytes(int slots, int rows, int heads, int dim) {
  return chunks_of(rows, slots, CHUNK) * heads * (int64_t)mix_words((dim + 15) / 16) * 4;
}
extern "C" int64_t iron_delta_rule_workspace_bytes(int slots, int rows, int heads) {
  return chunks_of(rows, slots, CHUNK) * heads * (int64_t)DELTA_WORDS * 4;
}

#define IRON_CHUNKED_REQUIRE(name)                                                                        \
  IRON_REQUIRE(spans && ((uintptr_t)spans & 15) == 0, name ": spans must be there and 16-byte aligned");    \
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0, name ": slots (%d) and rows (%d) must be positive", slots, rows)

extern "C" int iron_time_mix_chunked(const void* r, const void* k, const void* v, const float* log_decay, const uint16_t* u,
                                     float* state, const int* spans, float* o, void* workspace, int slots, int rows, int heads,
                                     int dim, int is_float, void* stream) {
  IRON_REQUIRE(r && k && v && log_decay && u && state && o && workspace, "time_mix_chunked: null operand");
  IRON_CHUNKED_REQUIRE("time_mix_chunked");
  IRON_REQUIRE(heads > 0 && heads <= 65535 && dim > 0 && dim <= 256, "time_mix_chunked: heads (%d) positive, dim (%d) from 1 to 256", heads, dim);
  IRON_REQUIRE(((uintptr_t)workspace & 15) == 0, "time_mix_chunked: the workspace must be 16-byte aligned");
  IRON_REQUIRE((long)rows * heads * dim < (1L << 28), "time_mix_chunked: the batch's rows are addressed with 32-bit offsets");
  hipStream_t s = (hipStream_t)stream;
  const int tiles = (dim + 15) / 16, pitch = tiles * 16 + 4;
  const size_t lds = ((size_t)(3 * CHUNK + 1) * pitch + CHUNK * 17) * 4;
  const dim3 all((rows + CHUNK - 1) / CHUNK, heads, slots), walk(heads, tiles, slots);
  float* work = (float*)workspace;
  const WalkShape shape{rows, slots, heads, dim, dim, heads * dim, heads * dim};
#define IRON_MIX_WALK(T, NT, DEPTH) \
  hipLaunchKernelGGL((time_mix_walk_kernel<T, NT, DEPTH>), walk, dim3(256), 0, s, (const T*)v, state, spans, work, o, shape)
#define IRON_MIX(T)                                                                                                             \
  hipLaunchKernelGGL((time_mix_chunks_kernel<T>), all, dim3(256), lds, s, (const T*)r, (const T*)k, log_decay, u, spans, work, rows, \
                     slots, heads, dim);                                                                                        \
  if (tiles <= 4) IRON_MIX_WALK(T, 1, 6);                                                                                          \
  else if (tiles <= 8) IRON_MIX_WALK(T, 2, 4);                                                                                     \
  else IRON_MIX_WALK(T, 4, 2);
  if (is_float) { IRON_MIX(float) }
  else { IRON_MIX(bf16_t) }
#undef IRON_MIX
#undef IRON_MIX_WALK
  IRON_LAUNCH_CHECK();
}

extern "C" int64_t iron_hgrn2_workspace_bytes(int slots, int rows, int heads, int dim) {
  return chunks_of(rows, slots, CHUNK) * heads * (int64_t)mix_words((dim + 15) / 16) * 4;
}

extern "C" int iron_hgrn2_chunked(const void* x, const uint16_t* f_bias, const uint16_t* lower, float* state, const int* spans, float* o, void* workspace,
                                  int slots, int rows, int stride, int heads, int dim, int vdim, int is_float, void* stream) {
  IRON_REQUIRE(x && f_bias && lower && state && o && workspace, "hgrn2_chunked: null operand");
  IRON_CHUNKED_REQUIRE("hgrn2_chunked");
  IRON_REQUIRE(heads > 0 && heads <= 65535 && dim > 0 && dim <= 256 && vdim > 0, "hgrn2_chunked: heads (%d) and vdim (%d) positive, dim (%d) from 1 to 256",
               heads, vdim, dim);
  IRON_REQUIRE(stride >= heads * (2 * dim + vdim), "hgrn2_chunked: a row of %d holds no q, f and v of %d heads", stride, heads);
  IRON_REQUIRE(((uintptr_t)workspace & 15) == 0, "hgrn2_chunked: the workspace must be 16-byte aligned");
  IRON_REQUIRE((long)rows * stride < (1L << 28) && (long)rows * heads * vdim < (1L << 28), "hgrn2_chunked: the batch's rows are addressed with 32-bit offsets");
  hipStream_t s = (hipStream_t)stream;
  const int tiles = (dim + 15) / 16, pitch = tiles * 16 + 4;
  const size_t lds = ((size_t)3 * CHUNK * pitch + CHUNK * 17) * 4;
  const dim3 all((rows + CHUNK - 1) / CHUNK, heads, slots), walk(heads, (vdim + 15) / 16, slots);
  float* work = (float*)workspace;
  const FadeGates g{f_bias, lower};
  const bool vec = dim % 8 == 0 && stride % 8 == 0 && (((uintptr_t)x | (uintptr_t)f_bias | (uintptr_t)lower) & 15) == 0;
  const WalkShape shape{rows, slots, heads, dim, vdim, stride, heads * vdim};
#define IRON_FADE_WALK(T, NT, DEPTH) \
  hipLaunchKernelGGL((time_mix_walk_kernel<T, NT, DEPTH>), walk, dim3(256), 0, s, (const T*)x + 2 * heads * dim, state, spans, work, o, shape)
#define IRON_FADE(T)                                                                                                                        \
  if (vec) hipLaunchKernelGGL((hgrn2_chunks_kernel<T, 8>), all, dim3(256), lds, s, (const T*)x, g, spans, work, rows, slots, stride, heads, dim); \
  else hipLaunchKernelGGL((hgrn2_chunks_kernel<T, 1>), all, dim3(256), lds, s, (const T*)x, g, spans, work, rows, slots, stride, heads, dim); \
  if (tiles <= 4) IRON_FADE_WALK(T, 1, 6);                                                                                                  \
  else if (tiles <= 8) IRON_FADE_WALK(T, 2, 4);                                                                                             \
  else IRON_FADE_WALK(T, 4, 2);
  if (is_float) { IRON_FADE(float) }
  else { IRON_FADE(bf16_t) }
#undef IRON_FADE
#undef IRON_FADE_WALK
  IRON_LAUNCH_CHECK();
}

extern "C" int64_t iron_matrix_memory_workspace_bytes(int slots, int rows, int heads, int dim) {
  return chunks_of(rows, slots, CHUNK) * heads * (int64_t)(mix_words((dim + 15) / 16) * 4 + 4);
}

extern "C" int iron_matrix_memory_chunked(const void* x, const uint16_t* i_bias, const uint16_t* f_bias, float* state, float* tops,
                                          const int* spans, float* o, void* workspace, int slots, int rows, int stride, int heads, int dim,
                                          int vdim, int i_at, int f_at, float cap, int is_float, void* stream) {
  IRON_REQUIRE(x && i_bias && f_bias && state && tops && o && workspace, "matrix_memory_chunked: null operand");
  IRON_CHUNKED_REQUIRE("matrix_memory_chunked");
  IRON_REQUIRE(heads > 0 && heads <= 65535 && dim > 0 && dim <= 256 && vdim > 0,
               "matrix_memory_chunked: heads (%d) and vdim (%d) positive, dim (%d) from 1 to 256", heads, vdim, dim);
  const int packed = heads * (2 * dim + vdim);
  IRON_REQUIRE(i_at >= packed && f_at >= packed && i_at + heads <= stride && f_at + heads <= stride,
               "matrix_memory_chunked: the gates (%d, %d) lie behind q, k, v (%d) in a row of %d", i_at, f_at, packed, stride);
  IRON_REQUIRE(cap > 0.f, "matrix_memory_chunked: a cap (%g) above 0", (double)cap);
  IRON_REQUIRE(((uintptr_t)workspace & 15) == 0, "matrix_memory_chunked: the workspace must be 16-byte aligned");
  IRON_REQUIRE((long)rows * stride < (1L << 28) && (long)rows * heads * (vdim + 2) < (1L << 28),
               "matrix_memory_chunked: the batch's rows are addressed with 32-bit offsets");
  hipStream_t s = (hipStream_t)stream;
  const int tiles = (dim + 15) / 16;
  const size_t lds = (size_t)2 * CHUNK * (tiles * 16 + 4) * 4;
  const dim3 all((rows + CHUNK - 1) / CHUNK, heads, slots), walk(heads, (vdim + 1 + 15) / 16, slots);
  float *work = (float*)workspace, *starts = work + chunks_of(rows, slots, CHUNK) * heads * (size_t)mix_words(tiles);
  const MemoryGates g{i_bias, f_bias, i_at, f_at, cap};
  const WalkShape shape{rows, slots, heads, dim, vdim, stride, heads * vdim + 2 * heads};
#define IRON_MEMORY_WALK(T, NT, DEPTH) \
  hipLaunchKernelGGL((time_mix_walk_kernel<T, NT, DEPTH, true>), walk, dim3(256), 0, s, (const T*)x + 2 * heads * dim, state, spans, work, o, shape)
#define IRON_MEMORY(T)                                                                                                                  \
  hipLaunchKernelGGL((memory_tops_kernel<T>), dim3(heads, slots), dim3(TOPS_THREADS), 0, s, (const T*)x, g, tops, spans, starts, rows,  \
                     slots, stride, heads);                                                                                             \
  hipLaunchKernelGGL((memory_chunks_kernel<T>), all, dim3(256), lds, s, (const T*)x, g, spans, starts, work, o, rows, slots, stride,    \
                     heads, dim, vdim);                                                                                                 \
  if (tiles <= 4) IRON_MEMORY_WALK(T, 1, 6);                                                                                            \
  else if (tiles <= 8) IRON_MEMORY_WALK(T, 2, 4);                                                                                       \
  else IRON_MEMORY_WALK(T, 4, 2);
  if (is_float) { IRON_MEMORY(float) }
  else { IRON_MEMORY(bf16_t) }
#undef IRON_MEMORY
#undef IRON_MEMORY_WALK
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_delta_rule_chunked(const float* x, float* state, const int* spans, float* o, void* workspace, int slots,
                                       int rows, int heads, int kv_heads, int dim, int vdim, void* stream) {
  IRON_REQUIRE(x && state && o && workspace, "delta_rule_chunked: null operand");
  IRON_CHUNKED_REQUIRE("delta_rule_chunked");
  IRON_REQUIRE(heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0,
               "delta_rule_chunked: kv_heads (%d) must divide heads (%d)", kv_heads, heads);
  IRON_REQUIRE(dim > 0 && dim <= 256 && vdim > 0, "delta_rule_chunked: dim (%d) from 1 to 256, vdim (%d) positive", dim, vdim);
  IRON_REQUIRE(((uintptr_t)workspace & 15) == 0, "delta_rule_chunked: the workspace must be 16-byte aligned");
  IRON_REQUIRE((long)rows * (2 * kv_heads * dim + heads * (vdim + 2)) < (1L << 28),
               "delta_rule_chunked: the batch's rows are addressed with 32-bit offsets");
  hipStream_t s = (hipStream_t)stream;
  const dim3 all((rows + CHUNK - 1) / CHUNK, heads, slots), walk(heads, (vdim + 15) / 16, slots);
  const bool vec = dim % 4 == 0 && (heads * vdim + 2 * heads) % 4 == 0 && ((uintptr_t)x & 15) == 0;   // (2 kv_heads dim is whole then)
  float* work = (float*)workspace;
#define IRON_DELTA_WALK(NT, DEPTH)                                                                                                    \
  {                                                                                                                              \
    hipLaunchKernelGGL((delta_chunks_kernel<NT>), all, dim3(256), 0, s, x, spans, work, rows, slots, heads, kv_heads, dim, vdim); \
    if (vec)                                                                                                                     \
      hipLaunchKernelGGL((delta_walk_kernel<NT, DEPTH, true>), walk, dim3(256), 0, s, x, state, spans, work, o, rows, slots, heads, \
                         kv_heads, dim, vdim);                                                                                   \
    else                                                                                                                         \
      hipLaunchKernelGGL((delta_walk_kernel<NT, DEPTH, false>), walk, dim3(256), 0, s, x, state, spans, work, o, rows, slots,    \
                         heads, kv_heads, dim, vdim);                                                                            \
  }
  if (dim <= 64) IRON_DELTA_WALK(1, 3)
  else if (dim <= 128) IRON_DELTA_WALK(2, 2)
  else IRON_DELTA_WALK(4, 2)
#undef IRON_DELTA_WALK
  IRON_LAUNCH_CHECK();
}
