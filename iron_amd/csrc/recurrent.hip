// Layers that carry a state from token to token, over a batch of rows whose spans say which rows are
// which sequence's: the token shift, a low-rank decay, the time-mixing recurrence, the short causal
// convolution, the gated delta rule, and the per-head norm and gate behind either recurrence.
//
// A slot's state belongs to the sequence in it.  A span that starts at position 0 reads no state (it
// counts as zeros), so a slot needs no clearing between sequences.  States that the rows of a span
// both read and replace are replaced by the thread that read them, after it read them.
//
// The recurrences run in float32 throughout.  The state of a head, (dim, columns), is split by
// columns: a wave holds 4 columns, 16 lanes to a column, NI consecutive rows of it a lane, so that a
// sum along dim is a sum in a lane and four steps of the DPP path.  A block (16 columns) stages 16
// tokens of its head in LDS while the next 16 are on their way from memory.
#include "../../include/iron_hip.h"
#include "rows.h"

namespace iron {

constexpr int SCAN_TOKENS = 16;    // tokens staged at a time
constexpr int SCAN_COLUMNS = 16;   // state columns a block holds

__device__ __forceinline__ float sigmoid_exact(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_exact(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// ------------------------------------------------------------- token shift
// mixed[s] = h + (before - h) * mu[s], `before` the row ahead of h in its sequence.
constexpr int SHIFT_TILE = 4;
template <typename T, int VEC>
__global__ __launch_bounds__(256) void token_shift_kernel(const T* __restrict__ h, const bf16_t* __restrict__ mu,
                                                          T* __restrict__ carry, const int* __restrict__ spans,
                                                          T* __restrict__ mixed, int rows, int cols, int mixes) {
  const Span s = span_of(spans, blockIdx.y, rows);
  const int first = blockIdx.x * SHIFT_TILE;
  if (first >= s.rows) return;
  const int last = min(s.rows, first + SHIFT_TILE);
  // Two rows a slot, by a position's parity: a decode step's launch reads one and leaves the other.
  T* held = carry + (size_t)blockIdx.y * 2 * cols;
  const int old_row = (s.start - 1) & 1, new_row = (s.start + s.rows - 1) & 1;
  for (int c = threadIdx.x * VEC; c < cols; c += 256 * VEC) {
    float before[VEC];
    if (first > 0) load_vec<VEC>(h + (size_t)(s.row0 + first - 1) * cols + c, before);
    else if (s.start > 0) load_vec<VEC>(held + old_row * cols + c, before);
    else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) before[j] = 0.f;
    }
    if (first == 0) {   // the span's last row is what the next one starts from
      float end[VEC];
      load_vec<VEC>(h + (size_t)(s.row0 + s.rows - 1) * cols + c, end);
      store_vec<VEC>(held + new_row * cols + c, end);
    }
    for (int i = first; i < last; ++i) {
      float now[VEC];
      load_vec<VEC>(h + (size_t)(s.row0 + i) * cols + c, now);
      for (int m = 0; m < mixes; ++m) {
        float g[VEC];
        load_vec<VEC>(mu + (size_t)m * cols + c, g);
#pragma unroll
        for (int j = 0; j < VEC; ++j) g[j] = now[j] + (before[j] - now[j]) * g[j];
        store_vec<VEC>(mixed + ((size_t)m * rows + s.row0 + i) * cols + c, g);
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) before[j] = now[j];
    }
  }
}

// --------------------------------------------------------- low-rank decay
// log decay = -exp(W2 tanh(z) + w0), in float32: what the recurrence takes the exponential of.
constexpr int DECAY_ROWS = 16;
template <typename T>
__global__ __launch_bounds__(256) void low_rank_decay_kernel(const T* __restrict__ z, const bf16_t* __restrict__ w2,
                                                             const bf16_t* __restrict__ w0, float* __restrict__ out,
                                                             int rows, int n, int rank, const int* __restrict__ valid) {
  extern __shared__ __align__(16) float zt[];   // [rank][DECAY_ROWS]
  const int live = bound_or(valid, rows);
  const int r0 = blockIdx.y * DECAY_ROWS;
  if (r0 >= live) return;
  for (int i = threadIdx.x; i < rank * DECAY_ROWS; i += 256) {
    const int r = i / rank, k = i - r * rank;
    zt[k * DECAY_ROWS + r] = r0 + r < live ? tanhf(load_one(z + (size_t)(r0 + r) * rank + k)) : 0.f;
  }
  __syncthreads();
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= n) return;
  float acc[DECAY_ROWS];
  const float bias = bf16_to_f32(w0[c]);
#pragma unroll
  for (int r = 0; r < DECAY_ROWS; ++r) acc[r] = 0.f;
  const bf16_t* wr = w2 + (size_t)c * rank;
  int k = 0;
  if (rank % 8 == 0 && ((uintptr_t)w2 & 15) == 0)
    for (; k < rank; k += 8) {
      float w[8];
      unpack8(*reinterpret_cast<const uint4*>(wr + k), w);
#pragma unroll
      for (int j = 0; j < 8; ++j)
#pragma unroll
        for (int r = 0; r < DECAY_ROWS; r += 4) {
          const float4 z4 = *reinterpret_cast<const float4*>(zt + (k + j) * DECAY_ROWS + r);
          acc[r] = fmaf(w[j], z4.x, acc[r]);
          acc[r + 1] = fmaf(w[j], z4.y, acc[r + 1]);
          acc[r + 2] = fmaf(w[j], z4.z, acc[r + 2]);
          acc[r + 3] = fmaf(w[j], z4.w, acc[r + 3]);
        }
    }
  for (; k < rank; ++k) {
    const float w = bf16_to_f32(wr[k]);
#pragma unroll
    for (int r = 0; r < DECAY_ROWS; ++r) acc[r] = fmaf(w, zt[k * DECAY_ROWS + r], acc[r]);
  }
#pragma unroll
  for (int r = 0; r < DECAY_ROWS; ++r)
    if (r0 + r < live) out[(size_t)(r0 + r) * n + c] = -expf(acc[r] + bias);
}

// -------------------------------------------------------------- time mixing
template <int NI>
__device__ __forceinline__ void lds_run(const float* __restrict__ p, float (&f)[NI]) {
  if constexpr (NI % 4 == 0) {
#pragma unroll
    for (int e = 0; e < NI; e += 4) {
      const float4 v = *reinterpret_cast<const float4*>(p + e);
      f[e] = v.x; f[e + 1] = v.y; f[e + 2] = v.z; f[e + 3] = v.w;
    }
  } else {
#pragma unroll
    for (int e = 0; e < NI; ++e) f[e] = p[e];
  }
}

// o_t = (S + diag(u) k v^T)^T r;  S <- diag(exp(log decay)) S + k v^T.  The bonus term is the scalar
// sum(r u k) times v.
template <typename T, int NI>
__global__ __launch_bounds__(256) void time_mix_kernel(const T* __restrict__ r, const T* __restrict__ k, const T* __restrict__ v,
                                                       const float* __restrict__ log_decay, const bf16_t* __restrict__ u,
                                                       float* __restrict__ state, const int* __restrict__ spans,
                                                       float* __restrict__ o, int rows, int heads, int dim) {
  constexpr int WIDE = 16 * NI;
  __shared__ __align__(16) float rs[SCAN_TOKENS][WIDE], ks[SCAN_TOKENS][WIDE], ds[SCAN_TOKENS][WIDE];
  __shared__ float vs[SCAN_TOKENS][SCAN_COLUMNS], os[SCAN_TOKENS][SCAN_COLUMNS + 1], bonus[SCAN_TOKENS];
  const int head = blockIdx.y, slot = blockIdx.z;
  const Span s = span_of(spans, slot, rows);
  if (s.rows == 0) return;
  const int t = threadIdx.x, lane = t & 63, ig = t & 15, tok = t >> 4;   // staging: 16 threads a token
  const int col = blockIdx.x * SCAN_COLUMNS + (t >> 4);                  // scanning: 16 lanes a column
  const int width = heads * dim;
  float* sp = state + ((size_t)slot * heads + head) * dim * dim;
  float S[NI], gain[NI];
#pragma unroll
  for (int e = 0; e < NI; ++e) {
    const int i = ig * NI + e;
    S[e] = (s.start > 0 && i < dim && col < dim) ? sp[(size_t)i * dim + col] : 0.f;
    gain[e] = i < dim ? bf16_to_f32(u[head * dim + i]) : 0.f;
  }
  float rn[NI], kn[NI], dn[NI], vn;
  const int vcol = blockIdx.x * SCAN_COLUMNS + ig;
  auto fetch = [&](int base) {
    const bool live = base + tok < s.rows;
    const size_t at = (size_t)(s.row0 + base + tok) * width + head * dim;
#pragma unroll
    for (int e = 0; e < NI; ++e) {
      const int i = ig * NI + e;
      const bool in = live && i < dim;
      rn[e] = in ? load_one(r + at + i) : 0.f;
      kn[e] = in ? load_one(k + at + i) : 0.f;
      dn[e] = in ? log_decay[at + i] : 0.f;
    }
    vn = live && vcol < dim ? load_one(v + at + vcol) : 0.f;
  };
  fetch(0);
  for (int base = 0; base < s.rows; base += SCAN_TOKENS) {
    float b = 0.f;
#pragma unroll
    for (int e = 0; e < NI; ++e) {
      rs[tok][ig * NI + e] = rn[e];
      ks[tok][ig * NI + e] = kn[e];
      ds[tok][ig * NI + e] = expf(dn[e]);
      b = fmaf(rn[e] * gain[e], kn[e], b);
    }
    vs[tok][ig] = vn;
    b = group16_sum(b);
    if (ig == 0) bonus[tok] = b;
    __syncthreads();
    if (base + SCAN_TOKENS < s.rows) fetch(base + SCAN_TOKENS);
    const int n = min(SCAN_TOKENS, (s.rows - base + 3) & ~3);   // past the last row: r, k, v 0, decay 1
    for (int q = 0; q < n; q += 4) {
#pragma unroll
      for (int p = q; p < q + 4; ++p) {
        float rr[NI], kk[NI], dd[NI];
        lds_run<NI>(&rs[p][ig * NI], rr);
        lds_run<NI>(&ks[p][ig * NI], kk);
        lds_run<NI>(&ds[p][ig * NI], dd);
        const float vv = vs[p][t >> 4];
        float acc = 0.f;
#pragma unroll
        for (int e = 0; e < NI; ++e) {
          acc = fmaf(rr[e], S[e], acc);
          S[e] = fmaf(dd[e], S[e], kk[e] * vv);
        }
        acc = group16_sum(acc);
        if (ig == 0) os[p][t >> 4] = fmaf(bonus[p], vv, acc);
      }
    }
    __syncthreads();
    if (base + tok < s.rows && vcol < dim) o[(size_t)(s.row0 + base + tok) * width + head * dim + vcol] = os[tok][ig];
  }
#pragma unroll
  for (int e = 0; e < NI; ++e) {
    const int i = ig * NI + e;
    if (i < dim && col < dim) sp[(size_t)i * dim + col] = S[e];
  }
  (void)lane;
}

// ------------------------------------------------------- short convolution
// The packed projection's rows [q | k | v | ... | b | a] -> float32 rows [unit q / sqrt(dim) | unit k |
// v | log decay | beta]: a causal convolution a channel and SiLU on q, k, v; unit q and k a head; the
// step's log decay -exp(A_log) softplus(a + dt_bias) and beta = sigmoid(b) a value head.
struct ConvShape {
  int rows, stride;                 // the projection's rows, and their length
  int heads, kv_heads, dim, vdim;
  int taps, b_at, a_at;             // columns of b and a in a projection row
};
constexpr int CONV_TILE = 16;
template <typename T, int TAPS>   // TAPS: the number of taps where it is a small one, else 0
__global__ __launch_bounds__(256) void short_conv_kernel(const T* __restrict__ x, const bf16_t* __restrict__ taps,
                                                         const bf16_t* __restrict__ a_log, const bf16_t* __restrict__ dt_bias,
                                                         T* __restrict__ state, const int* __restrict__ spans,
                                                         float* __restrict__ out, ConvShape c) {
  const int seg = blockIdx.y, slot = blockIdx.z, first = blockIdx.x * CONV_TILE;
  const Span s = span_of(spans, slot, c.rows);
  if (first >= s.rows) return;
  const int last = min(s.rows, first + CONV_TILE);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int qk = c.kv_heads * c.dim, channels = 2 * qk + c.heads * c.vdim, wide = channels + 2 * c.heads;
  if (seg == 2 * c.kv_heads + c.heads) {   // the heads' decays and betas
    const int count = (last - first) * c.heads;
    for (int i = threadIdx.x; i < count; i += 256) {
      const int p = first + i / c.heads, h = i % c.heads;
      const T* row = x + (size_t)(s.row0 + p) * c.stride;
      float* to = out + (size_t)(s.row0 + p) * wide + channels;
      const float a = load_one(row + c.a_at + h) + bf16_to_f32(dt_bias[h]);
      to[h] = -expf(bf16_to_f32(a_log[h])) * softplus_exact(a);
      to[c.heads + h] = sigmoid_exact(load_one(row + c.b_at + h));
    }
    return;
  }
  const bool is_v = seg >= 2 * c.kv_heads;
  const int len = is_v ? c.vdim : c.dim;
  const int at = is_v ? 2 * qk + (seg - 2 * c.kv_heads) * c.vdim : seg * c.dim;
  const int past = c.taps - 1;
  T* held = state + (size_t)slot * c.taps * channels;   // position p's input in row p % taps
  // The input at place p of the span: a row of this call, the slot's state before it, zero before 0.
  auto input = [&](int p, int ch) -> float {
    if (p >= 0) return load_one(x + (size_t)(s.row0 + p) * c.stride + ch);
    return s.start + p >= 0 ? load_one(held + (size_t)((s.start + p) % c.taps) * channels + ch) : 0.f;
  };
  // A wave makes four rows one after the other; where the taps are few their inputs slide through
  // registers, so that each is read once for the four.
  const int p0 = first + wave * 4;
  if (p0 < last) {
    float f[4][4], ss[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int j = lane + 64 * e;
      if (64 * e >= len) continue;
      const bool in = j < len;
      const bf16_t* tw = taps + (size_t)(at + (in ? j : 0)) * c.taps;
      if (TAPS > 0) {
        float w[TAPS > 0 ? TAPS : 1], win[TAPS + 3];
#pragma unroll
        for (int i = 0; i < TAPS; ++i) w[i] = in ? bf16_to_f32(tw[i]) : 0.f;
#pragma unroll
        for (int i = 0; i < TAPS + 3; ++i) win[i] = (in && p0 - (TAPS - 1) + i < last) ? input(p0 - (TAPS - 1) + i, at + j) : 0.f;
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          float acc = 0.f;
#pragma unroll
          for (int i = 0; i < TAPS; ++i) acc = fmaf(w[i], win[q + i], acc);
          f[q][e] = acc * sigmoid_exact(acc);
        }
      } else {
        for (int q = 0; q < 4; ++q) {
          float acc = 0.f;
          if (in && p0 + q < last)
            for (int i = 0; i < c.taps; ++i) acc = fmaf(bf16_to_f32(tw[i]), input(p0 + q - past + i, at + j), acc);
          f[q][e] = acc * sigmoid_exact(acc);
        }
      }
#pragma unroll
      for (int q = 0; q < 4; ++q) ss[q] = fmaf(f[q][e], f[q][e], ss[q]);
    }
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      float scale = 1.f;
      if (!is_v) {
        scale = 1.0f / sqrtf(wave_sum(ss[q]) + 1e-6f);
        if (seg < c.kv_heads) scale *= 1.0f / sqrtf((float)c.dim);
      }
      if (p0 + q >= last) continue;
      float* to = out + (size_t)(s.row0 + p0 + q) * wide + at;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (lane + 64 * e < len) to[lane + 64 * e] = f[q][e] * scale;
    }
  }
  if (first == 0) {   // no other block reads these channels' state
    __syncthreads();
    for (int j = threadIdx.x; j < len; j += 256)
      for (int p = max(0, s.rows - past); p < s.rows; ++p)
        store_one(held + (size_t)((s.start + p) % c.taps) * channels + at + j, input(p, at + j));
  }
}

// ----------------------------------------------------------- the delta rule
// S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  Both sums along dim are taken of the old
// state, so that they run side by side: o = g (S^T q) + (k . q) u.
template <int NI>
__global__ __launch_bounds__(256) void delta_rule_kernel(const float* __restrict__ x, float* __restrict__ state,
                                                         const int* __restrict__ spans, float* __restrict__ o, int rows,
                                                         int heads, int kv_heads, int dim, int vdim) {
  constexpr int WIDE = 16 * NI;
  __shared__ __align__(16) float qs[SCAN_TOKENS][WIDE], ks[SCAN_TOKENS][WIDE];
  __shared__ float vs[SCAN_TOKENS][SCAN_COLUMNS], os[SCAN_TOKENS][SCAN_COLUMNS + 1];
  __shared__ float gs[SCAN_TOKENS], bs[SCAN_TOKENS], kq[SCAN_TOKENS];
  const int head = blockIdx.y, slot = blockIdx.z;
  const Span s = span_of(spans, slot, rows);
  if (s.rows == 0) return;
  const int t = threadIdx.x, ig = t & 15, tok = t >> 4;
  const int col = blockIdx.x * SCAN_COLUMNS + (t >> 4), vcol = blockIdx.x * SCAN_COLUMNS + ig;
  const int qk = kv_heads * dim, channels = 2 * qk + heads * vdim, wide = channels + 2 * heads;
  const int group = head / (heads / kv_heads);
  float* sp = state + ((size_t)slot * heads + head) * dim * vdim;
  float S[NI];
#pragma unroll
  for (int e = 0; e < NI; ++e) {
    const int i = ig * NI + e;
    S[e] = (s.start > 0 && i < dim && col < vdim) ? sp[(size_t)i * vdim + col] : 0.f;
  }
  float qn[NI], kn[NI], vn, gn, bn;
  auto fetch = [&](int base) {
    const bool live = base + tok < s.rows;
    const float* row = x + (size_t)(s.row0 + base + tok) * wide;
#pragma unroll
    for (int e = 0; e < NI; ++e) {
      const int i = ig * NI + e;
      const bool in = live && i < dim;
      qn[e] = in ? row[group * dim + i] : 0.f;
      kn[e] = in ? row[qk + group * dim + i] : 0.f;
    }
    vn = live && vcol < vdim ? row[2 * qk + head * vdim + vcol] : 0.f;
    gn = live ? row[channels + head] : 0.f;
    bn = live ? row[channels + heads + head] : 0.f;
  };
  fetch(0);
  for (int base = 0; base < s.rows; base += SCAN_TOKENS) {
    float b = 0.f;
#pragma unroll
    for (int e = 0; e < NI; ++e) {
      qs[tok][ig * NI + e] = qn[e];
      ks[tok][ig * NI + e] = kn[e];
      b = fmaf(qn[e], kn[e], b);
    }
    vs[tok][ig] = vn;
    b = group16_sum(b);
    if (ig == 0) {
      kq[tok] = b;
      gs[tok] = expf(gn);
      bs[tok] = bn;
    }
    __syncthreads();
    if (base + SCAN_TOKENS < s.rows) fetch(base + SCAN_TOKENS);
    const int n = min(SCAN_TOKENS, (s.rows - base + 3) & ~3);   // past the last row: q, k, v, beta 0, decay 1
    for (int q = 0; q < n; q += 4) {
#pragma unroll
      for (int p = q; p < q + 4; ++p) {
        float qq[NI], kk[NI];
        lds_run<NI>(&qs[p][ig * NI], qq);
        lds_run<NI>(&ks[p][ig * NI], kk);
        const float g = gs[p];
        float read = 0.f, out = 0.f;
#pragma unroll
        for (int e = 0; e < NI; ++e) {
          read = fmaf(kk[e], S[e], read);
          out = fmaf(qq[e], S[e], out);
        }
        read = group16_sum(read);
        out = group16_sum(out);
        const float u = bs[p] * fmaf(-g, read, vs[p][t >> 4]);
#pragma unroll
        for (int e = 0; e < NI; ++e) S[e] = fmaf(kk[e], u, g * S[e]);
        if (ig == 0) os[p][t >> 4] = fmaf(kq[p], u, g * out);
      }
    }
    __syncthreads();
    if (base + tok < s.rows && vcol < vdim) o[(size_t)(s.row0 + base + tok) * (heads * vdim) + head * vdim + vcol] = os[tok][ig];
  }
#pragma unroll
  for (int e = 0; e < NI; ++e) {
    const int i = ig * NI + e;
    if (i < dim && col < vdim) sp[(size_t)i * vdim + col] = S[e];
  }
}

// ------------------------------------------------------- per-head norm, gate
// out = (o / rms(o)) * gain * silu(gate) * scale, the mean over one head's columns; without a gate, that factor is 1.
// LANES lanes to a head's row of up to 4 LANES columns, four a lane where VEC (else one of every LANES).
template <typename T, int LANES, bool VEC>
__global__ __launch_bounds__(256) void head_gate_kernel(const float* __restrict__ o, const T* __restrict__ gate,
                                                        const bf16_t* __restrict__ gain, T* __restrict__ out, int rows,
                                                        int heads, int dim, int gate_stride, int gate_at, int gain_shared,
                                                        int out_stride, int out_at, float eps, float scale,
                                                        const int* __restrict__ valid) {
  const long item = ((long)blockIdx.x * 256 + threadIdx.x) / LANES;
  const int row = (int)(item / heads), head = (int)(item - (long)row * heads), lane = threadIdx.x % LANES;
  if (row >= bound_or(valid, rows)) return;
  const float* src = o + ((size_t)row * heads + head) * dim;
  const T* gr = gate + (size_t)row * gate_stride + gate_at + head * dim;
  const bf16_t* wr = gain + (gain_shared ? 0 : head * dim);
  T* to = out + (size_t)row * out_stride + out_at + head * dim;
  float f[4] = {0.f, 0.f, 0.f, 0.f}, z[4], g[4], ss = 0.f;
  const int c0 = lane * 4;
  if (VEC && c0 < dim) {
    const float4 v = *reinterpret_cast<const float4*>(src + c0);
    f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w;
    if (gate == nullptr) {
      z[0] = z[1] = z[2] = z[3] = 0.f;
    } else if constexpr (sizeof(T) == 2) {
      const uint2 w = *reinterpret_cast<const uint2*>(gr + c0);
      z[0] = bf16_lo(w.x); z[1] = bf16_hi(w.x); z[2] = bf16_lo(w.y); z[3] = bf16_hi(w.y);
    } else {
      const float4 w = *reinterpret_cast<const float4*>(gr + c0);
      z[0] = w.x; z[1] = w.y; z[2] = w.z; z[3] = w.w;
    }
    const uint2 w = *reinterpret_cast<const uint2*>(wr + c0);
    g[0] = bf16_lo(w.x); g[1] = bf16_hi(w.x); g[2] = bf16_lo(w.y); g[3] = bf16_hi(w.y);
  } else if (!VEC) {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (lane + LANES * e < dim) {
        f[e] = src[lane + LANES * e];
        z[e] = gate != nullptr ? load_one(gr + lane + LANES * e) : 0.f;
        g[e] = bf16_to_f32(wr[lane + LANES * e]);
      }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) ss = fmaf(f[e], f[e], ss);
#pragma unroll
  for (int mask = 1; mask < LANES; mask <<= 1) ss += __shfl_xor(ss, mask, 64);
  const float inv = 1.0f / sqrtf(ss / (float)dim + eps);
  auto through = [&](float v) { return gate != nullptr ? v * sigmoid_exact(v) : 1.f; };
  if (VEC) {
    if (c0 >= dim) return;
#pragma unroll
    for (int e = 0; e < 4; ++e) f[e] = f[e] * inv * g[e] * through(z[e]) * scale;
    if constexpr (sizeof(T) == 2) *reinterpret_cast<uint2*>(to + c0) = make_uint2(pack_bf16(f[0], f[1]), pack_bf16(f[2], f[3]));
    else *reinterpret_cast<float4*>(to + c0) = make_float4(f[0], f[1], f[2], f[3]);
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (lane + LANES * e < dim) store_one(to + lane + LANES * e, f[e] * inv * g[e] * through(z[e]) * scale);
  }
}

}  // namespace iron

using namespace iron;

static int per_lane(int dim) {   // state rows a lane holds: the power of two that covers dim over 16 lanes
  int ni = 1;
  while (16 * ni < dim) ni *= 2;
  return ni;
}

#define IRON_SPANS_REQUIRE(name)                                                                       \
  IRON_REQUIRE(spans && ((uintptr_t)spans & 15) == 0, name ": spans must be there and 16-byte aligned"); \
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0, name ": slots (%d) and rows (%d) must be positive", slots, rows)

extern "C" int iron_token_shift(const void* h, const uint16_t* mu, void* carry, const int* spans, void* mixed, int slots,
                                int rows, int cols, int mixes, int is_float, void* stream) {
  IRON_REQUIRE(h && mu && carry && mixed, "token_shift: null operand");
  IRON_SPANS_REQUIRE("token_shift");
  IRON_REQUIRE(cols > 0 && mixes > 0, "token_shift: cols (%d) and mixes (%d) must be positive", cols, mixes);
  const dim3 grid((rows + SHIFT_TILE - 1) / SHIFT_TILE, slots);
  hipStream_t s = (hipStream_t)stream;
  const bool vec = cols % 8 == 0 && (((uintptr_t)h | (uintptr_t)mu | (uintptr_t)carry | (uintptr_t)mixed) & 15) == 0;
#define IRON_SHIFT(T, V) \
  hipLaunchKernelGGL((token_shift_kernel<T, V>), grid, dim3(256), 0, s, (const T*)h, mu, (T*)carry, spans, (T*)mixed, rows, cols, mixes)
  if (is_float) { if (vec) IRON_SHIFT(float, 8); else IRON_SHIFT(float, 1); }
  else { if (vec) IRON_SHIFT(bf16_t, 8); else IRON_SHIFT(bf16_t, 1); }
#undef IRON_SHIFT
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_low_rank_decay(const void* z, const uint16_t* w2, const uint16_t* w0, float* out, int rows, int n,
                                   int rank, int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(z && w2 && w0 && out, "low_rank_decay: null operand");
  IRON_REQUIRE(rows > 0 && n > 0 && rank > 0 && rank <= 512, "low_rank_decay: rows (%d), n (%d) positive, rank (%d) from 1 to 512",
               rows, n, rank);
  const dim3 grid((n + 255) / 256, (rows + DECAY_ROWS - 1) / DECAY_ROWS);
  IRON_REQUIRE(grid.y <= 65535, "low_rank_decay: rows (%d) exceed the grid's y extent", rows);
  const size_t lds = (size_t)rank * DECAY_ROWS * 4;
  if (is_float)
    hipLaunchKernelGGL((low_rank_decay_kernel<float>), grid, dim3(256), lds, (hipStream_t)stream, (const float*)z, w2, w0, out, rows, n, rank, valid);
  else
    hipLaunchKernelGGL((low_rank_decay_kernel<bf16_t>), grid, dim3(256), lds, (hipStream_t)stream, (const bf16_t*)z, w2, w0, out, rows, n, rank, valid);
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_time_mix(const void* r, const void* k, const void* v, const float* log_decay, const uint16_t* u,
                             float* state, const int* spans, float* o, int slots, int rows, int heads, int dim, int is_float,
                             void* stream) {
  IRON_REQUIRE(r && k && v && log_decay && u && state && o, "time_mix: null operand");
  IRON_SPANS_REQUIRE("time_mix");
  IRON_REQUIRE(heads > 0 && heads <= 65535 && dim > 0 && dim <= 256, "time_mix: heads (%d) positive, dim (%d) from 1 to 256", heads, dim);
  const dim3 grid((dim + SCAN_COLUMNS - 1) / SCAN_COLUMNS, heads, slots);
  hipStream_t s = (hipStream_t)stream;
#define IRON_TIME_MIX(T, NI)                                                                                              \
  hipLaunchKernelGGL((time_mix_kernel<T, NI>), grid, dim3(256), 0, s, (const T*)r, (const T*)k, (const T*)v, log_decay, u, \
                     state, spans, o, rows, heads, dim)
#define IRON_TIME_MIX_NI(NI) { if (is_float) IRON_TIME_MIX(float, NI); else IRON_TIME_MIX(bf16_t, NI); break; }
  switch (per_lane(dim)) {
    case 1: IRON_TIME_MIX_NI(1)
    case 2: IRON_TIME_MIX_NI(2)
    case 4: IRON_TIME_MIX_NI(4)
    case 8: IRON_TIME_MIX_NI(8)
    default: IRON_TIME_MIX_NI(16)
  }
#undef IRON_TIME_MIX_NI
#undef IRON_TIME_MIX
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_short_conv(const void* x, const uint16_t* taps_w, const uint16_t* a_log, const uint16_t* dt_bias,
                               void* state, const int* spans, float* out, int slots, int rows, int stride, int heads,
                               int kv_heads, int dim, int vdim, int taps, int b_at, int a_at, int is_float, void* stream) {
  IRON_REQUIRE(x && taps_w && a_log && dt_bias && out && state, "short_conv: null operand");
  IRON_SPANS_REQUIRE("short_conv");
  IRON_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "short_conv: kv_heads (%d) must divide heads (%d)", kv_heads, heads);
  IRON_REQUIRE(dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256, "short_conv: dim (%d) and vdim (%d) from 1 to 256", dim, vdim);
  IRON_REQUIRE(taps >= 1 && taps <= CONV_TILE + 1, "short_conv: taps (%d) from 1 to %d", taps, CONV_TILE + 1);
  const int channels = 2 * kv_heads * dim + heads * vdim;
  IRON_REQUIRE(b_at >= channels && a_at >= channels && b_at + heads <= stride && a_at + heads <= stride,
               "short_conv: b (%d) and a (%d) lie behind q, k, v (%d) in a row of %d", b_at, a_at, channels, stride);
  const ConvShape c{rows, stride, heads, kv_heads, dim, vdim, taps, b_at, a_at};
  const dim3 grid((rows + CONV_TILE - 1) / CONV_TILE, 2 * kv_heads + heads + 1, slots);
  IRON_REQUIRE(grid.y <= 65535, "short_conv: %d heads exceed the grid's y extent", heads);
#define IRON_CONV(T, N)                                                                                                  \
  hipLaunchKernelGGL((short_conv_kernel<T, N>), grid, dim3(256), 0, (hipStream_t)stream, (const T*)x, taps_w, a_log, dt_bias, \
                     (T*)state, spans, out, c)
#define IRON_CONVS(T)                     \
  {                                       \
    if (taps == 2) IRON_CONV(T, 2);       \
    else if (taps == 3) IRON_CONV(T, 3);  \
    else if (taps == 4) IRON_CONV(T, 4);  \
    else IRON_CONV(T, 0);                 \
  }
  if (is_float) IRON_CONVS(float)
  else IRON_CONVS(bf16_t)
#undef IRON_CONVS
#undef IRON_CONV
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_delta_rule(const float* x, float* state, const int* spans, float* o, int slots, int rows, int heads,
                               int kv_heads, int dim, int vdim, void* stream) {
  IRON_REQUIRE(x && state && o, "delta_rule: null operand");
  IRON_SPANS_REQUIRE("delta_rule");
  IRON_REQUIRE(heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0, "delta_rule: kv_heads (%d) must divide heads (%d)",
               kv_heads, heads);
  IRON_REQUIRE(dim > 0 && dim <= 256 && vdim > 0, "delta_rule: dim (%d) from 1 to 256, vdim (%d) positive", dim, vdim);
  const dim3 grid((vdim + SCAN_COLUMNS - 1) / SCAN_COLUMNS, heads, slots);
#define IRON_DELTA(NI)                                                                                                     \
  {                                                                                                                        \
    hipLaunchKernelGGL((delta_rule_kernel<NI>), grid, dim3(256), 0, (hipStream_t)stream, x, state, spans, o, rows, heads, \
                       kv_heads, dim, vdim);                                                                               \
    break;                                                                                                                 \
  }
  switch (per_lane(dim)) {
    case 1: IRON_DELTA(1)
    case 2: IRON_DELTA(2)
    case 4: IRON_DELTA(4)
    case 8: IRON_DELTA(8)
    default: IRON_DELTA(16)
  }
#undef IRON_DELTA
  IRON_LAUNCH_CHECK();
}

extern "C" int iron_head_gate(const float* o, const void* gate, const uint16_t* gain, void* out, int rows, int heads, int dim,
                              int gate_stride, int gate_at, int gain_shared, int out_stride, int out_at, float eps,
                              float scale, int is_float, const int* valid, void* stream) {
  IRON_REQUIRE(o && gain && out, "head_gate: null operand");
  IRON_REQUIRE(rows > 0 && heads > 0 && dim > 0 && dim <= 256, "head_gate: rows (%d), heads (%d) positive, dim (%d) from 1 to 256",
               rows, heads, dim);
  IRON_REQUIRE((gate == nullptr || (gate_at >= 0 && gate_at + heads * dim <= gate_stride)) && out_at >= 0 && out_at + heads * dim <= out_stride,
               "head_gate: %d columns from %d of a gate row of %d, from %d of an output row of %d", heads * dim, gate_at,
               gate_stride, out_at, out_stride);
  const long items = (long)rows * heads;
  const bool vec = dim % 4 == 0 && gate_stride % 4 == 0 && gate_at % 4 == 0 && out_stride % 4 == 0 && out_at % 4 == 0 &&
                   (((uintptr_t)o | (uintptr_t)gate | (uintptr_t)gain | (uintptr_t)out) & 15) == 0;
  const int lanes = !vec ? 64 : (dim <= 64 ? 16 : (dim <= 128 ? 32 : 64));
  const dim3 grid((unsigned)((items * lanes + 255) / 256));
#define IRON_HEAD_GATE(T, L, V)                                                                                              \
  hipLaunchKernelGGL((head_gate_kernel<T, L, V>), grid, dim3(256), 0, (hipStream_t)stream, o, (const T*)gate, gain, (T*)out, rows, \
                     heads, dim, gate_stride, gate_at, gain_shared, out_stride, out_at, eps, scale, valid)
#define IRON_HEAD_GATES(T)                                   \
  {                                                          \
    if (!vec) IRON_HEAD_GATE(T, 64, false);                  \
    else if (lanes == 16) IRON_HEAD_GATE(T, 16, true);       \
    else if (lanes == 32) IRON_HEAD_GATE(T, 32, true);       \
    else IRON_HEAD_GATE(T, 64, true);                        \
  }
  if (is_float) IRON_HEAD_GATES(float)
  else IRON_HEAD_GATES(bf16_t)
#undef IRON_HEAD_GATES
#undef IRON_HEAD_GATE
  IRON_LAUNCH_CHECK();
}
