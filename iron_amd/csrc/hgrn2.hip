// HGRN2: a matrix a head whose rows fade by a forget gate a channel and are written what the gate leaves,
// S <- diag(f) S + (1 - f) v^T, read behind that by o = S^T silu(q).  Token by token, over a batch of spans; float32 throughout.
//
// The state of a head, (dim, vdim), is split by columns: a wave holds 4 columns, 16 lanes to a column, NI consecutive rows of it a
// lane; a block (16 columns) stages 16 tokens of its head in LDS while the next 16 are on their way from memory.
#include "../../include/iron_hip.h"
#include "hgrn2.h"

namespace iron {

constexpr int FADE_TOKENS = 16, FADE_COLUMNS = 16;

template <typename T, int NI>
__global__ __launch_bounds__(256) void hgrn2_kernel(const T* __restrict__ x, FadeGates g, float* __restrict__ state,
                                                    const int* __restrict__ spans, float* __restrict__ o, int rows, int stride, int heads,
                                                    int dim, int vdim) {
  constexpr int WIDE = 16 * NI;
  __shared__ __align__(16) float qs[FADE_TOKENS][WIDE], fs[FADE_TOKENS][WIDE], ws[FADE_TOKENS][WIDE];
  __shared__ float vs[FADE_TOKENS][FADE_COLUMNS], os[FADE_TOKENS][FADE_COLUMNS + 1];
  const int head = blockIdx.y, slot = blockIdx.z;
  const Span s = span_of(spans, slot, rows);
  if (s.rows == 0) return;
  const int t = threadIdx.x, ig = t & 15, tok = t >> 4;   // staging: 16 threads a token
  const int col = blockIdx.x * FADE_COLUMNS + (t >> 4), vcol = blockIdx.x * FADE_COLUMNS + ig;   // scanning: 16 lanes a column
  float* sp = state + ((size_t)slot * heads + head) * dim * vdim;
  float S[NI], bias[NI], lower[NI];
#pragma unroll
  for (int e = 0; e < NI; ++e) {
    const int i = ig * NI + e;
    S[e] = (s.start > 0 && i < dim && col < vdim) ? sp[(size_t)i * vdim + col] : 0.f;
    bias[e] = i < dim ? bf16_to_f32(g.bias[head * dim + i]) : 0.f;
    lower[e] = i < dim ? bf16_to_f32(g.lower[head * dim + i]) : 0.f;
  }
  float qn[NI], zn[NI], vn;
  auto fetch = [&](int base) {
    const bool live = base + tok < s.rows;
    const T* row = x + (size_t)(s.row0 + base + tok) * stride;
#pragma unroll
    for (int e = 0; e < NI; ++e) {
      const int i = ig * NI + e;
      const bool in = live && i < dim;
      qn[e] = in ? load_one(row + head * dim + i) : 0.f;
      zn[e] = in ? load_one(row + (heads + head) * dim + i) : 0.f;
    }
    vn = live && vcol < vdim ? load_one(row + 2 * heads * dim + head * vdim + vcol) : 0.f;
  };
  fetch(0);
  for (int base = 0; base < s.rows; base += FADE_TOKENS) {
#pragma unroll
    for (int e = 0; e < NI; ++e) {
      const int i = ig * NI + e;
      const bool in = i < dim && base + tok < s.rows;   // past the last row: the state stays
      const Fade f = fade_of<T>(zn[e], bias[e], lower[e]);
      qs[tok][i] = silu_read<T>(qn[e]);
      fs[tok][i] = in ? f.keep : 1.f;
      ws[tok][i] = in ? f.write : 0.f;
    }
    vs[tok][ig] = vn;
    __syncthreads();
    if (base + FADE_TOKENS < s.rows) fetch(base + FADE_TOKENS);
    const int n = min(FADE_TOKENS, s.rows - base);
    for (int p = 0; p < n; ++p) {
      const float vv = vs[p][t >> 4];
      float acc = 0.f;
#pragma unroll
      for (int e = 0; e < NI; ++e) {
        S[e] = fmaf(fs[p][ig * NI + e], S[e], ws[p][ig * NI + e] * vv);
        acc = fmaf(qs[p][ig * NI + e], S[e], acc);
      }
      acc = group16_sum(acc);
      if (ig == 0) os[p][t >> 4] = acc;
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

}  // namespace iron

using namespace iron;

extern "C" int iron_hgrn2(const void* x, const uint16_t* f_bias, const uint16_t* lower, float* state, const int* spans, float* o, int slots, int rows,
                          int stride, int heads, int dim, int vdim, int is_float, void* stream) {
  IRON_REQUIRE(x && f_bias && lower && state && o, "hgrn2: null operand");
  IRON_REQUIRE(spans && ((uintptr_t)spans & 15) == 0, "hgrn2: spans must be there and 16-byte aligned");
  IRON_REQUIRE(slots > 0 && slots <= 65535 && rows > 0, "hgrn2: slots (%d) and rows (%d) must be positive", slots, rows);
  IRON_REQUIRE(heads > 0 && heads <= 65535 && dim > 0 && dim <= 256 && vdim > 0, "hgrn2: heads (%d) and vdim (%d) positive, dim (%d) from 1 to 256",
               heads, vdim, dim);
  IRON_REQUIRE(stride >= heads * (2 * dim + vdim), "hgrn2: a row of %d holds no q, f and v of %d heads", stride, heads);
  const dim3 grid((vdim + FADE_COLUMNS - 1) / FADE_COLUMNS, heads, slots);
  const FadeGates g{f_bias, lower};
#define IRON_HGRN2(T, NI) \
  hipLaunchKernelGGL((hgrn2_kernel<T, NI>), grid, dim3(256), 0, (hipStream_t)stream, (const T*)x, g, state, spans, o, rows, stride, heads, dim, vdim)
#define IRON_HGRN2S(T)                        \
  {                                           \
    if (dim <= 16) IRON_HGRN2(T, 1);          \
    else if (dim <= 32) IRON_HGRN2(T, 2);     \
    else if (dim <= 64) IRON_HGRN2(T, 4);     \
    else if (dim <= 128) IRON_HGRN2(T, 8);    \
    else IRON_HGRN2(T, 16);                   \
  }
  if (is_float) IRON_HGRN2S(float)
  else IRON_HGRN2S(bf16_t)
#undef IRON_HGRN2S
#undef IRON_HGRN2
  IRON_LAUNCH_CHECK();
}
