// C = A B^T for a few rows of A (a batch's decode step): bound by streaming B, (N, K), once.
//
// A block takes 16 rows of B -- the 16x16x32 MFMA's first operand -- and its eight waves deal K in pieces
// of 64 columns (a whole 128-byte line of each row), all of A's rows (up to 16 * MT) the second operand.
// The waves' sums meet in LDS.  With GATED a second matrix is streamed beside the first and the output is
// act(A B^T) * (A B2^T), rounded where the separate steps round.
#include "../../include/iron_hip.h"
#include "common.h"

namespace iron {

constexpr int FEW_WAVES = 8, FEW_STEP = 64;   // K columns a wave takes at a time

// MODE: one tile of 16 rows of B a block, two of them (a tall B), or one of each of two matrices.
enum { FEW_ONE = 0, FEW_TWO = 1, FEW_GATED = 2 };
template <int MT, int MODE>
__global__ __launch_bounds__(FEW_WAVES * 64) void gemm_few_kernel(const bf16_t* __restrict__ A, const bf16_t* __restrict__ B,
                                                                  const bf16_t* __restrict__ B2, bf16_t* __restrict__ C, int M,
                                                                  int N, int K, int activation) {
  constexpr int MATS = MODE == FEW_ONE ? 1 : 2, DEPTH = MT == 1 ? 4 : (MT == 2 ? 2 : 1);
  constexpr bool GATED = MODE == FEW_GATED;
  __shared__ float4 part[FEW_WAVES][MATS][MT][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, quad = lane >> 4;
  const int n0 = blockIdx.x * (MODE == FEW_TWO ? 32 : 16), steps = (K + FEW_WAVES * FEW_STEP - 1) / (FEW_WAVES * FEW_STEP);
  // Bounded buffers: a piece past K reads as zeros (of a row's own end, whatever follows it meets zeros of A).
  const __amdgpu_buffer_rsrc_t ab = bounded_bytes(A, M * K * 2);
  const size_t row = (size_t)min(n0 + l16, N - 1) * K;
  const bf16_t* w[MATS] = {B + row};
  if (MODE != FEW_ONE) w[MATS - 1] = GATED ? B2 + row : B + (size_t)min(n0 + 16 + l16, N - 1) * K;
  int a_row[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) a_row[m] = min(m * 16 + l16, M - 1) * K * 2;
  f32x4 acc[MATS][MT];
#pragma unroll
  for (int x = 0; x < MATS; ++x)
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[x][m] = f32x4{0.f, 0.f, 0.f, 0.f};
  struct Piece {
    u32x4 b[MATS][2], a[MT][2];
  } held[DEPTH];
  auto fetch = [&](Piece& p, int step) {
    // (a lane takes 32 consecutive bytes of its row: which of the 64 columns meet in which product is free)
    const int k = (step * FEW_WAVES + wave) * FEW_STEP + quad * 16;
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      const int kh = k + h * 8, in = min(kh, K - 8);   // past K: B's last piece, against zeros of A
#pragma unroll
      for (int x = 0; x < MATS; ++x) p.b[x][h] = *reinterpret_cast<const u32x4*>(w[x] + in);
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        // A row past the last reads the last again (its results are not stored).
        const int past = (K - 1 - kh) >> 31 & 0x40000000;   // past K: outside the buffer
        p.a[m][h] = __builtin_amdgcn_raw_buffer_load_b128(ab, a_row[m] + 2 * kh + past, 0, 0);
      }
    }
  };
#pragma unroll
  for (int d = 0; d < DEPTH; ++d) {
    fetch(held[d], d);
    __builtin_amdgcn_sched_barrier(0);
  }
  auto add = [&](const Piece& p) {
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int x = 0; x < MATS; ++x)
#pragma unroll
        for (int m = 0; m < MT; ++m)
          acc[x][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, p.b[x][h]), __builtin_bit_cast(bf16x8, p.a[m][h]), acc[x][m], 0, 0, 0);
  };
  for (int s = 0; s + DEPTH < steps; s += DEPTH) {   // (a step past the last adds zeros)
#pragma unroll
    for (int d = 0; d < DEPTH; ++d) {
      add(held[d]);
      fetch(held[d], s + d + DEPTH);
      __builtin_amdgcn_sched_barrier(0);
    }
  }
#pragma unroll
  for (int d = 0; d < DEPTH; ++d) add(held[d]);
#pragma unroll
  for (int x = 0; x < MATS; ++x)
#pragma unroll
    for (int m = 0; m < MT; ++m) part[wave][x][m][lane] = make_float4(acc[x][m][0], acc[x][m][1], acc[x][m][2], acc[x][m][3]);
  __syncthreads();
  // Lane (quad, l16) of a tile: columns n0 + quad * 4 .. + 3 of row m * 16 + l16.
  for (int e = threadIdx.x; e < MT * 64; e += FEW_WAVES * 64) {
    const int m = e >> 6, l = e & 63, r = m * 16 + (l & 15), n = n0 + (l >> 4) * 4;
    if (r >= M) continue;
    float v[MATS][4];
#pragma unroll
    for (int x = 0; x < MATS; ++x) {
      float4 sum = part[0][x][m][l];
#pragma unroll
      for (int q = 1; q < FEW_WAVES; ++q) {
        const float4 o = part[q][x][m][l];
        sum.x += o.x; sum.y += o.y; sum.z += o.z; sum.w += o.w;
      }
      v[x][0] = sum.x; v[x][1] = sum.y; v[x][2] = sum.z; v[x][3] = sum.w;
    }
    if (GATED) {
#pragma unroll
      for (int j = 0; j < 4; ++j) v[0][j] = round_bf16(gate_of(activation, round_bf16(v[0][j]))) * round_bf16(v[MATS - 1][j]);
    }
    bf16_t* to = C + (size_t)r * N + n;
#pragma unroll
    for (int x = 0; x < (MODE == FEW_TWO ? 2 : 1); ++x)
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (n + 16 * x + j < N) to[16 * x + j] = f32_to_bf16(v[x][j]);
  }
}

template <int MODE>
static int launch_gemm_few(const bf16_t* A, const bf16_t* B, const bf16_t* B2, bf16_t* C, int M, int N, int K, int activation, hipStream_t s) {
  const int per = MODE == FEW_TWO ? 32 : 16;
  const dim3 grid((N + per - 1) / per);
#define IRON_FEW(MT) \
  hipLaunchKernelGGL((gemm_few_kernel<MT, MODE>), grid, dim3(FEW_WAVES * 64), 0, s, A, B, B2, C, M, N, K, activation)
  if (M <= 16) IRON_FEW(1);
  else if (M <= 32) IRON_FEW(2);
  else IRON_FEW(4);
#undef IRON_FEW
  IRON_LAUNCH_CHECK();
}

}  // namespace iron

using namespace iron;

extern "C" int iron_gemm_few_bf16(const uint16_t* A, const uint16_t* B, const uint16_t* B2, uint16_t* C, int M, int N, int K,
                                  int activation, void* stream) {
  IRON_REQUIRE(A && B && C, "gemm_few: null operand");
  IRON_REQUIRE(M > 0 && M <= 64 && N > 0, "gemm_few: M (%d) from 1 to 64, N (%d) positive", M, N);
  IRON_REQUIRE(K >= 8 && K % 8 == 0 && K <= (1 << 22), "gemm_few: K (%d) is a positive multiple of 8 up to 2^22", K);
  IRON_REQUIRE((((uintptr_t)A | (uintptr_t)B | (uintptr_t)B2) & 15) == 0, "gemm_few: operands must be 16-byte aligned");
  IRON_REQUIRE(B2 == nullptr || (activation >= 1 && activation <= 3), "gemm_few: activation (%d) is 1 (SiLU), 2 (GELU, tanh form) or 3 (ReLU)",
               activation);
  hipStream_t s = (hipStream_t)stream;
  if (B2 != nullptr) return launch_gemm_few<FEW_GATED>(A, B, B2, C, M, N, K, activation, s);
  if (N >= 8192) return launch_gemm_few<FEW_TWO>(A, B, nullptr, C, M, N, K, 0, s);
  return launch_gemm_few<FEW_ONE>(A, B, nullptr, C, M, N, K, 0, s);
}
