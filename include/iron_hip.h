/* libiron_hip.so -- C ABI of the hand-written gfx950 (MI355X) kernels behind the
 * IRON operator hot path.
 *
 * Every entry point: plain pointers and sizes, all data pointers are DEVICE
 * pointers owned by the caller, bf16 is 16-bit storage (uint16_t), one HIP
 * stream is passed in (void* = hipStream_t, NULL = the default stream).  No
 * entry point allocates, frees or synchronizes, so each may be recorded into a
 * HIP graph.  Return value: 0 = launched, 1 = arguments refused (the text is
 * in iron_last_error()), any other value = the hipError_t the launch raised.
 *
 * "const int* valid"-style arguments are per-call bounds read on the device at
 * run time (the reference's per-call scratchpad words,
 * iron/common/image/packaging.py:20); NULL means the whole extent.
 *
 * Citations are into the reference tree (amd/IRON).
 */
#ifndef IRON_HIP_H
#define IRON_HIP_H

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

/* Library version (major*10000 + minor*100 + patch). */
int iron_version(void);
/* Text of the last refusal on this thread ("" if none). */
const char* iron_last_error(void);

/* C = A @ B, f32 accumulation, one rounding to bf16.
 * A (M,K) row-major.  B (K,N) row-major, or (N,K) row-major if b_col_maj.
 * C (M,N) row-major, or (N,M) if c_col_maj.  K % 8 == 0.
 * valid: rows of A computed (others of C untouched); valid_k: K actually summed.
 * Replaces GEMM.build()/kernels.linalg.mm: iron/operators/gemm.py:143,397-410,696-702. */
int iron_gemm_bf16(const uint16_t* A, const uint16_t* B, uint16_t* C, int M, int N, int K,
                   int b_col_maj, int c_col_maj, const int* valid, const int* valid_k,
                   void* stream);

/* y[b] = W[b / repeat] @ x[b] for b in [0, batches): W (batches/repeat, M, K), x (batches, K),
 * y (batches, M); f32 accumulation, one rounding.  K % 8 == 0.
 * valid: rows of W computed.
 * Replaces GEMV.build()/linalg.mv: iron/operators/gemv.py:79,267-275,408-417. */
int iron_gemv_bf16(const uint16_t* W, const uint16_t* x, uint16_t* y, int M, int K, int batches,
                   int repeat, const int* valid, void* stream);
/* The same with the launch shape forced (rows a wave takes, waves splitting K); 0 = heuristic. */
int iron_gemv_bf16_tuned(const uint16_t* W, const uint16_t* x, uint16_t* y, int M, int K,
                         int batches, int repeat, const int* valid, int rows_per_wave,
                         int k_split, void* stream);

/* C = bf16(residual_scale * bf16(A B^T) + R) for the rows under *valid (or M): a projection over many
 * rows with its residual (a scale of 1: the plain sum; another: AXPY's) in the product's epilogue.
 * A (M,K), B (N,K), R and C (M,N); K % 64 == 0, M, N >= 64.  C may be R.
 * Replaces GEMM followed by ElementwiseAdd / AXPY (iron/lm/blocks.py:386-391,723-733), rounding
 * where they round. */
int iron_gemm_residual_bf16(const uint16_t* A, const uint16_t* B, const uint16_t* R, uint16_t* C, int M,
                            int N, int K, float residual_scale, const int* valid, void* stream);

/* The same product and sum for few rows over a long K, and the RMSNorm of the rows it leaves:
 * C = bf16(residual_scale * bf16(A B^T) + R), Y = RMSNorm(C) * gain as iron_rmsnorm_bf16 computes it
 * (Y is bit for bit what that call makes of C), for the rows under *valid (or M), in two launches.
 * While the bound leaves 128 x 128 tiles for no more than half the chip (512 live rows of a 2048-row
 * prompt chunk at N = 2048), each tile's K is dealt over 4 or 2 blocks that leave float32 sums in
 * `workspace`, and the second launch adds a row's slices in slice order before it rounds: the sums
 * are the same whatever ran first, and differ from iron_gemm_residual_bf16's in the last bits of the
 * float32 sum only.  A (M,K), B (N,K), R and C (M,N), gain (N), Y (M,N); C may be R, Y neither.
 * iron_gemm_residual_norm_workspace_bytes(M, N, K): the workspace's size (any contents), 0 for a
 * shape this entry refuses (M < 128, N not a multiple of 128 up to 8192, K under 4096 or not a
 * multiple of 256).
 * Replaces GEMM (down_proj), ElementwiseAdd / AXPY and the next RMSNorm
 * (iron/lm/blocks.py:723-733, then :688 of the next layer or the final norm). */
int64_t iron_gemm_residual_norm_workspace_bytes(int M, int N, int K);
int iron_gemm_residual_norm_bf16(const uint16_t* A, const uint16_t* B, const uint16_t* R,
                                 const uint16_t* gain, uint16_t* C, uint16_t* Y, int M, int N, int K,
                                 float residual_scale, float eps, const int* valid, void* workspace,
                                 void* stream);

/* C = bf16(bf16(act(G)) * bf16(A B^T)) for the rows under *valid (or M): a gated feed-forward's second
 * projection with the activated gate in its epilogue; activation 1: SiLU, 2: GELU by its tanh form.
 * A (M,K), B (N,K), G and C (M,N); K % 64 == 0, M, N >= 64.  C may be G.
 * Replaces GEMM (up_proj), SiLU or GELU (of gate_proj's product G) and ElementwiseMul
 * (iron/lm/blocks.py:688,697-699), rounding where they round. */
int iron_gemm_gated_bf16(const uint16_t* A, const uint16_t* B, const uint16_t* G, uint16_t* C, int M,
                         int N, int K, int activation, const int* valid, void* stream);
/* Both first projections of a gated feed-forward and the gate in one launch:
 * G = bf16(A Bg^T), C = bf16(bf16(act(G)) * bf16(A Bu^T)) for the rows under *valid (or M) -- what
 * iron_gemm_bf16 (gate_proj) followed by iron_gemm_gated_bf16 (up_proj) compute, bit for bit; a block
 * reads back only the tile of G it wrote itself.  A (M,K); Bg, Bu (N,K); G, C (M,N), distinct.
 * Replaces GEMM, GEMM, SiLU or GELU, ElementwiseMul (iron/lm/blocks.py:688,697-699). */
int iron_gemm_gated_pair_bf16(const uint16_t* A, const uint16_t* Bg, const uint16_t* Bu, uint16_t* G,
                              uint16_t* C, int M, int N, int K, int activation, const int* valid,
                              void* stream);

/* One-row fusions of a decoder layer (no single counterpart in the reference: each replaces a run
 * of its steps, iron/lm/blocks.py:627-648,697-699,723-733, and rounds where those steps round).
 *   y = E(W @ N(x)):  N = RMSNorm(x, eps) * norm_w when norm_w is not NULL (else x itself);
 *   epilogue 0: y = bf16(W N(x));  1: y = bf16(residual_scale * bf16(W N(x)) + residual), one fused
 *   multiply-add (a scale of 1 is the plain sum; another is AXPY's, iron/lm/blocks.py:386-391);
 *   2: y = bf16(bf16(silu(bf16(W N(x)))) * bf16(W2 N(x)))   (gate, up -> SiLU -> Mul);
 *   3: the same with GELU by its tanh form for SiLU (Gemma's feed-forward);
 *   4: y = bf16(bf16(gelu_tanh(bf16(W N(x)))) * residual), 5: the same with SiLU: a projection, its
 *   activation and the product with a given row (`residual` holds it; Gemma 4's per-layer input gate,
 *   iron/lm/blocks.py:793-796; norm_w must be NULL).
 * W, W2 (M,K); x, norm_w (K); residual, y (M).  K % 8 == 0. */
int iron_gemv_fused_bf16(const uint16_t* W, const uint16_t* W2, const uint16_t* x,
                         const uint16_t* norm_w, float eps, const uint16_t* residual,
                         float residual_scale, uint16_t* y, int M, int K, int epilogue, void* stream);

/* Attention's first half for one token: n = RMSNorm(x) * norm_w; q = Wq n, k = Wk n, v = Wv n
 * (each rounded to bf16); q and k rotated by the RoPE row `angles` (d bf16, cos/sin interleaved,
 * two halves); q -> q_out (heads*d), k -> keys[*position], v -> values[*position], caches
 * (cache_rows, kv_heads, d).  With angle_row not NULL, `angles` is a whole RoPE table of angle_rows
 * rows and the row is angles[*angle_row] (held inside the table): the step's copy of its table row
 * (iron/lm/blocks.py:394-431) then needs no launch of its own.  Replaces RMSNorm, 3 GEMV, 2 RoPE and
 * 2 Copy steps (iron/lm/blocks.py:472-502,627-648). */
int iron_decode_qkv_bf16(const uint16_t* x, const uint16_t* norm_w, float eps, const uint16_t* Wq,
                         const uint16_t* Wk, const uint16_t* Wv, const uint16_t* angles,
                         uint16_t* q_out, uint16_t* keys, uint16_t* values, int hidden, int heads,
                         int kv_heads, int d, int cache_rows, const int* position, const int* angle_row,
                         int angle_rows, void* stream);
/* The same for a decoder's first layer, whose input is the token's row of the embedding table
 * (table_rows, hidden): the row is read at table[*token] (held inside the table), and also written to
 * x (hidden), which the layer's residual sum reads -- the step's embedding lookup
 * (iron/lm/blocks.py:349-383, iron/lm/causal.py:292-299) then needs no launch of its own. */
int iron_decode_qkv_embed_bf16(const uint16_t* table, const int* token, int table_rows, uint16_t* x,
                               const uint16_t* norm_w, float eps, const uint16_t* Wq, const uint16_t* Wk,
                               const uint16_t* Wv, const uint16_t* angles, uint16_t* q_out, uint16_t* keys,
                               uint16_t* values, int hidden, int heads, int kv_heads, int d, int cache_rows,
                               const int* position, const int* angle_row, int angle_rows, void* stream);

/* Between a token's q/k/v projections and its attention where the heads are normed one by one
 * (Gemma's): RMSNorm of each q head (bit 0 of norms; gain q_gain or none), k head (bit 1; k_gain) and v
 * head (bit 2; no gain), RoPE on q and k by the call's angle rows (q_angles, k_angles: `rotary`
 * columns, cos/sin interleaved; the columns of a head past them pass through; NULL: not rotated), q ->
 * q_out (heads, d), k -> keys[*row0] and v -> values[*row0], caches (cache_rows, kv_heads, d), and
 * again at [*row1] where row1 is not NULL (a ring cache's mirror row).  k, v NULL: the layer reads
 * another layer's cache and only q is done.  Each step computed as its own kernel computes it.
 * Replaces up to 3 RMSNorm, 2 RoPE and 4 Copy steps (iron/lm/blocks.py:563-660,434-529). */
int iron_decode_heads_bf16(const uint16_t* q, const uint16_t* k, const uint16_t* v, const uint16_t* q_gain,
                           const uint16_t* k_gain, int norms, float eps, const uint16_t* q_angles,
                           const uint16_t* k_angles, int rotary, int two_halves, uint16_t* q_out,
                           uint16_t* keys, uint16_t* values, const int* row0, const int* row1,
                           int cache_rows, int heads, int kv_heads, int d, void* stream);

/* A prompt chunk's three projections and the rotation of q and k in one launch (no single
 * counterpart in the reference: replaces 3 GEMM and 2 RoPE steps, iron/lm/blocks.py:617-648, and
 * rounds where those steps round): q = x Wq^T, k = x Wk^T, v = x Wv^T, each rounded to bf16; q and k
 * then turned by RoPE (two halves) with row r's angles `angles[r]` (rows, 64; cos and sin interleaved)
 * and rounded again.  x (rows, hidden); Wq (heads*d, hidden), Wk, Wv (kv_heads*d, hidden);
 * q_out (rows, heads*d), k_out, v_out (rows, kv_heads*d).  d == 64; heads, kv_heads even;
 * hidden % 64 == 0; rows >= 64.  valid: rows computed. */
int iron_prefill_qkv_bf16(const uint16_t* x, const uint16_t* Wq, const uint16_t* Wk,
                          const uint16_t* Wv, const uint16_t* angles, uint16_t* q_out,
                          uint16_t* k_out, uint16_t* v_out, int rows, int hidden, int heads,
                          int kv_heads, int d, const int* valid, void* stream);
/* The same with k and v written straight into the chunk's rows of the layer's KV caches, rows
 * *start on of keys and values (cache_rows, kv_heads*d): replaces the two Copy steps that follow as
 * well (iron/lm/blocks.py:472-486).  The first row is held where the rows under the bound end inside
 * the cache; rows <= cache_rows. */
int iron_prefill_qkv_cache_bf16(const uint16_t* x, const uint16_t* Wq, const uint16_t* Wk,
                                const uint16_t* Wv, const uint16_t* angles, uint16_t* q_out,
                                uint16_t* keys, uint16_t* values, int rows, int hidden, int heads,
                                int kv_heads, int d, int cache_rows, const int* start,
                                const int* valid, void* stream);

/* y = bf16(bf16(x * rsqrt(mean(x^2) + eps)) * w) per row; w NULL = unweighted (one rounding).
 * x,y (rows, cols); w (cols).  cols % 8 == 0.  valid: rows computed.
 * Replaces norm.rms_norm_eps + eltwise.mul_sized: iron/operators/rms_norm.py:10,
 * iron/common/elementwise.py:619-682. */
int iron_rmsnorm_bf16(const uint16_t* x, const uint16_t* w, uint16_t* y, int rows, int cols,
                      float eps, const int* valid, void* stream);
/* y = bf16(residual + the row above): a block's output normed again before its residual, the
 * sandwich layer's RMSNorm and ElementwiseAdd in one pass (iron/lm/blocks.py:748-767), rounding
 * where the two steps round.  residual (rows, cols); y may be residual. */
int iron_rmsnorm_add_bf16(const uint16_t* x, const uint16_t* w, const uint16_t* residual, uint16_t* y,
                          int rows, int cols, float eps, const int* valid, void* stream);

/* Rotary embedding of x (rows, cols) by the packed table angles (angle_rows, cols), cos and
 * sin interleaved; row r uses angle row r / (rows / angle_rows).  two_halves: rotate the two
 * halves of a row (else interleaved pairs).  cols % 16 == 0.  valid: rows computed.
 * Replaces datamovement.rope: iron/operators/rope.py:58,161-184. */
int iron_rope_bf16(const uint16_t* x, const uint16_t* angles, uint16_t* y, int rows, int cols,
                   int angle_rows, int two_halves, const int* valid, void* stream);

/* The same over the first rotary_cols columns of rows row_cols wide (angles (angle_rows, rotary_cols));
 * the columns past them are copied as they are.  (row_cols - rotary_cols) % 8 == 0.  A decoder whose
 * RoPE covers part of each head: one launch for the reference's copy out, rotation and copy back
 * (Attention.rotate, iron/lm/blocks.py:612-620). */
int iron_rope_partial_bf16(const uint16_t* x, const uint16_t* angles, uint16_t* y, int rows, int row_cols,
                           int rotary_cols, int angle_rows, int two_halves, const int* valid, void* stream);

/* Elementwise over n elements (valid: elements computed), f32 math, one rounding each:
 *   silu: y = x*sigmoid(x)   mul: y = a*b   add: y = a+b
 *   silu_mul: y = bf16(bf16(silu(g)) * u)  -- SiLU then ElementwiseMul, rounded between,
 * as two reference steps are.
 * Replaces activation.silu / eltwise.mul_sized / eltwise.add_sized:
 * iron/operators/silu.py:12, elementwise_mul.py:11, elementwise_add.py:11,
 * iron/common/elementwise.py:255-285. */
int iron_silu_bf16(const uint16_t* x, uint16_t* y, int64_t n, const int* valid, void* stream);
int iron_mul_bf16(const uint16_t* a, const uint16_t* b, uint16_t* y, int64_t n, const int* valid,
                  void* stream);
int iron_add_bf16(const uint16_t* a, const uint16_t* b, uint16_t* y, int64_t n, const int* valid,
                  void* stream);
int iron_silu_mul_bf16(const uint16_t* g, const uint16_t* u, uint16_t* y, int64_t n,
                       const int* valid, void* stream);

/* y[r] = bf16(x[r] + row) (or x[r] * row if multiply) for r < *valid (or rows): one row met by
 * every row, f32 math, one rounding.  x,y (rows, cols); row (cols).  cols % 8 == 0.
 * Replaces RowwiseAdd (a projection's bias) / RowwiseMul: iron/operators/elementwise_add.py:18,
 * elementwise_mul.py:18, iron/common/elementwise.py:797-867. */
int iron_row_broadcast_bf16(const uint16_t* x, const uint16_t* row, uint16_t* y, int rows, int cols,
                            int multiply, const int* valid, void* stream);

/* y[i] = bf16(f(x[i])) for i < *valid (or n), f32 math, one rounding; kind names f:
 * GELU by its tanh approximation or exact (x Phi(x)), ReLU, sigmoid, tanh, or the clamp to
 * [p0, p1] (p0, p1 are read by the clamp alone; the caller rounds them to bf16).
 * Replaces GELU / ReLU / Sigmoid / Tanh / Clamp: iron/operators/gelu.py:13, relu.py:11,
 * sigmoid.py:9, tanh.py:9, clamp.py:14 (each a UnaryElementwise, iron/common/elementwise.py:494). */
#define IRON_UNARY_GELU_TANH 0
#define IRON_UNARY_GELU_ERF 1
#define IRON_UNARY_RELU 2
#define IRON_UNARY_SIGMOID 3
#define IRON_UNARY_TANH 4
#define IRON_UNARY_CLAMP 5
int iron_unary_bf16(const uint16_t* x, uint16_t* y, int64_t n, int kind, float p0, float p1,
                    const int* valid, void* stream);

/* out[i] = bf16(a * x[i] + y[i]) for i < *valid (or n): one fused multiply-add in f32.
 * Replaces AXPY: iron/operators/axpy.py:13. */
int iron_axpy_bf16(const uint16_t* x, const uint16_t* y, uint16_t* out, int64_t n, float a,
                   const int* valid, void* stream);

/* y[r] = bf16((x[r] - mean) / sqrt(var + eps)) per row r < *valid (or rows), mean and the
 * variance about it in f32 (beta 0); with w, that row times w rounded again, as RMSNorm.
 * x,y (rows, cols); w (cols) or NULL.  cols % 8 == 0.
 * Replaces LayerNorm: iron/operators/layer_norm.py:10 over iron/common/elementwise.py:676-682. */
int iron_layernorm_bf16(const uint16_t* x, const uint16_t* w, uint16_t* y, int rows, int cols,
                        float eps, const int* valid, void* stream);

/* y[r, c] = softmax over the first *length (or cols) columns of row r, 0 in the columns past them:
 * z = x + addend (addend float32 or NULL), capped as soft_cap * tanh(z / soft_cap) when
 * soft_cap > 0, exp(z - max) / sum in f32, one rounding.  x (rows, cols) bf16, or float32 when
 * x_is_f32; y (rows, cols) bf16.  cols % 8 == 0.
 * Replaces Softmax without its band (window, period): iron/operators/softmax.py:62,523-545. */
int iron_softmax_bf16(const void* x, int x_is_f32, const float* addend, uint16_t* y, int rows,
                      int cols, float soft_cap, const int* length, void* stream);

/* Attention, many queries (prefill / prompt chunk).  Q,O: (seq, heads, d) if q_interleaved
 * else (heads, seq, d); K,V: (kv_len, kv_heads, d) if kv_interleaved else (kv_heads, kv_len, d).
 * The queries are the last rows of the keys: query i sits at position kv_tokens - q_tokens + i,
 * q_tokens = *valid (or seq_len), kv_tokens = *kv_valid (or kv_len - seq + q_tokens).
 * causal masks key > position; window >= 0 also masks key < position - window (and, when not
 * causal, key > position + window); window < 0 = none.  Rows >= q_tokens of O are zeros.
 * d in {64, 128, 256, 512} (MFMA tiles throughout: 32 queries a wave on 32x32x16 tiles at 64 and
 * 128, groups of 16 on 16x16x32 tiles at 256 and 512); heads % kv_heads == 0.
 * Replaces kernels.linalg.mha + partial_softmax + matmul_PV:
 * iron/operators/mha.py:191,574-667,1073-1116. */
int iron_mha_prefill_bf16(const uint16_t* Q, const uint16_t* K, const uint16_t* V, uint16_t* O,
                          int heads, int kv_heads, int d, int seq, int seq_len, int kv_len,
                          float scale, int causal, int window, int q_interleaved,
                          int kv_interleaved, const int* valid, const int* kv_valid, void* stream);
/* The same over a window of a longer buffer of keys: K, V (kv_rows, kv_heads, d), of which the kv_len
 * rows from *kv_first on are the keys (the first row is held where they end inside the buffer).  What
 * a sliding-window layer's ring cache needs (iron/lm/blocks.py:504-529: the reference copies the
 * window into a staging tensor first; here attention reads it where it lies). */
int iron_mha_prefill_at_bf16(const uint16_t* Q, const uint16_t* K, const uint16_t* V, uint16_t* O,
                             int heads, int kv_heads, int d, int seq, int seq_len, int kv_len,
                             float scale, int causal, int window, int q_interleaved, const int* valid,
                             const int* kv_valid, const int* kv_first, int kv_rows, void* stream);

/* Attention, one query (decode; the reference's "packed" MHA, seq_len == 1).
 * Q,O: (heads, d).  K,V as above.  kv_tokens = *kv_valid (or kv_len); the query sits at
 * kv_tokens - 1.  workspace: iron_mha_decode_workspace_bytes(heads, d) bytes of device memory.
 * Q, K, V, O and workspace 16-byte aligned.
 * d in {64, 128} with up to 16 query heads a KV head, d = 256 with 1, 2, 3, 4, 5, 6 or 8, or d = 512
 * with any.  The launches depend on (heads, kv_heads, d) and on whether kv_len can pass 2048 rows;
 * what they read, and how the keys are dealt over the chip, follow *kv_valid (a cache's length only
 * sizes the buffers: the reference's "attention over a cache costs the context, not the cache",
 * iron/operators/mha.py:275-278).
 * Replaces the packed single-query MHA: iron/operators/mha.py:476-477,1073-1116. */
int iron_mha_decode_bf16(const uint16_t* Q, const uint16_t* K, const uint16_t* V, uint16_t* O,
                         int heads, int kv_heads, int d, int kv_len, float scale, int window,
                         int kv_interleaved, const int* kv_valid, void* workspace, void* stream);
int64_t iron_mha_decode_workspace_bytes(int heads, int d);
/* The same with the kernel form forced, for tests and measurements (as iron_gemv_bf16_tuned):
 * form 0 the default choice, 1 the lane-per-column scans, 2 the matrix-core scan (d = 64 or 128);
 * short_keys > 0: the live-key count up to which the matrix-core scan's one block a KV head writes
 * the output itself (beyond it the keys are dealt over every CU and a second launch merges). */
int iron_mha_decode_tuned_bf16(const uint16_t* Q, const uint16_t* K, const uint16_t* V, uint16_t* O,
                               int heads, int kv_heads, int d, int kv_len, float scale, int window,
                               int kv_interleaved, const int* kv_valid, void* workspace, int form,
                               int short_keys, void* stream);
/* iron_mha_decode_bf16 for callers that cannot allocate (code under HIP-graph capture, tight
 * serving loops, harnesses that forbid hipMalloc): the same kernels, their split-KV partial results
 * in a scratch array the library holds in device memory itself (iron_mha_decode_static_max_bytes()
 * bytes on each GPU it runs on, until the process ends), so no workspace is passed and nothing is
 * allocated or freed.  Refused (1) when iron_mha_decode_workspace_bytes(heads, d) exceeds that size.
 * Every call on a GPU shares that GPU's array: calls that overlap on one GPU race.  Nothing in it
 * has to start at zero.  The first call on a device asks the runtime for the array's address there
 * (hipGetSymbolAddress, which may load the code object): make one call per device outside any stream
 * capture before recording calls into a graph.  No counterpart in the reference. */
int iron_mha_decode_static_bf16(const uint16_t* Q, const uint16_t* K, const uint16_t* V, uint16_t* O,
                                int heads, int kv_heads, int d, int kv_len, float scale, int window,
                                int kv_interleaved, const int* kv_valid, void* stream);
int64_t iron_mha_decode_static_max_bytes(void);
/* One query over a window of a longer buffer of keys, as iron_mha_prefill_at_bf16. */
int iron_mha_decode_at_bf16(const uint16_t* Q, const uint16_t* K, const uint16_t* V, uint16_t* O,
                            int heads, int kv_heads, int d, int kv_len, float scale, int window,
                            const int* kv_valid, const int* kv_first, int kv_rows, void* workspace,
                            void* stream);

/* out[i] = table[ids[i]] for i < *valid (or n_ids); rows of row_bytes bytes (multiple of 4).
 * ids outside [0, table_rows) are skipped (the row is left untouched).
 * Replaces Copy's gather (embedding lookup): iron/operators/copy.py:72,546,839-902. */
int iron_gather_rows(const void* table, const int* ids, void* out, int n_ids, int table_rows,
                     int64_t row_bytes, const int* valid, void* stream);

/* dst[(*dst_row + i)] = src[(*src_row + i)] for i < *valid (or rows); NULL row index = 0.
 * Rows are row_bytes bytes (multiple of 4) at src_stride/dst_stride bytes apart; rows that
 * would land outside [0, src_rows) / [0, dst_rows) are skipped.
 * Replaces Copy between views with per-call offsets (KV-cache write, RoPE-table row,
 * last-row pick): iron/operators/copy.py:546,839-902. */
int iron_copy_rows(const void* src, void* dst, int rows, int64_t row_bytes, int64_t src_stride,
                   int64_t dst_stride, int src_rows, int dst_rows, const int* src_row,
                   const int* dst_row, const int* valid, void* stream);

/* Greedy draw: *token = index of the first largest logit among logits[0..n); when record is
 * not NULL also record[*at] = token (at NULL = 0; skipped if outside [0, record_len)), and when
 * token_copy is not NULL *token_copy = token (the carried `token` word of a decode loop: the draw
 * feeds the next step without a copy kernel between).
 * Replaces Sample with an all-zero draw row: iron/operators/sample.py:72-79,106,324-333. */
int iron_argmax_bf16(const uint16_t* logits, int n, int* token, int* record, int record_len,
                     const int* at, int* token_copy, void* stream);

/* The draw of one draw row: draws[*row .. *row+4) = {temperature as float32 bits, top-k, the low
 * and the high word of a 53-bit number} (row NULL = 0; draws NULL, a row outside
 * [0, draws_words) or a temperature that is not positive = the greedy draw above).  With a
 * temperature the candidates are the min(top-k, k_max) largest of logits[0..n), equals to the
 * lower index; candidate i weighs exp((l_i - l_0) / temperature) in float64 and the token is the
 * first whose running weight exceeds number * 2^-53 * total.  token, record, at, token_copy as
 * iron_argmax_bf16.  1 <= k_max <= 64; n <= 524288.  workspace: iron_sample_workspace_bytes(n)
 * bytes, 8-byte aligned (NULL allowed for n <= 2048); its first 16 bytes count the launch's blocks:
 * zero before the workspace's first launch, left zero by every launch; the rest may hold anything.
 * One launch; launches that share a workspace must not overlap.
 * Replaces Sample: iron/operators/sample.py:72-79,106-336 (its sample_ref is out of the
 * reference's tree; the arithmetic above is this library's own, fixed so a host computes the
 * same token bit for bit). */
int64_t iron_sample_workspace_bytes(int n);
int iron_sample_bf16(const uint16_t* logits, int n, const int* draws, int draws_words,
                     const int* row, int k_max, void* workspace, int* token, int* record,
                     int record_len, const int* at, int* token_copy, void* stream);

/* iron_sample_bf16 that ends a decode step: after the token is written (to token, record and
 * token_copy), the same launch evaluates the n_exprs word expressions of iron_eval_words over
 * words[0..n_words) -- the carried position and every word derived from it -- so a replayed step needs
 * no launch of its own for them.  Replaces Sample followed by the carry's Emit
 * (iron/operators/sample.py:106, iron/common/graph/carried.py:189-276). */
int iron_sample_advance_bf16(const uint16_t* logits, int n, const int* draws, int draws_words,
                             const int* row, int k_max, void* workspace, int* token, int* record,
                             int record_len, const int* at, int* token_copy, int* words, int n_words,
                             const int* exprs, int n_exprs, void* stream);

/* Evaluate n per-call word expressions in order, on the device, in one thread:
 *   words[e.dst] = (clamp(((words[e.src] * e.mul + e.add) >> e.shift), e.lo, e.hi) & e.mask) + e.post
 * exprs is n records of 9 int32 {dst, src, mul, add, shift, lo, hi, mask, post} in device memory
 * (mask -1 keeps every bit; 2^k - 1 is the remainder a ring of 2^k rows indexes by, post the
 * rows its mirror lies further on).
 * The device-side carry/Emit of a decode loop (position += 1, kv_valid = position + 1):
 * iron/common/graph/carried.py:189-276, iron/operators/emit.py. */
int iron_eval_words(int* words, int n_words, const int* exprs, int n, void* stream);

/* C = A B^T for up to 64 rows of A, or with B2 C = act(A B^T) * (A B2^T) (activation 1 SiLU, 2 GELU by its
 * tanh form, 3 ReLU; rounded where the separate steps round): bound by streaming B.  A (M, K), B and B2
 * (N, K), C (M, N); K % 8 == 0.  What iron_gemm_bf16 and iron_gemm_gated_pair_bf16 launch for fewer than 64
 * rows without a bound (the latter needs no G then). */
int iron_gemm_few_bf16(const uint16_t* A, const uint16_t* B, const uint16_t* B2, uint16_t* C, int M, int N, int K,
                       int activation, void* stream);

/* ---- decoders with a float32 residual stream and layers that carry a state, over a batch of rows.
 *
 * `spans` is an int32 (slots, 4) table in device memory, 16-byte aligned: {row0, rows, start, unused}
 * says that rows row0 .. row0 + rows - 1 of the batch are one sequence's tokens at positions start,
 * start + 1, ...; an idle slot has no rows.  Spans must not overlap.  States are kept a slot; a span
 * that starts at position 0 reads none, so a slot needs no clearing between sequences.
 * `is_float`: void* activations are float instead of bf16 (a model that runs in 32 bits throughout). */

/* x[i] = scale * table[ids[i]] in float, for i < *valid (or rows); ids outside the table are skipped.  also (may be
 * NULL): the same rows once more. */
int iron_stream_embed(const uint16_t* table, const int* ids, float* x, float* also, int rows, int table_rows, int cols,
                      float scale, const int* valid, void* stream);
/* The stream's rows: with y, x += rmsnorm(y + y_bias) * (unit + back_gain) in place (y_bias may be NULL); with h,
 * h = rmsnorm(x) * (unit + gain) of the rows as they then stand.  Float throughout, h rounded once. */
int iron_stream_rows(float* x, const void* y, const uint16_t* y_bias, const uint16_t* back_gain, const uint16_t* gain, void* h,
                     int rows, int cols, float eps, float unit, int is_float, const int* valid, void* stream);
/* The stream's rows: with y, as above; with planes (index + 1 or more planes of plane_rows rows), the rows as they then
 * stand become plane `index`, and the sum of weights[j] times plane j over j <= index takes their place; with h, h is
 * the rows as they then stand, rounded once. */
int iron_stream_depth_rows(float* x, const void* y, const uint16_t* y_bias, const uint16_t* back_gain, float* planes,
                           const uint16_t* weights, int plane_rows, int index, void* h, int rows, int cols, float eps,
                           float unit, int is_float, const int* valid, void* stream);
/* x += (y + y_bias) * sigmoid(gate + gate_bias) in place, gate columns gate_at .. of rows of gate_stride (y_bias
 * may be NULL); with h, h = rmsnorm(x) * gain of the rows as they then stand.  Float throughout, h rounded once. */
int iron_stream_gated_rows(float* x, const void* y, const uint16_t* y_bias, const void* gate, const uint16_t* gate_bias,
                           int gate_stride, int gate_at, const uint16_t* gain, void* h, int rows, int cols, float eps,
                           int is_float, const int* valid, void* stream);
/* The stream's rows: with y, x += y + y2 in place (y2 may be NULL); with h, each of the `groups` equal parts of a row as it
 * then stands over its own root mean square, times (unit + gain).  Float throughout, h rounded once. */
int iron_stream_groups(float* x, const void* y, const void* y2, const uint16_t* gain, void* h, int rows, int cols, int groups,
                       float eps, float unit, int is_float, const int* valid, void* stream);
/* Columns at .. + cols of y (rows of width) = act(g) * u, g and u the columns gate_at .. and gate_at + cols .. of x (rows of
 * stride).  kind: 0 the limited gate, g' sigmoid(1.702 g') (u' + 1) with g' = min(g, limit), u' = u within [-limit, limit]; 1
 * SiLU, 2 GELU (tanh form), 3 ReLU. */
int iron_gated_columns(const void* x, void* y, int rows, int cols, int stride, int gate_at, int width, int at, int kind,
                       float limit, int is_float, const int* valid, void* stream);
/* y = a N(z) + b N(z^2) + c N(z^3) + e, z columns at .. of x (rows, stride) plus bias (may be NULL), powers element
 * by element, N over a row's root mean square; coefficients {a, b, c, e}.  y (rows, cols); float, rounded once. */
int iron_poly_norm(const void* x, const uint16_t* bias, const uint16_t* coefficients, void* y, int rows, int cols,
                   int stride, int at, float eps, int is_float, const int* valid, void* stream);
/* out[slot] = the last row of the slot's span (left as it is for an idle slot). */
int iron_span_tails(const float* x, const int* spans, float* out, int slots, int rows, int cols, void* stream);
/* y = cap * tanh(scale x / cap) (cap 0: y = scale x) as float, and rounded to bf16 in rows of rounded_stride. */
int iron_softcap(const void* x, float* y, uint16_t* rounded, int rows, int cols, int rounded_stride, float cap,
                 float scale, int is_float, void* stream);
/* y = act(gate) * up in float; activation 1 SiLU, 2 GELU (tanh form), 3 ReLU. */
int iron_act_mul_f32(const float* gate, const float* up, float* y, int rows, int cols, int activation,
                     const int* valid, void* stream);
/* y = act(x), rounded once; activation as above. */
int iron_activation(const void* x, void* y, int rows, int cols, int activation, int is_float, const int* valid,
                    void* stream);
/* y = x w^T, x (rows, k), w (n, k) bf16, y (rows, n); float sums of float products, any sizes. */
int iron_linear_any(const void* x, const uint16_t* w, void* y, int rows, int n, int k, int is_float,
                    const int* valid, void* stream);

/* mixed[m] = h + (before - h) * mu[m] for m < mixes, `before` the row ahead of h in its sequence (zeros
 * ahead of the first).  carry (slots, 2, cols) keeps position p's row in row p % 2: read ahead of a span's
 * first row, and written with its last.  mu (mixes, cols), mixed (mixes, rows, cols). */
int iron_token_shift(const void* h, const uint16_t* mu, void* carry, const int* spans, void* mixed, int slots,
                     int rows, int cols, int mixes, int is_float, void* stream);
/* out = -exp(w2 tanh(z) + w0): the logarithm of a decay per channel.  z (rows, rank), w2 (n, rank). */
int iron_low_rank_decay(const void* z, const uint16_t* w2, const uint16_t* w0, float* out, int rows, int n,
                        int rank, int is_float, const int* valid, void* stream);
/* o_t = (S + diag(u) k_t v_t^T)^T r_t; S <- diag(exp(log_decay_t)) S + k_t v_t^T per head.
 * r, k, v, log_decay, o (rows, heads * dim); u (heads, dim); state (slots, heads, dim, dim).  dim <= 256. */
int iron_time_mix(const void* r, const void* k, const void* v, const float* log_decay, const uint16_t* u, float* state,
                  const int* spans, float* o, int slots, int rows, int heads, int dim, int is_float, void* stream);
/* x (rows, stride) = [q | k | v | .. b .. a ..]: a causal convolution of `taps` taps (channels, taps) a
 * channel and SiLU on q, k (kv_heads x dim) and v (heads x vdim); q and k made unit vectors a head
 * (eps 1e-6), q times dim^-1/2; log decay = -exp(a_log) softplus(a + dt_bias), beta = sigmoid(b).
 * out (rows, 2 kv_heads dim + heads vdim + 2 heads) = [q | k | v | log decay | beta] in float.
 * state (slots, taps, channels): position p's inputs in row p % taps. */
int iron_short_conv(const void* x, const uint16_t* taps_w, const uint16_t* a_log, const uint16_t* dt_bias, void* state,
                    const int* spans, float* out, int slots, int rows, int stride, int heads, int kv_heads, int dim,
                    int vdim, int taps, int b_at, int a_at, int is_float, void* stream);
/* x as iron_short_conv leaves it.  S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q per value
 * head (q/k head head / (heads / kv_heads)).  state (slots, heads, dim, vdim), o (rows, heads * vdim). */
int iron_delta_rule(const float* x, float* state, const int* spans, float* o, int slots, int rows, int heads,
                    int kv_heads, int dim, int vdim, void* stream);
/* iron_time_mix and iron_delta_rule over portions of many rows, sixteen tokens at a time on float32 MFMAs:
 * two launches, a workspace of the bytes given (any contents, 16-byte aligned).  The same sums in another
 * order. */
int64_t iron_time_mix_workspace_bytes(int slots, int rows, int heads, int dim);
int iron_time_mix_chunked(const void* r, const void* k, const void* v, const float* log_decay, const uint16_t* u,
                          float* state, const int* spans, float* o, void* workspace, int slots, int rows, int heads,
                          int dim, int is_float, void* stream);
int64_t iron_delta_rule_workspace_bytes(int slots, int rows, int heads);
int iron_delta_rule_chunked(const float* x, float* state, const int* spans, float* o, void* workspace, int slots, int rows,
                            int heads, int kv_heads, int dim, int vdim, void* stream);
/* out = o / rms(o, one head) * gain * silu(gate) * scale; gain (dim) if gain_shared, else (heads * dim).  gate NULL: that
 * factor is 1. */
int iron_head_gate(const float* o, const void* gate, const uint16_t* gain, void* out, int rows, int heads, int dim,
                   int gate_stride, int gate_at, int gain_shared, int out_stride, int out_at, float eps, float scale,
                   int is_float, const int* valid, void* stream);
/* x (rows, stride) = [q heads | k heads | v heads]; score = q . k * scale + bias[head][i - j] over
 * 0 <= i - j < window, softmax, the values' sum times out_scale into columns out_at .. of out.
 * bias (heads, window); keys (slots, ring, kv_heads, dim), values (.., vdim): position p in row p % ring,
 * ring >= window; they receive the spans' last rows.  single: no span has more than one row. */
int iron_mha_window(const void* x, void* keys, void* values, const float* bias, const int* spans, void* out, int slots,
                    int rows, int stride, int heads, int kv_heads, int dim, int vdim, int window, int ring, float scale,
                    int out_stride, int out_at, float out_scale, int single, int is_float, void* stream);
/* x (rows, stride) = [zx | ux | gx | ..] of `width` columns each.  Per channel z = sigmoid(zx + z_bias), u = ux + x_bias,
 * c = u + 1/2 where u >= 0, else sigmoid(u); S <- (1 - z) S + z c; y = S silu(gx), y (rows, width).  state (slots, 2, width): the
 * state behind position p in row p % 2.
 * With a workspace (the bytes given, any contents, 16-byte aligned) chunks of a portion run side by side; without, a
 * span's rows one after the other. */
int64_t iron_min_gru_workspace_bytes(int slots, int rows, int width);
int iron_min_gru(const void* x, const uint16_t* z_bias, const uint16_t* x_bias, float* state, const int* spans, void* y,
                 void* workspace, int slots, int rows, int stride, int width, int is_float, void* stream);
/* Latent attention.  latent_rows: x (rows, stride) = [query latent (q_rank) | latent (rank) | shared key part (rot) | ..];
 * both latents RMS-normed (gains q_gain, c_gain), the first `turned` of the rot columns turned in neighbouring pairs
 * by row p of angles (angle_rows, turned; cos and sin side by side); q_out (rows, q_rank), and position p's latent
 * and key part in row p % ring of latents (slots, ring, rank) and shared_keys (slots, ring, rot; NULL if rot is 0).
 * mha_latent: q (rows, heads * (dim + rot)), a head's rot columns turned here; up (heads * (dim + vdim), rank): U, V.
 * score = (q . U c + turned q . shared key) * scale over 0 <= i - j < window, softmax (exp(sink[head]) in its denominator
 * unless sink is NULL); y (rows, heads * vdim) the sum of V c.  The rows' own latents are in the caches already.
 * single: no span has more than one row.  Else `cap` key rows are expanded at most: the spans' rows and, of the
 * positions before them, the last window - 1 each; a span whose keys do not fit is left out.
 * workspace: the bytes given, any contents. */
int iron_latent_rows(const void* x, const uint16_t* q_gain, const uint16_t* c_gain, const float* angles, const int* spans,
                     void* q_out, void* latents, void* shared_keys, int slots, int rows, int stride, int q_rank, int rank,
                     int rot, int turned, int angle_rows, int ring, float eps, int is_float, void* stream);
int64_t iron_mha_latent_workspace_bytes(int slots, int rows, int heads, int dim, int rot, int vdim, int rank, int window, int ring,
                                        int cap, int single, int is_float);
int iron_mha_latent(const void* q, const void* latents, const void* shared_keys, const uint16_t* up, const uint16_t* sink,
                    const float* angles, const int* spans, void* y, void* workspace, int slots, int rows, int heads, int dim,
                    int rot, int vdim, int rank, int turned, int angle_rows, int window, int ring, int cap, float scale, int single,
                    int is_float, void* stream);
/* One token a slot (no span of more than one row) through a mixer, bf16, in one launch; each computes what
 * the entry points above compute in turn, on the same states.
 * decode_mixed (one slot): iron_token_shift and `count` (up to 8) products y[i] = W[i] (rows[i], K) times
 * the blend by mu[i], or the row itself (mu[i] NULL).  The four arrays are host memory, read at the call.
 * decode_parallel: iron_low_rank_decay, iron_time_mix and iron_head_gate (columns mix_at ..; mix_dim a
 * power of two from 16) beside iron_mha_window (columns win_at ..; widths multiples of 8).
 * decode_delta: iron_short_conv, iron_delta_rule and iron_head_gate (shared gain; vdim a power of two
 * from 16). */
int iron_decode_mixed_bf16(const uint16_t* h, uint16_t* carry, const int* spans, int K, int count, const void* const* W,
                           void* const* y, const void* const* mu, const int* rows, void* stream);
int iron_decode_parallel_bf16(const uint16_t* r, const uint16_t* k, const uint16_t* v, const uint16_t* gate,
                              const uint16_t* z, const uint16_t* w2, const uint16_t* w0, const uint16_t* u,
                              const uint16_t* norm, float* memory, int mix_heads, int mix_dim, int rank, float eps,
                              float mix_scale, int mix_at, const uint16_t* x, uint16_t* keys, uint16_t* values,
                              const float* bias, int stride, int heads, int kv_heads, int dim, int vdim, int window,
                              int ring, float scale, float out_scale, int win_at, const int* spans, uint16_t* out,
                              int slots, int rows, int out_stride, void* stream);
int iron_decode_delta_bf16(const uint16_t* x, const uint16_t* taps_w, const uint16_t* a_log, const uint16_t* dt_bias,
                           const uint16_t* norm, uint16_t* inputs, float* state, const int* spans, uint16_t* out,
                           int slots, int rows, int stride, int heads, int kv_heads, int dim, int vdim, int taps,
                           int gate_at, int b_at, int a_at, float eps, void* stream);
/* Rows [q heads | k heads | v heads] of a packed projection made ready to be attended: q and k (+ bias) RMS-normed a head
 * with q_gain / k_gain (dim), their first `turned` columns turned in neighbouring pairs by their position's row of angles
 * (cos and sin side by side; positions behind the table's last row read that), q times scale * temp[head]; v (+ bias), with
 * first (rows of first_stride, columns first_at ..) blended to (1 - share) v + share first. */
int iron_turned_heads(const void* x, void* y, const uint16_t* bias, const uint16_t* q_gain, const uint16_t* k_gain,
                      const uint16_t* temp, const float* angles, const uint16_t* share, const void* first,
                      int first_stride, int first_at, const int* spans, int slots, int rows, int stride, int heads,
                      int kv_heads, int dim, int vdim, int turned, int angle_rows, float scale, float eps,
                      int is_float, const int* valid, void* stream);
/* Attention of such rows within chunks of `chunk` positions: softmax a head over the chunk's positions up to the row's own,
 * the heads' weights mixed by talk (heads, heads), each head's mixed weights applied to its own values.  Position p's key
 * and value live in row p % ring of the slot's ring, ring = chunk.  single: every span is one row at most.  workspace: of
 * that many bytes, 16-byte aligned. */
int64_t iron_mha_talking_workspace_bytes(int slots, int rows, int heads, int vdim, int chunk, int single);
int iron_mha_talking(const void* x, void* keys, void* values, const uint16_t* talk, const int* spans, void* out,
                     void* workspace, int slots, int rows, int stride, int heads, int kv_heads, int dim, int vdim, int chunk, int ring, int single,
                     int is_float, void* stream);
/* mLSTM: per head S <- keep S + write k v^T, n <- keep n + write k with m' = max(f + m, i), keep = exp(f + m - m'), write =
 * exp(i - m'); i = cap tanh((gate + i_bias) / cap), f = log sigmoid of the same of its gate.  x: rows [q | k | v | ..],
 * gates at columns i_at and f_at.  state: (slots, heads, dim, vdim + 1), n the last column; tops: (slots, 2, heads), m behind
 * position p in row p % 2.  o: rows [S^T q dim^-1/2 (heads * vdim) | n . q dim^-1/2 (heads) | m (heads)], float. */
int iron_matrix_memory(const void* x, const uint16_t* i_bias, const uint16_t* f_bias, float* state, float* tops,
                       const int* spans, float* o, int slots, int rows, int stride, int heads, int dim, int vdim,
                       int i_at, int f_at, float cap, int is_float, void* stream);
/* The same sixteen tokens at a time (dim up to 256), with a workspace of that many bytes, 16-byte aligned. */
int64_t iron_matrix_memory_workspace_bytes(int slots, int rows, int heads, int dim);
int iron_matrix_memory_chunked(const void* x, const uint16_t* i_bias, const uint16_t* f_bias, float* state, float* tops,
                               const int* spans, float* o, void* workspace, int slots, int rows, int stride, int heads,
                               int dim, int vdim, int i_at, int f_at, float cap, int is_float, void* stream);
/* y = o / (max(|n . q|, exp(-m)) + floor), RMS-normed a head, times gain (heads * dim) and sigmoid(gate). */
int iron_memory_gate(const float* o, const void* gate, const uint16_t* gain, void* y, int rows, int heads, int dim,
                     int gate_stride, int gate_at, float floor, float eps, int is_float, const int* valid, void* stream);
/* A row's `top` experts by the largest of its logits w h + bias (float; bias may be NULL), and their shares, a softmax over the
 * chosen logits; or (scored) by the largest of the logits' softmax plus correction (may be NULL), and their shares, the softmax's
 * over their sum + 1e-20. */
int iron_router(const void* h, const uint16_t* w, const uint16_t* bias, const uint16_t* correction, int scored, int* ids,
                float* shares, int rows, int cols, int experts, int top, int is_float, const int* valid, void* stream);
/* y = sum over a row's experts e of share * down_e (act(gate_e h) * (up_e h)); gate and up (experts, ff, cols), down
 * (experts, cols, ff).  With identity > 0, ids from `experts` on stand for h itself.  activation: 1 SiLU, 2 GELU (tanh form),
 * 3 ReLU. */
int64_t iron_experts_workspace_bytes(int rows, int cols, int ff, int experts, int top, int is_float);
int iron_experts(const void* h, const uint16_t* gate, const uint16_t* up, const uint16_t* down, const int* ids,
                 const float* shares, void* y, void* workspace, int rows, int cols, int ff, int experts, int identity, int top,
                 int activation, int is_float, const int* valid, void* stream);
/* HGRN2: per head S <- diag(f) S + (1 - f) v^T, then o = S^T silu(q), f = lower + (1 - lower) sigmoid(z + f_bias).  x: rows
 * [q | z | v | ..]; f_bias, lower (heads * dim); state (slots, heads, dim, vdim); o (rows, heads * vdim), float.  dim <= 256. */
int iron_hgrn2(const void* x, const uint16_t* f_bias, const uint16_t* lower, float* state, const int* spans, float* o, int slots,
               int rows, int stride, int heads, int dim, int vdim, int is_float, void* stream);
/* The same sixteen tokens at a time, with a workspace of that many bytes, 16-byte aligned. */
int64_t iron_hgrn2_workspace_bytes(int slots, int rows, int heads, int dim);
int iron_hgrn2_chunked(const void* x, const uint16_t* f_bias, const uint16_t* lower, float* state, const int* spans, float* o,
                       void* workspace, int slots, int rows, int stride, int heads, int dim, int vdim, int is_float,
                       void* stream);
/* One token a slot, bf16, in one launch: iron_hgrn2, iron_head_gate without a gate (gains (vdim) shared by the heads) into columns
 * out_at .. of out, and beside it iron_gated_columns of the same rows into those from gated_at (cols 0: none), and, for one slot, iron_router's
 * scored choice from its logits z (NULL: none).  vdim a power of two from 16. */
int iron_decode_hgrn2_bf16(const uint16_t* x, const uint16_t* f_bias, const uint16_t* lower, const uint16_t* norm, float* state,
                           const int* spans, uint16_t* out, int slots, int rows, int stride, int heads, int dim, int vdim,
                           int out_stride, int out_at, float eps, int cols, int gate_at, int gated_at, int kind, float limit,
                           const float* z, const uint16_t* correction, int logits, int top, int* ids, float* shares,
                           void* stream);
/* Rows [q heads | k heads | v heads | ..] of a packed projection made ready to be attended: q and k RMS-normed a head with
 * q_gain / k_gain (dim), columns i and i + turned / 2 of the first `turned` turned together by their position's row of angles
 * (cos and sin side by side, multiplied in as they are); v, with value_norm, over its root mean square a head.  q (rows, heads *
 * dim); position p's key and value in row p of keys (slots, kv_heads, context, dim) and values (.., vdim). */
int iron_cached_heads(const void* x, void* q, void* keys, void* values, const uint16_t* q_gain, const uint16_t* k_gain,
                      const float* angles, const int* spans, int slots, int rows, int stride, int heads, int kv_heads, int dim,
                      int vdim, int context, int turned, int angle_rows, int value_norm, float eps, int is_float,
                      const int* valid, void* stream);
/* One token a slot, bf16, in one launch: iron_cached_heads, and beside it iron_gated_columns of the same rows into columns
 * gated_at .. of out (cols 0: none), and, for one slot, iron_router's scored choice from its logits z (NULL: none). */
int iron_decode_heads_global_bf16(const uint16_t* x, uint16_t* q, uint16_t* keys, uint16_t* values, const uint16_t* q_gain,
                                  const uint16_t* k_gain, const float* angles, const int* spans, int slots, int rows, int stride,
                                  int heads, int kv_heads, int dim, int vdim, int context, int turned, int angle_rows,
                                  int value_norm, float eps, uint16_t* out, int out_stride, int cols, int gate_at, int gated_at,
                                  int kind, float limit, const float* z, const uint16_t* correction, int logits, int top, int* ids,
                                  float* shares, void* stream);
/* Causal attention over such caches, the rows' own keys in them already: score = q . k * scale, with cap > 0 cap *
 * tanh(score / cap); softmax, with `sink` one more in its denominator; the values' sums in columns out_at .. of y (rows of
 * out_stride).  single: no span has more than one row.  workspace: of that many bytes (it may be none), 16-byte aligned. */
int64_t iron_mha_global_workspace_bytes(int slots, int heads, int kv_heads, int vdim, int context, int single);
int iron_mha_global(const void* q, const void* keys, const void* values, const int* spans, void* y, void* workspace, int slots,
                    int rows, int heads, int kv_heads, int dim, int vdim, int context, float scale, float cap, int sink,
                    int out_stride, int out_at, int single, int is_float, void* stream);

/* One row's product with its input made and its output taken in the same launch, bf16; each computes what the entry
 * points above and iron_gemv_bf16 compute in turn.
 * stream_product: input 0 the bf16 row x (K); 1 the float row x, 2 the bf16 row x, RMS-normed with unit + gain; 3 slot 0's
 * iron_min_gru over the row x = [zx | ux | gx] (width K, biases b0 and b1); 4 iron_poly_norm (bias b0, coefficients
 * gain).  Output: the row y (M), inputs 0 to 2; or iron_stream_gated_rows on stream_row (M), inputs 0, 3 and 4.
 * latent_query: iron_latent_rows of slot 0's one row x (whole 16-byte pieces), and q = W (M, q_rank) times the
 * query's latent. */
int iron_stream_product_bf16(int input, const void* x, const uint16_t* gain, const uint16_t* b0, const uint16_t* b1,
                             float* state, const int* spans, float eps, float unit, const uint16_t* W, int M,
                             int K, uint16_t* y, float* stream_row, const uint16_t* y_bias, const uint16_t* gate, const uint16_t* gate_bias,
                             void* stream);
/* norm_product: y = W (M, K) times h, the float row x normed in `groups` parts (iron_stream_groups); h (may be NULL) as well, and
 * with a router (logits, K) its logits in float to z.  product_sum: the stream's row += W (M, K) times x, plus also (may be NULL). */
int iron_norm_product_bf16(const float* x, const uint16_t* gain, int groups, float eps, float unit, const uint16_t* W, int M, int K,
                           uint16_t* y, uint16_t* h, const uint16_t* router, int logits, float* z, void* stream);
int iron_product_sum_bf16(const uint16_t* x, const uint16_t* W, int M, int K, const uint16_t* also, float* stream_row, void* stream);
/* One row through its experts (iron_experts; h, gate .. activation as there) and, in the launch that sums them, out (cols, inner)
 * times made: the stream's row += both, each rounded.  workspace: 2 top ff bytes.  Two launches. */
int iron_experts_tail_bf16(const uint16_t* h, const uint16_t* gate, const uint16_t* up, const uint16_t* down, const int* ids, const float* shares,
                           const uint16_t* out, const uint16_t* made, float* stream_row, void* workspace, int cols, int ff, int inner,
                           int experts, int identity, int top, int activation, void* stream);
int iron_latent_query_bf16(const uint16_t* x, const uint16_t* q_gain, const uint16_t* c_gain, const float* angles,
                           const int* spans, const uint16_t* W, uint16_t* q, uint16_t* latents, uint16_t* shared_keys,
                           int M, int stride, int q_rank, int rank, int rot, int turned, int angle_rows, int ring,
                           float eps, void* stream);
/* iron_sample_bf16 for every slot that has rows: logits (slots, logits_stride), drawn at the position p
 * of the span's last row by draw row slot * steps + p, recorded in record[slot * steps + p]; the span
 * then becomes {slot, 1, p + 1}.  workspace: slots times iron_sample_workspace_bytes(n). */
int iron_sample_slots_bf16(const uint16_t* logits, int n, int logits_stride, int* spans, int slots, int batch_rows,
                           int steps, const int* draws, int k_max, void* workspace, int* token, int* record,
                           void* stream);

#ifdef __cplusplus
}
#endif
#endif /* IRON_HIP_H */
