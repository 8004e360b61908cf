"""Thin, typed Python calls onto the C ABI: torch CUDA tensors in, launches out.

Each function checks what the C side cannot see (dtype, device, contiguity,
element counts), passes raw device pointers and the current HIP stream, and
raises ``IronHipError`` on refusal.  Nothing here computes.
"""

from __future__ import annotations

import ctypes
import math

import torch

from ._lib import check, current_stream, lib, ptr

BF16 = torch.bfloat16
GATES = {"silu": 1, "gelu_tanh": 2, "relu": 3}   # a gated feed-forward's activation, by the C ABI's number


def _dev(t, name, dtype=BF16):
    if not isinstance(t, torch.Tensor):
        raise TypeError(f"{name}: expected a torch tensor, got {type(t).__name__}")
    if not t.is_cuda:
        raise TypeError(f"{name}: expected a tensor on the GPU, got {t.device}")
    if dtype is not None and t.dtype != dtype:
        raise TypeError(f"{name}: expected {dtype}, got {t.dtype}")
    if not t.is_contiguous():
        raise ValueError(f"{name}: expected a contiguous tensor")
    return t


def _word(t, name):
    """An optional per-call word: a 1-element int32 device tensor, or None."""
    if t is None:
        return None
    _dev(t, name, torch.int32)
    if t.numel() < 1:
        raise ValueError(f"{name}: expected at least one int32 word")
    return t


def _numel(t, n, name):
    if t.numel() != n:
        raise ValueError(f"{name}: expected {n} elements, got {t.numel()} {tuple(t.shape)}")


def gemm(A, B, C, *, M, N, K, b_col_maj=False, c_col_maj=False, valid=None, valid_k=None):
    _numel(_dev(A, "A"), M * K, "A")
    _numel(_dev(B, "B"), K * N, "B")
    _numel(_dev(C, "C"), M * N, "C")
    check(
        lib().iron_gemm_bf16(
            ptr(A), ptr(B), ptr(C), M, N, K, int(b_col_maj), int(c_col_maj),
            ptr(_word(valid, "valid")), ptr(_word(valid_k, "valid_k")), current_stream(),
        ),
        "iron_gemm_bf16",
    )


def gemv(W, x, y, *, M, K, batches=1, repeat=1, valid=None, rows_per_wave=0, k_split=0):
    _numel(_dev(W, "A"), (batches // repeat) * M * K, "A")
    _numel(_dev(x, "B"), batches * K, "B")
    _numel(_dev(y, "C"), batches * M, "C")
    check(
        lib().iron_gemv_bf16_tuned(
            ptr(W), ptr(x), ptr(y), M, K, batches, repeat, ptr(_word(valid, "valid")),
            rows_per_wave, k_split, current_stream(),
        ),
        "iron_gemv_bf16",
    )


def gemm_residual(A, B, R, C, *, M, N, K, residual_scale=1.0, valid=None):
    """``C = residual_scale * (A @ B.T) + R`` over many rows, B stored ``(N, K)``."""
    _numel(_dev(A, "A"), M * K, "A")
    _numel(_dev(B, "B"), N * K, "B")
    _numel(_dev(R, "R"), M * N, "R")
    _numel(_dev(C, "C"), M * N, "C")
    check(lib().iron_gemm_residual_bf16(ptr(A), ptr(B), ptr(R), ptr(C), M, N, K, float(residual_scale),
                                        ptr(_word(valid, "valid")), current_stream()), "iron_gemm_residual_bf16")


def gemm_residual_norm_workspace_bytes(M, N, K) -> int:
    """Bytes of workspace ``gemm_residual_norm`` needs; 0 for a shape it refuses."""
    return int(lib().iron_gemm_residual_norm_workspace_bytes(M, N, K))


def gemm_residual_norm(A, B, R, gain, C, Y, workspace, *, M, N, K, eps, residual_scale=1.0, valid=None):
    """``C = residual_scale * (A @ B.T) + R`` and ``Y = rmsnorm(C) * gain`` over few rows and a long K:
    K dealt over several blocks a tile while the bound leaves the chip idle, float32 sums in
    ``workspace`` (any contents), the rows finished and normed by a second launch."""
    _numel(_dev(A, "A"), M * K, "A")
    _numel(_dev(B, "B"), N * K, "B")
    _numel(_dev(R, "R"), M * N, "R")
    _numel(_dev(gain, "gain"), N, "gain")
    _numel(_dev(C, "C"), M * N, "C")
    _numel(_dev(Y, "Y"), M * N, "Y")
    need = gemm_residual_norm_workspace_bytes(M, N, K)
    if need and _dev(workspace, "workspace", None).numel() * workspace.element_size() < need:
        raise ValueError(f"gemm_residual_norm: workspace holds {workspace.numel() * workspace.element_size()} bytes, "
                         f"{need} needed")
    check(lib().iron_gemm_residual_norm_bf16(ptr(A), ptr(B), ptr(R), ptr(gain), ptr(C), ptr(Y), M, N, K,
                                             float(residual_scale), float(eps), ptr(_word(valid, "valid")),
                                             ptr(workspace), current_stream()), "iron_gemm_residual_norm_bf16")


def gemm_gated(A, B, G, C, *, M, N, K, activation="silu", valid=None):
    """``C = act(G) * (A @ B.T)`` over many rows, B stored ``(N, K)``; ``activation`` "silu" or
    "gelu_tanh"."""
    kinds = GATES
    if activation not in kinds:
        raise ValueError(f"gemm_gated: activation {activation!r} is none of {sorted(kinds)}")
    _numel(_dev(A, "A"), M * K, "A")
    _numel(_dev(B, "B"), N * K, "B")
    _numel(_dev(G, "G"), M * N, "G")
    _numel(_dev(C, "C"), M * N, "C")
    check(lib().iron_gemm_gated_bf16(ptr(A), ptr(B), ptr(G), ptr(C), M, N, K, kinds[activation],
                                     ptr(_word(valid, "valid")), current_stream()), "iron_gemm_gated_bf16")


def gemm_gated_pair(A, Bg, Bu, G, C, *, M, N, K, activation="silu", valid=None):
    """``G = A @ Bg.T``, ``C = act(G) * (A @ Bu.T)`` over many rows in one launch (weights ``(N, K)``)."""
    kinds = GATES
    if activation not in kinds:
        raise ValueError(f"gemm_gated_pair: activation {activation!r} is none of {sorted(kinds)}")
    _numel(_dev(A, "A"), M * K, "A")
    _numel(_dev(Bg, "Bg"), N * K, "Bg")
    _numel(_dev(Bu, "Bu"), N * K, "Bu")
    _numel(_dev(G, "G"), M * N, "G")
    _numel(_dev(C, "C"), M * N, "C")
    check(lib().iron_gemm_gated_pair_bf16(ptr(A), ptr(Bg), ptr(Bu), ptr(G), ptr(C), M, N, K, kinds[activation],
                                          ptr(_word(valid, "valid")), current_stream()), "iron_gemm_gated_pair_bf16")


def gemv_fused(W, x, y, *, M, K, W2=None, norm_w=None, eps=0.0, residual=None, residual_scale=1.0, epilogue=0):
    """One-row fusion: ``[RMSNorm ->] GEMV [-> + residual | gate/up -> SiLU -> Mul]``."""
    _numel(_dev(W, "W"), M * K, "W")
    _numel(_dev(x, "x"), K, "x")
    _numel(_dev(y, "y"), M, "y")
    if W2 is not None:
        _numel(_dev(W2, "W2"), M * K, "W2")
    if norm_w is not None:
        _numel(_dev(norm_w, "norm_w"), K, "norm_w")
    if residual is not None:
        _numel(_dev(residual, "residual"), M, "residual")
    check(
        lib().iron_gemv_fused_bf16(ptr(W), ptr(W2), ptr(x), ptr(norm_w), float(eps), ptr(residual),
                                   float(residual_scale), ptr(y), M, K, int(epilogue), current_stream()),
        "iron_gemv_fused_bf16",
    )


def decode_qkv(x, norm_w, Wq, Wk, Wv, angles, q_out, keys, values, *, eps, hidden, heads, kv_heads, d,
               cache_rows, position, angle_row=None, table=None, token=None):
    """Attention's first half for one token: norm, q/k/v projections, RoPE, cache writes.  ``angles``
    is the token's row of the RoPE table, or with ``angle_row`` (a device word) the whole table.  With
    ``table`` and ``token`` (a device word) the input is that row of the embedding table, which the
    launch also writes to ``x``."""
    _numel(_dev(x, "x"), hidden, "x")
    _numel(_dev(norm_w, "norm_w"), hidden, "norm_w")
    _numel(_dev(Wq, "Wq"), heads * d * hidden, "Wq")
    _numel(_dev(Wk, "Wk"), kv_heads * d * hidden, "Wk")
    _numel(_dev(Wv, "Wv"), kv_heads * d * hidden, "Wv")
    _dev(angles, "angles")
    if angle_row is None:
        _numel(angles, d, "angles")
    elif angles.numel() % d or angles.numel() < d:
        raise ValueError(f"angles: a table of rows of {d}, got {angles.numel()} elements")
    _numel(_dev(q_out, "q_out"), heads * d, "q_out")
    _numel(_dev(keys, "keys"), cache_rows * kv_heads * d, "keys")
    _numel(_dev(values, "values"), cache_rows * kv_heads * d, "values")
    if table is not None:
        _dev(table, "table")
        if table.numel() % hidden or table.numel() < hidden:
            raise ValueError(f"table: rows of {hidden}, got {table.numel()} elements")
        check(
            lib().iron_decode_qkv_embed_bf16(ptr(table), ptr(_word(token, "token")), table.numel() // hidden, ptr(x),
                                             ptr(norm_w), float(eps), ptr(Wq), ptr(Wk), ptr(Wv), ptr(angles),
                                             ptr(q_out), ptr(keys), ptr(values), hidden, heads, kv_heads, d, cache_rows,
                                             ptr(_word(position, "position")), ptr(_word(angle_row, "angle_row")),
                                             angles.numel() // d, current_stream()),
            "iron_decode_qkv_embed_bf16",
        )
        return
    check(
        lib().iron_decode_qkv_bf16(ptr(x), ptr(norm_w), float(eps), ptr(Wq), ptr(Wk), ptr(Wv), ptr(angles),
                                   ptr(q_out), ptr(keys), ptr(values), hidden, heads, kv_heads, d, cache_rows,
                                   ptr(_word(position, "position")), ptr(_word(angle_row, "angle_row")),
                                   angles.numel() // d, current_stream()),
        "iron_decode_qkv_bf16",
    )


def decode_heads(q, q_out, *, heads, kv_heads, d, eps, norms=0, k=None, v=None, q_gain=None, k_gain=None,
                 q_angles=None, k_angles=None, rotary=0, two_halves=True, keys=None, values=None, row0=None,
                 row1=None, cache_rows=0):
    """Per-head norms, RoPE and the cache rows of one token's q, k, v (``iron_decode_heads_bf16``)."""
    _numel(_dev(q, "q"), heads * d, "q")
    _numel(_dev(q_out, "q_out"), heads * d, "q_out")
    for name, t, n in (("k", k, kv_heads * d), ("v", v, kv_heads * d), ("q_gain", q_gain, d), ("k_gain", k_gain, d),
                       ("q_angles", q_angles, rotary), ("k_angles", k_angles, rotary),
                       ("keys", keys, cache_rows * kv_heads * d), ("values", values, cache_rows * kv_heads * d)):
        if t is not None:
            _numel(_dev(t, name), n, name)
    check(
        lib().iron_decode_heads_bf16(ptr(q), ptr(k), ptr(v), ptr(q_gain), ptr(k_gain), int(norms), float(eps),
                                     ptr(q_angles), ptr(k_angles), int(rotary), int(two_halves), ptr(q_out), ptr(keys),
                                     ptr(values), ptr(_word(row0, "row0")), ptr(_word(row1, "row1")), int(cache_rows),
                                     heads, kv_heads, d, current_stream()),
        "iron_decode_heads_bf16",
    )


def prefill_qkv(x, Wq, Wk, Wv, angles, q_out, k_out, v_out, *, rows, hidden, heads, kv_heads, d, valid=None):
    """A prompt chunk's q/k/v projections with q and k turned by RoPE, one launch."""
    _numel(_dev(x, "x"), rows * hidden, "x")
    _numel(_dev(Wq, "Wq"), heads * d * hidden, "Wq")
    _numel(_dev(Wk, "Wk"), kv_heads * d * hidden, "Wk")
    _numel(_dev(Wv, "Wv"), kv_heads * d * hidden, "Wv")
    _numel(_dev(angles, "angles"), rows * d, "angles")
    _numel(_dev(q_out, "q_out"), rows * heads * d, "q_out")
    _numel(_dev(k_out, "k_out"), rows * kv_heads * d, "k_out")
    _numel(_dev(v_out, "v_out"), rows * kv_heads * d, "v_out")
    check(
        lib().iron_prefill_qkv_bf16(ptr(x), ptr(Wq), ptr(Wk), ptr(Wv), ptr(angles), ptr(q_out), ptr(k_out),
                                    ptr(v_out), rows, hidden, heads, kv_heads, d, ptr(_word(valid, "valid")),
                                    current_stream()),
        "iron_prefill_qkv_bf16",
    )


def prefill_qkv_cache(x, Wq, Wk, Wv, angles, q_out, keys, values, *, rows, hidden, heads, kv_heads, d, cache_rows,
                      start, valid=None):
    """``prefill_qkv`` with k and v written into rows ``start`` on of the layer's KV caches."""
    _numel(_dev(x, "x"), rows * hidden, "x")
    _numel(_dev(Wq, "Wq"), heads * d * hidden, "Wq")
    _numel(_dev(Wk, "Wk"), kv_heads * d * hidden, "Wk")
    _numel(_dev(Wv, "Wv"), kv_heads * d * hidden, "Wv")
    _numel(_dev(angles, "angles"), rows * d, "angles")
    _numel(_dev(q_out, "q_out"), rows * heads * d, "q_out")
    _numel(_dev(keys, "keys"), cache_rows * kv_heads * d, "keys")
    _numel(_dev(values, "values"), cache_rows * kv_heads * d, "values")
    check(
        lib().iron_prefill_qkv_cache_bf16(ptr(x), ptr(Wq), ptr(Wk), ptr(Wv), ptr(angles), ptr(q_out), ptr(keys),
                                          ptr(values), rows, hidden, heads, kv_heads, d, cache_rows,
                                          ptr(_word(start, "start")), ptr(_word(valid, "valid")), current_stream()),
        "iron_prefill_qkv_cache_bf16",
    )


def rmsnorm(x, w, y, *, rows, cols, eps, valid=None, residual=None):
    """``residual``: the normed rows are added to it (the sum rounded as the separate step rounds)."""
    _numel(_dev(x, "x"), rows * cols, "x")
    _numel(_dev(y, "y"), rows * cols, "y")
    if w is not None:
        _numel(_dev(w, "weight"), cols, "weight")
    if residual is not None:
        _numel(_dev(residual, "residual"), rows * cols, "residual")
        check(
            lib().iron_rmsnorm_add_bf16(ptr(x), ptr(w), ptr(residual), ptr(y), rows, cols, float(eps),
                                        ptr(_word(valid, "valid")), current_stream()),
            "iron_rmsnorm_add_bf16",
        )
        return
    check(
        lib().iron_rmsnorm_bf16(
            ptr(x), ptr(w), ptr(y), rows, cols, float(eps), ptr(_word(valid, "valid")),
            current_stream(),
        ),
        "iron_rmsnorm_bf16",
    )


def rope(x, angles, y, *, rows, cols, angle_rows, two_halves=True, valid=None, row_cols=None):
    """``cols`` columns of each row turn; ``row_cols`` (default: the same) is the whole row, whose
    remaining columns pass through."""
    row_cols = cols if row_cols is None else row_cols
    _numel(_dev(x, "x"), rows * row_cols, "x")
    _numel(_dev(angles, "angles"), angle_rows * cols, "angles")
    _numel(_dev(y, "y"), rows * row_cols, "y")
    if row_cols == cols:
        check(lib().iron_rope_bf16(ptr(x), ptr(angles), ptr(y), rows, cols, angle_rows, int(two_halves),
                                   ptr(_word(valid, "valid")), current_stream()), "iron_rope_bf16")
    else:
        check(lib().iron_rope_partial_bf16(ptr(x), ptr(angles), ptr(y), rows, row_cols, cols, angle_rows,
                                           int(two_halves), ptr(_word(valid, "valid")), current_stream()),
              "iron_rope_partial_bf16")


def _binary(name):
    def call(a, b, y, *, n=None, valid=None):
        n = y.numel() if n is None else n
        _numel(_dev(a, "a"), n, "a")
        _numel(_dev(b, "b"), n, "b")
        _numel(_dev(y, "y"), n, "y")
        check(
            getattr(lib(), name)(ptr(a), ptr(b), ptr(y), n, ptr(_word(valid, "valid")), current_stream()),
            name,
        )

    call.__name__ = name
    return call


mul = _binary("iron_mul_bf16")
add = _binary("iron_add_bf16")
silu_mul = _binary("iron_silu_mul_bf16")


def row_broadcast(x, row, y, *, rows, cols, multiply=False, valid=None):
    """``y[r] = x[r] + row`` (or ``* row``) for every row ``r`` under the bound."""
    _numel(_dev(x, "x"), rows * cols, "x")
    _numel(_dev(row, "row"), cols, "row")
    _numel(_dev(y, "y"), rows * cols, "y")
    check(
        lib().iron_row_broadcast_bf16(ptr(x), ptr(row), ptr(y), rows, cols, int(bool(multiply)),
                                      ptr(_word(valid, "valid")), current_stream()),
        "iron_row_broadcast_bf16",
    )


def silu(x, y, *, n=None, valid=None):
    n = y.numel() if n is None else n
    _numel(_dev(x, "x"), n, "x")
    _numel(_dev(y, "y"), n, "y")
    check(lib().iron_silu_bf16(ptr(x), ptr(y), n, ptr(_word(valid, "valid")), current_stream()), "iron_silu_bf16")


UNARY = {"gelu_tanh": 0, "gelu_erf": 1, "relu": 2, "sigmoid": 3, "tanh": 4, "clamp": 5}


def unary(x, y, kind, *, n=None, low=0.0, high=0.0, valid=None):
    """``y = f(x)``, ``kind`` one of ``UNARY``; ``low`` and ``high`` are the clamp's bounds."""
    n = y.numel() if n is None else n
    _numel(_dev(x, "x"), n, "x")
    _numel(_dev(y, "y"), n, "y")
    check(lib().iron_unary_bf16(ptr(x), ptr(y), n, UNARY[kind], float(low), float(high), ptr(_word(valid, "valid")),
                                current_stream()), "iron_unary_bf16")


def axpy(x, y, out, *, a, n=None, valid=None):
    n = out.numel() if n is None else n
    _numel(_dev(x, "x"), n, "x")
    _numel(_dev(y, "y"), n, "y")
    _numel(_dev(out, "out"), n, "out")
    check(lib().iron_axpy_bf16(ptr(x), ptr(y), ptr(out), n, float(a), ptr(_word(valid, "valid")), current_stream()),
          "iron_axpy_bf16")


def layernorm(x, w, y, *, rows, cols, eps, valid=None):
    _numel(_dev(x, "x"), rows * cols, "x")
    _numel(_dev(y, "y"), rows * cols, "y")
    if w is not None:
        _numel(_dev(w, "weight"), cols, "weight")
    check(lib().iron_layernorm_bf16(ptr(x), ptr(w), ptr(y), rows, cols, float(eps), ptr(_word(valid, "valid")),
                                    current_stream()), "iron_layernorm_bf16")


def softmax(x, y, *, rows, cols, addend=None, soft_cap=None, length=None):
    """Softmax of each row of ``x`` (bf16 or float32) over its first ``length`` columns (a device word)."""
    f32 = x.dtype == torch.float32
    _numel(_dev(x, "x", torch.float32 if f32 else torch.bfloat16), rows * cols, "x")
    _numel(_dev(y, "y"), rows * cols, "y")
    if addend is not None:
        _numel(_dev(addend, "addend", torch.float32), rows * cols, "addend")
    check(lib().iron_softmax_bf16(ptr(x), int(f32), ptr(addend), ptr(y), rows, cols, float(soft_cap or 0.0),
                                  ptr(_word(length, "length")), current_stream()), "iron_softmax_bf16")


def mha_prefill(
    Q, K, V, O, *, heads, kv_heads, d, seq, seq_len=None, kv_len, scale=None, causal=True,
    window=None, q_interleaved=False, kv_interleaved=False, valid=None, kv_valid=None, kv_first=None, kv_rows=None,
):
    """``kv_first`` (a device word) and ``kv_rows``: K and V are buffers of ``kv_rows`` rows (at the
    least; ``kv_interleaved``) of which the ``kv_len`` from row ``*kv_first`` on are the keys."""
    seq_len = seq if seq_len is None else seq_len
    scale = 1.0 / math.sqrt(d) if scale is None else scale
    _numel(_dev(Q, "Q"), seq * heads * d, "Q")
    _numel(_dev(O, "O"), seq * heads * d, "O")
    if kv_first is not None:
        _window(K, V, kv_rows, kv_len, kv_heads, d, kv_interleaved)
        check(
            lib().iron_mha_prefill_at_bf16(
                ptr(Q), ptr(K), ptr(V), ptr(O), heads, kv_heads, d, seq, seq_len, kv_len, float(scale),
                int(causal), -1 if window is None else int(window), int(q_interleaved),
                ptr(_word(valid, "valid")), ptr(_word(kv_valid, "kv_valid")), ptr(_word(kv_first, "kv_first")),
                int(kv_rows), current_stream(),
            ),
            "iron_mha_prefill_at_bf16",
        )
        return
    _numel(_dev(K, "K"), kv_len * kv_heads * d, "K")
    _numel(_dev(V, "V"), kv_len * kv_heads * d, "V")
    check(
        lib().iron_mha_prefill_bf16(
            ptr(Q), ptr(K), ptr(V), ptr(O), heads, kv_heads, d, seq, seq_len, kv_len, float(scale),
            int(causal), -1 if window is None else int(window), int(q_interleaved),
            int(kv_interleaved), ptr(_word(valid, "valid")), ptr(_word(kv_valid, "kv_valid")),
            current_stream(),
        ),
        "iron_mha_prefill_bf16",
    )


def _window(K, V, kv_rows, kv_len, kv_heads, d, kv_interleaved):
    if not kv_interleaved or kv_rows is None or kv_rows < kv_len:
        raise ValueError(f"a window of the keys takes them row by row (kv_interleaved) out of kv_rows ({kv_rows}) "
                         f">= kv_len ({kv_len})")
    for name, t in (("K", K), ("V", V)):
        if _dev(t, name).numel() < kv_rows * kv_heads * d:
            raise ValueError(f"{name}: expected {kv_rows * kv_heads * d} elements at the least, got {t.numel()}")


def mha_decode_workspace(heads, d, device="cuda"):
    n = lib().iron_mha_decode_workspace_bytes(heads, d)
    return torch.empty(n // 4, dtype=torch.float32, device=device)


def mha_decode(
    Q, K, V, O, *, heads, kv_heads, d, kv_len, scale=None, window=None, kv_interleaved=False,
    kv_valid=None, workspace, kv_first=None, kv_rows=None, form=0, short_keys=0,
):
    """``kv_first`` / ``kv_rows``: the keys are a window of a longer buffer, as ``mha_prefill``'s.
    ``form`` / ``short_keys`` force the kernel form (``iron_mha_decode_tuned_bf16``)."""
    scale = 1.0 / math.sqrt(d) if scale is None else scale
    _numel(_dev(Q, "Q"), heads * d, "Q")
    _numel(_dev(O, "O"), heads * d, "O")
    _dev(workspace, "workspace", torch.float32)
    need = lib().iron_mha_decode_workspace_bytes(heads, d)
    if workspace.numel() * 4 < need:
        raise ValueError(f"workspace: {workspace.numel() * 4} bytes, need {need}")
    if kv_first is not None:
        _window(K, V, kv_rows, kv_len, kv_heads, d, kv_interleaved)
        check(
            lib().iron_mha_decode_at_bf16(
                ptr(Q), ptr(K), ptr(V), ptr(O), heads, kv_heads, d, kv_len, float(scale),
                -1 if window is None else int(window), ptr(_word(kv_valid, "kv_valid")),
                ptr(_word(kv_first, "kv_first")), int(kv_rows), ptr(workspace), current_stream(),
            ),
            "iron_mha_decode_at_bf16",
        )
        return
    _numel(_dev(K, "K"), kv_len * kv_heads * d, "K")
    _numel(_dev(V, "V"), kv_len * kv_heads * d, "V")
    if form or short_keys:
        check(
            lib().iron_mha_decode_tuned_bf16(
                ptr(Q), ptr(K), ptr(V), ptr(O), heads, kv_heads, d, kv_len, float(scale),
                -1 if window is None else int(window), int(kv_interleaved),
                ptr(_word(kv_valid, "kv_valid")), ptr(workspace), int(form), int(short_keys), current_stream(),
            ),
            "iron_mha_decode_tuned_bf16",
        )
        return
    check(
        lib().iron_mha_decode_bf16(
            ptr(Q), ptr(K), ptr(V), ptr(O), heads, kv_heads, d, kv_len, float(scale),
            -1 if window is None else int(window), int(kv_interleaved),
            ptr(_word(kv_valid, "kv_valid")), ptr(workspace), current_stream(),
        ),
        "iron_mha_decode_bf16",
    )


def mha_decode_static(Q, K, V, O, *, heads, kv_heads, d, kv_len, scale=None, window=None, kv_interleaved=False,
                      kv_valid=None):
    """``mha_decode`` with the split-KV partial results in the library's own device scratch: no
    workspace, nothing allocated (for callers that cannot allocate); refused past its fixed size."""
    scale = 1.0 / math.sqrt(d) if scale is None else scale
    _numel(_dev(Q, "Q"), heads * d, "Q")
    _numel(_dev(O, "O"), heads * d, "O")
    _numel(_dev(K, "K"), kv_len * kv_heads * d, "K")
    _numel(_dev(V, "V"), kv_len * kv_heads * d, "V")
    check(
        lib().iron_mha_decode_static_bf16(
            ptr(Q), ptr(K), ptr(V), ptr(O), heads, kv_heads, d, kv_len, float(scale),
            -1 if window is None else int(window), int(kv_interleaved),
            ptr(_word(kv_valid, "kv_valid")), current_stream(),
        ),
        "iron_mha_decode_static_bf16",
    )


def gather_rows(table, ids, out, *, valid=None):
    _dev(table, "table", None)
    _dev(ids, "ids", torch.int32)
    _dev(out, "out", table.dtype)
    row_bytes = table[0].numel() * table.element_size()
    n_ids = ids.numel()
    _numel(out, n_ids * table[0].numel(), "out")
    check(
        lib().iron_gather_rows(
            ptr(table), ptr(ids), ptr(out), n_ids, table.shape[0], row_bytes,
            ptr(_word(valid, "valid")), current_stream(),
        ),
        "iron_gather_rows",
    )


def copy_rows(src, dst, *, rows, row_elems, src_rows, dst_rows, src_stride=None, dst_stride=None,
              src_row=None, dst_row=None, valid=None):
    """``dst[dst_row + i] = src[src_row + i]`` for ``i < rows``; strides in elements."""
    _dev(src, "src", None)
    _dev(dst, "dst", src.dtype)
    es = src.element_size()
    src_stride = row_elems if src_stride is None else src_stride
    dst_stride = row_elems if dst_stride is None else dst_stride
    if src.numel() < (src_rows - 1) * src_stride + row_elems:
        raise ValueError(f"src: {src.numel()} elements do not hold {src_rows} rows")
    if dst.numel() < (dst_rows - 1) * dst_stride + row_elems:
        raise ValueError(f"dst: {dst.numel()} elements do not hold {dst_rows} rows")
    check(
        lib().iron_copy_rows(
            ptr(src), ptr(dst), rows, row_elems * es, src_stride * es, dst_stride * es, src_rows,
            dst_rows, ptr(_word(src_row, "src_row")), ptr(_word(dst_row, "dst_row")),
            ptr(_word(valid, "valid")), current_stream(),
        ),
        "iron_copy_rows",
    )


def argmax(logits, token, *, n=None, record=None, at=None, token_copy=None):
    n = logits.numel() if n is None else n
    _dev(logits, "logits")
    _dev(token, "token", torch.int32)
    if record is not None:
        _dev(record, "record", torch.int32)
    check(
        lib().iron_argmax_bf16(
            ptr(logits), n, ptr(token), ptr(record), 0 if record is None else record.numel(),
            ptr(_word(at, "at")), ptr(_word(token_copy, "token_copy")), current_stream(),
        ),
        "iron_argmax_bf16",
    )


def sample_workspace(n, device="cuda"):
    """The draw's workspace, zeroed: its first words count a launch's blocks and start at zero."""
    return torch.zeros(lib().iron_sample_workspace_bytes(n) // 8, dtype=torch.int64, device=device)


def sample(logits, draws, token, *, n=None, row=None, k_max=64, workspace=None, record=None, at=None,
           token_copy=None, advance=None):
    """The draw of ``draws``' row at word ``row`` (a device word, or None for the first row).
    ``advance``: ``(words, exprs, n)`` -- word expressions the same launch evaluates once the token is
    written (``eval_words``'s, for the tail of a replayed decode step)."""
    n = logits.numel() if n is None else n
    _dev(logits, "logits")
    _dev(token, "token", torch.int32)
    if draws is not None:
        _dev(draws, "draws", torch.int32)
    if record is not None:
        _dev(record, "record", torch.int32)
    if workspace is None:
        workspace = sample_workspace(n, logits.device)
    need = lib().iron_sample_workspace_bytes(n)
    if workspace.numel() * workspace.element_size() < need:
        raise ValueError(f"workspace: {workspace.numel() * workspace.element_size()} bytes, need {need}")
    common = (ptr(logits), n, ptr(draws), 0 if draws is None else draws.numel(), ptr(_word(row, "row")), k_max,
              ptr(workspace), ptr(token), ptr(record), 0 if record is None else record.numel(),
              ptr(_word(at, "at")), ptr(_word(token_copy, "token_copy")))
    if advance is None:
        check(lib().iron_sample_bf16(*common, current_stream()), "iron_sample_bf16")
        return
    words, exprs, count = advance
    _dev(words, "words", torch.int32)
    _dev(exprs, "exprs", torch.int32)
    if exprs.numel() < 9 * count:
        raise ValueError(f"exprs: {exprs.numel()} words hold fewer than {count} expressions of 9")
    check(lib().iron_sample_advance_bf16(*common, ptr(words), words.numel(), ptr(exprs), count, current_stream()),
          "iron_sample_advance_bf16")


def eval_words(words, exprs, n=None):
    _dev(words, "words", torch.int32)
    _dev(exprs, "exprs", torch.int32)
    n = exprs.numel() // 9 if n is None else n  # nine words a record
    check(lib().iron_eval_words(ptr(words), words.numel(), ptr(exprs), n, current_stream()), "iron_eval_words")



# ---- the float32 stream and the layers that carry a state (rows of a batch told apart by spans)


def _act(t, n, name):
    """An activation operand, bf16 or float32: its number of elements checked, and whether it is float."""
    _dev(t, name, torch.float32 if t.dtype == torch.float32 else BF16)
    _numel(t, n, name)
    return t.dtype == torch.float32


def _same_kind(is_float, **tensors):
    for name, t in tensors.items():
        if (t.dtype == torch.float32) != is_float:
            raise TypeError(f"{name}: {t.dtype} beside {'float32' if is_float else 'bfloat16'} activations")


def _f32(t, n, name):
    _numel(_dev(t, name, torch.float32), n, name)


def _bf16(t, n, name):
    _numel(_dev(t, name), n, name)


def _spans(t, slots):
    _numel(_dev(t, "spans", torch.int32), 4 * slots, "spans")
    return ptr(t)


def stream_embed(table, ids, x, *, rows, table_rows, cols, scale=1.0, also=None, valid=None):
    _bf16(table, table_rows * cols, "table")
    _numel(_dev(ids, "ids", torch.int32), rows, "ids")
    _f32(x, rows * cols, "x")
    if also is not None:
        _f32(also, rows * cols, "also")
    check(lib().iron_stream_embed(ptr(table), ptr(ids), ptr(x), ptr(also), rows, table_rows, cols, float(scale),
                                  ptr(_word(valid, "valid")), current_stream()), "iron_stream_embed")


def _added(x, y, y_bias, back_gain, h, rows, cols):
    """The operands of a row that joins the stream and of one that leaves it; whether activations are float."""
    _f32(x, rows * cols, "x")
    is_float = False
    for t, name in ((y, "y"), (h, "h")):
        if t is not None:
            is_float = _act(t, rows * cols, name)
    for t, name in ((y_bias, "y_bias"), (back_gain, "the gain of y")):
        if t is not None:
            _bf16(t, cols, name)
    if y is not None and h is not None:
        _same_kind(is_float, y=y)
    return is_float


def stream_rows(x, *, rows, cols, eps, unit=0.0, y=None, y_bias=None, back_gain=None, h=None, gain=None, valid=None):
    """``x += rmsnorm(y + y_bias) * (unit + back_gain)`` (with ``y``) and ``h = rmsnorm(x) * (unit + gain)`` (with ``h``), one
    launch."""
    is_float = _added(x, y, y_bias, back_gain, h, rows, cols)
    if h is not None:
        _bf16(gain, cols, "the gain of h")
    check(lib().iron_stream_rows(ptr(x), ptr(y), ptr(y_bias), ptr(back_gain), ptr(gain), ptr(h), rows, cols, float(eps), float(unit),
                                 int(is_float), ptr(_word(valid, "valid")), current_stream()), "iron_stream_rows")


def stream_depth_rows(x, *, rows, cols, eps=0.0, unit=0.0, y=None, y_bias=None, back_gain=None, planes=None, weights=None, plane_rows=0,
                      index=0, h=None, valid=None):
    """``x += rmsnorm(y + y_bias) * (unit + back_gain)`` (with ``y``); with ``planes``, ``planes[index] = x`` and ``x`` the sum of
    ``weights[j] * planes[j]``; ``h = x`` (with ``h``), one launch."""
    is_float = _added(x, y, y_bias, back_gain, h, rows, cols)
    if planes is not None:
        _bf16(weights, index + 1, "weights")
        if _dev(planes, "planes", torch.float32).numel() < (index + 1) * plane_rows * cols:
            raise ValueError(f"planes: {planes.numel()} elements hold no {index + 1} planes of {plane_rows} rows of {cols}")
    check(lib().iron_stream_depth_rows(ptr(x), ptr(y), ptr(y_bias), ptr(back_gain), ptr(planes), ptr(weights), plane_rows, index, ptr(h),
                                       rows, cols, float(eps), float(unit), int(is_float), ptr(_word(valid, "valid")), current_stream()),
          "iron_stream_depth_rows")


def stream_groups(x, *, rows, cols, groups=1, eps=0.0, unit=0.0, y=None, y2=None, h=None, gain=None, valid=None):
    """``x += y + y2`` (with ``y``; ``y2`` may be missing) and ``h``, the norm by ``groups`` of a row times ``unit + gain`` (with
    ``h``), one launch."""
    is_float = _added(x, y, None, None, h, rows, cols)
    if y2 is not None:
        _same_kind(is_float, y2=y2)
        _act(y2, rows * cols, "y2")
    if h is not None:
        _bf16(gain, cols, "the gain of h")
    check(lib().iron_stream_groups(ptr(x), ptr(y), ptr(y2), ptr(gain), ptr(h), rows, cols, groups, float(eps), float(unit), int(is_float),
                                   ptr(_word(valid, "valid")), current_stream()), "iron_stream_groups")


COLUMN_GATES = {"limited": 0, **GATES}   # by the C ABI's number


def gated_columns(x, y, *, rows, cols, stride, gate_at, width, at, kind, limit=0.0, valid=None):
    is_float = _act(x, rows * stride, "x")
    _same_kind(is_float, y=y)
    _act(y, rows * width, "y")
    check(lib().iron_gated_columns(ptr(x), ptr(y), rows, cols, stride, gate_at, width, at, COLUMN_GATES[kind], float(limit), int(is_float),
                                   ptr(_word(valid, "valid")), current_stream()), "iron_gated_columns")


def hgrn2(x, f_bias, lower, state, spans, o, *, slots, rows, stride, heads, dim, vdim, workspace=None):
    """The recurrence token by token, or with ``workspace`` sixteen tokens at a time."""
    is_float = _act(x, rows * stride, "x")
    _bf16(f_bias, heads * dim, "f_bias")
    _bf16(lower, heads * dim, "lower")
    _f32(state, slots * heads * dim * vdim, "state")
    _f32(o, rows * heads * vdim, "o")
    sizes = (slots, rows, stride, heads, dim, vdim, int(is_float), current_stream())
    if workspace is not None:
        work = _work(workspace, int(lib().iron_hgrn2_workspace_bytes(slots, rows, heads, dim)), "hgrn2: workspace")
        check(lib().iron_hgrn2_chunked(ptr(x), ptr(f_bias), ptr(lower), ptr(state), _spans(spans, slots), ptr(o), work, *sizes), "iron_hgrn2_chunked")
        return
    check(lib().iron_hgrn2(ptr(x), ptr(f_bias), ptr(lower), ptr(state), _spans(spans, slots), ptr(o), *sizes), "iron_hgrn2")


def _choice(z, correction, logits, top, ids, shares):
    """A router's choice beside a step's mixer: the C ABI's arguments for it."""
    if z is None:
        return None, None, 0, 0, None, None
    _f32(z, logits, "z")
    if correction is not None:
        _bf16(correction, logits, "correction")
    _numel(_dev(ids, "ids", torch.int32), top, "ids")
    _f32(shares, top, "shares")
    return ptr(z), ptr(correction), logits, top, ptr(ids), ptr(shares)


def decode_hgrn2(x, f_bias, lower, norm, state, spans, out, *, slots, rows, stride, heads, dim, vdim, out_stride, out_at, eps, cols=0, gate_at=0,
                 gated_at=0, kind="limited", limit=0.0, z=None, correction=None, logits=0, top=0, ids=None, shares=None):
    """A decode step's forget gate, fading memory and head norm beside a feed-forward's gated columns and a router's choice."""
    _bf16(x, rows * stride, "x")
    _bf16(f_bias, heads * dim, "f_bias")
    _bf16(lower, heads * dim, "lower")
    _bf16(norm, vdim, "norm")
    _f32(state, slots * heads * dim * vdim, "state")
    _bf16(out, rows * out_stride, "out")
    check(lib().iron_decode_hgrn2_bf16(ptr(x), ptr(f_bias), ptr(lower), ptr(norm), ptr(state), _spans(spans, slots), ptr(out), slots, rows, stride,
                                       heads, dim, vdim, out_stride, out_at, float(eps), cols, gate_at, gated_at, COLUMN_GATES[kind], float(limit),
                                       *_choice(z, correction, logits, top, ids, shares), current_stream()), "iron_decode_hgrn2_bf16")


def decode_heads_global(x, q, keys, values, q_gain, k_gain, spans, *, slots, rows, stride, heads, kv_heads, dim, vdim, context, eps, turned=0,
                        angle_rows=1, angles=None, value_norm=False, out=None, out_stride=0, cols=0, gate_at=0, gated_at=0, kind="limited", limit=0.0,
                        z=None, correction=None, logits=0, top=0, ids=None, shares=None):
    """A decode step's heads into their caches beside a feed-forward's gated columns and a router's choice."""
    _bf16(x, rows * stride, "x")
    _bf16(q, rows * heads * dim, "q")
    _bf16(keys, slots * kv_heads * context * dim, "keys")
    _bf16(values, slots * kv_heads * context * vdim, "values")
    _bf16(q_gain, dim, "q_gain")
    _bf16(k_gain, dim, "k_gain")
    if cols:
        _bf16(out, rows * out_stride, "out")
    check(lib().iron_decode_heads_global_bf16(ptr(x), ptr(q), ptr(keys), ptr(values), ptr(q_gain), ptr(k_gain), _turned(angles, angle_rows, turned),
                                              _spans(spans, slots), slots, rows, stride, heads, kv_heads, dim, vdim, context, turned, angle_rows,
                                              int(value_norm), float(eps), ptr(out), out_stride, cols, gate_at, gated_at, COLUMN_GATES[kind],
                                              float(limit), *_choice(z, correction, logits, top, ids, shares), current_stream()),
          "iron_decode_heads_global_bf16")


def norm_product(x, gain, W, y, *, M, K, groups, eps, unit=0.0, h=None, router=None, z=None, logits=0):
    """One row: the stream's, normed in groups, through ``W``; the normed row to ``h`` too, and with ``router`` its logits to ``z``."""
    _f32(x, K, "x")
    _bf16(gain, K, "gain")
    _bf16(W, M * K, "W")
    _bf16(y, M, "y")
    if h is not None:
        _bf16(h, K, "h")
    if router is not None:
        _bf16(router, logits * K, "router")
        _f32(z, logits, "z")
    check(lib().iron_norm_product_bf16(ptr(x), ptr(gain), groups, float(eps), float(unit), ptr(W), M, K, ptr(y), ptr(h), ptr(router), logits, ptr(z),
                                       current_stream()), "iron_norm_product_bf16")


def product_sum(x, W, stream, *, M, K, also=None):
    """One row: ``stream += W x + also``."""
    _bf16(x, K, "x")
    _bf16(W, M * K, "W")
    _f32(stream, M, "stream")
    if also is not None:
        _bf16(also, M, "also")
    check(lib().iron_product_sum_bf16(ptr(x), ptr(W), M, K, ptr(also), ptr(stream), current_stream()), "iron_product_sum_bf16")


def experts_tail(h, gate, up, down, ids, shares, out, made, stream, workspace, *, cols, ff, inner, experts, top, activation, identity=0):
    """One row: its experts, and with their sums ``out`` times ``made``, both onto the stream's row."""
    _bf16(h, cols, "h")
    for t, name in ((gate, "gate"), (up, "up"), (down, "down")):
        _bf16(t, experts * ff * cols, name)
    _numel(_dev(ids, "ids", torch.int32), top, "ids")
    _f32(shares, top, "shares")
    _bf16(out, cols * inner, "out")
    _bf16(made, inner, "made")
    _f32(stream, cols, "stream")
    check(lib().iron_experts_tail_bf16(ptr(h), ptr(gate), ptr(up), ptr(down), ptr(ids), ptr(shares), ptr(out), ptr(made), ptr(stream),
                                       _work(workspace, 2 * top * ff, "experts_tail: workspace"), cols, ff, inner, experts, identity, top,
                                       GATES[activation], current_stream()), "iron_experts_tail_bf16")


def cached_heads(x, q, keys, values, q_gain, k_gain, spans, *, slots, rows, stride, heads, kv_heads, dim, vdim, context, eps, turned=0,
                 angle_rows=1, angles=None, value_norm=False, valid=None):
    is_float = _act(x, rows * stride, "x")
    _same_kind(is_float, q=q, keys=keys, values=values)
    _act(q, rows * heads * dim, "q")
    _act(keys, slots * kv_heads * context * dim, "keys")
    _act(values, slots * kv_heads * context * vdim, "values")
    _bf16(q_gain, dim, "q_gain")
    _bf16(k_gain, dim, "k_gain")
    check(lib().iron_cached_heads(ptr(x), ptr(q), ptr(keys), ptr(values), ptr(q_gain), ptr(k_gain), _turned(angles, angle_rows, turned),
                                  _spans(spans, slots), slots, rows, stride, heads, kv_heads, dim, vdim, context, turned, angle_rows,
                                  int(value_norm), float(eps), int(is_float), ptr(_word(valid, "valid")), current_stream()), "iron_cached_heads")


def mha_global(q, keys, values, spans, y, *, slots, rows, heads, kv_heads, dim, vdim, context, scale, cap=0.0, sink=False, out_stride, out_at=0,
               single=False, workspace=None):
    is_float = _act(q, rows * heads * dim, "q")
    _same_kind(is_float, keys=keys, values=values, y=y)
    _act(keys, slots * kv_heads * context * dim, "keys")
    _act(values, slots * kv_heads * context * vdim, "values")
    _act(y, rows * out_stride, "y")
    need = int(lib().iron_mha_global_workspace_bytes(slots, heads, kv_heads, vdim, context, int(single)))
    work = _work(workspace, need, "mha_global: workspace") if need else None
    check(lib().iron_mha_global(ptr(q), ptr(keys), ptr(values), _spans(spans, slots), ptr(y), work, slots, rows, heads, kv_heads, dim, vdim,
                                context, float(scale), float(cap), int(sink), out_stride, out_at, int(single), int(is_float), current_stream()),
          "iron_mha_global")


def activation(x, y, *, rows, cols, kind, valid=None):
    is_float = _act(x, rows * cols, "x")
    _same_kind(is_float, y=y)
    _act(y, rows * cols, "y")
    check(lib().iron_activation(ptr(x), ptr(y), rows, cols, GATES[kind], int(is_float), ptr(_word(valid, "valid")), current_stream()),
          "iron_activation")


def turned_heads(x, y, bias, q_gain, k_gain, temp, spans, *, slots, rows, stride, heads, kv_heads, dim, vdim, scale, eps, turned=0,
                 angle_rows=1, angles=None, share=None, first=None, first_stride=0, first_at=0, valid=None):
    is_float = _act(x, rows * stride, "x")
    _same_kind(is_float, y=y)
    _act(y, rows * stride, "y")
    _bf16(bias, heads * dim + kv_heads * (dim + vdim), "bias")
    for t, n, name in ((q_gain, dim, "q_gain"), (k_gain, dim, "k_gain"), (temp, heads, "temp")):
        _bf16(t, n, name)
    if first is not None:
        _same_kind(is_float, first=first)
        _act(first, rows * first_stride, "first")
        _bf16(share, 1, "share")
    check(lib().iron_turned_heads(ptr(x), ptr(y), ptr(bias), ptr(q_gain), ptr(k_gain), ptr(temp), _turned(angles, angle_rows, turned),
                                  ptr(share), ptr(first), first_stride, first_at, _spans(spans, slots), slots, rows, stride, heads, kv_heads,
                                  dim, vdim, turned, angle_rows, float(scale), float(eps), int(is_float), ptr(_word(valid, "valid")),
                                  current_stream()), "iron_turned_heads")


def mha_talking(x, keys, values, talk, spans, y, workspace, *, slots, rows, stride, heads, kv_heads, dim, vdim, chunk, ring, single=False):
    is_float = _act(x, rows * stride, "x")
    _same_kind(is_float, keys=keys, values=values, y=y)
    _act(keys, slots * ring * kv_heads * dim, "keys")
    _act(values, slots * ring * kv_heads * vdim, "values")
    _bf16(talk, heads * heads, "talk")
    _act(y, rows * heads * vdim, "y")
    need = int(lib().iron_mha_talking_workspace_bytes(slots, rows, heads, vdim, chunk, int(single)))
    work = _work(workspace, need, "mha_talking: workspace")
    check(lib().iron_mha_talking(ptr(x), ptr(keys), ptr(values), ptr(talk), _spans(spans, slots), ptr(y), work, slots, rows, stride, heads, kv_heads,
                                 dim, vdim, chunk, ring, int(single), int(is_float), current_stream()), "iron_mha_talking")


def matrix_memory(x, i_bias, f_bias, state, tops, spans, o, *, slots, rows, stride, heads, dim, vdim, i_at, f_at, cap, workspace=None):
    """The recurrence token by token, or with ``workspace`` sixteen tokens at a time."""
    is_float = _act(x, rows * stride, "x")
    _bf16(i_bias, heads, "i_bias")
    _bf16(f_bias, heads, "f_bias")
    _f32(state, slots * heads * dim * (vdim + 1), "state")
    _f32(tops, slots * 2 * heads, "tops")
    _f32(o, rows * heads * (vdim + 2), "o")
    if workspace is not None:
        work = _work(workspace, int(lib().iron_matrix_memory_workspace_bytes(slots, rows, heads, dim)), "matrix_memory: workspace")
        check(lib().iron_matrix_memory_chunked(ptr(x), ptr(i_bias), ptr(f_bias), ptr(state), ptr(tops), _spans(spans, slots), ptr(o), work,
                                               slots, rows, stride, heads, dim, vdim, i_at, f_at, float(cap), int(is_float), current_stream()),
              "iron_matrix_memory_chunked")
        return
    check(lib().iron_matrix_memory(ptr(x), ptr(i_bias), ptr(f_bias), ptr(state), ptr(tops), _spans(spans, slots), ptr(o), slots, rows, stride,
                                   heads, dim, vdim, i_at, f_at, float(cap), int(is_float), current_stream()), "iron_matrix_memory")


def memory_gate(o, gate, gain, y, *, rows, heads, dim, gate_stride, gate_at, floor, eps, valid=None):
    _f32(o, rows * heads * (dim + 2), "o")
    is_float = _act(gate, rows * gate_stride, "gate")
    _bf16(gain, heads * dim, "gain")
    _same_kind(is_float, y=y)
    _act(y, rows * heads * dim, "y")
    check(lib().iron_memory_gate(ptr(o), ptr(gate), ptr(gain), ptr(y), rows, heads, dim, gate_stride, gate_at, float(floor), float(eps),
                                 int(is_float), ptr(_word(valid, "valid")), current_stream()), "iron_memory_gate")


def router(h, w, bias, ids, shares, *, rows, cols, experts, top, correction=None, scored=False, valid=None):
    is_float = _act(h, rows * cols, "h")
    _bf16(w, experts * cols, "w")
    for t, name in ((bias, "bias"), (correction, "correction")):
        if t is not None:
            _bf16(t, experts, name)
    _numel(_dev(ids, "ids", torch.int32), rows * top, "ids")
    _f32(shares, rows * top, "shares")
    check(lib().iron_router(ptr(h), ptr(w), ptr(bias), ptr(correction), int(scored), ptr(ids), ptr(shares), rows, cols, experts, top, int(is_float),
                            ptr(_word(valid, "valid")), current_stream()), "iron_router")


def experts(h, gate, up, down, ids, shares, y, workspace, *, rows, cols, ff, experts, top, activation, identity=0, valid=None):
    is_float = _act(h, rows * cols, "h")
    for t, name in ((gate, "gate"), (up, "up"), (down, "down")):
        _bf16(t, experts * ff * cols, name)
    _numel(_dev(ids, "ids", torch.int32), rows * top, "ids")
    _f32(shares, rows * top, "shares")
    _same_kind(is_float, y=y)
    _act(y, rows * cols, "y")
    need = int(lib().iron_experts_workspace_bytes(rows, cols, ff, experts, top, int(is_float)))
    check(lib().iron_experts(ptr(h), ptr(gate), ptr(up), ptr(down), ptr(ids), ptr(shares), ptr(y), _work(workspace, need, "experts: workspace"),
                             rows, cols, ff, experts, identity, top, GATES[activation], int(is_float), ptr(_word(valid, "valid")),
                             current_stream()), "iron_experts")


def stream_gated_rows(x, y, gate, gate_bias, *, rows, cols, eps=0.0, gate_stride, gate_at, y_bias=None, h=None, gain=None, valid=None):
    """``x += (y + y_bias) * sigmoid(gate + gate_bias)`` and, with ``h``, ``h = rmsnorm(x) * gain``, one launch."""
    _f32(x, rows * cols, "x")
    is_float = _act(y, rows * cols, "y")
    _same_kind(is_float, gate=gate)
    _act(gate, rows * gate_stride, "gate")
    _bf16(gate_bias, cols, "gate_bias")
    if y_bias is not None:
        _bf16(y_bias, cols, "y_bias")
    if h is not None:
        _same_kind(is_float, h=h)
        _act(h, rows * cols, "h")
        _bf16(gain, cols, "gain")
    check(lib().iron_stream_gated_rows(ptr(x), ptr(y), ptr(y_bias), ptr(gate), ptr(gate_bias), gate_stride, gate_at, ptr(gain), ptr(h),
                                       rows, cols, float(eps), int(is_float), ptr(_word(valid, "valid")), current_stream()),
          "iron_stream_gated_rows")


def poly_norm(x, coefficients, y, *, rows, cols, stride, at, eps, bias=None, valid=None):
    is_float = _act(x, rows * stride, "x")
    _bf16(coefficients, 4, "coefficients")
    if bias is not None:
        _bf16(bias, cols, "bias")
    _same_kind(is_float, y=y)
    _act(y, rows * cols, "y")
    check(lib().iron_poly_norm(ptr(x), ptr(bias), ptr(coefficients), ptr(y), rows, cols, stride, at, float(eps), int(is_float),
                               ptr(_word(valid, "valid")), current_stream()), "iron_poly_norm")


def span_tails(x, spans, out, *, slots, rows, cols):
    _f32(x, rows * cols, "x")
    _f32(out, slots * cols, "out")
    check(lib().iron_span_tails(ptr(x), _spans(spans, slots), ptr(out), slots, rows, cols, current_stream()),
          "iron_span_tails")


def softcap(x, y, rounded, *, rows, cols, stride, cap, scale=1.0):
    is_float = _act(x, rows * cols, "x")
    _f32(y, rows * cols, "y")
    _bf16(rounded, rows * stride, "rounded")
    check(lib().iron_softcap(ptr(x), ptr(y), ptr(rounded), rows, cols, stride, float(cap), float(scale), int(is_float),
                             current_stream()), "iron_softcap")


def act_mul_f32(gate, up, y, *, rows, cols, activation, valid=None):
    for t, name in ((gate, "gate"), (up, "up"), (y, "y")):
        _f32(t, rows * cols, name)
    check(lib().iron_act_mul_f32(ptr(gate), ptr(up), ptr(y), rows, cols, GATES[activation], ptr(_word(valid, "valid")),
                                 current_stream()), "iron_act_mul_f32")


def linear_any(x, w, y, *, rows, n, k, valid=None):
    is_float = _act(x, rows * k, "x")
    _bf16(w, n * k, "w")
    _same_kind(is_float, y=y)
    _act(y, rows * n, "y")
    check(lib().iron_linear_any(ptr(x), ptr(w), ptr(y), rows, n, k, int(is_float), ptr(_word(valid, "valid")),
                                current_stream()), "iron_linear_any")


def token_shift(h, mu, carry, spans, mixed, *, slots, rows, cols, mixes):
    is_float = _act(h, rows * cols, "h")
    _bf16(mu, mixes * cols, "mu")
    _same_kind(is_float, carry=carry, mixed=mixed)
    _act(carry, slots * 2 * cols, "carry")
    _act(mixed, mixes * rows * cols, "mixed")
    check(lib().iron_token_shift(ptr(h), ptr(mu), ptr(carry), _spans(spans, slots), ptr(mixed), slots, rows, cols, mixes,
                                 int(is_float), current_stream()), "iron_token_shift")


def low_rank_decay(z, w2, w0, out, *, rows, n, rank, valid=None):
    is_float = _act(z, rows * rank, "z")
    _bf16(w2, n * rank, "w2")
    _bf16(w0, n, "w0")
    _f32(out, rows * n, "out")
    check(lib().iron_low_rank_decay(ptr(z), ptr(w2), ptr(w0), ptr(out), rows, n, rank, int(is_float),
                                    ptr(_word(valid, "valid")), current_stream()), "iron_low_rank_decay")


def _work(t, nbytes, name):
    if _dev(t, name, None).numel() * t.element_size() < nbytes:
        raise ValueError(f"{name}: {t.numel() * t.element_size()} bytes, {nbytes} needed")
    return ptr(t)


def time_mix(r, k, v, log_decay, u, state, spans, o, *, slots, rows, heads, dim, workspace=None):
    """The recurrence token by token, or with ``workspace`` sixteen tokens at a time."""
    n = rows * heads * dim
    is_float = _act(r, n, "r")
    _same_kind(is_float, k=k, v=v)
    _act(k, n, "k")
    _act(v, n, "v")
    _f32(log_decay, n, "log_decay")
    _bf16(u, heads * dim, "u")
    _f32(state, slots * heads * dim * dim, "state")
    _f32(o, n, "o")
    if workspace is not None:
        work = _work(workspace, int(lib().iron_time_mix_workspace_bytes(slots, rows, heads, dim)), "time_mix: workspace")
        check(lib().iron_time_mix_chunked(ptr(r), ptr(k), ptr(v), ptr(log_decay), ptr(u), ptr(state), _spans(spans, slots),
                                          ptr(o), work, slots, rows, heads, dim, int(is_float), current_stream()),
              "iron_time_mix_chunked")
        return
    check(lib().iron_time_mix(ptr(r), ptr(k), ptr(v), ptr(log_decay), ptr(u), ptr(state), _spans(spans, slots), ptr(o), slots,
                              rows, heads, dim, int(is_float), current_stream()), "iron_time_mix")


def short_conv(x, taps_w, a_log, dt_bias, state, spans, out, *, slots, rows, stride, heads, kv_heads, dim, vdim, taps,
               b_at, a_at):
    channels = 2 * kv_heads * dim + heads * vdim
    is_float = _act(x, rows * stride, "x")
    _bf16(taps_w, channels * taps, "taps_w")
    _bf16(a_log, heads, "a_log")
    _bf16(dt_bias, heads, "dt_bias")
    _same_kind(is_float, state=state)
    _act(state, slots * taps * channels, "state")
    _f32(out, rows * (channels + 2 * heads), "out")
    check(lib().iron_short_conv(ptr(x), ptr(taps_w), ptr(a_log), ptr(dt_bias), ptr(state), _spans(spans, slots), ptr(out),
                                slots, rows, stride, heads, kv_heads, dim, vdim, taps, b_at, a_at, int(is_float),
                                current_stream()), "iron_short_conv")


def delta_rule(x, state, spans, o, *, slots, rows, heads, kv_heads, dim, vdim, workspace=None):
    """The recurrence token by token, or with ``workspace`` sixteen tokens at a time."""
    _f32(x, rows * (2 * kv_heads * dim + heads * vdim + 2 * heads), "x")
    _f32(state, slots * heads * dim * vdim, "state")
    _f32(o, rows * heads * vdim, "o")
    if workspace is not None:
        work = _work(workspace, int(lib().iron_delta_rule_workspace_bytes(slots, rows, heads)), "delta_rule: workspace")
        check(lib().iron_delta_rule_chunked(ptr(x), ptr(state), _spans(spans, slots), ptr(o), work, slots, rows, heads, kv_heads,
                                            dim, vdim, current_stream()), "iron_delta_rule_chunked")
        return
    check(lib().iron_delta_rule(ptr(x), ptr(state), _spans(spans, slots), ptr(o), slots, rows, heads, kv_heads, dim, vdim,
                                current_stream()), "iron_delta_rule")


def head_gate(o, gate, gain, out, *, rows, heads, dim, gate_stride, gate_at, gain_shared, out_stride, out_at, eps, scale,
              valid=None):
    _f32(o, rows * heads * dim, "o")
    is_float = _act(out, rows * out_stride, "out")
    _bf16(gain, dim if gain_shared else heads * dim, "gain")
    if gate is not None:
        _same_kind(is_float, gate=gate)
        _act(gate, rows * gate_stride, "gate")
    check(lib().iron_head_gate(ptr(o), ptr(gate), ptr(gain), ptr(out), rows, heads, dim, gate_stride, gate_at,
                               int(gain_shared), out_stride, out_at, float(eps), float(scale), int(is_float),
                               ptr(_word(valid, "valid")), current_stream()), "iron_head_gate")


def mha_window(x, keys, values, bias, spans, out, *, slots, rows, stride, heads, kv_heads, dim, vdim, window, ring, scale,
               out_stride, out_at=0, out_scale=1.0, single=False):
    is_float = _act(x, rows * stride, "x")
    _same_kind(is_float, keys=keys, values=values, out=out)
    _act(keys, slots * ring * kv_heads * dim, "keys")
    _act(values, slots * ring * kv_heads * vdim, "values")
    _f32(bias, heads * window, "bias")
    _act(out, rows * out_stride, "out")
    check(lib().iron_mha_window(ptr(x), ptr(keys), ptr(values), ptr(bias), _spans(spans, slots), ptr(out), slots, rows, stride,
                                heads, kv_heads, dim, vdim, window, ring, float(scale), out_stride, out_at, float(out_scale),
                                int(single), int(is_float), current_stream()), "iron_mha_window")


def min_gru(x, z_bias, x_bias, state, spans, y, *, slots, rows, stride, width, workspace=None):
    """The gated recurrence a span's rows in turn, or with ``workspace`` its chunks side by side."""
    is_float = _act(x, rows * stride, "x")
    _bf16(z_bias, width, "z_bias")
    _bf16(x_bias, width, "x_bias")
    _f32(state, slots * 2 * width, "state")
    _same_kind(is_float, y=y)
    _act(y, rows * width, "y")
    work = None if workspace is None else _work(workspace, int(lib().iron_min_gru_workspace_bytes(slots, rows, width)), "min_gru: workspace")
    check(lib().iron_min_gru(ptr(x), ptr(z_bias), ptr(x_bias), ptr(state), _spans(spans, slots), ptr(y), work, slots, rows, stride,
                             width, int(is_float), current_stream()), "iron_min_gru")


def _turned(angles, angle_rows, turned):
    if turned:
        _f32(angles, angle_rows * turned, "angles")
    return ptr(angles)


def latent_rows(x, q_gain, c_gain, spans, q_out, latents, *, slots, rows, stride, q_rank, rank, ring, eps, rot=0, turned=0,
                angle_rows=0, angles=None, shared_keys=None):
    is_float = _act(x, rows * stride, "x")
    _bf16(q_gain, q_rank, "q_gain")
    _bf16(c_gain, rank, "c_gain")
    _same_kind(is_float, q_out=q_out, latents=latents)
    _act(q_out, rows * q_rank, "q_out")
    _act(latents, slots * ring * rank, "latents")
    if rot:
        _same_kind(is_float, shared_keys=shared_keys)
        _act(shared_keys, slots * ring * rot, "shared_keys")
    check(lib().iron_latent_rows(ptr(x), ptr(q_gain), ptr(c_gain), _turned(angles, angle_rows, turned), _spans(spans, slots), ptr(q_out),
                                 ptr(latents), ptr(shared_keys), slots, rows, stride, q_rank, rank, rot, turned, angle_rows, ring,
                                 float(eps), int(is_float), current_stream()), "iron_latent_rows")


def mha_latent(q, latents, up, spans, y, workspace, *, slots, rows, heads, dim, vdim, rank, window, ring, cap, scale, rot=0, turned=0,
               angle_rows=0, angles=None, shared_keys=None, sink=None, single=False):
    is_float = _act(q, rows * heads * (dim + rot), "q")
    _same_kind(is_float, latents=latents, y=y)
    _act(latents, slots * ring * rank, "latents")
    if rot:
        _same_kind(is_float, shared_keys=shared_keys)
        _act(shared_keys, slots * ring * rot, "shared_keys")
    _bf16(up, heads * (dim + vdim) * rank, "up")
    if sink is not None:
        _bf16(sink, heads, "sink")
    _act(y, rows * heads * vdim, "y")
    need = int(lib().iron_mha_latent_workspace_bytes(slots, rows, heads, dim, rot, vdim, rank, window, ring, cap, int(single), int(is_float)))
    check(lib().iron_mha_latent(ptr(q), ptr(latents), ptr(shared_keys), ptr(up), ptr(sink), _turned(angles, angle_rows, turned),
                                _spans(spans, slots), ptr(y), _work(workspace, need, "mha_latent: workspace"), slots, rows, heads, dim,
                                rot, vdim, rank, turned, angle_rows, window, ring, cap, float(scale), int(single), int(is_float),
                                current_stream()), "iron_mha_latent")


STREAM_INPUTS = {"row": 0, "stream_norm": 1, "row_norm": 2, "min_gru": 3, "poly_norm": 4}   # by the C ABI's number


def stream_product(W, x, *, input, M, K, y=None, stream=None, y_bias=None, gate=None, gate_bias=None, gain=None, b0=None, b1=None,
                   state=None, spans=None, eps=0.0, unit=0.0):
    """One row's product: ``input`` says how its input is made of ``x``; the output is the row ``y``, or joins the
    stream's row ``stream`` through ``gate`` (its first M elements)."""
    _bf16(W, M * K, "W")
    if input == "stream_norm":
        _f32(x, K, "x")
    elif _dev(x, "x").numel() < (3 * K if input == "min_gru" else K):
        raise ValueError(f"stream_product: x holds {x.numel()} elements")
    for t, n, name in ((y, M, "y"), (y_bias, M, "y_bias"), (gate_bias, M, "gate_bias"), (gain, 4 if input == "poly_norm" else K, "gain"),
                       (b0, K, "b0"), (b1, K, "b1")):
        if t is not None:
            _bf16(t, n, name)
    if state is not None:
        _f32(state, 2 * K, "state")
    if stream is not None:
        _f32(stream, M, "stream")
        if _dev(gate, "gate").numel() < M:
            raise ValueError(f"stream_product: a gate of {gate.numel()} elements for {M}")
    check(lib().iron_stream_product_bf16(STREAM_INPUTS[input], ptr(x), ptr(gain), ptr(b0), ptr(b1), ptr(state),
                                         None if spans is None else _spans(spans, 1), float(eps), float(unit), ptr(W), M, K, ptr(y), ptr(stream), ptr(y_bias),
                                         ptr(gate), ptr(gate_bias), current_stream()), "iron_stream_product_bf16")


def latent_query(x, q_gain, c_gain, spans, W, q, latents, *, M, stride, q_rank, rank, ring, eps, rot=0, turned=0, angle_rows=0,
                 angles=None, shared_keys=None):
    """A single slot's row: its latents normed, stored and turned, and the queries' product."""
    _bf16(x, stride, "x")
    _bf16(q_gain, q_rank, "q_gain")
    _bf16(c_gain, rank, "c_gain")
    _bf16(W, M * q_rank, "W")
    _bf16(q, M, "q")
    _bf16(latents, ring * rank, "latents")
    if rot:
        _bf16(shared_keys, ring * rot, "shared_keys")
    check(lib().iron_latent_query_bf16(ptr(x), ptr(q_gain), ptr(c_gain), _turned(angles, angle_rows, turned), _spans(spans, 1), ptr(W), ptr(q),
                                       ptr(latents), ptr(shared_keys), M, stride, q_rank, rank, rot, turned, angle_rows, ring, float(eps),
                                       current_stream()), "iron_latent_query_bf16")


def decode_mixed(h, carry, spans, products, *, k):
    """A token shift and the projections of its blends, one row, one launch.  ``products``: (weight, output,
    mu row or None) each."""
    _bf16(h, k, "h")
    _bf16(carry, 2 * k, "carry")
    n = len(products)
    for w, y, mu in products:
        _dev(w, "weight")
        if w.numel() != y.numel() * k:
            raise ValueError(f"decode_mixed: a weight of {w.numel()} elements for {y.numel()} rows of {k}")
        _dev(y, "output")
        if mu is not None:
            _bf16(mu, k, "mu")
    pointers = ctypes.c_void_p * n
    check(lib().iron_decode_mixed_bf16(ptr(h), ptr(carry), _spans(spans, 1), k, n, pointers(*(ptr(w) for w, _, _ in products)),
                                       pointers(*(ptr(y) for _, y, _ in products)), pointers(*(ptr(m) for _, _, m in products)),
                                       (ctypes.c_int * n)(*(y.numel() for _, y, _ in products)), current_stream()),
          "iron_decode_mixed_bf16")


def decode_parallel(r, k, v, gate, z, w2, w0, u, norm, memory, x, keys, values, bias, spans, out, *, slots, rows, mix_heads,
                    mix_dim, rank, eps, mix_scale, mix_at, stride, heads, kv_heads, dim, vdim, window, ring, scale, out_scale,
                    win_at, out_stride):
    """A decode step's decay, time mixing, head norm and gate beside its windowed attention."""
    inner = mix_heads * mix_dim
    for t, name in ((r, "r"), (k, "k"), (v, "v"), (gate, "gate")):
        _bf16(t, rows * inner, name)
    _bf16(z, rows * rank, "z")
    _bf16(w2, inner * rank, "w2")
    for t, name in ((w0, "w0"), (u, "u"), (norm, "norm")):
        _bf16(t, inner, name)
    _f32(memory, slots * inner * mix_dim, "memory")
    _bf16(x, rows * stride, "x")
    _bf16(keys, slots * ring * kv_heads * dim, "keys")
    _bf16(values, slots * ring * kv_heads * vdim, "values")
    _f32(bias, heads * window, "bias")
    _bf16(out, rows * out_stride, "out")
    check(lib().iron_decode_parallel_bf16(ptr(r), ptr(k), ptr(v), ptr(gate), ptr(z), ptr(w2), ptr(w0), ptr(u), ptr(norm),
                                          ptr(memory), mix_heads, mix_dim, rank, float(eps), float(mix_scale), mix_at, ptr(x),
                                          ptr(keys), ptr(values), ptr(bias), stride, heads, kv_heads, dim, vdim, window, ring,
                                          float(scale), float(out_scale), win_at, _spans(spans, slots), ptr(out), slots, rows,
                                          out_stride, current_stream()), "iron_decode_parallel_bf16")


def decode_delta(x, taps_w, a_log, dt_bias, norm, inputs, state, spans, out, *, slots, rows, stride, heads, kv_heads, dim, vdim,
                 taps, gate_at, b_at, a_at, eps):
    """A decode step's short convolution, gated delta rule, head norm and gate."""
    channels = 2 * kv_heads * dim + heads * vdim
    _bf16(x, rows * stride, "x")
    _bf16(taps_w, channels * taps, "taps_w")
    _bf16(a_log, heads, "a_log")
    _bf16(dt_bias, heads, "dt_bias")
    _bf16(norm, vdim, "norm")
    _bf16(inputs, slots * taps * channels, "inputs")
    _f32(state, slots * heads * dim * vdim, "state")
    _bf16(out, rows * heads * vdim, "out")
    check(lib().iron_decode_delta_bf16(ptr(x), ptr(taps_w), ptr(a_log), ptr(dt_bias), ptr(norm), ptr(inputs), ptr(state),
                                       _spans(spans, slots), ptr(out), slots, rows, stride, heads, kv_heads, dim, vdim, taps,
                                       gate_at, b_at, a_at, float(eps), current_stream()), "iron_decode_delta_bf16")


def sample_slots(logits, spans, draws, token, record, workspace, *, n, stride, slots, batch_rows, steps, k_max=64):
    _bf16(logits, slots * stride, "logits")
    for t, count, name in ((draws, 4 * slots * steps, "draws"), (token, slots, "token"), (record, slots * steps, "record")):
        _numel(_dev(t, name, torch.int32), count, name)
    need = slots * int(lib().iron_sample_workspace_bytes(n))
    if _dev(workspace, "workspace", None).numel() * workspace.element_size() < need:
        raise ValueError(f"sample_slots: the workspace is smaller than {need} bytes")
    check(lib().iron_sample_slots_bf16(ptr(logits), n, stride, _spans(spans, slots), slots, batch_rows, steps, ptr(draws),
                                       k_max, ptr(workspace), ptr(token), ptr(record), current_stream()),
          "iron_sample_slots_bf16")
