"""Step fusion for the versions of a graph.

The recorded steps stay what the reference records -- one operator per step, which is
what ``Graph.reference`` and check mode run.  When a version is loaded for the GPU, runs
of single-row steps that a decoder layer always records together are launched as one
fused kernel each (``iron_amd/csrc/fused.hip``), which rounds wherever the separate steps
round:

  RMSNorm, GEMV q/k/v, RoPE q/k, Copy k/v -> cache      => iron_decode_qkv_bf16
  RMSNorm, GEMV gate, GEMV up, SiLU, ElementwiseMul      => iron_gemv_fused_bf16 (epilogue 2)
  ... with GELU (tanh) for SiLU                          => iron_gemv_fused_bf16 (epilogue 3)
  GEMV, ElementwiseAdd / AXPY (the residual)             => iron_gemv_fused_bf16 (epilogue 1)
  RMSNorm, GEMV (the head; or a layer's q, k, v)         => iron_gemv_fused_bf16 (epilogue 0) each
  GEMV, GELU (tanh) or SiLU, Mul by a given row          => iron_gemv_fused_bf16 (epilogue 4 / 5)
  RMSNorm per head of q/k/v, RoPE q/k, Copy k/v -> cache => iron_decode_heads_bf16

in a prompt chunk's version (several rows, 64-wide heads),

  GEMM q/k/v (one input), RoPE q/k                       => iron_prefill_qkv_bf16
  ... and Copy k/v -> the chunk's cache rows             => iron_prefill_qkv_cache_bf16
  GEMM (gate), GEMM (up), SiLU or GELU (tanh), Mul       => iron_gemm_gated_pair_bf16
  GEMM (up), SiLU or GELU (tanh) of the gate, Mul        => iron_gemm_gated_bf16
  SiLU, ElementwiseMul (no such product before them)     => iron_silu_mul_bf16
  GEMM, ElementwiseAdd / AXPY (the residual)             => iron_gemm_residual_bf16
  ... few rows over a long K, and the RMSNorm after them => iron_gemm_residual_norm_bf16

in a batched decoder's decode step (bf16; a float32 stream, layers with a state),

  [GEMV,] TokenShift, GEMV of its blends (one slot)      => iron_decode_mixed_bf16
  LowRankDecay, TimeMix, HeadGate, WindowMHA             => iron_decode_parallel_bf16
  ShortConv, DeltaRule, HeadGate                         => iron_decode_delta_bf16
  GEMV gate, GEMV up, SiLU / GELU (tanh) / ReLU, Mul     => iron_gemv_fused_bf16 (epilogue 2 / 3 / 6)
  StreamNorm, GEMV (one slot, as the rest here)          => iron_stream_product_bf16 (input 1)
  [MinGRU / PolyNorm,] GEMV, StreamGatedAdd              => iron_stream_product_bf16 (input 0 / 3 / 4)
  LatentRows, GEMV (the queries)                         => iron_latent_query_bf16
  StreamNorm (groups), GEMV                              => iron_norm_product_bf16
  Hgrn2, HeadGate [, GatedColumns] (any slots)           => iron_decode_hgrn2_bf16
  CachedHeads, GlobalMHA [, GatedColumns] (any slots)    => iron_decode_heads_global_bf16, iron_mha_global
  ... either behind StreamNorm, GEMV, Router             => iron_norm_product_bf16 with the logits; the choice beside the mixer
  GEMV, StreamSum                                        => iron_product_sum_bf16
  Experts, GEMV, StreamSum                               => iron_experts_tail_bf16

and in either,

  StreamAdd, StreamNorm                                  => iron_stream_rows
  StreamSum, StreamNorm                                  => iron_stream_groups
  [StreamAdd,] [DepthAverage,] [StreamCast] (two of them) => iron_stream_depth_rows
  StreamGatedAdd, StreamNorm                             => iron_stream_gated_rows
  RMSNorm, ElementwiseAdd (a sandwich layer's residual)  => iron_rmsnorm_add_bf16

A run is fused only if every intermediate it hides is read by nothing else.
"""

from __future__ import annotations

import dataclasses
from collections import Counter
from collections.abc import Callable
from typing import Any

from ..bf16 import bfloat16


@dataclasses.dataclass
class Fused:
    """One launch standing for ``steps`` consecutive recorded steps."""

    kind: str
    first: int
    count: int
    launch: Callable[[], None]
    launches: int = 1      # 0: a step other launches made needless (nothing runs for it)
    scratch_bytes: int = 0  # device memory of its own the launch needs, live over the run


# a gated feed-forward's activation steps: the C ABI's name, and gemv_fused's epilogue
_GATES = {"SiLU": ("silu", 2), "GELU": ("gelu_tanh", 3), "ReLU": ("relu", 6)}


def _gate(step) -> tuple[str, int] | None:
    """The fused launches' names for an activation step they compute, or None."""
    name = type(step.op).__name__
    if name not in _GATES or (name == "GELU" and step.op.approximate != "tanh"):
        return None
    return _GATES[name]


class _Anything:
    """Stands for a tensor while runs are only being matched (before the arena is loaded)."""

    def reshape(self, *a):
        return self

    def __getitem__(self, key):
        return self


def match(recording) -> list[Fused]:
    """The runs ``plan`` would fuse, without binding any tensor: for the arena plan, which must
    keep every buffer a run touches alive across the whole run."""
    return plan(recording, lambda h: _Anything(), lambda e: None, lambda first, nbytes: _Anything())


def _plain(h) -> bool:
    return h.index is None and h.ids is None and not h.valid


def _name(step) -> str:
    return type(step.op).__name__


def _same(a, b) -> bool:
    """Two handles that are the same elements of the same buffer."""
    return a.buffer is b.buffer and a.offset == b.offset and a.elements == b.elements and _plain(a) and _plain(b)


def _same_view(a, b) -> bool:
    """The same elements of the same buffer, whatever bound each carries."""
    return (a.buffer is b.buffer and a.offset == b.offset and a.elements == b.elements
            and a.index is None and a.ids is None and b.index is None and b.ids is None)


def plan(recording, tensor: Callable[[Any], Any], word: Callable[[Any], Any],
         scratch: Callable[[int, int], Any] | None = None) -> list[Fused]:
    """The fused launches of ``recording``'s steps, by the first step each covers.

    ``tensor(handle)`` is the device tensor behind a handle, ``word(expr)`` the device word
    of a per-call expression, ``scratch(first, nbytes)`` the device memory placed for the run
    that starts at step ``first`` (``Fused.scratch_bytes`` of it); without ``scratch`` no run
    that needs memory of its own is planned.
    """
    from .. import kernels

    steps = recording.steps
    reads: Counter = Counter()
    for s in steps:
        for h in s.inputs.values():
            reads[id(h.buffer)] += 1
            if h.ids is not None:
                reads[id(h.ids.buffer)] += 1
    for h in recording.outputs:
        reads[id(h.buffer)] += 1
    for v in (recording.carry or {}).values():
        if hasattr(v, "buffer"):
            reads[id(v.buffer)] += 1

    def once(h, n=1) -> bool:
        return h.buffer.kind == "transient" and reads[id(h.buffer)] == n

    def norm_row(s) -> bool:
        return (_name(s) == "RMSNorm" and s.op.rows == 1 and s.op.weighted and not s.values
                and all(_plain(h) for h in (*s.inputs.values(), *s.outputs.values())))

    def gemv_row(s, x=None) -> bool:
        ok = (_name(s) == "GEMV" and s.op.num_batches is None and not s.values
              and all(_plain(h) for h in (*s.inputs.values(), *s.outputs.values())))
        return ok and (x is None or _same(s.inputs["B"], x))

    def gated_at(j, before=None):
        """``(args, kw)`` of ``iron_gemm_gated_bf16`` where steps j, j + 1, j + 2 are a many-row product, the
        activation of an earlier product of the same shape (the gate) and their Mul, or None.  With
        ``before``, the step right ahead of them must be the product that made the gate, of the same
        rows by the same bound and read by the activation alone."""
        if j + 2 >= len(steps):
            return None
        s, sl, ml = steps[j], steps[j + 1], steps[j + 2]
        if not (_name(s) == "GEMM"
                and _gate(sl) is not None
                and _name(ml) == "ElementwiseMul"
                and s.op.b_col_maj and not s.op.c_col_maj and "valid_k" not in s.values
                and ((s.op.M >= 64 and s.op.N >= 64 and s.op.K % 64 == 0)
                     or (s.op.M < 64 and before is not None and "valid" not in s.values))):   # a batch's few rows
            return None
        up, gate, act = s.outputs["C"], sl.inputs["x"], sl.outputs["y"]
        a, b = ml.inputs["a"], ml.inputs["b"]
        paired = (_same_view(a, act) and _same_view(b, up)) or (_same_view(a, up) and _same_view(b, act))
        gv, sv, mv = s.values.get("valid"), sl.values.get("valid"), ml.values.get("valid")
        # the elementwise bounds count elements, the product's rows
        bounds_agree = sv == mv and ((gv is None and sv is None) or (
            gv is not None and sv is not None and gv.value == sv.value and gv.linear and sv.linear
            and sv.scale == gv.scale * s.op.N and sv.bias == gv.bias * s.op.N))
        flat = all(h.index is None and h.ids is None
                   for h in (*s.inputs.values(), up, gate, act, a, b, ml.outputs["y"]))
        if not (paired and flat and once(up) and once(act) and bounds_agree and gate.buffer is not up.buffer
                and gate.elements == up.elements and sl.op.size == up.elements and ml.op.size == up.elements
                and ml.outputs["y"].elements == up.elements
                and set(sl.values) <= {"valid"} and set(ml.values) <= {"valid"}):
            return None
        if before is not None:
            g = before
            if not (_name(g) == "GEMM" and g.op.b_col_maj and not g.op.c_col_maj and "valid_k" not in g.values
                    and (g.op.M, g.op.N, g.op.K) == (s.op.M, s.op.N, s.op.K) and g.values.get("valid") == gv
                    and _same_view(g.inputs["A"], s.inputs["A"]) and _same_view(g.outputs["C"], gate) and once(gate)
                    and gate.buffer is not ml.outputs["y"].buffer
                    and all(h.index is None and h.ids is None for h in (*g.inputs.values(), g.outputs["C"]))):
                return None
        args = dict(A=tensor(s.inputs["A"]), B=tensor(s.inputs["B"]), G=tensor(gate), C=tensor(ml.outputs["y"]))
        kw = dict(M=s.op.M, N=s.op.N, K=s.op.K, valid=word(gv),
                  activation=_gate(sl)[0])
        return args, kw

    def gated_rows_at(j):
        """``(args, kw)`` of ``iron_gemv_fused_bf16`` where the four steps from ``j`` are one row's gate and up
        projections (of one input), the gate's activation and the product, or None."""
        if j + 3 >= len(steps):
            return None
        gg, gu, si, mu = steps[j : j + 4]
        if not (gemv_row(gg) and gemv_row(gu, gg.inputs["B"]) and _gate(si) is not None and _name(mu) == "ElementwiseMul"):
            return None
        g, u = gg.outputs["C"], gu.outputs["C"]
        if not (_same(si.inputs["x"], g) and once(g) and once(u) and once(si.outputs["y"]) and not si.values and not mu.values
                and _same(mu.inputs["a"], si.outputs["y"]) and _same(mu.inputs["b"], u) and gg.op.M == gu.op.M
                and gg.op.K == gu.op.K and _plain(mu.outputs["y"])):
            return None
        args = dict(W=tensor(gg.inputs["A"]), W2=tensor(gu.inputs["A"]), x=tensor(gg.inputs["B"]).reshape(-1),
                    y=tensor(mu.outputs["y"]).reshape(-1))
        return args, dict(M=gg.op.M, K=gg.op.K, epilogue=_gate(si)[1])

    def mixed_at(j):
        """The launch for a token shift of one row from step ``j`` on, with a projection of the shift's own input
        ahead of it (if there is one) and those of its blends behind it -- or None."""
        ahead = gemv_row(steps[j])
        at = j + 1 if ahead else j
        shift = steps[at] if at < len(steps) else None
        if (shift is None or _name(shift) != "TokenShift" or shift.op.rows != 1 or shift.op.slots != 1
                or shift.op.dtype is not bfloat16 or shift.op.cols % 8):
            return None
        h, blends, K = shift.inputs["h"], shift.outputs["mixed"], shift.op.cols
        if ahead and not _same(steps[j].inputs["B"], h):
            return None
        behind = steps[at + 1 : at + 1 + shift.op.mixes]
        if (len(behind) != shift.op.mixes or shift.op.mixes > 7 or not once(blends, shift.op.mixes)
                or not all(gemv_row(g) and g.inputs["B"].buffer is blends.buffer and g.inputs["B"].elements == K
                           and g.inputs["B"].offset % K == 0 and g.op.K == K for g in behind)):
            return None
        mu = tensor(shift.inputs["mu"])
        gemvs = ([steps[j]] if ahead else []) + behind
        products = [(tensor(g.inputs["A"]), tensor(g.outputs["C"]).reshape(-1),
                     mu[g.inputs["B"].offset // K] if g is not steps[j] or not ahead else None) for g in gemvs]
        args = dict(h=tensor(h).reshape(-1), carry=tensor(shift.inputs["carry"]).reshape(-1),
                    spans=tensor(shift.inputs["spans"]), products=products)
        return Fused("decode_mixed", j, len(gemvs) + 1, lambda a=args: kernels.decode_mixed(**a, k=K))

    def gate_behind(o, gate):
        """Whether ``gate`` is the head norm and gate of a recurrence's output, read by nothing else."""
        return (_name(gate) == "HeadGate" and _same(gate.inputs["o"], o) and once(o) and not gate.values
                and gate.op.dtype is bfloat16)

    def parallel_at(j):
        """The launch for a decode step's time mixing beside its windowed attention -- or None."""
        if j + 3 >= len(steps):
            return None
        decay, mix, gate, win = steps[j : j + 4]
        if [_name(t) for t in (mix, gate, win)] != ["TimeMix", "HeadGate", "WindowMHA"] or decay.values or not win.op.single:
            return None
        D, w = mix.op.dim, win.op
        if not (_same(mix.inputs["log_decay"], decay.outputs["y"]) and once(decay.outputs["y"])
                and gate_behind(mix.outputs["o"], gate) and mix.op.dtype is bfloat16 and w.dtype is bfloat16
                and 16 <= D <= 256 and D & (D - 1) == 0 and w.dim % 8 == 0 and w.vdim % 8 == 0 and w.stride % 8 == 0
                and gate.op.gains == gate.op.o_width and gate.op.gate_at == 0 and gate.op.gate_width == gate.op.o_width
                and _same(win.inputs["y"], gate.outputs["y"]) and win.inputs["spans"].buffer is mix.inputs["spans"].buffer):
            return None
        flat = dict(r=mix.inputs["r"], k=mix.inputs["k"], v=mix.inputs["v"], gate=gate.inputs["gate"], z=decay.inputs["z"],
                    w2=decay.inputs["up"], w0=decay.inputs["base"], u=mix.inputs["u"], norm=gate.inputs["gain"],
                    memory=mix.inputs["state"], x=win.inputs["x"], keys=win.inputs["keys"], values=win.inputs["values"],
                    bias=win.inputs["bias"], spans=win.inputs["spans"], out=win.inputs["y"])
        args = {n: tensor(h) for n, h in flat.items()}
        kw = dict(slots=w.slots, rows=w.rows, mix_heads=mix.op.heads, mix_dim=D, rank=decay.op.rank,
                  eps=float(gate.op.epsilon), mix_scale=float(gate.op.scale), mix_at=gate.op.at, stride=w.stride, heads=w.heads,
                  kv_heads=w.kv_heads, dim=w.dim, vdim=w.vdim, window=w.window, ring=w.ring, scale=float(w.scale),
                  out_scale=float(w.out_scale), win_at=w.at, out_stride=w.width)
        return Fused("decode_parallel", j, 4, lambda a=args, kw=kw: kernels.decode_parallel(**a, **kw))

    def delta_at(j):
        """The launch for a decode step's convolution, delta rule, head norm and gate -- or None.  The step is
        told by its rows: one a slot (a prompt's portion carries a bound)."""
        if j + 2 >= len(steps):
            return None
        conv, rule, gate = steps[j : j + 3]
        c = conv.op
        if not (_name(rule) == "DeltaRule" and not conv.values and c.rows == c.slots and c.dtype is bfloat16
                and _same(rule.inputs["x"], conv.outputs["y"]) and once(conv.outputs["y"]) and gate_behind(rule.outputs["o"], gate)
                and 16 <= c.vdim <= 256 and c.vdim & (c.vdim - 1) == 0 and gate.op.gains == c.vdim and gate.op.at == 0
                and gate.op.width == gate.op.o_width and gate.op.scale == 1.0
                and _same(gate.inputs["gate"], conv.inputs["x"])
                and rule.inputs["spans"].buffer is conv.inputs["spans"].buffer):
            return None
        flat = dict(x=conv.inputs["x"], taps_w=conv.inputs["weight"], a_log=conv.inputs["a_log"], dt_bias=conv.inputs["dt_bias"],
                    norm=gate.inputs["gain"], inputs=conv.inputs["state"], state=rule.inputs["state"],
                    spans=conv.inputs["spans"], out=gate.outputs["y"])
        args = {n: tensor(h) for n, h in flat.items()}
        kw = dict(slots=c.slots, rows=c.rows, stride=c.stride, heads=c.heads, kv_heads=c.kv_heads, dim=c.dim, vdim=c.vdim,
                  taps=c.taps, gate_at=gate.op.gate_at, b_at=c.b_at, a_at=c.a_at, eps=float(gate.op.epsilon))
        return Fused("decode_delta", j, 3, lambda a=args, kw=kw: kernels.decode_delta(**a, **kw))

    def bare(s) -> bool:
        return not s.values and all(_plain(h) for h in (*s.inputs.values(), *s.outputs.values()))

    def gated_end(j, x):
        """``(product, add)`` where step ``j`` is one row's product of ``x`` and the next adds it, gated, to the
        stream -- or None."""
        if j + 1 >= len(steps):
            return None
        g, add = steps[j], steps[j + 1]
        if not (gemv_row(g) and (x is None or _same(g.inputs["B"], x)) and g.op.K % 8 == 0 and g.op.K <= 16384 and _name(add) == "StreamGatedAdd"
                and add.op.rows == 1 and add.op.dtype is bfloat16 and bare(add) and _same(add.inputs["y"], g.outputs["C"])
                and once(g.outputs["C"])):
            return None
        return g, add

    def into_stream(g, add):
        at = add.op.gate_at
        args = dict(W=tensor(g.inputs["A"]), stream=tensor(add.inputs["x"]).reshape(-1),
                    gate=tensor(add.inputs["gate"]).reshape(-1)[at : at + add.op.cols], gate_bias=tensor(add.inputs["gate_bias"]))
        if "y_bias" in add.inputs:
            args["y_bias"] = tensor(add.inputs["y_bias"])
        return args, dict(M=g.op.M, K=g.op.K)

    def stream_product_at(j):
        """The launch for a single row's product with what makes its input ahead of it (a norm of the stream, a
        gated recurrence's step, an activation over normed powers) or what takes its output behind it (the stream,
        through a gate) -- or None."""
        s = steps[j]
        if _name(s) == "StreamNorm":
            g = steps[j + 1] if j + 1 < len(steps) else None
            h = s.outputs["y"]
            if not (g is not None and s.op.rows == 1 and s.op.groups == 1 and s.op.dtype is bfloat16 and s.op.cols % 8 == 0 and s.op.cols <= 16384 and bare(s)
                    and gemv_row(g, h) and once(h)):
                return None
            args = dict(W=tensor(g.inputs["A"]), x=tensor(s.inputs["x"]).reshape(-1), gain=tensor(s.inputs["weight"]),
                        y=tensor(g.outputs["C"]).reshape(-1))
            kw = dict(input="stream_norm", M=g.op.M, K=g.op.K, eps=float(s.op.epsilon), unit=float(s.op.unit))
            return Fused("stream_norm_gemv", j, 2, lambda a=args, kw=kw: kernels.stream_product(**a, **kw))
        if _name(s) == "MinGRU":
            y = s.outputs["y"]
            end = gated_end(j + 1, y)
            if not (end and s.op.rows == 1 and s.op.slots == 1 and s.op.dtype is bfloat16 and s.op.width % 8 == 0 and bare(s) and once(y)):
                return None
            args, kw = into_stream(*end)
            args |= dict(x=tensor(s.inputs["x"]).reshape(-1), b0=tensor(s.inputs["z_bias"]), b1=tensor(s.inputs["x_bias"]),
                         state=tensor(s.inputs["state"]).reshape(-1), spans=tensor(s.inputs["spans"]))
            kw["input"] = "min_gru"
            return Fused("min_gru_gated_product", j, 3, lambda a=args, kw=kw: kernels.stream_product(**a, **kw))
        if _name(s) == "PolyNorm":
            y = s.outputs["y"]
            end = gated_end(j + 1, y)
            if not (end and s.op.rows == 1 and s.op.biased and s.op.dtype is bfloat16 and s.op.cols % 8 == 0 and s.op.at % 8 == 0 and bare(s)
                    and once(y)):
                return None
            args, kw = into_stream(*end)
            args |= dict(x=tensor(s.inputs["x"]).reshape(-1)[s.op.at : s.op.at + s.op.cols], b0=tensor(s.inputs["bias"]),
                         gain=tensor(s.inputs["coefficients"]))
            kw |= dict(input="poly_norm", eps=float(s.op.epsilon))
            return Fused("poly_norm_gated_product", j, 3, lambda a=args, kw=kw: kernels.stream_product(**a, **kw))
        if (end := gated_end(j, None)) is not None:
            args, kw = into_stream(*end)
            args["x"] = tensor(s.inputs["B"]).reshape(-1)
            return Fused("gated_product", j, 2, lambda a=args, kw=kw: kernels.stream_product(input="row", **a, **kw))
        return None

    def depth_rows_at(j):
        """The launch for a block's output into the stream, the average over what it was behind every layer and the row a
        block reads of it, where two or three of them follow each other on the same rows -- or None."""
        found, at = {}, j
        for name in ("StreamAdd", "DepthAverage", "StreamCast"):
            st = steps[at] if at < len(steps) else None
            if st is None or _name(st) != name or set(st.values) - {"valid"}:
                continue
            if found:
                ahead = next(iter(found.values()))
                if not (_same_view(st.inputs["x"], ahead.outputs["x"]) and st.values.get("valid") == ahead.values.get("valid")
                        and (st.op.rows, st.op.cols) == (ahead.op.rows, ahead.op.cols)):
                    break
            found[name] = st
            at += 1
        add, depth, cast = (found.get(n) for n in ("StreamAdd", "DepthAverage", "StreamCast"))
        if len(found) < 2 or (add is not None and cast is not None and add.op.dtype is not cast.op.dtype):
            return None
        first = next(iter(found.values()))
        args = dict(x=tensor(first.inputs["x"]))
        kw = dict(rows=first.op.rows, cols=first.op.cols, valid=word(first.values.get("valid")))
        if add is not None:
            args |= dict(y=tensor(add.inputs["y"]), back_gain=tensor(add.inputs["weight"]))
            if "y_bias" in add.inputs:
                args["y_bias"] = tensor(add.inputs["y_bias"])
            kw |= dict(eps=float(add.op.epsilon), unit=float(add.op.unit))
        if depth is not None:
            args |= dict(planes=tensor(depth.inputs["planes"]), weights=tensor(depth.inputs["weights"]))
            kw |= dict(plane_rows=depth.op.plane_rows, index=depth.op.count - 1)
        if cast is not None:
            args["h"] = tensor(cast.outputs["y"])
        return Fused("stream_depth_rows", j, at - j, lambda a=args, kw=kw: kernels.stream_depth_rows(**a, **kw))

    def step_mixer_at(j):
        """``(steps, launch)`` where a decode step's mixer with what it needs ahead and behind, and a feed-forward's gated columns
        beside it (if there are any), start at step ``j``; ``launch(**choice)`` runs them, a router's choice beside -- or None."""
        first, second = steps[j : j + 2] if j + 1 < len(steps) else (None, None)
        if first is None or first.op.dtype is not bfloat16 or first.values or second.values:
            return None
        o = first.op
        if _name(first) == "Hgrn2" and _name(second) == "HeadGate":
            ok = (o.rows == o.slots and 16 <= o.vdim <= 256 and o.vdim & (o.vdim - 1) == 0 and not second.op.gated and second.op.gains == o.vdim
                  and second.op.dtype is bfloat16 and second.op.scale == 1.0 and _same(second.inputs["o"], first.outputs["o"])
                  and once(first.outputs["o"]))
        elif _name(first) == "CachedHeads" and _name(second) == "GlobalMHA":
            ok = (o.rows == o.slots and second.op.single and not any(n % 8 for n in (o.dim, o.vdim, o.stride)) and max(o.dim, o.vdim) <= 256
                  and _same(second.inputs["q"], first.outputs["q"]) and second.op.dtype is bfloat16)
        else:
            return None
        if not ok:
            return None
        made, count = second.outputs["y"], 2
        columns = steps[j + 2] if j + 2 < len(steps) and _name(steps[j + 2]) == "GatedColumns" else None
        if (columns is not None and not columns.values and columns.op.dtype is bfloat16 and _same(columns.inputs["x"], first.inputs["x"])
                and _same(columns.inputs["y"], made)):
            count, c = 3, columns.op
            beside = dict(cols=c.cols, gate_at=c.gate_at, gated_at=c.at, kind=c.kind, limit=float(c.limit))
        else:
            beside = {}
        if _name(first) == "Hgrn2":
            args = {n: tensor(first.inputs[n]) for n in ("x", "f_bias", "lower", "state", "spans")}
            args |= dict(norm=tensor(second.inputs["gain"]), out=tensor(made))
            kw = {n: getattr(o, n) for n in ("slots", "rows", "stride", "heads", "dim", "vdim")}
            kw |= dict(out_stride=second.op.width, out_at=second.op.at, eps=float(second.op.epsilon), **beside)
            return count, 1, lambda **choice: kernels.decode_hgrn2(**args, **kw, **choice)
        heads = {n: tensor(first.inputs[n]) for n in ("x", "q_gain", "k_gain", "spans", "keys", "values", "angles") if n in first.inputs}
        heads |= dict(q=tensor(first.outputs["q"]), out=tensor(made))
        kw = {n: getattr(o, n) for n in ("slots", "rows", "stride", "heads", "kv_heads", "dim", "vdim", "context", "turned", "angle_rows", "value_norm")}
        kw |= dict(eps=float(o.epsilon), out_stride=second.op.width, **beside)
        m = second.op
        attend = dict(q=heads["q"], keys=heads["keys"], values=heads["values"], spans=heads["spans"], y=heads["out"],
                      workspace=tensor(second.outputs["workspace"]))
        attend |= {n: getattr(m, n) for n in ("slots", "rows", "heads", "kv_heads", "dim", "vdim", "context", "sink")}
        attend |= dict(scale=float(m.scale), cap=float(m.cap), out_stride=m.width, out_at=m.at, single=True)

        def launch(**choice):
            kernels.decode_heads_global(**heads, **kw, **choice)
            kernels.mha_global(**attend)

        return count, 3, launch

    def step_mixer(j):
        found = step_mixer_at(j)
        return None if found is None else Fused("step_mixer", j, found[0], found[2], launches=found[1])

    def norm_product_at(j):
        """The launch for a single row's grouped norm and the product of it -- with a router's logits and, beside the mixer behind
        it, the router's choice, where they follow -- or None."""
        s = steps[j]
        g = steps[j + 1] if j + 1 < len(steps) else None
        h, o = s.outputs["y"], s.op
        if not (g is not None and o.rows == 1 and o.dtype is bfloat16 and o.cols % (8 * o.groups) == 0 and o.cols <= 16384 and o.groups <= 256
                and bare(s) and gemv_row(g, h)):
            return None
        args = dict(W=tensor(g.inputs["A"]), x=tensor(s.inputs["x"]).reshape(-1), gain=tensor(s.inputs["weight"]),
                    y=tensor(g.outputs["C"]).reshape(-1))
        kw = dict(M=g.op.M, K=g.op.K, groups=o.groups, eps=float(o.epsilon), unit=float(o.unit))
        if once(h):
            return Fused("norm_product", j, 2, lambda: kernels.norm_product(**args, **kw))
        args["h"] = tensor(h).reshape(-1)
        r = steps[j + 2] if j + 2 < len(steps) and _name(steps[j + 2]) == "Router" else None
        if (r is not None and scratch is not None and bare(r) and r.op.scored and not r.op.biased and r.op.dtype is bfloat16 and _same(r.inputs["h"], h)
                and (mixer := step_mixer_at(j + 3)) is not None):
            need = 4 * r.op.experts
            z = scratch(j, need)
            logits = dict(router=tensor(r.inputs["weight"]), z=z, logits=r.op.experts)
            choice = dict(z=z, logits=r.op.experts, top=r.op.top, ids=tensor(r.outputs["ids"]).reshape(-1), shares=tensor(r.outputs["shares"]).reshape(-1))
            if "correction" in r.inputs:
                choice["correction"] = tensor(r.inputs["correction"])
            count, launches, run = mixer

            def launch():
                kernels.norm_product(**args, **kw, **logits)
                run(**choice)

            return Fused("norm_product_router_mixer", j, 3 + count, launch, launches=1 + launches, scratch_bytes=need)
        return Fused("norm_product", j, 2, lambda: kernels.norm_product(**args, **kw))

    def stream_end(j):
        """``(product, sum)`` where step ``j`` is one row's product and the next adds it to the stream -- or None."""
        g, add = steps[j : j + 2] if j + 1 < len(steps) else (None, None)
        if not (g is not None and gemv_row(g) and g.op.K % 8 == 0 and g.op.K <= 32768 and _name(add) == "StreamSum" and add.op.rows == 1
                and add.op.dtype is bfloat16 and bare(add) and _same(add.inputs["y"], g.outputs["C"]) and once(g.outputs["C"])):
            return None
        return g, add

    def product_sum_at(j):
        if (end := stream_end(j)) is None:
            return None
        g, add = end
        args = dict(x=tensor(g.inputs["B"]).reshape(-1), W=tensor(g.inputs["A"]), stream=tensor(add.inputs["x"]).reshape(-1))
        if "also" in add.inputs:
            args["also"] = tensor(add.inputs["also"]).reshape(-1)
        return Fused("product_sum", j, 2, lambda: kernels.product_sum(**args, M=g.op.M, K=g.op.K))

    def experts_tail_at(j):
        """The launches for one row's experts, and the product and the sum that join the stream with them -- or None."""
        s = steps[j]
        o, y, end = s.op, s.outputs["y"], stream_end(j + 1)
        if not (end and o.rows == 1 and o.dtype is bfloat16 and bare(s) and once(y) and "also" in end[1].inputs and _same(end[1].inputs["also"], y)
                and not any(n % 8 for n in (o.cols, o.ff)) and o.top <= 64 and end[0].op.K // 8 + o.top * o.ff // 8 <= 4096):
            return None
        g, add = end
        args = {n: tensor(s.inputs[n]) for n in ("gate", "up", "down")}
        args |= {n: tensor(s.inputs[n]).reshape(-1) for n in ("h", "ids", "shares")}
        args |= dict(out=tensor(g.inputs["A"]), made=tensor(g.inputs["B"]).reshape(-1), stream=tensor(add.inputs["x"]).reshape(-1),
                     workspace=tensor(s.outputs["workspace"]))
        kw = dict(cols=o.cols, ff=o.ff, inner=g.op.K, experts=o.experts, identity=o.identity, top=o.top, activation=o.activation)
        return Fused("experts_tail", j, 3, lambda: kernels.experts_tail(**args, **kw), launches=2)

    def latent_query_at(j):
        """The launch for a single slot's latents and the product of its queries -- or None."""
        s = steps[j]
        g = steps[j + 1] if j + 1 < len(steps) else None
        o, q = s.op, s.outputs["q"]
        if not (g is not None and o.rows == 1 and o.slots == 1 and o.dtype is bfloat16 and bare(s) and gemv_row(g, q) and once(q)
                and not any(n % 8 for n in (o.stride, o.q_rank, o.rank, o.rot, o.turned)) and o.rank + o.rot <= 4096
                and o.q_rank + o.rank + o.rot <= 8192):
            return None
        args = dict(x=tensor(s.inputs["x"]).reshape(-1), q_gain=tensor(s.inputs["q_gain"]), c_gain=tensor(s.inputs["c_gain"]),
                    spans=tensor(s.inputs["spans"]), W=tensor(g.inputs["A"]), q=tensor(g.outputs["C"]).reshape(-1),
                    latents=tensor(s.inputs["latents"]))
        args |= {n: tensor(s.inputs[n]) for n in ("shared_keys", "angles") if n in s.inputs}
        kw = {n: getattr(o, n) for n in ("stride", "q_rank", "rank", "rot", "turned", "angle_rows", "ring")}
        kw |= dict(M=g.op.M, eps=float(o.epsilon))
        return Fused("latent_query", j, 2, lambda a=args, kw=kw: kernels.latent_query(**a, **kw))

    def same_data(a, b) -> bool:
        return (a is not None and b is not None and a.buffer is b.buffer and a.offset == b.offset
                and a.elements == b.elements and _plain(a) and _plain(b))

    def heads_finish_at(j):
        """The launch for the steps from ``j`` on where they are what lies between a token's q/k/v
        projections and its attention in a layer that norms its heads one by one: RMSNorm per head of
        q (of k, of v), RoPE on q (and k), k's and v's copies into their cache rows -- or None."""
        first = steps[j]
        # the projections just ahead: q's product is what this norm reads; k's and v's follow it
        back = j
        while back > 0 and j - back < 3 and gemv_row(steps[back - 1]):
            back -= 1
        made = [g.outputs["C"] for g in steps[back:j]]
        at = next((n for n, h in enumerate(made) if same_data(h, first.inputs["x"])), None)
        if at is None or len(made) - at not in (1, 3):
            return None
        cur = {"q": made[at], "k": made[at + 1] if len(made) - at == 3 else None,
               "v": made[at + 2] if len(made) - at == 3 else None}
        d = first.op.tile_size
        if any(h is not None and h.elements % d for h in cur.values()) or d % 16 or d > 2048:
            return None
        heads = cur["q"].elements // d
        kv_heads = cur["k"].elements // d if cur["k"] is not None else 1
        if cur["k"] is not None and cur["v"].elements != cur["k"].elements:
            return None
        p, norms, eps, gains = j, 0, None, {"q": None, "k": None}
        for bit, name in enumerate(("q", "k", "v")):
            st = steps[p] if p < len(steps) else None
            if (cur[name] is None or st is None or _name(st) != "RMSNorm" or st.values or st.op.tile_size != d
                    or not same_data(st.inputs["x"], cur[name]) or not once(cur[name]) or not _plain(st.outputs["y"])
                    or (eps is not None and float(st.op.epsilon) != eps) or (name == "v" and st.op.weighted)):
                continue
            if st.op.weighted:
                if not _plain(st.inputs["weight"]) or st.inputs["weight"].elements != d:
                    return None
                gains[name] = st.inputs["weight"]
            norms |= 1 << bit
            eps = float(st.op.epsilon)
            cur[name] = st.outputs["y"]
            p += 1
        if not norms & 1:
            return None
        angles, rotary, two_halves = {"q": None, "k": None}, 0, True
        for name in ("q", "k"):
            st = steps[p] if p < len(steps) else None
            if (cur[name] is None or st is None or _name(st) != "RoPE" or st.values or st.op.angle_rows != 1
                    or st.op.row != d or st.op.cols % 16 or not same_data(st.inputs["x"], cur[name])
                    or not once(cur[name]) or not _plain(st.inputs["angles"]) or not _plain(st.outputs["y"])
                    or (rotary and (st.op.cols, st.op.two_halves) != (rotary, two_halves))):
                continue
            angles[name], rotary, two_halves = st.inputs["angles"], st.op.cols, bool(st.op.two_halves)
            cur[name] = st.outputs["y"]
            p += 1
        # k's copies into its cache rows (the slot and, in a ring, its mirror), then v's into the same rows
        caches, rows_at = {}, None
        for name in ("k", "v"):
            if cur[name] is None:
                continue
            found = []
            while p < len(steps) and len(found) < 2 and _name(steps[p]) == "Copy" and not steps[p].values:
                cp = steps[p]
                src, dst = cp.inputs["src"], cp.outputs["dst"]
                if not (same_data(src, cur[name]) and dst.index is not None and dst.ids is None and not dst.valid
                        and dst.offset == 0 and dst.index_stride == cur[name].elements
                        and dst.elements == cur[name].elements
                        and (not found or dst.buffer is found[0].buffer)):
                    break
                found.append(dst)
                p += 1
            if not found or not once(cur[name], len(found)):
                return None
            if rows_at is None:
                rows_at = [f.index for f in found]
            elif [f.index for f in found] != rows_at or found[0].index_rows != caches["k"].index_rows:
                return None
            caches[name] = found[0]
        if p - j < 2:
            return None
        args = dict(q=tensor(made[at]).reshape(-1), q_out=tensor(cur["q"]).reshape(-1))
        kw = dict(heads=heads, kv_heads=kv_heads, d=d, eps=eps, norms=norms, rotary=rotary, two_halves=two_halves)
        for name in ("q", "k"):
            if gains[name] is not None:
                args[f"{name}_gain"] = tensor(gains[name]).reshape(-1)
            if angles[name] is not None:
                args[f"{name}_angles"] = tensor(angles[name]).reshape(-1)
        if caches:
            kd, vd = caches["k"], caches["v"]
            args |= dict(k=tensor(made[at + 1]).reshape(-1), v=tensor(made[at + 2]).reshape(-1),
                         keys=tensor(kd)[: kd.index_rows * kd.index_stride],
                         values=tensor(vd)[: vd.index_rows * vd.index_stride])
            kw |= dict(cache_rows=kd.index_rows, row0=word(rows_at[0]),
                       row1=word(rows_at[1]) if len(rows_at) > 1 else None)
        return Fused("decode_heads", j, p - j, lambda a=args, kw=kw: kernels.decode_heads(**a, **kw))

    fused: list[Fused] = []
    # decode_qkv launches whose RoPE row is a copy of one table row: (producing step, args, kw)
    rope_rows: list[tuple[int, dict, dict]] = []
    # decode_qkv launches whose input row is a copy of one row of a table (the token's embedding)
    embed_rows: list[tuple[int, dict, dict]] = []
    i = 0
    while i < len(steps):
        s = steps[i]
        got = None
        if norm_row(s):
            n = s.outputs["y"]
            rest = steps[i + 1 :]
            # attention's first half
            if (len(rest) >= 7 and all(gemv_row(g, n) for g in rest[:3]) and once(n, 3)
                    and _name(rest[3]) == "RoPE" and _name(rest[4]) == "RoPE"
                    and _name(rest[5]) == "Copy" and _name(rest[6]) == "Copy"):
                gq, gk, gv, rq, rk, ck, cv = rest[:7]
                q, k, v = (g.outputs["C"] for g in (gq, gk, gv))
                d = rq.op.cols
                kd, vd = ck.outputs["dst"], cv.outputs["dst"]
                ok = (
                    _same(rq.inputs["x"], q) and _same(rk.inputs["x"], k) and once(q) and once(k) and once(v)
                    and rq.op.two_halves and rk.op.two_halves and rq.op.angle_rows == 1 and rk.op.angle_rows == 1
                    and rq.op.row == rq.op.cols and rk.op.row == rk.op.cols
                    and rk.op.cols == d and d in (64, 128) and not rq.values and not rk.values
                    and rq.inputs["angles"].buffer is rk.inputs["angles"].buffer and _plain(rq.inputs["angles"])
                    and _same(ck.inputs["src"], rk.outputs["y"]) and once(rk.outputs["y"])
                    and _same(cv.inputs["src"], v)
                    and kd.index is not None and vd.index is not None and kd.index == vd.index
                    and kd.ids is None and vd.ids is None and not kd.valid and not vd.valid
                    and kd.offset == 0 and vd.offset == 0
                    and kd.index_stride == k.elements and vd.index_stride == v.elements
                    and k.elements == v.elements and k.elements % d == 0 and q.elements % d == 0
                )
                if ok:
                    args = dict(
                        x=tensor(s.inputs["x"]).reshape(-1), norm_w=tensor(s.inputs["weight"]).reshape(-1),
                        Wq=tensor(gq.inputs["A"]), Wk=tensor(gk.inputs["A"]), Wv=tensor(gv.inputs["A"]),
                        angles=tensor(rq.inputs["angles"]).reshape(-1), q_out=tensor(rq.outputs["y"]).reshape(-1),
                        keys=tensor(kd)[: kd.index_rows * kd.index_stride],
                        values=tensor(vd)[: vd.index_rows * vd.index_stride],
                    )
                    kw = dict(eps=float(s.op.epsilon), hidden=s.op.tile_size, heads=q.elements // d,
                              kv_heads=k.elements // d, d=d, cache_rows=kd.index_rows, position=word(kd.index))
                    got = Fused("decode_qkv", i, 8, lambda a=args, kw=kw: kernels.decode_qkv(**a, **kw))
                    made_by = _row_copy(steps, i, rq.inputs["angles"], d)
                    if made_by is not None:
                        rope_rows.append((made_by, args, kw))
                    # ... and the layer's input where it is one row of an embedding table
                    looked_up = _row_copy(steps, i, s.inputs["x"], s.op.tile_size)
                    if looked_up is not None and not any(
                            h.buffer is s.inputs["x"].buffer for t in steps[looked_up + 1 : i] for h in t.inputs.values()):
                        embed_rows.append((looked_up, args, kw))
            # the gated MLP's first half
            if (got is None and len(rest) >= 4 and gemv_row(rest[0], n) and gemv_row(rest[1], n) and once(n, 2)
                    and (_name(rest[2]) == "SiLU" or (_name(rest[2]) == "GELU" and rest[2].op.approximate == "tanh"))
                    and _name(rest[3]) == "ElementwiseMul"):
                gg, gu, si, mu = rest[:4]
                g, u = gg.outputs["C"], gu.outputs["C"]
                ok = (_same(si.inputs["x"], g) and once(g) and once(u) and once(si.outputs["y"])
                      and not si.values and not mu.values
                      and _same(mu.inputs["a"], si.outputs["y"]) and _same(mu.inputs["b"], u)
                      and gg.op.M == gu.op.M and gg.op.K == gu.op.K and _plain(mu.outputs["y"]))
                if ok:
                    args = dict(W=tensor(gg.inputs["A"]), W2=tensor(gu.inputs["A"]),
                                x=tensor(s.inputs["x"]).reshape(-1), norm_w=tensor(s.inputs["weight"]).reshape(-1),
                                y=tensor(mu.outputs["y"]).reshape(-1))
                    kw = dict(M=gg.op.M, K=gg.op.K, eps=float(s.op.epsilon), epilogue=2 if _name(si) == "SiLU" else 3)
                    got = Fused("norm_gate_up_silu_mul" if _name(si) == "SiLU" else "norm_gate_up_gelu_mul", i, 5, lambda a=args, kw=kw: kernels.gemv_fused(**a, **kw))
            # the head: norm, then one projection -- or a layer's q, k, v projections where something
            # other than RoPE follows them (heads normed one by one): the norm rides each one's prologue
            if got is None:
                count = 0
                while count < 3 and count < len(rest) and gemv_row(rest[count], n):
                    count += 1
                if count and once(n, count):
                    calls = []
                    for g0 in rest[:count]:
                        args = dict(W=tensor(g0.inputs["A"]), x=tensor(s.inputs["x"]).reshape(-1),
                                    norm_w=tensor(s.inputs["weight"]).reshape(-1), y=tensor(g0.outputs["C"]).reshape(-1))
                        calls.append((args, dict(M=g0.op.M, K=g0.op.K, eps=float(s.op.epsilon), epilogue=0)))

                    def norm_gemvs(calls=calls):
                        for a, kw in calls:
                            kernels.gemv_fused(**a, **kw)

                    got = Fused("norm_gemv", i, 1 + count, norm_gemvs, launches=count)
        elif (_name(s) == "GEMM" and len(steps) - i >= 5
              and [_name(t) for t in steps[i + 1 : i + 5]] == ["GEMM", "GEMM", "RoPE", "RoPE"]):
            # a prompt chunk's projections and rotations
            gq, gk, gv, rq, rk = steps[i : i + 5]
            a = gq.inputs["A"]

            def rows_gemm(g):
                return (g.op.b_col_maj and not g.op.c_col_maj and "valid_k" not in g.values
                        and _same_view(g.inputs["A"], a) and g.op.M == gq.op.M and g.op.K == gq.op.K
                        and all(h.index is None and h.ids is None for h in (*g.inputs.values(), *g.outputs.values())))

            q, k, v = (g.outputs["C"] for g in (gq, gk, gv))
            M, d = gq.op.M, 64
            ok = (
                all(rows_gemm(g) for g in (gq, gk, gv)) and once(q) and once(k)
                and M >= 64 and gq.op.K % 64 == 0 and gq.op.N % 128 == 0 and gk.op.N % 128 == 0
                and gk.op.N == gv.op.N
                and _same_view(rq.inputs["x"], q) and _same_view(rk.inputs["x"], k)
                and all(r.op.two_halves and r.op.cols == d and r.op.row == d and r.op.angle_rows == M for r in (rq, rk))
                and rq.op.rows * d == M * gq.op.N and rk.op.rows * d == M * gk.op.N
                and rq.inputs["angles"].buffer is rk.inputs["angles"].buffer
                and _same_view(rq.inputs["angles"], rk.inputs["angles"])
                and all(h.index is None and h.ids is None for h in (rq.outputs["y"], rk.outputs["y"]))
            )
            if ok:
                args = dict(x=tensor(a), Wq=tensor(gq.inputs["B"]), Wk=tensor(gk.inputs["B"]), Wv=tensor(gv.inputs["B"]),
                            angles=tensor(rq.inputs["angles"]), q_out=tensor(rq.outputs["y"]),
                            k_out=tensor(rk.outputs["y"]), v_out=tensor(v))
                kw = dict(rows=M, hidden=gq.op.K, heads=gq.op.N // d, kv_heads=gk.op.N // d, d=d,
                          valid=word(gq.values.get("valid")))
                got = Fused("prefill_qkv", i, 5, lambda a=args, kw=kw: kernels.prefill_qkv(**a, **kw))
                # ... and the two copies of k and v into the chunk's rows of the layer's caches
                ck, cv = (steps[i + 5], steps[i + 6]) if i + 6 < len(steps) else (None, None)
                if ck is not None and _name(ck) == "Copy" and _name(cv) == "Copy":
                    kd, vd = ck.outputs["dst"], cv.outputs["dst"]
                    gvalid = gq.values.get("valid")
                    cached = (
                        _same_view(ck.inputs["src"], rk.outputs["y"]) and _same_view(cv.inputs["src"], v)
                        and once(rk.outputs["y"]) and once(v)
                        and all(h.index is not None and h.ids is None and h.offset == 0
                                and h.index_stride == gk.op.N and h.elements == M * gk.op.N for h in (kd, vd))
                        and kd.index == vd.index and kd.index_rows == vd.index_rows
                        and kd.valid.get(0) == gvalid and vd.valid.get(0) == gvalid
                        and ck.inputs["src"].valid.get(0) == gvalid and cv.inputs["src"].valid.get(0) == gvalid
                        and M <= kd.index_rows
                    )
                    if cached:
                        args = {k_: t for k_, t in args.items() if k_ not in ("k_out", "v_out")}
                        args |= dict(keys=tensor(kd)[: kd.index_rows * kd.index_stride],
                                     values=tensor(vd)[: vd.index_rows * vd.index_stride])
                        kw = dict(kw, cache_rows=kd.index_rows, start=word(kd.index))
                        got = Fused("prefill_qkv_cache", i, 7,
                                    lambda a=args, kw=kw: kernels.prefill_qkv_cache(**a, **kw))
        elif (_name(s) == "GEMM" and i + 1 < len(steps) and _name(steps[i + 1]) in ("ElementwiseAdd", "AXPY")
              and s.op.b_col_maj and not s.op.c_col_maj and "valid_k" not in s.values
              and s.op.M >= 64 and s.op.N >= 64 and s.op.K % 64 == 0):
            # a projection over many rows and its residual: the sum rides the product's epilogue
            ad = steps[i + 1]
            c = s.outputs["C"]
            a, b = ad.inputs["a"], ad.inputs["b"]
            if _name(ad) == "AXPY":   # scalar_factor * a + b: the product is the one scaled
                other, scale = (b if _same_view(a, c) else None), float(ad.op.scalar_factor)
            else:
                other, scale = (a if _same_view(b, c) else (b if _same_view(a, c) else None)), 1.0
            gv, av = s.values.get("valid"), ad.values.get("valid")
            # the sum's bound counts elements, the product's rows
            bounds_agree = (gv is None and av is None) or (
                gv is not None and av is not None and gv.value == av.value and gv.linear and av.linear
                and av.scale == gv.scale * s.op.N and av.bias == gv.bias * s.op.N)
            flat = all(h.index is None and h.ids is None
                       for h in (*s.inputs.values(), c, a, b, ad.outputs["y"]))
            if (other is not None and flat and once(c) and bounds_agree and other.elements == c.elements
                    and ad.outputs["y"].elements == c.elements and set(ad.values) <= {"valid"}):
                args = dict(A=tensor(s.inputs["A"]), B=tensor(s.inputs["B"]), R=tensor(other), C=tensor(ad.outputs["y"]))
                kw = dict(M=s.op.M, N=s.op.N, K=s.op.K, residual_scale=scale, valid=word(gv))
                got = Fused("gemm_add", i, 2, lambda a=args, kw=kw: kernels.gemm_residual(**a, **kw))
                # ... and the norm of the rows it leaves (the next layer's input norm after a down
                # projection): few rows over a long K are dealt over several blocks a tile, and the
                # launch that adds their sums up stands where the norm's stood
                nm = steps[i + 2] if i + 2 < len(steps) else None
                need = kernels.gemm_residual_norm_workspace_bytes(s.op.M, s.op.N, s.op.K) if scratch and nm else 0
                if (need and _name(nm) == "RMSNorm" and nm.op.weighted and nm.op.rows == s.op.M
                        and nm.op.tile_size == s.op.N and set(nm.values) <= {"valid"} and nm.values.get("valid") == gv
                        and _same_view(nm.inputs["x"], ad.outputs["y"])
                        and all(h.index is None and h.ids is None for h in (*nm.inputs.values(), nm.outputs["y"]))
                        and nm.outputs["y"].buffer is not ad.outputs["y"].buffer
                        and nm.outputs["y"].buffer is not other.buffer):
                    args = dict(args, gain=tensor(nm.inputs["weight"]), Y=tensor(nm.outputs["y"]),
                                workspace=scratch(i, need))
                    kw = dict(kw, eps=float(nm.op.epsilon))
                    got = Fused("gemm_add_norm", i, 3, lambda a=args, kw=kw: kernels.gemm_residual_norm(**a, **kw),
                                launches=2, scratch_bytes=need)
        elif _name(s) == "GEMM" and (gated := gated_at(i + 1, s)) is not None:
            # a gated feed-forward's two first projections over many rows: one launch computes both
            # products tile by tile, the activated gate riding the second one's epilogue
            args, kw = gated
            args = dict(A=args["A"], Bg=tensor(s.inputs["B"]), Bu=args["B"], G=args["G"], C=args["C"])
            got = Fused("gemm_gated_pair", i, 4, lambda a=args, kw=kw: kernels.gemm_gated_pair(**a, **kw))
        elif _name(s) == "GEMM" and (gated := gated_at(i)) is not None:
            # a gated feed-forward's second projection over many rows: the activated gate rides its epilogue
            args, kw = gated
            got = Fused("gemm_gated", i, 3, lambda a=args, kw=kw: kernels.gemm_gated(**a, **kw))
        elif _name(s) == "SiLU" and i + 1 < len(steps) and _name(steps[i + 1]) == "ElementwiseMul":
            # a gated feed-forward's activation and gate over many rows: one pass instead of two
            m = steps[i + 1]
            act = s.outputs["y"]
            a, b = m.inputs["a"], m.inputs["b"]
            other = b if _same_view(a, act) else (a if _same_view(b, act) else None)
            flat = all(h.index is None and h.ids is None for h in (s.inputs["x"], act, a, b, m.outputs["y"]))
            if (other is not None and flat and once(act) and s.op.size == m.op.size
                    and s.values.get("valid") == m.values.get("valid") and other.elements == act.elements):
                args = dict(a=tensor(s.inputs["x"]).reshape(-1), b=tensor(other).reshape(-1),
                            y=tensor(m.outputs["y"]).reshape(-1))
                kw = dict(n=s.op.size, valid=word(m.values.get("valid")))
                got = Fused("silu_mul", i, 2, lambda a=args, kw=kw: kernels.silu_mul(**a, **kw))
        elif (gemv_row(s) and i + 2 < len(steps) and _name(steps[i + 2]) in ("RowwiseMul", "ElementwiseMul")
              and (_name(steps[i + 1]) == "SiLU"
                   or (_name(steps[i + 1]) == "GELU" and steps[i + 1].op.approximate == "tanh"))):
            # a projection, its activation and the product with a given row (a per-layer input's gate)
            ac, mu = steps[i + 1], steps[i + 2]
            c, act = s.outputs["C"], ac.outputs["y"]
            if _name(mu) == "RowwiseMul":   # one row of x by the row: the same product element by element
                a, b = mu.inputs["x"], mu.inputs["row"]
                other = None if mu.op.rows != 1 else (b if same_data(a, act) else (a if same_data(b, act) else None))
            else:
                a, b = mu.inputs["a"], mu.inputs["b"]
                other = b if same_data(a, act) else (a if same_data(b, act) else None)
            if (other is not None and same_data(ac.inputs["x"], c) and once(c) and once(act) and not ac.values
                    and not mu.values and _plain(other) and other.elements == c.elements and _plain(mu.outputs["y"])
                    and mu.outputs["y"].elements == c.elements and other.buffer is not act.buffer):
                args = dict(W=tensor(s.inputs["A"]), x=tensor(s.inputs["B"]).reshape(-1),
                            residual=tensor(other).reshape(-1), y=tensor(mu.outputs["y"]).reshape(-1))
                kw = dict(M=s.op.M, K=s.op.K, epilogue=5 if _name(ac) == "SiLU" else 4)
                got = Fused("gemv_act_mul", i, 3, lambda a=args, kw=kw: kernels.gemv_fused(**a, **kw))
        elif _name(s) in ("StreamAdd", "DepthAverage") and (got := depth_rows_at(i)) is not None:
            pass
        elif _name(s) == "StreamNorm" and (s.op.groups > 1 or (i + 2 < len(steps) and _name(steps[i + 2]) == "Router")):
            got = norm_product_at(i)
        elif _name(s) in ("Hgrn2", "CachedHeads"):
            got = step_mixer(i)
        elif _name(s) == "Experts":
            got = experts_tail_at(i)
        elif gemv_row(s) and (got := product_sum_at(i)) is not None:
            pass
        elif _name(s) == "StreamSum" and i + 1 < len(steps) and _name(steps[i + 1]) == "StreamNorm":
            # what blocks made joins the stream, and the next blocks' norm leaves it: one pass over the row
            nm = steps[i + 1]
            if (_same_view(nm.inputs["x"], s.outputs["x"]) and nm.op.dtype is s.op.dtype and (nm.op.rows, nm.op.cols) == (s.op.rows, s.op.cols)
                    and nm.values.get("valid") == s.values.get("valid") and set(nm.values) <= {"valid"} and set(s.values) <= {"valid"}):
                args = dict(x=tensor(s.inputs["x"]), y=tensor(s.inputs["y"]), h=tensor(nm.outputs["y"]), gain=tensor(nm.inputs["weight"]))
                if "also" in s.inputs:
                    args["y2"] = tensor(s.inputs["also"])
                kw = dict(rows=s.op.rows, cols=s.op.cols, groups=nm.op.groups, eps=float(nm.op.epsilon), unit=float(nm.op.unit),
                          valid=word(s.values.get("valid")))
                got = Fused("stream_sum_norm", i, 2, lambda a=args, kw=kw: kernels.stream_groups(**a, **kw))
        elif _name(s) == "StreamAdd" and i + 1 < len(steps) and _name(steps[i + 1]) == "StreamNorm":
            # a block's output into the stream and the next block's norm out of it: one pass over the row
            nm = steps[i + 1]
            if (_same_view(nm.inputs["x"], s.outputs["x"]) and nm.op.dtype is s.op.dtype
                    and (nm.op.epsilon, nm.op.unit, nm.op.groups) == (s.op.epsilon, s.op.unit, 1)
                    and (nm.op.rows, nm.op.cols) == (s.op.rows, s.op.cols) and nm.values.get("valid") == s.values.get("valid")
                    and set(nm.values) <= {"valid"} and set(s.values) <= {"valid"}):
                args = dict(x=tensor(s.inputs["x"]), y=tensor(s.inputs["y"]), back_gain=tensor(s.inputs["weight"]),
                            h=tensor(nm.outputs["y"]), gain=tensor(nm.inputs["weight"]))
                if "y_bias" in s.inputs:
                    args["y_bias"] = tensor(s.inputs["y_bias"])
                kw = dict(rows=s.op.rows, cols=s.op.cols, eps=float(s.op.epsilon), unit=float(s.op.unit), valid=word(s.values.get("valid")))
                got = Fused("stream_add_norm", i, 2, lambda a=args, kw=kw: kernels.stream_rows(**a, **kw))
        elif (_name(s) in ("StreamNorm", "MinGRU", "PolyNorm") or gemv_row(s)) and (got := stream_product_at(i)) is not None:
            pass
        elif _name(s) == "LatentRows" and (got := latent_query_at(i)) is not None:
            pass
        elif _name(s) == "StreamGatedAdd" and i + 1 < len(steps) and _name(steps[i + 1]) == "StreamNorm":
            # a block's gated output into the stream and the next block's norm out of it: one pass over the row
            nm = steps[i + 1]
            if (_same_view(nm.inputs["x"], s.outputs["x"]) and nm.op.dtype is s.op.dtype and (nm.op.rows, nm.op.cols) == (s.op.rows, s.op.cols)
                    and nm.op.groups == 1 and nm.values.get("valid") == s.values.get("valid") and set(nm.values) <= {"valid"} and set(s.values) <= {"valid"}):
                args = dict(x=tensor(s.inputs["x"]), y=tensor(s.inputs["y"]), gate=tensor(s.inputs["gate"]), gate_bias=tensor(s.inputs["gate_bias"]),
                            h=tensor(nm.outputs["y"]), gain=tensor(nm.inputs["weight"]))
                if "y_bias" in s.inputs:
                    args["y_bias"] = tensor(s.inputs["y_bias"])
                kw = dict(rows=s.op.rows, cols=s.op.cols, eps=float(nm.op.epsilon), gate_stride=s.op.gate_width, gate_at=s.op.gate_at,
                          valid=word(s.values.get("valid")))
                got = Fused("stream_gated_add_norm", i, 2, lambda a=args, kw=kw: kernels.stream_gated_rows(**a, **kw))
        elif _name(s) == "LowRankDecay":
            got = parallel_at(i)
        elif _name(s) == "ShortConv":
            got = delta_at(i)
        elif (_name(s) == "TokenShift" or gemv_row(s)) and (got := mixed_at(i)) is not None:
            pass
        elif gemv_row(s) and (gated := gated_rows_at(i)) is not None:
            args, kw = gated
            got = Fused("gemv_gate_up_mul", i, 4, lambda a=args, kw=kw: kernels.gemv_fused(**a, **kw))
        elif gemv_row(s) and i + 1 < len(steps) and _name(steps[i + 1]) in ("ElementwiseAdd", "AXPY"):
            ad = steps[i + 1]
            c = s.outputs["C"]
            a, b = ad.inputs["a"], ad.inputs["b"]
            if _name(ad) == "AXPY":   # scalar_factor * a + b: the GEMV's row is the one scaled
                other, scale = (b if _same(a, c) else None), float(ad.op.scalar_factor)
            else:
                other, scale = (a if _same(b, c) else (b if _same(a, c) else None)), 1.0
            if other is not None and once(c) and _plain(other) and not ad.values and _plain(ad.outputs["y"]) \
                    and other.elements == c.elements:
                args = dict(W=tensor(s.inputs["A"]), x=tensor(s.inputs["B"]).reshape(-1),
                            residual=tensor(other).reshape(-1), y=tensor(ad.outputs["y"]).reshape(-1))
                kw = dict(M=s.op.M, K=s.op.K, epilogue=1, residual_scale=scale)
                got = Fused("gemv_add", i, 2, lambda a=args, kw=kw: kernels.gemv_fused(**a, **kw))
        if got is None and _name(s) == "RMSNorm" and s.op.rows >= 1 and not s.values:
            got = heads_finish_at(i)
        if (got is None and _name(s) == "RMSNorm" and i + 1 < len(steps) and _name(steps[i + 1]) == "ElementwiseAdd"
                and set(s.values) <= {"valid"}):
            # a block's output normed again before its residual (a sandwich layer): the sum rides the norm's pass
            ad = steps[i + 1]
            n = s.outputs["y"]
            a, b = ad.inputs["a"], ad.inputs["b"]
            other = a if _same_view(b, n) else (b if _same_view(a, n) else None)
            nv, av = s.values.get("valid"), ad.values.get("valid")
            cols = s.op.tile_size
            bounds_agree = (nv is None and av is None) or (
                nv is not None and av is not None and nv.value == av.value and nv.linear and av.linear
                and av.scale == nv.scale * cols and av.bias == nv.bias * cols)
            flat = all(h.index is None and h.ids is None
                       for h in (*s.inputs.values(), n, a, b, ad.outputs["y"]))
            if (other is not None and flat and once(n) and bounds_agree and other.elements == n.elements
                    and ad.outputs["y"].elements == n.elements and set(ad.values) <= {"valid"}):
                args = dict(x=tensor(s.inputs["x"]), w=tensor(s.inputs["weight"]) if s.op.weighted else None,
                            y=tensor(ad.outputs["y"]), residual=tensor(other))
                kw = dict(rows=s.op.rows, cols=cols, eps=float(s.op.epsilon), valid=word(nv))
                got = Fused("norm_add", i, 2, lambda a=args, kw=kw: kernels.rmsnorm(**a, **kw))
        if got is not None:
            fused.append(got)
            i += got.count
        else:
            i += 1
    # A RoPE row copied out of its table for nobody but these launches: they read the table at the
    # call's row themselves, and the copy is not launched.
    for producer in sorted({p for p, _, _ in rope_rows}):
        users = [(a, kw) for p, a, kw in rope_rows if p == producer]
        row = steps[producer].outputs["dst"]
        if reads[id(row.buffer)] != 2 * len(users) or any(f.first <= producer < f.first + f.count for f in fused):
            continue
        table = steps[producer].inputs["src"]
        for a, kw in users:
            a["angles"] = tensor(table).reshape(-1)[: table.index_rows * table.index_stride]
            kw["angle_row"] = word(table.index)
        fused.append(Fused("elided_rope_row", producer, 1, lambda: None, launches=0))
    # The token's embedding row, copied out of its table for a first layer whose fused projections can
    # read the table at the token themselves (and leave the copy where the residual sum reads it).
    for producer, a, kw in embed_rows:
        if any(f.first <= producer < f.first + f.count for f in fused):
            continue
        table = steps[producer].inputs["src"]
        a["table"] = tensor(table).reshape(-1)[: table.index_rows * table.index_stride]
        kw["token"] = word(table.index)
        fused.append(Fused("elided_embedding_row", producer, 1, lambda: None, launches=0))
    return sorted(fused, key=lambda f: f.first)


def _row_copy(steps, before: int, row, width: int):
    """The step before ``before`` that made ``row`` by copying one table row a per-call word names
    (``Copy(table[position])``), or None."""
    for j in range(before - 1, -1, -1):
        s = steps[j]
        if any(h.buffer is row.buffer for h in s.outputs.values()):
            if _name(s) != "Copy":
                return None
            src, dst = s.inputs["src"], s.outputs["dst"]
            ok = (_same(dst, row) and src.index is not None and src.ids is None and not src.valid and src.offset == 0
                  and src.index_stride == width and src.elements == width and src.buffer.kind == "resident"
                  and not s.values)
            return j if ok else None
    return None
