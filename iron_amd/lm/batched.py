"""A decoder that serves several sequences at once: its graph over a batch of rows, the slots its
sequences' states live in, and the scheduler that turns requests into launches.

Rows of a batch are packed, never padded: a *span* (``row0, rows, start``) a slot says which rows are
which sequence's tokens and at which positions.  A prompt is run in portions of at most
``prefill_chunk`` rows, several sequences' portions side by side in one launch; a decode step is one row
a slot.  Both read the spans from device memory and end with a draw a slot, which moves every span to the
one row behind it, so a captured decode step replays with no host round trip.  The residual stream stays
where it is after a portion: the ``readout`` version gives the logits of any of its rows.
"""

from __future__ import annotations

import dataclasses
from collections.abc import Hashable, Iterator, Sequence
from typing import Any

import numpy as np

from ..common import graph as iron
from ..common.graph import Scratchpad
from ..operators.copy import Copy
from ..operators.sample import ROW_WORDS, SampleSlots
from ..operators.stream import Softcap, SpanTails, StreamEmbed
from .causal import CausalLM, Decoder, OnHost, _HostOutput, _HostVersion
from .mixers import StreamRMSNorm, as_rows
from .session import Session

READOUT_ROWS = 64   # rows whose logits one launch of the readout gives


@dataclasses.dataclass(kw_only=True)
class BatchCall:
    """What one recording of a batched body gives its layers: the spans, in a prompt's portion the bound on its
    rows, and what they hand on to each other."""

    prompt: bool
    spans: Any
    rows: Any = None
    planes: Any = None                                   # what the stream was behind every layer, where layers look back
    kept: dict = dataclasses.field(default_factory=dict)   # what a layer leaves for later ones of the same call

    def bound(self, x):
        """``x`` as far as this call's rows go."""
        return x[: self.rows] if self.prompt else x


@dataclasses.dataclass
class Entry:
    """A request's next tokens, and the places among them whose logits are asked for."""

    key: Hashable
    tokens: Sequence[int]
    want: Sequence[int] = ()


class Batch:
    """The requests a model's slots hold, by key.  ``step`` runs the next tokens of any of them as one
    batch; ``end`` gives back what one holds; ``generate`` and ``draw`` are the serving loops on top.

    Raises (all before anything is launched):
        IndexError: a token outside the vocabulary.
        ValueError: no free slot, no tokens, or more of them than the model holds positions.
    """

    def __init__(self, lm):
        self.lm = lm
        self.slots: dict[Hashable, int] = {}
        self.held: dict[Hashable, int] = {}     # tokens of each request that have been run
        self._free = list(range(lm.config.slots))
        self._rows: np.ndarray | None = None    # the draw rows as the device has them

    # ------------------------------------------------------------------ slots
    def _claim(self) -> None:
        if self.lm.holder is not self:   # the versions were (re)loaded: the states hold nobody
            self.lm.holder = self
            self.slots.clear()
            self.held.clear()
            self._free = list(range(self.lm.config.slots))
            self._rows = None

    @property
    def free(self) -> int:
        self._claim()
        return len(self._free)

    def end(self, key: Hashable) -> None:
        """Give back the request's slot.  Its states need no clearing: the next sequence there starts at
        position 0 and reads none of them."""
        slot = self.slots.pop(key, None)
        if slot is not None:
            self.held.pop(key)
            self._free.append(slot)

    def _admit(self, entries: Sequence[Entry], more: int = 0) -> list[np.ndarray]:
        model = self.lm
        if model.decode_step is None:
            raise RuntimeError(f"{type(model).__name__}: load_versions() first")
        self._claim()
        keys = [e.key for e in entries]
        if len(set(keys)) != len(keys):
            raise ValueError(f"a request comes once a step, not as {keys}")
        ids = []
        for e in entries:
            tokens = np.asarray(e.tokens, dtype=np.int64).ravel()
            bad = tokens[(tokens < 0) | (tokens >= model.config.vocab_size)]
            if bad.size:
                raise IndexError(f"tokens {bad} are outside [0, {model.config.vocab_size})")
            total = self.held.get(e.key, 0) + tokens.size
            if tokens.size == 0 or total + more > model.config.max_seq_len:
                raise ValueError(f"{total} tokens{f' and {more} more' if more else ''} of request {e.key!r} do not fit "
                                 f"{model.config.max_seq_len} positions")
            if any(not 0 <= w < tokens.size for w in e.want):
                raise IndexError(f"request {e.key!r}: wanted places {list(e.want)} of {tokens.size} tokens")
            ids.append(tokens)
        new = [k for k in keys if k not in self.slots]
        if len(new) > len(self._free):
            raise ValueError(f"{len(new)} new requests for {len(self._free)} free slots")
        for key in new:
            self.slots[key] = self._free.pop(0)
            self.held[key] = 0
        return ids

    # ------------------------------------------------------------------ steps
    def step(self, entries: Sequence[Entry]) -> list[np.ndarray]:
        """Run every entry's tokens after what its request holds.  Returns, an entry, the logits at its
        wanted places: float32 ``(len(want), vocab)``."""
        ids = self._admit(entries)
        if all(t.size == 1 for t in ids):
            return self._decode(entries, ids)
        return self._portions(entries, ids)

    def _spans(self, spans: np.ndarray) -> None:
        self.lm.decode_step.write(self.lm.spans, spans)

    def _decode(self, entries, ids) -> list[np.ndarray]:
        model, c = self.lm, self.lm.config
        spans, tokens = np.zeros((c.slots, 4), np.int32), np.zeros(c.slots, np.int32)
        for e, t in zip(entries, ids):
            slot = self.slots[e.key]
            spans[slot, :3] = slot, 1, self.held[e.key]
            tokens[slot] = t[0]
        self._spans(spans)
        model.decode_step.write(model.token, tokens)
        logits = model()
        for e in entries:
            self.held[e.key] += 1
        if not any(len(e.want) for e in entries):
            return [np.empty((0, c.vocab_size), np.float32) for _ in entries]
        rows = logits.numpy()
        return [rows[[self.slots[e.key]] * len(e.want)] for e in entries]

    def _portions(self, entries, ids) -> list[np.ndarray]:
        model, c = self.lm, self.lm.config
        done = [0] * len(entries)
        room = c.key_room
        out = [np.empty((len(e.want), c.vocab_size), np.float32) for e in entries]
        while True:
            row, keys, spans, portion, asked = 0, 0, np.zeros((c.slots, 4), np.int32), np.zeros(c.prefill_chunk, np.int32), []
            for i, (e, t) in enumerate(zip(entries, ids)):
                n = min(t.size - done[i], c.prefill_chunk - row)
                if n > 0 and room is not None:   # (a request alone always fits: it has no more keys than positions)
                    n = min(n, room - keys - self.held[e.key])
                if n <= 0:
                    continue
                keys += self.held[e.key] + n
                spans[self.slots[e.key], :3] = row, n, self.held[e.key]
                portion[row : row + n] = t[done[i] : done[i] + n]
                asked += [(i, k, row + w - done[i]) for k, w in enumerate(e.want) if done[i] <= w < done[i] + n]
                done[i] += n
                self.held[e.key] += n
                row += n
            if row == 0:
                return out
            self._spans(spans)
            tails = model(portion, rows=row)
            at_tail = {int(s[0] + s[1] - 1): slot for slot, s in enumerate(spans) if s[1]}
            if all(r in at_tail for _, _, r in asked):
                got = tails.numpy() if asked else None
                for i, k, r in asked:
                    out[i][k] = got[at_tail[r]]
                continue
            for first in range(0, len(asked), READOUT_ROWS):
                some = asked[first : first + READOUT_ROWS]
                picks = np.zeros(READOUT_ROWS, np.int32)
                picks[: len(some)] = [r for _, _, r in some]
                got = model.readout(picks).numpy()
                for (i, k, _), line in zip(some, got):
                    out[i][k] = line

    # ------------------------------------------------------------------ serving
    def _stage_draws(self, slot: int, sampler, start: int, count: int) -> None:
        """The slot's draw rows for positions ``start`` onwards; all zero draws greedily."""
        model, c = self.lm, self.lm.config
        if sampler is None and (self._rows is None or not self._rows[slot].any()):
            return
        if self._rows is None:
            self._rows = np.zeros((c.slots, c.max_seq_len, ROW_WORDS), np.int32)
        self._rows[slot] = 0
        if sampler is not None:
            self._rows[slot, start : start + count] = sampler.rows(count, model.k_max)
        model.decode_step.write(model.draws, self._rows)

    def _prefill(self, key, tokens, count: int, sampler) -> None:
        entry = Entry(key, tokens)
        (ids,) = self._admit([entry], more=count - 1)
        last = self.held[key] + ids.size - 1
        self._stage_draws(self.slots[key], sampler, last, count)
        self._portions([entry], [ids])

    def _drawn(self) -> np.ndarray:
        return self.lm.decode_step.read(self.lm.drawn)

    def _run(self, last: dict[Hashable, int], steps: int) -> None:
        """``steps`` decode steps of the requests in ``last`` (each one's last drawn token), nothing read
        back between them where the step is captured."""
        model, c = self.lm, self.lm.config
        spans, tokens = np.zeros((c.slots, 4), np.int32), np.zeros(c.slots, np.int32)
        for key, token in last.items():
            slot = self.slots[key]
            spans[slot, :3] = slot, 1, self.held[key]
            tokens[slot] = token
        self._spans(spans)
        model.decode_step.write(model.token, tokens)
        if model.decode_step.captured:
            model.decode_step.start()
            model.decode_step.replay(steps - 1)
        else:
            for _ in range(steps):
                model()
        for key in last:
            self.held[key] += steps

    def draw(self, key: Hashable, tokens, max_tokens: int, sampler=None, each: bool = False) -> Iterator[int]:
        """Yield ``max_tokens`` tokens drawn on the device after ``tokens`` of one request."""
        self._prefill(key, tokens, max_tokens, sampler)
        slot = self.slots[key]
        token = int(self._drawn()[slot, self.held[key] - 1])
        yield token
        left = max_tokens - 1
        while left:
            n = 1 if each else left
            at = self.held[key]
            self._run({key: token}, n)
            for token in self._drawn()[slot, at : at + n]:
                token = int(token)
                yield token
            left -= n

    def generate(self, prompts: Sequence[Sequence[int]], max_tokens: int, samplers=None, round_steps: int = 32) -> list[list[int]]:
        """Up to ``max_tokens`` tokens after each of the prompts, as many of them in flight as there are
        free slots; a prompt that has its tokens, or drew an end-of-sequence id, makes room for the next
        one every ``round_steps`` steps."""
        if max_tokens <= 0:
            raise ValueError(f"{max_tokens} tokens to draw")
        eos = self.lm.eos
        out: list[list[int]] = [[] for _ in prompts]
        waiting, running = list(range(len(prompts))), {}
        if not self.free:
            raise ValueError("no free slot")
        try:
            while waiting or running:
                while waiting and self._free:
                    i = waiting.pop(0)
                    key = ("generate", id(out), i)
                    running[key] = i
                    self._prefill(key, prompts[i], max_tokens, None if samplers is None else samplers[i])
                    out[i].append(int(self._drawn()[self.slots[key], self.held[key] - 1]))
                for key, i in list(running.items()):
                    if len(out[i]) >= max_tokens or out[i][-1] in eos:
                        self.end(key)
                        del running[key]
                if not running:
                    continue
                steps = min(round_steps, min(max_tokens - len(out[i]) for i in running.values()))
                starts = {key: self.held[key] for key in running}
                self._run({key: out[i][-1] for key, i in running.items()}, steps)
                record = self._drawn()
                for key, i in running.items():
                    for token in record[self.slots[key], starts[key] : starts[key] + steps]:
                        out[i].append(int(token))
                        if out[i][-1] in eos:
                            break
        finally:
            for key in running:
                self.end(key)
        return out


class SlotSession(Session):
    """A conversation as one request of the model's batch.  A recurrent state cannot be rewound, so a
    history that is not the cached one plus more tokens is run from its start."""

    def _reusable(self, ids: np.ndarray) -> int:
        batch = self.lm.batch
        batch._claim()
        if batch.held.get(self) != self.cached.size:
            self.cached = self.cached[:0]
        shared = super()._reusable(ids)
        return shared if shared == self.cached.size else 0

    def _start(self, ids: np.ndarray) -> np.ndarray:
        """The tokens of ``ids`` the request does not hold yet, its slot given back first if it must
        start over."""
        begin = self._reusable(ids)
        if begin == 0:
            self.lm.batch.end(self)
        return ids[begin:]

    def forget(self, position: int) -> None:
        if position < self.cached.size:
            self.lm.batch.end(self)
            self.cached = self.cached[:0]

    def resume(self, held: int) -> int:
        return held if held == self.cached.size else 0

    def logits(self, tokens) -> np.ndarray:
        ids = self._checked(tokens)
        self._fits(ids.size)
        rest = self._start(ids)
        self.cached = self.cached[:0]
        (row,) = self.lm.batch.step([Entry(self, rest, [rest.size - 1])])
        self.cached = ids
        return row[0]

    def draw(self, tokens, max_tokens: int, sampler=None, each: bool = False) -> Iterator[int]:
        model, ids = self.lm, self._checked(tokens)
        if max_tokens <= 0:
            raise ValueError(f"{ids.size} tokens and {max_tokens} more to draw do not fit {model.config.max_seq_len} rows")
        self._fits(ids.size, max_tokens - 1)
        if model.decode_step is None:
            raise RuntimeError(f"{type(model).__name__}: load_versions() first")
        rest = self._start(ids)
        self.cached = self.cached[:0]
        out: list[int] = []
        for token in model.batch.draw(self, rest, max_tokens, sampler, each):
            out.append(token)
            yield token
        self.cached = np.concatenate([ids, np.asarray(out[:-1], dtype=np.int64)])


class StreamDecoder(Decoder):
    """The trunk of a decoder with a float32 stream: embedding, layers, final norm."""

    def __init__(self, c, layer):
        super().__init__(c, layer)
        self.norm = StreamRMSNorm(c.hidden_size, c.eps, c.activations, c.norm_unit, c.norm_groups)


class BatchedLM(CausalLM):
    """A ``CausalLM`` whose graph runs a batch of spans over a float32 residual stream.  ``runs`` lists the
    layer runs in order, each the index of its layer and the states of that run alone.

    The config is a ``LayerListConfig``: it adds to a decoder's ``slots`` (sequences served at once),
    ``activations`` (bf16, or float32 for a model in 32 bits throughout), ``order`` (layer indices in running
    order), ``norm_unit`` (what the final norm's gains are stored around), ``norm_groups`` (parts of a row it norms by themselves),
    ``embed_scale``, ``looks_back`` (layers read the stream behind every earlier one), ``logit_scale``, ``logit_softcap`` and ``key_room`` (keys a portion's layers may attend in all)."""

    decoder_class = StreamDecoder
    session_class = SlotSession

    def __init__(self, config, weights):
        super().__init__(config, weights)
        c = config
        self.residual = iron.state((max(c.prefill_chunk, c.slots), c.hidden_size), np.float32)
        self.planes = iron.state((len(c.order) + 1, *self.residual.shape), np.float32) if c.looks_back else None
        self.spans = iron.state((c.slots, 4), np.int32)
        self.token = iron.state((c.slots,), np.int32)
        self.runs = [(i, self.layers[i].mixer.states(c.slots)) for i in c.order]
        self.readout = None
        self.batch = Batch(self)

    @staticmethod
    def draw_shape(config) -> tuple[int, ...]:
        return (config.slots, config.max_seq_len)

    # ------------------------------------------------------------------ the recorded body
    def body(self, ids=None, picks=None, *, rows: Scratchpad[np.int32] = np.int32(1)):
        c = self.config
        if picks is not None:
            return self.head(Copy.step(self.residual[picks], dtype=np.float32))[0]
        call = BatchCall(prompt=ids is not None, spans=self.spans, rows=rows, planes=self.planes)
        count = c.prefill_chunk if call.prompt else c.slots
        x = call.bound(self.residual[:count])
        ids = call.bound(ids) if call.prompt else self.token
        first = [] if self.planes is None else [call.bound(self.planes[0][:count])]
        StreamEmbed.step(self.model.embed_tokens.weight, ids, x, *first, twice=bool(first), scale=c.embed_scale)
        for index, states in self.runs:
            x = self.layers[index](x, call, states)
        last = SpanTails.step(x, self.spans) if call.prompt else x
        logits, rounded = self.head(last)
        SampleSlots.step(rounded, self.draws, self.spans, self.token, self.drawn, vocab=c.vocab_size, batch_rows=count,
                         k_max=min(self.k_max, c.vocab_size))
        return logits

    def head(self, x):
        """Final norm, output projection, scale and soft cap: float32 logits, and the draw's rounded ones."""
        logits = as_rows(self.lm_head(self.model.norm(x)), x.shape[0])
        return Softcap.step(logits, cap=self.config.logit_softcap or 0.0, scale=self.config.logit_scale,
                            dtype=self.config.activations)

    # ------------------------------------------------------------------ versions
    def shapes(self) -> list[dict]:
        """``[decode step, prompt portion (ids), readout (picks)]``."""
        return [{}, {"ids": ((self.config.prefill_chunk,), np.int32)}, {"picks": ((READOUT_ROWS,), np.int32)}]

    def load_versions(self, *, capture: bool = True, check: bool = False, fuse: bool = True) -> None:
        try:
            versions = [self.compile(capture=capture, check=check, fuse=fuse, **shape) for shape in self.shapes()]
            for version in versions:
                version.load()
        except Exception:
            self.release()
            raise
        self.use(*versions)

    def use(self, decode, prompt, readout) -> None:
        super().use(decode, prompt)
        self.readout = readout

    def release(self) -> None:
        self.readout = None
        super().release()

    def generate_batch(self, prompts, max_tokens: int, samplers=None) -> list[list[int]]:
        """``generate`` for several prompts of token ids at once (see ``Batch.generate``)."""
        return self.batch.generate([self._prompt_ids(p) for p in prompts], max_tokens, samplers)


class _HostBatchVersion(_HostVersion):
    """A batched version stood in by the graph's host reference."""

    def __init__(self, graph, name: str | None = None):
        super().__init__(graph, name is not None)
        self.name = name

    def __call__(self, *tensors, **values):
        lead = (None,) if self.name == "picks" else ()
        outs, _ = iron.Graph.reference(self.graph, *lead, *tensors, **values)
        return _HostOutput(outs[0])


class BatchedOnHost(OnHost):
    """``OnHost`` for a batched model."""

    def load_versions(self, **_):
        self.use(_HostBatchVersion(self), _HostBatchVersion(self, "ids"), _HostBatchVersion(self, "picks"))
