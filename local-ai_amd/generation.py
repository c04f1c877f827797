"""Generation over any pipeline that serves sequences: sampler, requests and the scheduler that shares the pipeline's
sequence slots among them.

A model here has ``vocab_size``, ``new_sequence() -> seq``, ``step(seq, tokens, want) -> logits``, ``end_sequence(seq)`` and
``slots`` (kv_cache.SlotPool); ``StackPipeline`` is one, ``PipelineSequences`` makes one of a ``DecodePipeline``."""
from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field
from typing import Deque, List, Optional, Sequence

import numpy as np

from . import InvalidArgument
from .kv_cache import SlotPool


@dataclass
class Sampler:
    """Picks the next token from logits.  temperature 0 is greedy (ties: the lower index)."""
    temperature: float = 0.0
    top_k: int = 0
    top_p: float = 1.0
    seed: int = 0

    def __post_init__(self):
        self._rng = np.random.default_rng(self.seed)

    def pick(self, logits: np.ndarray) -> int:
        if self.temperature <= 0.0:
            return int(np.argmax(logits))
        z = logits.astype(np.float64) / self.temperature
        order = np.argsort(-z, kind="stable")
        if self.top_k > 0:
            order = order[:self.top_k]
        p = np.exp(z[order] - z[order[0]])
        p /= p.sum()
        if self.top_p < 1.0:                       # the shortest prefix that reaches top_p
            keep = int(np.searchsorted(np.cumsum(p), self.top_p)) + 1
            order, p = order[:keep], p[:keep] / p[:keep].sum()
        return int(self._rng.choice(order, p=p))


@dataclass(eq=False)
class Request:
    prompt: Sequence[int]
    max_new_tokens: int
    sampler: Sampler = field(default_factory=Sampler)
    stop_tokens: Sequence[int] = ()
    tokens: List[int] = field(default_factory=list)    # generated so far
    done: bool = False
    _seq: object = None
    _fed: int = 0                                       # prompt tokens that have run


class Scheduler:
    """First come, first served into the model's slots; the live requests take turns, a turn being one portion of the prompt
    (at most `portion` tokens) or one generated token."""

    def __init__(self, model, portion: int = 512):
        if portion < 1:
            raise InvalidArgument("a portion has at least one token")
        self.model, self.portion = model, portion
        self.waiting: Deque[Request] = deque()
        self.live: Deque[Request] = deque()

    def submit(self, request: Request) -> Request:
        if not request.prompt:
            raise InvalidArgument("the prompt is empty")
        limit = getattr(self.model, "max_tokens", None)
        if limit is not None and len(request.prompt) + max(request.max_new_tokens - 1, 0) > limit:
            raise InvalidArgument(f"{len(request.prompt)} + {request.max_new_tokens} tokens exceed the {limit} of a sequence")
        self.waiting.append(request)
        return request

    def turn(self) -> Optional[Request]:
        """Runs one turn of the request whose turn it is; None when there is nothing to do."""
        while self.waiting and self.model.slots.available() > 0:
            r = self.waiting.popleft()
            r._seq = self.model.new_sequence()
            self.live.append(r)
        if not self.live:
            return None
        r = self.live.popleft()
        try:
            self._advance(r)
        except BaseException:
            self._finish(r)
            raise
        if not r.done:
            self.live.append(r)
        return r

    def _advance(self, r: Request) -> None:
        if r.max_new_tokens <= 0:
            return self._finish(r)
        if r._fed < len(r.prompt):
            part = list(r.prompt[r._fed:r._fed + self.portion])
            last = r._fed + len(part) == len(r.prompt)
            logits = self.model.step(r._seq, part, [len(part) - 1] if last else [])
            r._fed += len(part)
            if not last:
                return
            token = r.sampler.pick(logits[0])
        elif r.sampler.temperature <= 0.0 and hasattr(self.model, "greedy"):
            token = self.model.greedy(r._seq, r.tokens[-1])
        else:
            token = r.sampler.pick(self.model.step(r._seq, [r.tokens[-1]], [0])[0])
        r.tokens.append(token)
        if len(r.tokens) >= r.max_new_tokens or token in r.stop_tokens:
            self._finish(r)

    def _finish(self, r: Request) -> None:
        r.done = True
        if r._seq is not None:
            self.model.end_sequence(r._seq)
            r._seq = None

    def run(self) -> None:
        while self.turn() is not None:
            pass


def generate(model, prompt: Sequence[int], max_new_tokens: int, sampler: Optional[Sampler] = None,
             stop_tokens: Sequence[int] = (), portion: int = 512) -> List[int]:
    """The tokens that follow `prompt`."""
    scheduler = Scheduler(model, portion)
    r = scheduler.submit(Request(prompt, max_new_tokens, sampler or Sampler(), stop_tokens))
    scheduler.run()
    return r.tokens


class PipelineSequences:
    """A ``pipeline.DecodePipeline`` (one sequence at a time over its own caches) as a sequence model."""

    def __init__(self, pipeline):
        self.pipeline, self.vocab_size, self.max_tokens = pipeline, pipeline.config.vocab_size, pipeline.max_context
        self.slots = SlotPool(lambda: pipeline, 1)

    def new_sequence(self):
        self.pipeline.reset()
        return self.slots.acquire()

    def end_sequence(self, seq) -> None:
        self.slots.release(seq)

    def step(self, seq, tokens, want=()) -> np.ndarray:
        out = np.empty((len(want), self.vocab_size), np.float32)
        last, lo = len(tokens) - 1, 0
        while lo <= last:
            if any(p == lo for p in want) or lo == last:
                seq.decode_step(int(tokens[lo]))
                for i, p in enumerate(want):
                    if p == lo:
                        out[i] = seq.logits()
                lo += 1
                continue
            hi = min([p for p in want if p > lo] + [last, lo + seq.max_batch])
            seq.forward_tokens_batch(list(tokens[lo:hi]), seq.position)
            seq.position += hi - lo
            lo = hi
        return out
