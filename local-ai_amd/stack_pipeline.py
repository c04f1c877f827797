"""Pipeline of a stack of layers with bf16 weights (mixers.py): embedding, layer runs in order -- a range of layers may run
several times in a row -- final norm and head, over the caches and states of sequence slots."""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Sequence, Tuple, Type

import numpy as np

from . import BF16, F32, Buffer, CommandBatch, InvalidArgument, Kernels
from .kv_cache import SequenceSlot, SlotPool
from .linear_weight import Segment, StackedLinear
from .mixers import LatentAttentionSpec, LayerSpec, Norm, OutputNormLayer, PreNormLayer, Run, Workspace

DEFAULT_MAX_ROWS = 2048     # rows of one pass; longer portions go through in pieces


@dataclass
class Loop:
    """The range [start, stop) of layers is walked `times` times; every repetition begins by adding the embedded tokens again."""
    start: int
    stop: int
    times: int


@dataclass
class StackConfig:
    vocab: int
    width: int
    eps: float
    layers: List[LayerSpec]
    loop: Optional[Loop] = None
    layer: Type[PreNormLayer] = PreNormLayer     # where the norms are
    softcap: Optional[float] = None              # logits become softcap * tanh(logits / softcap)

    def runs(self) -> List[Tuple[int, bool]]:
        """[(layer, whether the embedding output is added before it)] in running order."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, False) for i in range(n)]
        a, b, t = self.loop.start, self.loop.stop, self.loop.times
        if not (0 <= a <= b <= n and t >= 0):
            raise InvalidArgument(f"loop over layers {a}..{b} of {n}, {t} times")
        return ([(i, False) for i in range(a)] + [(i, p > 0 and i == a) for p in range(t) for i in range(a, b)]
                + [(i, False) for i in range(b, n)])

    def check(self) -> None:
        """Refuses what no pipeline can run."""
        if self.loop is not None and issubclass(self.layer, OutputNormLayer):
            raise InvalidArgument("layers with norms behind the branches do not repeat")
        if self.softcap is not None and not self.softcap > 0:
            raise InvalidArgument(f"logits capped at {self.softcap}")
        for i, l in enumerate(self.layers):
            m = l.mixer
            if not isinstance(m, LatentAttentionSpec) or m.kv_from is None:
                continue
            j = self.layers[m.kv_from].mixer if 0 <= m.kv_from < i else None
            if not isinstance(j, LatentAttentionSpec) or j.kv_from is not None:
                raise InvalidArgument(f"layer {i} reads the cache of layer {m.kv_from}, which is no earlier layer with one of its own")
            if (j.kv_rank, j.rot_dim, j.rot_base) != (m.kv_rank, m.rot_dim, m.rot_base):
                raise InvalidArgument(f"layer {i} reads the cache of layer {m.kv_from}, whose rows are others")
            if self.loop is not None:
                raise InvalidArgument("layers that share a cache do not repeat")


class StackPipeline:
    """Serves one sequence per slot; the calls are those of generation.SequenceModel."""

    def __init__(self, ctx, kernels: Kernels, config: StackConfig, tensors, max_tokens: int, dtype: int = BF16,
                 max_sequences: int = 1, max_rows: int = DEFAULT_MAX_ROWS, graphs: bool = True):
        if dtype not in (BF16, F32):
            raise InvalidArgument("activations are bf16 or f32")
        config.check()
        self.ctx, self.kernels, self.config, self.dtype, self.graphs = ctx, kernels, config, dtype, graphs
        self.vocab_size, self.max_rows = config.vocab, max_rows
        self.max_tokens = max(max_tokens, 1)
        w = config.width
        self.layers = [config.layer(ctx, kernels, s, w, config.eps, tensors, f"l{i}.") for i, s in enumerate(config.layers)]
        self.runs = config.runs()
        self.embed = Buffer.from_slice(ctx, tensors.bf16("embed", (config.vocab, w)))
        self.final_norm = Norm(ctx, tensors.f32("final.norm", (w,)), config.eps)
        self.head = StackedLinear(ctx, [tensors.bf16("head", (config.vocab, w))], [Segment(config.vocab)])
        self.ws = Workspace(ctx)
        self.tokens_buf = Buffer.empty(ctx, 4 * max_rows)
        self.logits_buf = Buffer.empty(ctx, 4 * config.vocab)
        self.next_buf = Buffer.empty(ctx, 4)
        self.slots = SlotPool(self._new_slot, max_sequences)
        self.observe = None          # called with (run index, residual stream buffer, rows) after every layer run

    def _new_slot(self) -> SequenceSlot:
        memories = []
        for i, _ in self.runs:
            mixer = self.layers[i].mixer
            source = getattr(mixer, "source", None)         # the layer whose memory this one reads
            memories.append(mixer.memory(self.ctx, self.kernels, self.max_tokens, self.dtype) if source is None else memories[source])
        return SequenceSlot(self.ctx, memories)

    # ---- sequences ------------------------------------------------------------------------------------------------------
    def new_sequence(self) -> SequenceSlot:
        return self.slots.acquire()

    def end_sequence(self, seq: SequenceSlot) -> None:
        self.slots.release(seq)

    def step(self, seq: SequenceSlot, tokens: Sequence[int], want: Sequence[int] = ()) -> np.ndarray:
        """Runs `tokens` at the sequence's next positions; logits f32 [len(want), vocab] at those places among them."""
        n = len(tokens)
        if n == 0:
            raise InvalidArgument("a step needs at least one token")
        if seq.position + n > self.max_tokens:
            raise InvalidArgument(f"position {seq.position + n} beyond the {self.max_tokens} tokens of a sequence")
        if any(not 0 <= int(t) < self.vocab_size for t in tokens):
            raise InvalidArgument("token id outside the vocabulary")
        if any(not 0 <= int(p) < n for p in want):
            raise InvalidArgument("wanted place outside the step")
        out = np.empty((len(want), self.vocab_size), np.float32)
        for lo in range(0, n, self.max_rows):
            hi = min(lo + self.max_rows, n)
            at = [i for i, p in enumerate(want) if lo <= p < hi]
            got = self._forward(seq, tokens[lo:hi], [want[i] - lo for i in at])
            if at:
                out[at] = got
        return out

    def greedy(self, seq: SequenceSlot, token: int) -> int:
        """One decoded token whose successor is picked on the device."""
        if seq.position + 1 > self.max_tokens:
            raise InvalidArgument(f"position {seq.position + 1} beyond the {self.max_tokens} tokens of a sequence")
        self._decode(seq, token)
        return int(self.next_buf.as_array(np.uint32, 1)[0])

    # ---- encoding -------------------------------------------------------------------------------------------------------
    def _encode_stack(self, batch, seq: SequenceSlot, n: int, max_position: int) -> Buffer:
        """Embedding and all layer runs of the n tokens in tokens_buf; returns the residual stream.  The embedding output
        stays as it is (later passes of a loop add it): the first norm leaves the stream in a buffer of its own.  For one
        token a norm may not write what other workgroups still read, so the stream alternates between two buffers."""
        K, width = self.kernels, self.config.width
        x0 = self.ws.get("embedded", n * width * 4)
        x, y = self.ws.get("stream", n * width * 4), self.ws.get("stream.other", width * 4)
        K.embed_rows_bf16_into(batch, self.embed, self.vocab_size, width, self.tokens_buf, n, x0)
        r = Run(K, batch, n, self.ws, self.dtype, seq.position_buf, max_position, x0, None, x)
        for i, ((layer, add), memory) in enumerate(zip(self.runs, seq.memories)):
            if add:
                r.add = x0
                r.store = (y if r.x is x else x) if n == 1 else r.x
            self.layers[layer].run(r, memory)
            if self.observe is not None:
                Norm.flush(r)
                self.observe(i, r.x, n)
        Norm.flush(r)
        return r.x

    def _forward(self, seq: SequenceSlot, tokens, want) -> Optional[np.ndarray]:
        n = len(tokens)
        if n == 1 and self.observe is None:
            self._decode(seq, int(tokens[0]))
            return np.repeat(self.logits_buf.as_array(np.float32, self.vocab_size)[None], len(want), 0) if want else None
        K, width = self.kernels, self.config.width
        self.tokens_buf.copy_from_bytes(np.asarray(tokens, np.uint32))
        batch = CommandBatch(self.ctx)
        x = self._encode_stack(batch, seq, n, seq.position)
        K.advance_position_into(batch, seq.position_buf, n)
        logits = None
        if len(want) == 1:
            logits = self.logits_buf
            self._encode_head(batch, x.view(want[0] * width * 4, width * 4))
        elif want:
            m = len(want)
            index = self.ws.get("want", 4 * self.max_rows)
            index.copy_from_bytes(np.asarray(want, np.uint32))
            logits = self.ws.get("logits", m * self.vocab_size * 4)
            size = 4 if self.dtype == F32 else 2
            h = self.ws.get("wanted", m * width * size)
            K.norm_rows_f32_into(batch, x, None, self.final_norm.weight, None, index, h, self.dtype, width, m, self.config.eps)
            self.head.rows_into(batch, K, h, self.dtype, m, [logits], F32)
            self._encode_cap(batch, logits, m)
        batch.commit_and_wait()
        seq.position += n
        return logits.as_array(np.float32, len(want) * self.vocab_size).reshape(len(want), -1) if want else None

    def _encode_head(self, batch, row: Buffer) -> None:
        self.head.normed_vector_into(batch, self.kernels, row, self.final_norm.weight, self.config.eps, [self.logits_buf], F32)
        self._encode_cap(batch, self.logits_buf, 1)

    def _encode_cap(self, batch, logits: Buffer, rows: int) -> None:
        if self.config.softcap is not None:
            self.kernels.softcap_f32_into(batch, logits, rows * self.vocab_size, self.config.softcap)

    def _encode_decode(self, batch, seq: SequenceSlot, max_position: int) -> None:
        self._encode_head(batch, self._encode_stack(batch, seq, 1, max_position))
        self.kernels.argmax_rows_f32_into(batch, self.logits_buf, self.next_buf, 1, self.vocab_size)
        self.kernels.advance_position_into(batch, seq.position_buf, 1)

    def _decode(self, seq: SequenceSlot, token: int) -> None:
        """One token: logits in logits_buf, the largest one's index in next_buf.  The first decoded token of a slot runs
        dispatch by dispatch, the next one records the step into a graph that later ones replay as long as the scratch buffers
        stay where they are (everything that changes from step to step is in device memory)."""
        self.tokens_buf.copy_from_bytes(np.asarray([token], np.uint32))
        batch = CommandBatch(self.ctx)
        if seq.graph is not None and seq.graph_version == self.ws.version:
            seq.graph.launch()
        elif self.graphs and seq.graph_ready:
            seq.graph = None
            batch.begin_capture()
            try:
                self._encode_decode(batch, seq, self.max_tokens - 1)
            except BaseException:
                batch.end_capture()
                raise
            seq.graph, seq.graph_version = batch.end_capture(), self.ws.version
            seq.graph.launch()
        else:
            self._encode_decode(batch, seq, seq.position)
            seq.graph_ready = True
        batch.commit_and_wait()
        seq.position += 1
