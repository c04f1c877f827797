"""The parts of a decoder layer with bf16 weights: token mixers (softmax attention with one or two score maps, linear
attention with a fixed decay), feed-forwards (dense, mixture of experts), and the pre-norm layer that joins them.  Every
part has two encodings of the same computation: ``rows`` for a portion of several tokens, and ``vector`` for a single token,
where norms, gates and expert selection ride in the products that need them.  All constants come with the specs.

A spec is what a configuration says about a part; it also names the tensors the part loads.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional

import numpy as np

from . import (ACT_GELU_TANH, ACT_NONE, ACT_RELU_SQUARED, ACT_SILU, BLOCKS_AT_POSITION, F32, ROWS_AT_POSITION, Buffer,
               InvalidArgument, Kernels)
from .kv_cache import BlockKvCache, RecurrentState
from .linear_weight import Segment, StackedLinear

CHUNK = 64                 # rows per chunk of lh_linear_attention_chunked_into
CHUNKED_MIN_ROWS = 17      # below this a portion walks the recurrence
MAX_CHUNKED_DIM = 256


class Workspace:
    """Scratch buffers by name, grown to the largest request.  Layers of a stack run one after the other and share them.
    ``version`` changes whenever a buffer is replaced: a step recorded before that must not be replayed."""

    def __init__(self, ctx):
        self.ctx, self._buffers, self.version = ctx, {}, 0

    def get(self, name: str, nbytes: int) -> Buffer:
        b = self._buffers.get(name)
        if b is None or b.length() < nbytes:
            self.version += 1
            b = self._buffers[name] = Buffer.empty(self.ctx, max(nbytes, 16))
        return b


@dataclass
class Run:
    """One pass of a portion through the stack: where the residual stream is and what the next norm adds to it first."""
    kernels: Kernels
    batch: object
    rows: int
    ws: Workspace
    dtype: int                       # activations and caches: bf16, or f32
    position: Buffer                 # device word: position of the portion's first token
    max_position: int                # bound on it that holds whenever this encoding runs
    x: Buffer                        # residual stream, f32 [rows, width]
    add: Optional[Buffer] = None     # rows the next norm adds to x before it
    store: Optional[Buffer] = None   # where the next norm leaves the (summed) stream; None: x stays as it is

    @property
    def size(self) -> int:
        return 4 if self.dtype == F32 else 2

    def scratch(self, name: str, values: int, f32: bool = False) -> Buffer:
        return self.ws.get(name + (".f32" if f32 else ""), values * (4 if f32 else self.size))

    def take_input(self):
        """(x, add, store) for the norm that runs now; the stream is in ``store`` afterwards if there is one."""
        x, add, store = self.x, self.add, self.store
        self.add = self.store = None
        if store is not None:
            self.x = store
        return x, add, store


class Norm:
    def __init__(self, ctx, weight: np.ndarray, eps: float):
        self.weight, self.dim, self.eps = Buffer.from_slice(ctx, np.asarray(weight, np.float32)), weight.size, eps

    def rows(self, r: Run) -> Buffer:
        x, add, store = r.take_input()
        out = r.scratch("normed", r.rows * self.dim)
        r.kernels.norm_rows_f32_into(r.batch, x, add, self.weight, store, None, out, r.dtype, self.dim, r.rows, self.eps)
        return out

    def vector_into(self, r: Run, linear: StackedLinear, outputs, dtype: int) -> None:
        """The norm of the stream, then `linear` on it, in one step."""
        x, add, store = r.take_input()
        linear.normed_vector_into(r.batch, r.kernels, x, self.weight, self.eps, outputs, dtype, r.position, add, store)


# ---- softmax attention, one or two maps ---------------------------------------------------------------------------------
@dataclass
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    maps: int = 1
    diff: float = 0.0        # two maps: the constant part of lambda, and 1 - diff scales the output
    bias: bool = False


def difference_lambda(lq1, lk1, lq2, lk2, diff: float) -> float:
    """The weight of the second map, one number per layer, from four learned vectors (32-bit)."""
    f = np.float32
    a = np.exp(np.sum(np.asarray(lq1, f) * np.asarray(lk1, f), dtype=f))
    b = np.exp(np.sum(np.asarray(lq2, f) * np.asarray(lk2, f), dtype=f))
    return float(f(a) - f(b) + f(diff))


class SoftmaxAttention:
    def __init__(self, ctx, kernels: Kernels, spec: AttentionSpec, width: int, eps: float, tensors, prefix: str):
        s = self.spec = spec
        if s.heads % s.kv_heads:
            raise InvalidArgument(f"{s.heads} heads over {s.kv_heads} key/value heads")
        dq, dv = kernels.attention_padded_dim(s.dim), kernels.attention_padded_vdim(s.vdim)
        self.dq = dq
        nq, nk, nv = s.heads * s.maps * s.dim, s.kv_heads * s.maps * s.dim, s.kv_heads * s.vdim
        names = [(prefix + n, c) for n, c in (("q", nq), ("k", nk), ("v", nv))]
        self.qkv = StackedLinear(ctx, [tensors.bf16(n, (c, width)) for n, c in names],
                                 [Segment(nq, head=s.dim, padded=dq), Segment(nk, head=s.dim, padded=dq, layout=ROWS_AT_POSITION),
                                  Segment(nv, head=s.vdim, padded=dv, layout=BLOCKS_AT_POSITION)],
                                 [tensors.f32(n + ".b", (c,)) for n, c in names] if s.bias else None)
        self.out = StackedLinear(ctx, [tensors.bf16(prefix + "o", (width, s.heads * s.vdim))], [Segment(width)])
        self.eps, self.lam, self.out_scale = eps, 0.0, 1.0
        if s.maps == 2:
            self.lam = difference_lambda(*(tensors.f32(prefix + n, (s.dim,)) for n in ("lq1", "lk1", "lq2", "lk2")), s.diff)
            self.out_scale = 1.0 - s.diff

    def memory(self, ctx, kernels: Kernels, capacity: int, dtype: int) -> BlockKvCache:
        s = self.spec
        return BlockKvCache(ctx, kernels, s.kv_heads, s.maps, s.dim, s.vdim, capacity, dtype)

    def run(self, r: Run, norm: Norm, memory: BlockKvCache) -> None:
        s = self.spec
        q = r.scratch("q", r.rows * s.heads * s.maps * self.dq)
        outputs = [q, memory.keys, memory.values]
        if r.rows == 1:
            norm.vector_into(r, self.qkv, outputs, r.dtype)
        else:
            self.qkv.rows_into(r.batch, r.kernels, norm.rows(r), r.dtype, r.rows, outputs, r.dtype, r.position)
        mixed = r.scratch("mixed", r.rows * s.heads * s.vdim)
        r.kernels.attention_rows_into(r.batch, q, memory.keys, memory.values, mixed, r.dtype, r.position, r.max_position, r.rows,
                                      s.heads, s.kv_heads, s.maps, s.dim, s.vdim, memory.capacity, s.scale, self.lam,
                                      self.out_scale, self.eps)
        if r.rows == 1:
            self.out.vector_add_into(r.batch, r.kernels, mixed, r.dtype, r.x)
        else:
            self.out.rows_add_into(r.batch, r.kernels, mixed, r.dtype, r.rows, r.x)


# ---- linear attention with a fixed decay per head -----------------------------------------------------------------------
@dataclass
class LinearAttentionSpec:
    heads: int
    dim: int
    vdim: int
    decay: List[float]
    act: int = ACT_SILU      # of q, k and v


class LinearAttention:
    def __init__(self, ctx, kernels: Kernels, spec: LinearAttentionSpec, width: int, eps: float, tensors, prefix: str):
        s = self.spec = spec
        if len(s.decay) != s.heads:
            raise InvalidArgument(f"{len(s.decay)} decays for {s.heads} heads")
        dq = self.dq = kernels.linear_attention_padded_dim(s.dim)
        nk, nv = s.heads * s.dim, s.heads * s.vdim
        self.qkvg = StackedLinear(ctx, [tensors.bf16(prefix + n, (c, width)) for n, c in (("q", nk), ("k", nk), ("v", nv), ("g", nv))],
                                  [Segment(nk, s.act, s.dim, dq), Segment(nk, s.act, s.dim, dq), Segment(nv, s.act),
                                   Segment(nv, ACT_NONE)])
        self.norm = Norm(ctx, tensors.f32(prefix + "norm", (nv,)), eps)
        self.out = StackedLinear(ctx, [tensors.bf16(prefix + "o", (width, nv))], [Segment(width)])
        decay = np.asarray(s.decay, np.float64)
        self.decay = Buffer.from_slice(ctx, decay.astype(np.float32))
        self.powers = Buffer.from_slice(ctx, (decay[:, None] ** np.arange(CHUNK + 1)).astype(np.float32))

    def memory(self, ctx, kernels: Kernels, capacity: int, dtype: int) -> RecurrentState:
        return RecurrentState(ctx, kernels, self.spec.heads, self.spec.dim, self.spec.vdim)

    def run(self, r: Run, norm: Norm, memory: RecurrentState) -> None:
        s, K, b, n = self.spec, r.kernels, r.batch, r.rows
        nk, nv = s.heads * self.dq, s.heads * s.vdim
        q, k = r.scratch("lin.q", n * nk), r.scratch("lin.k", n * nk)
        v, g = r.scratch("lin.v", n * nv), r.scratch("lin.g", n * nv)
        o = r.scratch("lin.o", n * nv, f32=True)
        if n == 1:
            norm.vector_into(r, self.qkvg, [q, k, v, g], r.dtype)
        else:
            self.qkvg.rows_into(b, K, norm.rows(r), r.dtype, n, [q, k, v, g], r.dtype)
        if n >= CHUNKED_MIN_ROWS and r.dtype != F32 and s.dim <= MAX_CHUNKED_DIM:
            work = r.ws.get("lin.work", K.linear_attention_workspace_bytes(n, s.heads, s.dim, s.vdim))
            K.linear_attention_chunked_into(b, q, k, v, memory.state, self.powers, work, o, n, s.heads, s.dim, s.vdim)
        else:
            K.linear_attention_recurrent_into(b, q, k, v, r.dtype, memory.state, self.decay, o, n, s.heads, s.dim, s.vdim)
        if n == 1:
            K.linear_gated_vector_into(b, o, g, r.dtype, self.norm.weight, self.norm.eps, self.out.weight, None, nv,
                                       self.out.segments, [r.x], F32, True)
        else:
            y = r.scratch("mixed", n * nv)
            K.gated_norm_rows_into(b, o, g, self.norm.weight, y, r.dtype, nv, n, self.norm.eps)
            self.out.rows_add_into(b, K, y, r.dtype, n, r.x)


# ---- feed-forwards ------------------------------------------------------------------------------------------------------
@dataclass
class DenseSpec:
    ff: int
    act: int = ACT_GELU_TANH


class DenseFeedForward:
    def __init__(self, ctx, kernels: Kernels, spec: DenseSpec, width: int, tensors, prefix: str):
        self.spec = spec
        self.up = StackedLinear(ctx, [tensors.bf16(prefix + "up", (spec.ff, width))], [Segment(spec.ff, spec.act)])
        self.down = StackedLinear(ctx, [tensors.bf16(prefix + "down", (width, spec.ff))], [Segment(width)])

    def run(self, r: Run, norm: Norm) -> None:
        h = r.scratch("hidden", r.rows * self.spec.ff)
        if r.rows == 1:
            norm.vector_into(r, self.up, [h], r.dtype)
            self.down.vector_add_into(r.batch, r.kernels, h, r.dtype, r.x)
        else:
            self.up.rows_into(r.batch, r.kernels, norm.rows(r), r.dtype, r.rows, [h], r.dtype)
            self.down.rows_add_into(r.batch, r.kernels, h, r.dtype, r.rows, r.x)


@dataclass
class MoeSpec:
    experts: int
    top: int
    ff: int
    act: int = ACT_RELU_SQUARED


class MoeFeedForward:
    """Sigmoid gates: a token goes to its ``top`` best experts, scaled by the gate on the way in."""

    def __init__(self, ctx, kernels: Kernels, spec: MoeSpec, width: int, tensors, prefix: str):
        s = self.spec = spec
        self.width = width
        if not 1 <= s.top <= s.experts:
            raise InvalidArgument(f"top {s.top} of {s.experts} experts")
        self.router = StackedLinear(ctx, [tensors.bf16(prefix + "router", (s.experts, width))], [Segment(s.experts)])
        names = [f"{prefix}e{e}." for e in range(s.experts)]
        self.up = Buffer.from_slice(ctx, np.stack([tensors.bf16(n + "up", (s.ff, width)) for n in names]))
        self.down = Buffer.from_slice(ctx, np.stack([tensors.bf16(n + "down", (width, s.ff)) for n in names]))

    def run(self, r: Run, norm: Norm) -> None:
        s, K, b, n = self.spec, r.kernels, r.batch, r.rows
        logits = r.scratch("router", n * s.experts, f32=True)
        if n == 1:
            norm.vector_into(r, self.router, [logits], F32)
            h = r.scratch("expert", s.top * s.ff, f32=True)
            K.moe_vector_up_into(b, r.x, norm.weight, norm.eps, logits, self.up, h, s.experts, s.top, self.width, s.ff, s.act)
            K.moe_vector_down_into(b, h, logits, self.down, r.x, s.experts, s.top, self.width, s.ff)
            return
        x = norm.rows(r)
        self.router.rows_into(b, K, x, r.dtype, n, [logits], F32)
        plan = r.ws.get("plan", 4 * K.moe_plan_words(n, s.experts, s.top))
        K.moe_route_into(b, logits, plan, n, s.experts, s.top)
        h = r.scratch("hidden", n * s.top * s.ff)
        K.moe_up_into(b, x, r.dtype, plan, self.up, h, n, s.experts, s.top, self.width, s.ff, s.act)
        slots = r.scratch("slots", n * s.top * self.width, f32=True) if s.top > 1 else None
        K.moe_down_into(b, h, r.dtype, plan, self.down, slots, r.x, n, s.experts, s.top, self.width, s.ff)


# ---- the layer ----------------------------------------------------------------------------------------------------------
MIXERS = {AttentionSpec: SoftmaxAttention, LinearAttentionSpec: LinearAttention}
FEED_FORWARDS = {DenseSpec: DenseFeedForward, MoeSpec: MoeFeedForward}


@dataclass
class LayerSpec:
    mixer: object
    ff: Optional[object] = None


class PreNormLayer:
    """Two residual branches, each on a norm of the stream: the mixer, and the feed-forward where the layer has one."""

    def __init__(self, ctx, kernels: Kernels, spec: LayerSpec, width: int, eps: float, tensors, prefix: str):
        self.norm1 = Norm(ctx, tensors.f32(prefix + "norm1", (width,)), eps)
        self.mixer = MIXERS[type(spec.mixer)](ctx, kernels, spec.mixer, width, eps, tensors, prefix + "mix.")
        self.norm2 = self.ff = None
        if spec.ff is not None:
            self.norm2 = Norm(ctx, tensors.f32(prefix + "norm2", (width,)), eps)
            self.ff = FEED_FORWARDS[type(spec.ff)](ctx, kernels, spec.ff, width, tensors, prefix + "mlp.")

    def run(self, r: Run, memory) -> None:
        self.mixer.run(r, self.norm1, memory)
        if self.ff is not None:
            self.ff.run(r, self.norm2)
