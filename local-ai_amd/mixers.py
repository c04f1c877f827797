"""The parts of a decoder layer with bf16 weights: token mixers (softmax attention with one or two score maps, latent
attention, linear attention with a fixed decay, selective state space), feed-forwards (dense, gated, mixture of experts), and
the layers that join them, with norms in front of the residual branches or behind them.  Every part has two encodings of the
same computation: one for a portion of several rows, and one for a single row, where norms, gates and expert selection ride in
the products that need them.  All constants come with the specs.

A residual branch begins with a projection of the stream and ends with a product into it.  Where the norms are is the affair
of ``Norm`` (in front) and ``OutputNorm`` (behind): the parts call ``project`` and ``finish``.

A spec is what a configuration says about a part; it also names the tensors the part loads.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional

import numpy as np

from . import (ACT_GELU_TANH, ACT_NONE, ACT_RELU_SQUARED, ACT_SIGMOID, ACT_SILU, ACT_SILU_PAIRS, BLOCKS_AT_POSITION, F32,
               ROWS_AT_POSITION, ROWS_F32, Buffer, InvalidArgument, Kernels)
from .kv_cache import BlockKvCache, LatentCache, RecurrentState, SelectiveState
from .linear_weight import Segment, Segments, StackedLinear

CHUNK = 64                 # rows per chunk of lh_linear_attention_chunked_into and lh_selective_chunked_into
CHUNKED_MIN_ROWS = 17      # below this a portion walks the recurrence
MAX_CHUNKED_DIM = 256
GATED_IN_PRODUCT = 2048    # longer gated norms are a step of their own: every wave of the product would repeat them
EXPANDED_MIN_ROWS = 65     # from here on latent attention makes keys and values of every head out of its cache


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
    other: Optional[Buffer] = None   # norms behind the branches: the stream's second buffer
    pending: Optional[tuple] = None  # norms behind the branches: (branch output, its norm) still to be added to x

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

    def project(self, r: Run, linear: StackedLinear, outputs, dtype: int, segments: Optional[Segments] = None) -> None:
        """The branch's first product; `dtype` is that of the outputs, `segments` overrides where they go."""
        if r.rows == 1:
            x, add, store = r.take_input()
            linear.normed_vector_into(r.batch, r.kernels, x, self.weight, self.eps, outputs, dtype, r.position, add, store, segments)
        else:
            linear.rows_into(r.batch, r.kernels, self.rows(r), r.dtype, r.rows, outputs, dtype, r.position, segments)

    def destination(self, r: Run):
        """Where the branch's last product goes, and whether it adds to what is there."""
        return r.x, True

    def finish(self, r: Run, linear: StackedLinear, x: Buffer, x_dtype: int) -> None:
        """The branch's last product."""
        dest, add = self.destination(r)
        if r.rows == 1:
            r.kernels.linear_vector_into(r.batch, x, x_dtype, linear.weight, linear.bias, linear.k, linear.segments, [dest], F32, add)
        else:
            r.kernels.linear_rows_into(r.batch, x, x_dtype, linear.weight, linear.bias, r.rows, linear.k, linear.segments, [dest], F32, add)

    @staticmethod
    def flush(r: Run) -> None:
        """Leaves the whole stream in ``r.x``."""
        if r.pending is not None:
            branch, norm = r.pending
            r.kernels.residual_rows_into(r.batch, r.x, branch, norm.weight, r.x, None, F32, norm.dim, r.rows, norm.eps)
            r.pending = None


class OutputNorm(Norm):
    """The norm behind a branch: x <- x + norm(branch(x)).  It is computed by whatever reads the stream next."""

    def project(self, r: Run, linear: StackedLinear, outputs, dtype: int, segments: Optional[Segments] = None) -> None:
        K, b = r.kernels, r.batch
        if r.add is not None:
            raise InvalidArgument("layers with norms behind the branches do not repeat")
        if r.rows == 1:
            if r.pending is None:
                return linear.vector_into(b, K, r.x, F32, outputs, dtype, r.position, segments)
            (branch, norm), dest = r.pending, r.store or r.other      # (other workgroups still read x)
            linear.residual_vector_into(b, K, r.x, branch, dest, norm.weight, norm.eps, outputs, dtype, r.position, segments)
            r.other, r.x, r.store, r.pending = r.x, dest, None, None
            return
        if r.dtype == F32:
            self.flush(r)
            return linear.rows_into(b, K, r.x, F32, r.rows, outputs, dtype, r.position, segments)
        copy, (branch, norm) = r.scratch("normed", r.rows * self.dim), r.pending or (None, None)
        K.residual_rows_into(b, r.x, branch, norm and norm.weight, branch and r.x, copy, r.dtype, self.dim, r.rows, (norm or self).eps)
        r.pending = None
        linear.rows_into(b, K, copy, r.dtype, r.rows, outputs, dtype, r.position, segments)

    def destination(self, r: Run):
        y = r.scratch("branch", r.rows * self.dim, f32=True)
        r.pending = (y, self)
        return y, False


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
        norm.project(r, self.qkv, outputs, r.dtype)
        mixed = r.scratch("mixed", r.rows * s.heads * s.vdim)
        r.kernels.attention_rows_into(r.batch, q, memory.keys, memory.values, mixed, r.dtype, r.position, r.max_position, r.rows,
                                      s.heads, s.kv_heads, s.maps, s.dim, s.vdim, memory.capacity, s.scale, self.lam,
                                      self.out_scale, self.eps)
        norm.finish(r, self.out, mixed, r.dtype)


# ---- latent attention ---------------------------------------------------------------------------------------------------
@dataclass
class LatentAttentionSpec:
    heads: int
    dim: int                 # unrotated dimensions of a head's query and key
    rot_dim: int             # rotated ones, shared by all heads on the key's side
    vdim: int
    kv_rank: int
    rot_base: float
    scale: float
    kv_from: Optional[int] = None    # the layer whose cache this one reads; None: its own


class LatentAttention:
    """Keys and values of all heads are projections of one cached latent per position.  Few rows: the key projection goes to
    the queries and the value projection to the output.  Many rows: keys and values are made from the cache, layer by layer, in
    scratch memory.  A learned sink joins every softmax, a gate per head multiplies the outputs."""

    def __init__(self, ctx, kernels: Kernels, spec: LatentAttentionSpec, width: int, eps: float, tensors, prefix: str):
        s = self.spec = spec
        if s.rot_dim < 2 or s.rot_dim % 2:
            raise InvalidArgument(f"{s.rot_dim} rotated dimensions do not make pairs")
        self.eps, self.source = eps, s.kv_from
        H, d, e, r = s.heads, s.dim, s.rot_dim, s.kv_rank
        self.row = kernels.latent_row(r, e)
        self.dq, self.dv = kernels.attention_padded_dim(d + e), kernels.attention_padded_vdim(s.vdim)
        q = tensors.bf16(prefix + "q", (H * (d + e), width)).reshape(H, d + e, width)
        weights = [np.ascontiguousarray(q[:, :d]).reshape(H * d, width), np.ascontiguousarray(q[:, d:]).reshape(H * e, width),
                   tensors.bf16(prefix + "g", (H, width))]
        rest = [Segment(H * e, layout=ROWS_F32), Segment(H, layout=ROWS_F32)]
        if s.kv_from is None:
            weights.append(tensors.bf16(prefix + "dkv", (r + e, width)))
            rest.append(Segment(r + e, layout=ROWS_F32))
            self.latent_norm = Buffer.from_slice(ctx, np.asarray(tensors.f32(prefix + "dkv.norm", (r,)), np.float32))
        else:
            self.latent_norm = None
        self.qkvg = StackedLinear(ctx, weights, [Segment(H * d, head=d, padded=d)] + rest)
        self.padded = Segments([Segment(H * d, head=d, padded=self.dq)] + rest)     # as the expanded form wants the queries
        uk, uv = tensors.bf16(prefix + "uk", (H * d, r)), tensors.bf16(prefix + "uv", (H * s.vdim, r))
        self.up = Buffer.from_slice(ctx, np.concatenate([uk, uv]))
        self.key_up = Buffer.from_slice(ctx, np.ascontiguousarray(uk.reshape(H, d, r).transpose(0, 2, 1)))      # [head][rank][dim]
        self.value_up = self.up.view(H * d * r * 2, H * s.vdim * r * 2)
        self.sink = Buffer.from_slice(ctx, np.asarray(tensors.f32(prefix + "sink", (H,)), np.float32))
        self.frequencies = Buffer.from_slice(ctx, (float(s.rot_base) ** (-2.0 * np.arange(e // 2) / e)).astype(np.float32))
        self.out = StackedLinear(ctx, [tensors.bf16(prefix + "o", (width, H * s.vdim))], [Segment(width)])

    def memory(self, ctx, kernels: Kernels, capacity: int, dtype: int) -> LatentCache:
        return LatentCache(ctx, kernels, self.spec.kv_rank, self.spec.rot_dim, capacity, dtype)

    def run(self, r: Run, norm: Norm, memory: LatentCache) -> None:
        s, K, b, n = self.spec, r.kernels, r.batch, r.rows
        H, expanded = s.heads, n >= EXPANDED_MIN_ROWS
        q_rot, gate = r.scratch("latent.rot", n * H * s.rot_dim, f32=True), r.scratch("latent.gate", n * H, f32=True)
        down = r.scratch("latent.down", n * (s.kv_rank + s.rot_dim), f32=True) if self.source is None else None
        q = r.scratch("q", n * H * (self.dq if expanded else s.dim))
        norm.project(r, self.qkvg, [q, q_rot, gate] + ([down] if down else []), r.dtype, self.padded if expanded else None)
        mixed = r.scratch("mixed", n * H * s.vdim)
        if expanded:
            K.latent_prepare_into(b, q_rot, down, self.latent_norm, self.frequencies, r.position, q, r.dtype, memory.rows, r.dtype, n, H,
                                  s.kv_rank, s.rot_dim, self.dq, s.dim, s.dim, memory.capacity, self.eps)
            positions = (r.max_position + n + 31) // 32 * 32
            keys, values = r.scratch("latent.keys", positions * H * self.dq), r.scratch("latent.values", positions * H * self.dv)
            K.latent_expand_into(b, memory.rows, r.dtype, self.up, keys, values, positions, H, s.dim, s.rot_dim, s.vdim, s.kv_rank)
            K.attention_rows_into(b, q, keys, values, mixed, r.dtype, r.position, r.max_position, n, H, H, 1, s.dim + s.rot_dim, s.vdim,
                                  positions, s.scale, sink=self.sink, gate=gate)
        else:
            ql = r.scratch("latent.q", n * H * self.row, f32=True)
            K.latent_queries_into(b, q, self.key_up, q_rot, down, self.latent_norm, self.frequencies, r.position, ql, memory.rows, r.dtype,
                                  n, H, s.dim, s.kv_rank, s.rot_dim, memory.capacity, self.eps)
            ol = r.scratch("latent.out", n * H * s.kv_rank)
            K.latent_attention_rows_into(b, ql, memory.rows, ol, r.dtype, r.position, r.max_position, n, H, s.kv_rank, s.rot_dim,
                                         memory.capacity, s.scale, self.sink, gate)
            K.head_linear_into(b, ol, r.dtype, self.value_up, mixed, r.dtype, n, H, s.vdim, s.kv_rank, s.vdim)
        norm.finish(r, self.out, mixed, r.dtype)


# ---- linear attention with a fixed decay per head -----------------------------------------------------------------------
@dataclass
class LinearAttentionSpec:
    heads: int
    dim: int
    vdim: int
    decay: List[float]
    act: int = ACT_SILU      # of q, k and v
    scale: float = 1.0       # of the keys
    gate: int = ACT_SIGMOID
    head_norm: bool = False  # every head's output is normed by itself, without a weight; else all heads together, with one


def finish_gated(r: Run, norm: Norm, out: StackedLinear, o: Buffer, gate: Buffer, gate_dtype: int, weight, eps: float, group: int,
                 act: int, gate_first: bool) -> None:
    """Norm in parts of `group` values and gate of o (f32), then the branch's last product."""
    K, b, k = r.kernels, r.batch, out.k
    if r.rows == 1 and k <= GATED_IN_PRODUCT and K.gated_vector_fits(k, group):
        dest, add = norm.destination(r)
        K.linear_gated_vector_into(b, o, gate, gate_dtype, weight, eps, out.weight, None, k, out.segments, [dest], F32, add, None, group,
                                   act, gate_first)
        return
    y = r.scratch("mixed", r.rows * k, f32=gate_dtype == F32)
    K.gated_norm_rows_into(b, o, gate, weight, y, gate_dtype, k, r.rows, eps, group, act, gate_first)
    norm.finish(r, out, y, gate_dtype)


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
        self.eps, self.weight = eps, None if s.head_norm else Buffer.from_slice(ctx, np.asarray(tensors.f32(prefix + "norm", (nv,)), np.float32))
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
        norm.project(r, self.qkvg, [q, k, v, g], r.dtype)
        if n >= CHUNKED_MIN_ROWS and r.dtype != F32 and s.dim <= MAX_CHUNKED_DIM:
            work = r.ws.get("lin.work", K.linear_attention_workspace_bytes(n, s.heads, s.dim, s.vdim))
            K.linear_attention_chunked_into(b, q, k, v, memory.state, self.powers, work, o, n, s.heads, s.dim, s.vdim, s.scale)
        else:
            K.linear_attention_recurrent_into(b, q, k, v, r.dtype, memory.state, self.decay, o, n, s.heads, s.dim, s.vdim, s.scale)
        finish_gated(r, norm, self.out, o, g, r.dtype, self.weight, self.eps, s.vdim if s.head_norm else nv, s.gate, False)


# ---- selective state space ----------------------------------------------------------------------------------------------
@dataclass
class SelectiveSpec:
    heads: int
    vdim: int
    state: int
    groups: int              # heads in a row share one B and one C
    taps: int                # of the convolution
    norm_groups: int


class SelectiveStateSpace:
    """Linear attention whose decay and step size come from the token, behind a short causal convolution; the gate multiplies
    before the norm."""

    def __init__(self, ctx, kernels: Kernels, spec: SelectiveSpec, width: int, eps: float, tensors, prefix: str):
        s = self.spec = spec
        inner = self.inner = s.heads * s.vdim
        if s.heads % s.groups or inner % s.norm_groups:
            raise InvalidArgument(f"{s.heads} heads over {s.groups} groups, {inner} columns in {s.norm_groups} normed parts")
        channels = self.channels = inner + 2 * s.groups * s.state
        self.dq = kernels.linear_attention_padded_dim(s.state)
        self.proj = StackedLinear(ctx, [tensors.bf16(prefix + "in", (inner + channels + s.heads, width))[a:b] for a, b in
                                        ((0, inner), (inner, inner + channels), (inner + channels, None))],
                                  [Segment(inner), Segment(channels), Segment(s.heads, layout=ROWS_F32)])

        def f32(name, shape):
            return np.asarray(tensors.f32(prefix + name, shape), np.float32)
        self.taps = Buffer.from_slice(ctx, np.ascontiguousarray(f32("conv", (channels, s.taps)).T))
        self.conv_bias = Buffer.from_slice(ctx, f32("conv.b", (channels,)))
        self.dt_bias, self.a_log, self.skip = (Buffer.from_slice(ctx, f32(n, (s.heads,))) for n in ("dt_bias", "A_log", "D"))
        self.eps, self.weight = eps, Buffer.from_slice(ctx, f32("norm", (inner,)))
        self.out = StackedLinear(ctx, [tensors.bf16(prefix + "o", (width, inner))], [Segment(width)])

    def memory(self, ctx, kernels: Kernels, capacity: int, dtype: int) -> SelectiveState:
        s = self.spec
        return SelectiveState(ctx, kernels, s.heads, s.state, s.vdim, self.channels, s.taps)

    def run(self, r: Run, norm: Norm, memory: SelectiveState) -> None:
        s, K, b, n = self.spec, r.kernels, r.batch, r.rows
        wide = n == 1                                  # one row: the projections stay f32
        dtype = F32 if wide else r.dtype
        z, u = r.scratch("sel.z", n * self.inner, wide), r.scratch("sel.u", n * self.channels, wide)
        dt, o = r.scratch("sel.dt", n * s.heads, f32=True), r.scratch("sel.o", n * self.inner, f32=True)
        norm.project(r, self.proj, [z, u, dt], dtype)
        if n == 1:
            K.selective_step_into(b, u, memory.ring, self.taps, self.conv_bias, r.position, dt, self.dt_bias, self.a_log, self.skip,
                                  memory.state, o, s.heads, s.vdim, s.groups, s.state, s.taps)
        else:
            x, B, C = r.scratch("sel.x", n * self.inner), r.scratch("sel.b", n * s.groups * self.dq), r.scratch("sel.c", n * s.groups * self.dq)
            K.selective_conv_into(b, u, r.dtype, memory.ring, self.taps, self.conv_bias, r.position, x, B, C, n, s.heads, s.vdim, s.groups,
                                  s.state, s.taps)
            if n >= CHUNKED_MIN_ROWS and r.dtype != F32 and s.state <= MAX_CHUNKED_DIM:
                steps = r.ws.get("sel.steps", K.selective_steps_bytes(n, s.heads))
                work = r.ws.get("lin.work", K.linear_attention_workspace_bytes(n, s.heads, s.state, s.vdim))
                K.selective_chunked_into(b, x, B, C, dt, self.dt_bias, self.a_log, self.skip, memory.state, steps, work, o, n, s.heads,
                                         s.vdim, s.groups, s.state)
            else:
                K.selective_recurrent_into(b, x, B, C, r.dtype, dt, self.dt_bias, self.a_log, self.skip, memory.state, o, n, s.heads,
                                           s.vdim, s.groups, s.state)
        finish_gated(r, norm, self.out, o, z, dtype, self.weight, self.eps, self.inner // s.norm_groups, ACT_SILU, True)


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
        norm.project(r, self.up, [h], r.dtype)
        norm.finish(r, self.down, h, r.dtype)


@dataclass
class GatedSpec:
    ff: int                  # down(silu(gate x) * (up x))


class GatedFeedForward:
    """Gate and up projections are interleaved row by row, so that a product has both factors of a value side by side."""

    def __init__(self, ctx, kernels: Kernels, spec: GatedSpec, width: int, tensors, prefix: str):
        self.spec = spec
        gate, up = tensors.bf16(prefix + "gate", (spec.ff, width)), tensors.bf16(prefix + "up", (spec.ff, width))
        self.up = StackedLinear(ctx, [np.stack([gate, up], 1).reshape(2 * spec.ff, width)], [Segment(2 * spec.ff, ACT_SILU_PAIRS)])
        self.down = StackedLinear(ctx, [tensors.bf16(prefix + "down", (width, spec.ff))], [Segment(width)])

    def run(self, r: Run, norm: Norm) -> None:
        h = r.scratch("hidden", r.rows * self.spec.ff)
        norm.project(r, self.up, [h], r.dtype)
        norm.finish(r, self.down, h, r.dtype)


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
MIXERS = {AttentionSpec: SoftmaxAttention, LatentAttentionSpec: LatentAttention, LinearAttentionSpec: LinearAttention,
          SelectiveSpec: SelectiveStateSpace}
FEED_FORWARDS = {DenseSpec: DenseFeedForward, GatedSpec: GatedFeedForward, MoeSpec: MoeFeedForward}


@dataclass
class LayerSpec:
    mixer: object
    ff: Optional[object] = None


class PreNormLayer:
    """Two residual branches, each on a norm of the stream: the mixer, and the feed-forward where the layer has one."""
    norm = Norm

    def __init__(self, ctx, kernels: Kernels, spec: LayerSpec, width: int, eps: float, tensors, prefix: str):
        self.norm1 = self.norm(ctx, tensors.f32(prefix + "norm1", (width,)), eps)
        self.mixer = MIXERS[type(spec.mixer)](ctx, kernels, spec.mixer, width, eps, tensors, prefix + "mix.")
        self.norm2 = self.ff = None
        if spec.ff is not None:
            self.norm2 = self.norm(ctx, tensors.f32(prefix + "norm2", (width,)), eps)
            self.ff = FEED_FORWARDS[type(spec.ff)](ctx, kernels, spec.ff, width, tensors, prefix + "mlp.")

    def run(self, r: Run, memory) -> None:
        self.mixer.run(r, self.norm1, memory)
        if self.ff is not None:
            self.ff.run(r, self.norm2)


class OutputNormLayer(PreNormLayer):
    """The same two branches on the stream itself, each with its norm behind it."""
    norm = OutputNorm

    def __init__(self, ctx, kernels: Kernels, spec: LayerSpec, *rest):
        if isinstance(spec.ff, MoeSpec):
            raise InvalidArgument("a mixture of experts adds to the stream itself: no norm can follow it")
        super().__init__(ctx, kernels, spec, *rest)
