"""bf16 weight matrices and the column segments of their products (see include/local_hip.h): several projections of the
same input are stacked into one matrix, each a segment with its own activation, head padding and destination."""
from __future__ import annotations

import ctypes as C
from dataclasses import dataclass
from typing import List, Optional, Sequence

import numpy as np

from . import ACT_NONE, F32, ROWS, Buffer, InvalidArgument, Kernels


@dataclass
class Segment:
    columns: int
    act: int = ACT_NONE
    head: int = 0           # 0: the whole segment is one head
    padded: int = 0
    layout: int = ROWS


class Segments:
    """The segment arrays of the C ABI, built once."""

    def __init__(self, segments: Sequence[Segment]):
        if not 1 <= len(segments) <= 4:
            raise InvalidArgument(f"{len(segments)} segments")
        self.columns = sum(s.columns for s in segments)

        def arr(values):
            return (C.c_uint32 * len(segments))(*values)
        heads = [s.head or s.columns for s in segments]
        self._keep = (arr([s.columns for s in segments]), arr([s.act for s in segments]), arr(heads),
                      arr([s.padded or h for s, h in zip(segments, heads)]), arr([s.layout for s in segments]))
        self.args = (C.c_uint32(len(segments)), *self._keep)


class StackedLinear:
    """Projections [columns, k] of one input, one below the other, with optional f32 biases."""

    def __init__(self, ctx, weights: List[np.ndarray], segments: Sequence[Segment], biases: Optional[List[np.ndarray]] = None):
        k = weights[0].shape[1]
        for w, s in zip(weights, segments):
            if w.dtype != np.uint16 or w.shape != (s.columns, k):
                raise InvalidArgument(f"weight {w.dtype} {w.shape} for {s.columns} columns over {k}")
        self.k, self.segments = k, Segments(segments)
        self.weight = Buffer.from_slice(ctx, np.concatenate(weights) if len(weights) > 1 else weights[0])
        self.bias = Buffer.from_slice(ctx, np.concatenate(biases).astype(np.float32)) if biases else None

    @property
    def n(self) -> int:
        return self.segments.columns

    def bytes(self) -> int:
        return self.weight.length()

    def rows_into(self, batch, kernels: Kernels, x: Buffer, x_dtype: int, m: int, outputs, dtype: int, position=None,
                  segments: Optional[Segments] = None) -> None:
        kernels.linear_rows_into(batch, x, x_dtype, self.weight, self.bias, m, self.k, segments or self.segments, outputs, dtype,
                                 False, position)

    def rows_add_into(self, batch, kernels: Kernels, x: Buffer, x_dtype: int, m: int, residual: Buffer) -> None:
        kernels.linear_rows_into(batch, x, x_dtype, self.weight, self.bias, m, self.k, self.segments, [residual], F32, True)

    def vector_into(self, batch, kernels: Kernels, x: Buffer, x_dtype: int, outputs, dtype: int, position=None,
                    segments: Optional[Segments] = None) -> None:
        kernels.linear_vector_into(batch, x, x_dtype, self.weight, self.bias, self.k, segments or self.segments, outputs, dtype,
                                   False, position)

    def residual_vector_into(self, batch, kernels: Kernels, x: Buffer, branch: Buffer, store, norm: Buffer, eps: float, outputs,
                             dtype: int, position=None, segments: Optional[Segments] = None) -> None:
        kernels.linear_residual_vector_into(batch, x, branch, store, norm, eps, self.weight, self.bias, self.k,
                                            segments or self.segments, outputs, dtype, False, position)

    def normed_vector_into(self, batch, kernels: Kernels, x: Buffer, norm: Buffer, eps: float, outputs, dtype: int,
                           position=None, add=None, store=None, segments: Optional[Segments] = None) -> None:
        kernels.linear_norm_vector_into(batch, x, add, store, norm, eps, self.weight, self.bias, self.k,
                                        segments or self.segments, outputs, dtype, False, position)
