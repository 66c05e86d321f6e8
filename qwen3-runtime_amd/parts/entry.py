"""Parts that work on the residual stream between two layers.

``origin_mix``: the stream is replaced by a product of itself joined with the embedding's
output, ``x <- W [x; x0]`` with ``W`` ``[width, 2 width]`` (the stream's columns first): how a pass
over a looped span of layers begins. What the layer before left pending is added first
(``x + scale * delta``), in float32; the product's result is the new float32 stream.

``pass_vector``: pass ``t`` over a looped span begins with a vector of its own, ``x <- x + step[t]`` (the
row ``index`` of the tensor ``step``), and, with ``origin=True``, with the embedding's output added once
more. Both travel with what is pending as one ``ScaledUpdate``, so that the span's first norm adds all of
it in the pass in which it normalises.
"""

from __future__ import annotations

import torch

from ..registry import register_part
from .base import Entry, ScaledUpdate
from .plan import TensorDecl


@register_part("entry", "origin_mix")
class OriginMix(Entry):
    def __init__(self, hidden_size: int, delta_scale: float = 1.0, tensors=None):
        super().__init__(tensors)
        self.hidden_size = int(hidden_size)
        self.delta_scale = float(delta_scale)
        self.weight = None

    def tensor_decls(self):
        return [TensorDecl(self._name("weight"), (self.hidden_size, 2 * self.hidden_size))]

    def load(self, fetch):
        self.weight = fetch.matrix(self._name("weight"))

    def forward(self, ctx, residual, delta, origin):
        joined = ctx.ops.add_concat(residual, delta, self.delta_scale, origin, ctx.dtype)
        return ctx.ops.linear(joined, self.weight, out_f32=True), None


@register_part("entry", "pass_vector")
class PassVector(Entry):
    def __init__(self, hidden_size: int, times: int, index: int, origin: bool = False, tensors=None):
        super().__init__(tensors)
        self.hidden_size, self.times, self.index, self.origin = int(hidden_size), int(times), int(index), bool(origin)
        if not 0 <= self.index < self.times:
            raise ValueError(f"pass {index} of {times}")
        self.vector = self.ones = None

    def tensor_decls(self):
        return [TensorDecl(self._name("step"), (self.times, self.hidden_size))]

    def load(self, fetch):
        self.vector = fetch.constant(fetch.vector_f32(self._name("step"))[self.index])
        if self.origin:
            self.ones = fetch.constant(torch.ones(self.hidden_size, dtype=torch.float32))

    def step_cost(self, spans, rows, elem_bytes):
        cost = super().step_cost(spans, rows, elem_bytes)
        cost.flop = 0.0  # a vector, not a matrix that multiplies tokens
        return cost

    def forward(self, ctx, residual, delta, origin):
        if delta is not None and (not isinstance(delta, ScaledUpdate) or delta.vector is not None):
            raise NotImplementedError("a pass begins behind a block whose outputs travel as a scaled sum")
        parts = [] if delta is None else list(delta.parts)
        if self.origin:
            parts.append((origin, self.ones))
        return residual, ScaledUpdate(parts, self.vector)
