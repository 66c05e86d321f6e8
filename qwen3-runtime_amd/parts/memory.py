"""Matrix memory with exponential gates (the mLSTM of xLSTM): a recurrent mixer with a matrix state, a
normaliser and a running maximum per head.

From the mixer's input ``h``: ``q = W_q h * dim^(-1/2)`` and ``k = W_k h`` (``heads x dim``), ``v = W_v h``
(``heads x vdim``), an output gate ``g = W_g h`` (``heads * vdim``), and per head the logarithms of an input
gate, ``a = cap tanh((W_i h + b_i) / cap)``, and of a forget gate, ``log sigmoid(cap tanh((W_f h + b_f) / cap))``.
Per head and token, all from zero::

    top = max(f + m, a);  keep = exp(f + m - top);  write = exp(a - top);  m <- top
    S <- keep S + write k v^T;   n <- keep n + write k
    o = S^T q / (max(|n . q|, exp(-m)) + 1e-6)

Each head's ``o`` is divided by its root mean square; the heads, concatenated, are multiplied by one weight
vector and by ``sigmoid(g)`` and projected out. ``S``, ``n`` and ``m`` are float32 and the request's state,
kept in its slot from step to step; the gates' logits come out of their product in float32, and
everything after the projections up to the read-out's gate is float32 in every mode.

The normaliser is the state's column for a value channel that always reads 1 (``S`` has ``vdim + 1``
columns), so one recurrence carries both. The gates of a step come first: ``m`` depends on nothing else,
and what the recurrence needs of a token is the pair ``(log keep, log write)``.
"""

from __future__ import annotations

import torch

from ..registry import register_part
from .base import Mixer
from .plan import CacheSpec, TensorDecl


@register_part("mixer", "matrix_memory")
class MatrixMemory(Mixer):
    """``tensors``: ``q``, ``k``, ``v``, ``g``, ``i``, ``i_bias``, ``f``, ``f_bias``, ``norm``, ``o``."""

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, gate_cap: float, norm_eps: float,
                 tensors=None):
        super().__init__(tensors)
        self.hidden_size, self.heads = int(hidden_size), int(num_heads)
        self.dim, self.vdim = int(head_dim), int(value_dim)
        self.gate_cap, self.norm_eps = float(gate_cap), float(norm_eps)
        if not 1 <= self.dim <= 512:
            raise ValueError(f"the state's rows are held in registers: key size 1 to 512, not {head_dim}")
        if not self.gate_cap > 0.0:
            raise ValueError(f"the gates' logits are held to a positive number, not {gate_cap}")
        self.proj = self.gates = self.gate_bias = self.norm = self.o = None

    def cache_specs(self):
        # the state transposed, [heads, vdim + 1, dim]: a value channel's column of S is contiguous, the
        # normaliser is the last one; the running maximum
        return (CacheSpec("state", shape=(self.heads, self.vdim + 1, self.dim), dtype="float32"),
                CacheSpec("state", shape=(self.heads,), dtype="float32"))

    def tensor_decls(self):
        h, n = self.hidden_size, self.heads
        return [TensorDecl(self._name("q"), (n * self.dim, h)), TensorDecl(self._name("k"), (n * self.dim, h)),
                TensorDecl(self._name("v"), (n * self.vdim, h)), TensorDecl(self._name("g"), (n * self.vdim, h)),
                TensorDecl(self._name("i"), (n, h)), TensorDecl(self._name("i_bias"), (n,)),
                TensorDecl(self._name("f"), (n, h)), TensorDecl(self._name("f_bias"), (n,), init="open_gate"),
                TensorDecl(self._name("norm"), (n * self.vdim,), init="norm"),
                TensorDecl(self._name("o"), (h, n * self.vdim))]

    def load(self, fetch):
        self.proj = fetch.fused([self._name(n) for n in ("q", "k", "v", "g")], dim=0)
        self.gates = fetch.fused([self._name("i"), self._name("f")], dim=0)
        self.gate_bias = fetch.constant(torch.cat([fetch.vector_f32(self._name("i_bias")), fetch.vector_f32(self._name("f_bias"))]))
        self.norm = fetch.vector_f32(self._name("norm"))
        self.o = fetch.matrix(self._name("o"))

    def step_cost(self, spans, rows, elem_bytes):
        cost = super().step_cost(spans, rows, elem_bytes)
        tokens = sum(q for q, _ in spans)
        # per token and head: decay and write, and one sum over the state's rows: 2 passes over D x (Dv + 1)
        cost.flop += 2.0 * 2 * tokens * self.heads * self.dim * (self.vdim + 1)
        return cost

    def forward(self, ctx, x, cache):
        ops = ctx.ops
        state, top = cache
        n = self.heads
        y = ops.linear(x, self.proj)  # q | k | v | g, read where they lie
        gates = ops.memory_gates(ctx, ops.linear(x, self.gates, out_f32=True), self.gate_bias, self.gate_cap, top.state, n)
        read, floor = ops.matrix_memory(ctx, y, gates, state.state, n, self.dim, self.vdim)
        out_gate = y[:, 2 * n * self.dim + n * self.vdim:]
        out = ops.memory_out(read, floor, gates, self.norm, out_gate, self.norm_eps, self.dim ** -0.5, ctx.dtype)
        return ops.linear_for_residual(out, self.o)
