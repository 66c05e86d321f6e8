"""State-space mixer (Mamba-2): a recurrence with a scalar decay per head made from the input.

One product of the mixer's input gives ``[z | x | B | C | dt]``: a gate ``z`` and values ``x`` of
``heads * vdim`` channels each, input and output vectors ``B`` and ``C`` of ``state`` elements for each of
``groups`` groups of heads (head ``j`` uses group ``j // (heads / groups)``), and a step logit ``dt`` per
head. ``x``, ``B`` and ``C`` together pass a short causal convolution over time per channel (``taps`` taps,
the last one on the current token, zeros before the sequence's start, a bias) and silu. Per head and
token, with ``step = softplus(dt + dt_bias)``::

    S <- exp(-exp(A_log) step) S + (step x) B^T;   y = S C + D x

The heads' ``y`` are concatenated, multiplied by ``silu(z)``, RMS-normed in ``norm_groups`` equal parts
(eps inside the root, one weight vector over all channels) and projected out. ``S`` starts at zero and
is float32; it and the convolution's last ``taps - 1`` inputs are the request's state, kept in its slot
from step to step. Step sizes, decays, recurrence and norm are float32 in every mode; the convolution's
output is in the activations' type.
"""

from __future__ import annotations

from ..registry import register_part
from .base import Mixer
from .plan import CacheSpec, TensorDecl


@register_part("mixer", "state_space")
class StateSpace(Mixer):
    """``tensors``: ``in``, ``conv``, ``conv_bias``, ``dt_bias``, ``A_log``, ``D``, ``norm``, ``o``."""

    def __init__(self, hidden_size: int, num_heads: int, value_dim: int, state_dim: int, groups: int, taps: int,
                 norm_groups: int, norm_eps: float, tensors=None):
        super().__init__(tensors)
        self.hidden_size, self.heads = int(hidden_size), int(num_heads)
        self.vdim, self.state_dim, self.groups = int(value_dim), int(state_dim), int(groups)
        self.taps, self.norm_groups, self.norm_eps = int(taps), int(norm_groups), float(norm_eps)
        if self.groups < 1 or self.heads % self.groups:
            raise ValueError(f"{num_heads} heads do not divide into {groups} groups")
        if not 1 <= self.taps <= 16:
            raise ValueError(f"the convolution has 1 to 16 taps, not {taps}")
        if not 1 <= self.state_dim <= 512:
            raise ValueError(f"the state's rows are held in registers: state size 1 to 512, not {state_dim}")
        if self.norm_groups < 1 or self.inner % self.norm_groups:
            raise ValueError(f"{self.inner} channels do not divide into {norm_groups} parts of the norm")
        self.proj = self.conv = self.conv_bias = self.dt_bias = self.a_log = self.skip = self.norm = self.o = None

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        """Convolved channels: x, B, C."""
        return self.inner + 2 * self.groups * self.state_dim

    def cache_specs(self):
        # the state transposed, [heads, vdim, state]: a value channel's column is contiguous
        return (CacheSpec("state", shape=(self.heads, self.vdim, self.state_dim), dtype="float32"),
                CacheSpec("state", shape=(self.channels, max(self.taps - 1, 1)), dtype="float32"))

    def tensor_decls(self):
        h = self.hidden_size
        return [TensorDecl(self._name("in"), (self.inner + self.channels + self.heads, h)),
                TensorDecl(self._name("conv"), (self.channels, self.taps)),
                TensorDecl(self._name("conv_bias"), (self.channels,)),
                TensorDecl(self._name("dt_bias"), (self.heads,)),
                TensorDecl(self._name("A_log"), (self.heads,), init="log_rate"),
                TensorDecl(self._name("D"), (self.heads,), init="norm"),
                TensorDecl(self._name("norm"), (self.inner,), init="norm"),
                TensorDecl(self._name("o"), (h, self.inner))]

    def load(self, fetch):
        self.proj, self.o = fetch.matrix(self._name("in")), fetch.matrix(self._name("o"))
        self.conv, self.conv_bias = fetch.vector_f32(self._name("conv")), fetch.vector_f32(self._name("conv_bias"))
        self.dt_bias, self.a_log = fetch.vector_f32(self._name("dt_bias")), fetch.vector_f32(self._name("A_log"))
        self.skip, self.norm = fetch.vector_f32(self._name("D")), fetch.vector_f32(self._name("norm"))

    def step_cost(self, spans, rows, elem_bytes):
        cost = super().step_cost(spans, rows, elem_bytes)
        tokens = sum(q for q, _ in spans)
        # per token and head: decay and write, and one sum over the state's rows: 2 passes over N x P
        cost.flop += 2.0 * 2 * tokens * self.inner * self.state_dim
        return cost

    def forward(self, ctx, x, cache):
        ops = ctx.ops
        state, tail = cache
        inner = self.inner
        y = ops.linear(x, self.proj)  # z | x | B | C | dt, read where they lie
        whole, rest = divmod(self.channels, 128)  # what a wave of the convolution takes at a time
        segments = tuple(s for s in ((whole, 128, 0), (1, rest, 0)) if s[0] * s[1])
        xbc = ops.delta_conv(ctx, y, self.channels, self.conv, tail.state, segments, 0.0, first=inner, bias=self.conv_bias,
                             out_dtype=ctx.dtype)
        step = y[:, inner + self.channels:]
        out = ops.state_space(ctx, xbc, step, self.dt_bias, self.a_log, self.skip, state.state, self.heads, self.groups,
                              self.state_dim, self.vdim)
        out = ops.gated_group_norm(out, y[:, :inner], self.norm, self.norm_eps, self.norm_groups, ctx.dtype)
        return ops.linear_for_residual(out, self.o)
