"""Token embedding and output head.

``h0[t] = E[ids[t]]`` without scaling (reference: qwen3_runtime/models/qwen3.py:243);
``logits = x W^T`` where ``W`` is the embedding table when the head is tied,
no bias and no scaling of logits (reference: qwen3_runtime/models/qwen3.py:265-266).
The embedding starts the float32 residual stream; logits come out in float32.
``bigram_embedding`` adds a row of a second table that the pair (previous token, token) picks:
``h0[t] = E[ids[t]] + B[(prev * mul_prev + ids[t] * mul_cur) mod buckets]``, for a sequence's first token
the table's last row, number ``buckets``. The last token of a request's step is its state, kept in its
slot (int32) for the step that goes on from it.
Either takes a constant ``scale`` (1 by default): the embedding's rows times it, in float32, and
the float32 logits times it. The head's ``softcap``: the logits become ``cap * tanh(logits / cap)``, float32.
"""

from __future__ import annotations

from ..registry import register_part
from .base import Part, StepCost
from .plan import CacheSpec, TensorDecl


@register_part("embedding", "token_embedding")
class TokenEmbedding(Part):
    role = "embedding"

    def __init__(self, vocab_size: int, hidden_size: int, scale: float = 1.0, tensors=None):
        super().__init__(tensors)
        self.vocab_size = int(vocab_size)
        self.hidden_size = int(hidden_size)
        self.scale = float(scale)
        self.weight = None

    def tensor_decls(self):
        return [TensorDecl(self._name("weight"), (self.vocab_size, self.hidden_size), init="embedding")]

    def load(self, fetch):
        self.weight = fetch.matrix(self._name("weight"))

    def forward(self, ctx, ids):
        if self.scale != 1.0:
            return ctx.ops.embed(ids, self.weight, scale=self.scale)
        return ctx.ops.embed(ids, self.weight)

    def step_cost(self, spans, rows, elem_bytes):
        # a lookup: one row of the table per token, no arithmetic
        tokens = sum(q for q, _ in spans)
        return StepCost({self._name("weight"): min(tokens, self.vocab_size) * self.hidden_size * elem_bytes}, 0.0)


@register_part("embedding", "bigram_embedding")
class BigramEmbedding(TokenEmbedding):
    """``tensors``: ``weight`` [vocab, width], ``bigram`` [buckets + 1, width]."""

    def __init__(self, vocab_size: int, hidden_size: int, buckets: int, mul_prev: int, mul_cur: int, tensors=None):
        super().__init__(vocab_size, hidden_size, tensors=tensors)
        self.buckets, self.mul_prev, self.mul_cur = int(buckets), int(mul_prev), int(mul_cur)
        if self.buckets < 1:
            raise ValueError(f"a second table of {buckets} rows for pairs")
        self.bigram = None

    def cache_specs(self):
        return (CacheSpec("state", shape=(1,), dtype="int32"),)  # the request's last token

    def tensor_decls(self):
        return super().tensor_decls() + [TensorDecl(self._name("bigram"), (self.buckets + 1, self.hidden_size), init="embedding")]

    def load(self, fetch):
        super().load(fetch)
        self.bigram = fetch.matrix(self._name("bigram"))

    def forward(self, ctx, ids, cache):
        return ctx.ops.embed_pairs(ctx, ids, self.weight, self.bigram, self.mul_prev, self.mul_cur, cache[0].state)

    def step_cost(self, spans, rows, elem_bytes):
        cost = super().step_cost(spans, rows, elem_bytes)
        tokens = sum(q for q, _ in spans)
        cost.weight_bytes[self._name("bigram")] = min(tokens, self.buckets + 1) * self.hidden_size * elem_bytes
        return cost


@register_part("head", "linear_head")
class LinearHead(Part):
    """Projection to the vocabulary. A tied head names the embedding's tensor."""

    role = "head"

    def __init__(self, vocab_size: int, hidden_size: int, scale: float = 1.0, softcap: float | None = None, tensors=None):
        super().__init__(tensors)
        self.softcap = None if softcap is None else float(softcap)
        self.vocab_size = int(vocab_size)
        self.hidden_size = int(hidden_size)
        self.scale = float(scale)
        self.weight = None

    def tensor_decls(self):
        return [TensorDecl(self._name("weight"), (self.vocab_size, self.hidden_size), init="embedding")]

    def load(self, fetch):
        self.weight = fetch.matrix(self._name("weight"))

    def forward(self, ctx, x):
        logits = ctx.ops.linear(x, self.weight, out_f32=True)
        if self.scale != 1.0:
            logits = ctx.ops.scale(logits, self.scale)
        return logits if self.softcap is None else ctx.ops.softcap(logits, self.softcap)

    def step_cost(self, spans, rows, elem_bytes):
        # the whole matrix, multiplied with the wanted rows only
        n = self.vocab_size * self.hidden_size
        return StepCost({self._name("weight"): n * elem_bytes}, 2.0 * rows * n)
