"""A model as data: which parts make each layer, and the order layers run in.

An architecture (see ``registry.py``) turns its typed configuration into a
``ModelPlan``. The plan names, layer by layer, a mixer, a feed-forward, the
norms and the block arrangement, each as a ``PartSpec`` (a registered kind, its
sizes and constants, and the names of its tensors in the model file). The plan
also lists the caches the layers own and ``order``: the sequence of
``RunStep``s one forward pass executes. A layer may appear in ``order`` more
than once, and a step may read the cache another step writes.

Parts never see the plan or the configuration; they see only their own
``PartSpec.args``.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Mapping, Sequence


@dataclass(frozen=True)
class PartSpec:
    """One part to build: ``kind`` picks the class from the registry of its role."""

    kind: str
    args: Mapping[str, Any] = field(default_factory=dict)
    # logical tensor name of the part -> tensor name in the model file
    tensors: Mapping[str, str] = field(default_factory=dict)


@dataclass(frozen=True)
class TensorDecl:
    """One tensor a part reads from the model file.

    ``init`` tells the random-weights mode how to draw it: ``"matrix"`` and
    ``"embedding"`` are zero-mean normal, ``"norm"`` is a scale around one, ``"mixing"``
    a square matrix around the identity, ``"log_rate"`` the logarithm of a decay rate (around -2:
    a recurrent state that forgets over tens of tokens), ``"norm_zero"`` a norm's weight stored around
    zero, ``"taps"`` those of a short convolution, ``"open_gate"`` the bias of a forget gate (around 3: it stays nearly open).
    ``storage`` is ``"float"`` (stored as bfloat16, float32 or float16) or ``"int"``
    (an integer table, held as int32; drawn as zeros in the random-weights mode unless
    ``init`` is ``"index:<n>"``, uniform in ``[0, n)``).
    """

    file_name: str
    shape: tuple[int, ...]
    init: str = "matrix"
    storage: str = "float"


@dataclass(frozen=True)
class PagedStream:
    """One tensor a paged cache keeps for every token: ``heads`` x ``width`` elements.

    Within a page the tensor is ``[head, offset, width]``, or, ``transposed``,
    ``[head, width, offset]`` (the tokens of a page contiguous for one element: what a kernel
    wants that multiplies probabilities over keys with values)."""

    name: str
    heads: int
    width: int
    transposed: bool = False

    def page_shape(self, page_size: int) -> tuple[int, int, int]:
        return (self.heads, self.width, page_size) if self.transposed else (self.heads, page_size, self.width)

    def elements_per_token(self) -> int:
        return self.heads * self.width


@dataclass(frozen=True)
class CacheSpec:
    """What one cache owner keeps between steps.

    ``kind == "paged_kv"``: keys and values for every token (or the last
    ``window`` tokens, beside which the sequence's first ``keep_first`` stay for good, or,
    with ``chunk``, the tokens of the chunk of ``chunk``
    positions, counted from position 0, that the newest token lies in),
    ``heads`` x ``head_dim`` keys and ``heads`` x ``value_dim``
    values (``head_dim`` when None), held in pages; the values transposed within a
    page. ``kind == "paged"``: any other set of per-token tensors, named by
    ``streams`` (one latent vector per token, say), with the same pages, tables and
    window. ``kind == "state"``: a fixed-size tensor of ``shape`` per request, held
    in a slot; ``dtype`` is a torch dtype name or ``"model"`` for the model's dtype.
    """

    kind: str
    heads: int = 0
    head_dim: int = 0
    window: int | None = None
    shape: tuple[int, ...] = ()
    dtype: str = "model"
    value_dim: int | None = None
    streams: tuple[PagedStream, ...] = ()
    chunk: int | None = None
    keep_first: int = 0

    def __post_init__(self) -> None:
        if self.window is not None and self.chunk is not None:
            raise ValueError("a cache keeps a window of keys or a chunk of them, not both")
        if self.keep_first < 0 or (self.keep_first and self.window is None):
            raise ValueError("first tokens are kept beside a window, and their number is not negative")
        for name in ("window", "chunk"):
            if getattr(self, name) is not None and getattr(self, name) < 1:
                raise ValueError(f"{name} must be positive, got {getattr(self, name)}")

    @property
    def paged(self) -> bool:
        return self.kind in ("paged_kv", "paged")

    def page_streams(self) -> tuple[PagedStream, ...]:
        """The per-token tensors of a paged cache; a ``CacheView`` holds one device tensor for each,
        under the stream's name."""
        if self.kind == "paged_kv":
            return (PagedStream("k", self.heads, self.head_dim),
                    PagedStream("v", self.heads, self.head_dim if self.value_dim is None else self.value_dim, True))
        if self.kind == "paged":
            if not self.streams:
                raise ValueError("a cache of kind 'paged' names its streams")
            return tuple(self.streams)
        return ()

    def elements_per_token(self) -> int:
        return sum(s.elements_per_token() for s in self.page_streams())

    def group_key(self) -> tuple:
        """Caches with equal keys share pages' geometry and lifetime, hence a pool."""
        if self.paged:
            return ("paged", self.page_streams(), self.window, self.chunk, self.keep_first)
        return ("state", tuple(self.shape), self.dtype)


@dataclass(frozen=True)
class LayerSpec:
    """One layer: a block arrangement over a mixer, a feed-forward (None: the layer has
    none) and norms."""

    block: PartSpec
    mixer: PartSpec
    feed_forward: PartSpec | None
    norms: Mapping[str, PartSpec]


@dataclass(frozen=True)
class RunStep:
    """One entry of the execution order.

    ``layer`` indexes ``ModelPlan.layers``. ``cache`` indexes ``ModelPlan.caches``
    (or is None for a mixer without cache); a mixer that keeps several things (pages of keys
    and a recurrent state, say) names them all, as a tuple in the order of its
    ``cache_specs()``, and its ``forward`` receives as many views. ``writes_cache`` is False
    when the step only reads a cache that an earlier step of the same pass wrote.
    ``entry`` indexes ``ModelPlan.entries``: a part that works on the residual stream right
    before this step's layer (the start of a pass over a looped span, say).
    """

    layer: int
    cache: int | tuple[int, ...] | None = None
    writes_cache: bool = True
    entry: int | None = None

    def cache_ids(self) -> tuple[int, ...]:
        if self.cache is None:
            return ()
        return tuple(self.cache) if isinstance(self.cache, (tuple, list)) else (self.cache,)


@dataclass(frozen=True)
class ModelPlan:
    hidden_size: int
    vocab_size: int
    max_positions: int
    embedding: PartSpec
    layers: Sequence[LayerSpec]
    caches: Sequence[CacheSpec]
    order: Sequence[RunStep]
    final_norm: PartSpec
    head: PartSpec
    # tensors a model file may hold although the plan reads them from elsewhere
    ignorable: Sequence[str] = ()
    eos_token_id: int | None = None
    # parts of role "entry" that steps of the order may name (``RunStep.entry``)
    entries: Sequence[PartSpec] = ()
    # the caches of an embedding that keeps something per request (the last token it saw, say), in the
    # order of its ``cache_specs()``; no step of the order names them
    embedding_cache: Sequence[int] = ()

    def __post_init__(self) -> None:
        writers: set[int] = set(self.embedding_cache)
        if any(not 0 <= cache < len(self.caches) for cache in writers) or len(writers) != len(self.embedding_cache):
            raise ValueError(f"the embedding names caches {list(self.embedding_cache)}; the plan has {len(self.caches)}")
        for i, step in enumerate(self.order):
            if not 0 <= step.layer < len(self.layers):
                raise ValueError(f"order[{i}] names layer {step.layer}; the plan has {len(self.layers)}")
            if step.entry is not None and not 0 <= step.entry < len(self.entries):
                raise ValueError(f"order[{i}] names entry {step.entry}; the plan has {len(self.entries)}")
            for cache in step.cache_ids():
                if not 0 <= cache < len(self.caches):
                    raise ValueError(f"order[{i}] names cache {cache}; the plan has {len(self.caches)}")
                if step.writes_cache:
                    if cache in writers:
                        raise ValueError(f"cache {cache} is written by two steps of the order")
                    writers.add(cache)
                elif cache not in writers:
                    raise ValueError(f"order[{i}] reads cache {cache} before any step writes it")
