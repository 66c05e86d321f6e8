"""Typed configuration of a Dekinex decoder, read from a model folder's ``config.json``.

The file names the design under ``architecture`` and gives ``vocab``, ``width``, the norms' ``eps``
(``norm.eps``), ``residual_mult`` (what the sum of a layer's outputs is multiplied by before it joins the
stream), the embedding's second table (``embedding.bigram``: ``buckets`` rows and one more, picked by
``mul_prev`` and ``mul_cur``), optionally a ``loop`` (``start``, ``stop``, ``times``: the layers
``start .. stop-1`` run ``times`` times in a row, every pass begun with its row of ``loop.step``), and
``layers``: per layer its ``type`` (``attention``: windowed softmax attention behind short convolutions;
``mlstm``: a matrix memory with exponential gates), the mixer's sizes (``mixer``) and its feed-forward
(``mlp``: dense with a clamped gate, a routed mixture, or null). Every size and every constant that may
differ between two models of the design is read here. Absent options mean "not there": no ``kv_heads`` a
key head per query head, no ``vdim`` values as wide as keys, no ``mask`` every earlier key in sight, no
``rot`` no rotation, no ``conv`` no convolution, no ``router.scale`` weights as normalised, no ``shared``
no shared expert, no ``bigram`` the token's embedding alone.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .deginex import _positive, _unknown
from .model import ConfigError
from .zisedra import _number
from .zuvasun import _window


def _integer(where: str, key: str, raw: Mapping[str, Any]) -> int:
    value = raw.get(key)
    if isinstance(value, bool) or not isinstance(value, int):
        raise ConfigError(f"{where}: {key} must be an integer, got {value!r}")
    return value


@dataclass(frozen=True)
class PairTable:
    """A second embedding table of ``buckets`` rows and one for a sequence's first token: token ``c`` behind
    token ``p`` adds row ``(p * mul_prev + c * mul_cur) mod buckets``."""

    buckets: int
    mul_prev: int
    mul_cur: int

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "PairTable":
        _unknown(where, raw, {"buckets", "mul_prev", "mul_cur"})
        return cls(_positive(where, "buckets", raw.get("buckets")), _integer(where, "mul_prev", raw), _integer(where, "mul_cur", raw))

    def to_dict(self) -> dict[str, Any]:
        return {"buckets": self.buckets, "mul_prev": self.mul_prev, "mul_cur": self.mul_cur}


@dataclass(frozen=True)
class ConvolvedAttentionSizes:
    """``heads`` query heads on ``kv_heads`` key/value heads, keys of ``dim`` and values of ``vdim`` elements,
    each projected channel convolved over time with ``conv`` taps (None: not); the first ``rot_dims`` elements
    of queries and keys turn in neighbour pairs with frequencies ``rot_base^(-2i/rot_dims)``; scores times
    ``scale``; a query sees itself and the ``window - 1`` tokens before it (None: all)."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int | None
    conv: int | None
    rot_dims: int = 0
    rot_base: float = 1.0

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "ConvolvedAttentionSizes":
        for key in ("heads", "dim", "scale"):
            if key not in raw:
                raise ConfigError(f"{where}: the mixer lacks {key!r}")
        heads = _positive(where, "heads", raw["heads"])
        kv_heads = _positive(where, "kv_heads", raw.get("kv_heads", heads))
        if heads % kv_heads:
            raise ConfigError(f"{where}: {heads} query heads do not divide into {kv_heads} key/value heads")
        dim = _positive(where, "dim", raw["dim"])
        if dim % 2:
            raise ConfigError(f"{where}: query/key heads have an even size, got {dim}")
        rot = raw.get("rot") or {"dims": 0, "base": 1.0}
        _unknown(where + " rot", rot, {"dims", "base"})
        dims = _integer(where + " rot", "dims", rot)
        if dims % 2 or not 0 <= dims <= dim:
            raise ConfigError(f"{where}: {dims} rotated elements in heads of {dim}: even, and no more than the head")
        conv = raw.get("conv")
        if conv is not None and not 1 <= _positive(where, "conv", conv) <= 16:
            raise ConfigError(f"{where}: the convolutions have 1 to 16 taps, got {conv}")
        _unknown(where + " mixer", raw, {"heads", "kv_heads", "dim", "vdim", "scale", "mask", "rot", "conv"})
        return cls(heads, kv_heads, dim, _positive(where, "vdim", raw.get("vdim", dim)), _number(where, "scale", raw),
                   _window(raw, where), conv, dims, _number(where + " rot", "base", rot))

    def to_dict(self) -> dict[str, Any]:
        raw: dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
                               "scale": self.scale, "rot": {"dims": self.rot_dims, "base": self.rot_base}}
        if self.conv is not None:
            raw["conv"] = self.conv
        if self.window is not None:
            raw["mask"] = {"size": self.window}
        return raw


@dataclass(frozen=True)
class MatrixMemorySizes:
    """``heads`` memories of ``dim`` x ``vdim``; the gates' logits are softly held to ``gate_cap``."""

    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "MatrixMemorySizes":
        for key in ("heads", "dim", "gate_cap"):
            if key not in raw:
                raise ConfigError(f"{where}: the mixer lacks {key!r}")
        dim = _positive(where, "dim", raw["dim"])
        _unknown(where + " mixer", raw, {"heads", "dim", "vdim", "gate_cap"})
        return cls(_positive(where, "heads", raw["heads"]), dim, _positive(where, "vdim", raw.get("vdim", dim)),
                   _number(where, "gate_cap", raw))

    def to_dict(self) -> dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "gate_cap": self.gate_cap}


@dataclass(frozen=True)
class ClampedSizes:
    """A dense feed-forward of inner width ``ff`` whose gate and other half are clamped at ``limit``."""

    ff: int
    limit: float

    def to_dict(self) -> dict[str, Any]:
        return {"kind": "dense", "ff": self.ff, "limit": self.limit}


@dataclass(frozen=True)
class SharedMixtureSizes:
    """``experts`` experts of inner width ``ff``, ``top`` a token by corrected sigmoid scores, weights times
    ``scale``; a shared expert of ``shared_ff`` (0: none) behind a gate of its own."""

    ff: int
    experts: int
    top: int
    scale: float = 1.0
    shared_ff: int = 0

    def to_dict(self) -> dict[str, Any]:
        raw: dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff},
                               "router": {"experts": self.experts, "top": self.top, "scale": self.scale}}
        if self.shared_ff:
            raw["shared"] = {"ff": self.shared_ff}
        return raw


def feed_forward_from_dict(raw: Mapping[str, Any], where: str) -> ClampedSizes | SharedMixtureSizes:
    kind = raw.get("kind")
    if kind == "dense":
        _unknown(where + " mlp", raw, {"kind", "ff", "limit"})
        return ClampedSizes(_positive(where, "mlp.ff", raw.get("ff")), _number(where + " mlp", "limit", raw))
    if kind != "moe":
        raise ConfigError(f"{where}: unknown feed-forward kind {kind!r} (dense, moe)")
    router, expert, shared = raw.get("router") or {}, raw.get("expert") or {}, raw.get("shared")
    experts = _positive(where, "mlp.router.experts", router.get("experts"))
    top = _positive(where, "mlp.router.top", router.get("top"))
    if top > experts:
        raise ConfigError(f"{where}: {top} of {experts} experts")
    _unknown(where + " mlp", raw, {"kind", "router", "expert", "shared"})
    _unknown(where + " mlp.router", router, {"experts", "top", "scale"})
    _unknown(where + " mlp.expert", expert, {"ff"})
    _unknown(where + " mlp.shared", shared or {}, {"ff"})
    return SharedMixtureSizes(_positive(where, "mlp.expert.ff", expert.get("ff")), experts, top,
                              _number(where + " mlp.router", "scale", router) if "scale" in router else 1.0,
                              0 if shared is None else _positive(where, "mlp.shared.ff", shared.get("ff")))


MIXERS = {"attention": ConvolvedAttentionSizes, "mlstm": MatrixMemorySizes}


@dataclass(frozen=True)
class DekinexLayer:
    kind: str  # a key of MIXERS
    mixer: Any
    feed_forward: ClampedSizes | SharedMixtureSizes | None


@dataclass(frozen=True)
class DekinexConfig:
    vocab: int
    width: int
    eps: float
    layers: tuple[DekinexLayer, ...]
    pairs: PairTable | None = None
    residual_mult: float = 1.0
    loop: tuple[int, int, int] | None = None  # (start, stop, times)
    max_positions: int = 1 << 20
    eos_token_id: int | None = None

    architecture = "Dekinex"

    def __post_init__(self) -> None:
        _positive("config", "vocab", self.vocab)
        _positive("config", "width", self.width)
        if not self.eps > 0.0:
            raise ConfigError(f"norm.eps must be positive, got {self.eps!r}")
        if not self.layers:
            raise ConfigError("the model has no layers")
        if self.loop is not None:
            start, stop, times = self.loop
            if not (0 <= start < stop <= len(self.layers)) or times < 1:
                raise ConfigError(f"loop {self.loop} does not fit {len(self.layers)} layers")

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "DekinexConfig":
        if raw.get("architecture") != cls.architecture and cls.architecture not in (raw.get("architectures") or []):
            raise ConfigError(f"unsupported architecture: {raw.get('architecture')!r}")
        for key in ("vocab", "width", "layers", "norm"):
            if key not in raw:
                raise ConfigError(f"config.json lacks {key!r}")
        layers = []
        for i, spec in enumerate(raw["layers"]):
            where = f"layer {i}"
            kind = spec.get("type")
            if kind not in MIXERS:
                raise ConfigError(f"{where}: unknown mixer type {kind!r} ({', '.join(MIXERS)})")
            mlp = spec.get("mlp")
            _unknown(where, spec, {"type", "mixer", "mlp"})
            layers.append(DekinexLayer(kind, MIXERS[kind].from_dict(spec.get("mixer") or {}, where),
                                       None if mlp is None else feed_forward_from_dict(mlp, where)))
        embedding = raw.get("embedding") or {}
        _unknown("embedding", embedding, {"bigram"})
        pairs = embedding.get("bigram")
        loop = raw.get("loop")
        if loop is not None:
            _unknown("loop", loop, {"start", "stop", "times"})
            loop = tuple(_integer("loop", key, loop) for key in ("start", "stop", "times"))
        eos = raw.get("eos_token_id")
        _unknown("config", raw, {"architecture", "architectures", "vocab", "width", "layers", "norm", "embedding", "loop",
                                 "residual_mult", "max_positions", "eos_token_id"})
        return cls(vocab=raw["vocab"], width=raw["width"], eps=float((raw["norm"] or {}).get("eps", 0.0)), layers=tuple(layers),
                   pairs=None if pairs is None else PairTable.from_dict(pairs, "embedding.bigram"),
                   residual_mult=float(raw.get("residual_mult", 1.0)), loop=loop,
                   max_positions=int(raw.get("max_positions", 1 << 20)), eos_token_id=None if eos is None else int(eos))

    def to_dict(self) -> dict[str, Any]:
        """The config.json a model folder of this configuration carries."""
        raw: dict[str, Any] = {
            "architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
            "residual_mult": self.residual_mult,
            "layers": [{"type": layer.kind, "mixer": layer.mixer.to_dict(),
                        "mlp": None if layer.feed_forward is None else layer.feed_forward.to_dict()} for layer in self.layers]}
        if self.pairs is not None:
            raw["embedding"] = {"bigram": self.pairs.to_dict()}
        if self.loop is not None:
            raw["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.max_positions != 1 << 20:
            raw["max_positions"] = self.max_positions
        if self.eos_token_id is not None:
            raw["eos_token_id"] = self.eos_token_id
        return raw

    def run_order(self) -> list[tuple[int, int | None]]:
        """(layer, number of the pass over the looped span that begins with it, or None), in the order a
        pass over the model runs them."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        start, stop, times = self.loop
        order: list[tuple[int, int | None]] = [(i, None) for i in range(start)]
        for t in range(times):
            order += [(i, t if i == start else None) for i in range(start, stop)]
        return order + [(i, None) for i in range(stop, n)]
