"""Typed configuration of a Sarudra decoder, read from a model folder's ``config.json``.

The file names the design under ``architecture`` and gives ``vocab``, ``width``, the norms'
``norm.eps`` and ``norm.groups`` (equal parts of the width, each with its own root mean square),
``embedding.scale``, ``logit_softcap`` and ``layers``: per layer its ``type`` (``mamba2``: a state-space
mixer; ``attention``: softmax attention over a sliding window with rotated values), the mixer's
sizes (``mixer``) and its feed-forward (``mlp``: dense, a routed mixture, or null). Every size and
every constant that may differ between two models of the design is read here. What a file leaves out
is not there: a key head per query head, values as wide as keys, no cap, one group, no shared expert.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .deginex import _positive, _unknown
from .model import ConfigError
from .zisedra import _number


def _optional_positive(where: str, key: str, raw: Mapping[str, Any]) -> float | None:
    return None if raw.get(key) is None else _number(where, key, raw)


@dataclass(frozen=True)
class StateSpaceSizes:
    """``heads`` heads of ``vdim`` channels with a state of ``state`` x ``vdim`` each; ``groups`` groups of
    heads share their input and output vectors; a convolution of ``conv`` taps; the read-out is normed in
    ``norm_groups`` equal parts."""

    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int = 1

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "StateSpaceSizes":
        for key in ("heads", "vdim", "state", "conv"):
            if key not in raw:
                raise ConfigError(f"{where}: the mixer lacks {key!r}")
        _unknown(where + " mixer", raw, {"heads", "vdim", "state", "groups", "conv", "norm_groups"})
        sizes = cls(*(_positive(where, key, raw[key]) for key in ("heads", "vdim", "state")),
                    _positive(where, "groups", raw.get("groups", 1)), _positive(where, "conv", raw["conv"]),
                    _positive(where, "norm_groups", raw.get("norm_groups", 1)))
        if sizes.heads % sizes.groups:
            raise ConfigError(f"{where}: {sizes.heads} heads do not divide into {sizes.groups} groups")
        if sizes.heads * sizes.vdim % sizes.norm_groups:
            raise ConfigError(f"{where}: {sizes.heads * sizes.vdim} channels do not divide into {sizes.norm_groups} parts of the norm")
        return sizes

    def to_dict(self) -> dict[str, Any]:
        return {"heads": self.heads, "vdim": self.vdim, "state": self.state, "groups": self.groups, "conv": self.conv,
                "norm_groups": self.norm_groups}


@dataclass(frozen=True)
class TurnedAttentionSizes:
    """``heads`` query heads on ``kv_heads`` key/value heads, keys of ``dim`` (the first ``rot_dims`` of them
    turn) and values of ``vdim`` elements (all of them turn), scores times ``scale`` and capped at ``softcap``
    (None: no cap), a query sees itself and the ``window - 1`` tokens before it (None: all of them)."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int
    rot_base: float
    window: int | None = None
    softcap: float | None = None

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "TurnedAttentionSizes":
        for key in ("heads", "dim", "scale", "rot"):
            if key not in raw:
                raise ConfigError(f"{where}: the mixer lacks {key!r}")
        heads = _positive(where, "heads", raw["heads"])
        kv_heads = _positive(where, "kv_heads", raw.get("kv_heads", heads))
        if heads % kv_heads:
            raise ConfigError(f"{where}: {heads} query heads do not divide into {kv_heads} key/value heads")
        dim = _positive(where, "dim", raw["dim"])
        vdim = _positive(where, "vdim", raw.get("vdim", dim))
        if dim % 2 or vdim % 2:
            raise ConfigError(f"{where}: turned heads have an even size, got keys of {dim} and values of {vdim}")
        rot = raw["rot"]
        _unknown(where + " rot", rot, {"dims", "base"})
        dims = rot.get("dims", dim)
        if isinstance(dims, bool) or not isinstance(dims, int) or not 0 <= dims <= dim or dims % 2:
            raise ConfigError(f"{where}: rot.dims must be an even number of the {dim} elements, got {dims!r}")
        mask = raw.get("mask") or {}
        _unknown(where + " mask", mask, {"size"})
        _unknown(where + " mixer", raw, {"heads", "kv_heads", "dim", "vdim", "scale", "mask", "rot", "softcap"})
        return cls(heads, kv_heads, dim, vdim, _number(where, "scale", raw), dims, _number(where + " rot", "base", rot),
                   None if mask.get("size") is None else _positive(where, "mask.size", mask["size"]),
                   _optional_positive(where, "softcap", raw))

    def to_dict(self) -> dict[str, Any]:
        raw: dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
                               "scale": self.scale, "rot": {"dims": self.rot_dims, "base": self.rot_base}}
        if self.window is not None:
            raw["mask"] = {"size": self.window}
        if self.softcap is not None:
            raw["softcap"] = self.softcap
        return raw


@dataclass(frozen=True)
class DenseSizes:
    ff: int

    def to_dict(self) -> dict[str, Any]:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class InputWeightedMixtureSizes:
    """``experts`` experts of inner width ``ff``, ``top`` a token by sigmoid scores; a shared expert of
    ``shared_ff`` (0: none)."""

    ff: int
    experts: int
    top: int
    shared_ff: int = 0

    def to_dict(self) -> dict[str, Any]:
        raw: dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff:
            raw["shared"] = {"ff": self.shared_ff}
        return raw


def _feed_forward(raw: Mapping[str, Any] | None, where: str):
    if raw is None:
        return None
    if raw.get("kind") == "dense":
        _unknown(where + " mlp", raw, {"kind", "ff"})
        return DenseSizes(_positive(where, "mlp.ff", raw.get("ff")))
    if raw.get("kind") != "moe":
        raise ConfigError(f"{where}: unknown feed-forward kind {raw.get('kind')!r} (dense, moe)")
    router, expert, shared = raw.get("router") or {}, raw.get("expert") or {}, raw.get("shared")
    _unknown(where + " mlp", raw, {"kind", "router", "expert", "shared"})
    _unknown(where + " mlp.router", router, {"experts", "top"})
    _unknown(where + " mlp.expert", expert, {"ff"})
    _unknown(where + " mlp.shared", shared or {}, {"ff"})
    experts, top = _positive(where, "mlp.router.experts", router.get("experts")), _positive(where, "mlp.router.top", router.get("top"))
    if top > experts:
        raise ConfigError(f"{where}: each token takes {top} of {experts} experts")
    return InputWeightedMixtureSizes(_positive(where, "mlp.expert.ff", expert.get("ff")), experts, top,
                                     0 if shared is None else _positive(where, "mlp.shared.ff", shared.get("ff")))


@dataclass(frozen=True)
class SarudraLayer:
    """``kind`` "mamba2": ``mixer`` is a ``StateSpaceSizes``. ``kind`` "attention": a ``TurnedAttentionSizes``."""

    kind: str
    mixer: Any
    feed_forward: Any


MIXERS = {"mamba2": StateSpaceSizes, "attention": TurnedAttentionSizes}


@dataclass(frozen=True)
class SarudraConfig:
    vocab: int
    width: int
    eps: float
    layers: tuple[SarudraLayer, ...]
    norm_groups: int = 1
    embedding_scale: float = 1.0
    logit_softcap: float | None = None
    max_positions: int = 1 << 20
    eos_token_id: int | None = None

    architecture = "Sarudra"

    def __post_init__(self) -> None:
        _positive("config", "vocab", self.vocab)
        _positive("config", "width", self.width)
        if not self.eps > 0.0:
            raise ConfigError(f"norm.eps must be positive, got {self.eps!r}")
        if self.width % _positive("config", "norm.groups", self.norm_groups):
            raise ConfigError(f"a width of {self.width} does not divide into {self.norm_groups} parts of the norm")
        if not self.layers:
            raise ConfigError("the model has no layers")

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "SarudraConfig":
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
            layers.append(SarudraLayer(kind, MIXERS[kind].from_dict(spec.get("mixer") or {}, where),
                                       _feed_forward(spec.get("mlp"), where)))
        norm, embedding = raw["norm"] or {}, raw.get("embedding") or {}
        _unknown("norm", norm, {"eps", "groups"})
        _unknown("embedding", embedding, {"scale"})
        _unknown("config", raw, {"architecture", "architectures", "vocab", "width", "layers", "norm", "embedding",
                                 "logit_softcap", "max_positions", "eos_token_id"})
        eos = raw.get("eos_token_id")
        return cls(vocab=raw["vocab"], width=raw["width"], eps=float(norm.get("eps", 0.0)), layers=tuple(layers),
                   norm_groups=norm.get("groups", 1), embedding_scale=float(embedding.get("scale", 1.0)),
                   logit_softcap=_optional_positive("config", "logit_softcap", raw),
                   max_positions=int(raw.get("max_positions", 1 << 20)), eos_token_id=None if eos is None else int(eos))

    def to_dict(self) -> dict[str, Any]:
        """The config.json a model folder of this configuration carries."""
        raw: dict[str, Any] = {
            "architecture": self.architecture, "vocab": self.vocab, "width": self.width,
            "norm": {"eps": self.eps, "groups": self.norm_groups}, "embedding": {"scale": self.embedding_scale},
            "layers": [{"type": layer.kind, "mixer": layer.mixer.to_dict(),
                        "mlp": None if layer.feed_forward is None else layer.feed_forward.to_dict()} for layer in self.layers]}
        for key, value, default in (("logit_softcap", self.logit_softcap, None), ("max_positions", self.max_positions, 1 << 20),
                                    ("eos_token_id", self.eos_token_id, None)):
            if value != default:
                raw[key] = value
        return raw
