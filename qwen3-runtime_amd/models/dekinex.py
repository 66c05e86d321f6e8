"""The Dekinex decoder as a plan of parts.

One residual stream that starts as the token's embedding plus a row picked by the token and the one before
it. A layer has one RMS norm (its weight stored around zero) that mixer and feed-forward both read; the
sum of their outputs joins the stream times ``residual_mult``. A layer's mixer is attention over a sliding
window (a short convolution over time behind every projection, queries and keys turned in neighbour pairs
and divided by their root mean square) or a matrix memory with exponential gates (mLSTM) whose state lives
in the request's slot; its feed-forward is dense with a clamped gate, a mixture chosen by corrected sigmoid
scores beside a gated shared expert, or nothing. A span of layers may run several times in a row; every
pass begins with a vector of its own, every pass but the first with the embedding's output added once
more, and every run of a layer has caches of its own. The head has a matrix of its own. Tensor names are
those of the model file: ``embed``, ``bigram``, ``loop.step``, ``l<i>.norm1``, ``l<i>.mix.*``,
``l<i>.mlp.gate|up|down`` or ``l<i>.mlp.router|correction``, ``l<i>.mlp.e<j>.gate|up|down`` and
``l<i>.mlp.shared.gate|up|down|sg``, ``final.norm``, ``head``.
"""

from __future__ import annotations

from ..config.dekinex import (ClampedSizes, ConvolvedAttentionSizes, DekinexConfig, DekinexLayer, MatrixMemorySizes,
                              PairTable, SharedMixtureSizes)
from ..parts.plan import LayerSpec, ModelPlan, PartSpec, RunStep
from ..registry import part_class, register_architecture, register_preset


def _norm(cfg: DekinexConfig, name: str) -> PartSpec:
    return PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.eps, "weight_offset": 1.0}, {"weight": name})


def _mixer(cfg: DekinexConfig, layer: DekinexLayer, p: str) -> PartSpec:
    s = layer.mixer
    if layer.kind == "mlstm":
        names = {n: f"{p}.{n}" for n in ("q", "k", "v", "g", "i", "f", "norm", "o")}
        names.update(i_bias=f"{p}.i.b", f_bias=f"{p}.f.b")
        return PartSpec("matrix_memory", {"hidden_size": cfg.width, "num_heads": s.heads, "head_dim": s.dim, "value_dim": s.vdim,
                                          "gate_cap": s.gate_cap, "norm_eps": cfg.eps}, names)
    tensors = {n: f"{p}.{n}" for n in ("q", "k", "v", "o")}
    if s.conv is not None:
        tensors.update({f"{n}_conv": f"{p}.{n}.conv" for n in ("q", "k", "v")})
    position = PartSpec("rope_half", {"head_dim": s.dim, "dims": s.rot_dims, "base": s.rot_base}) if s.rot_dims else None
    return PartSpec("gqa_attention", {"hidden_size": cfg.width, "num_heads": s.heads, "num_kv_heads": s.kv_heads,
                                      "head_dim": s.dim, "value_dim": s.vdim, "scale": s.scale, "window": s.window,
                                      "qk_norm_eps": cfg.eps, "qk_norm_weight": False, "position": position,
                                      "neighbour_pairs": True, "conv": s.conv}, tensors)


def _feed_forward(cfg: DekinexConfig, s, p: str) -> PartSpec | None:
    if s is None:
        return None
    if isinstance(s, ClampedSizes):
        return PartSpec("swiglu", {"hidden_size": cfg.width, "intermediate_size": s.ff, "activation": "clamped", "limit": s.limit},
                        {n: f"{p}.mlp.{n}" for n in ("gate", "up", "down")})
    tensors = {n: f"{p}.mlp.e{{e}}.{n}" for n in ("gate", "up", "down")}
    tensors.update(router=f"{p}.mlp.router", correction=f"{p}.mlp.correction")
    if s.shared_ff:
        tensors.update({f"shared_{n}": f"{p}.mlp.shared.{n}" for n in ("gate", "up", "down", "sg")})
    return PartSpec("routed_experts", {"hidden_size": cfg.width, "intermediate_size": s.ff, "num_experts": s.experts,
                                       "top": s.top, "router_bias": False, "scoring": "sigmoid", "correction": True,
                                       "renormalise": True, "weight_scale": s.scale, "shared_size": s.shared_ff or None,
                                       "shared_gate": bool(s.shared_ff)}, tensors)


def plan_dekinex(cfg: DekinexConfig) -> ModelPlan:
    layers = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        block = PartSpec("parallel_scaled", {"hidden_size": cfg.width, "layer_scale": False, "mult": cfg.residual_mult})
        layers.append(LayerSpec(block, _mixer(cfg, layer, f"{p}.mix"), _feed_forward(cfg, layer.feed_forward, p),
                                {"input": _norm(cfg, f"{p}.norm1")}))
    entries = []
    if cfg.loop is not None:
        times = cfg.loop[2]
        entries = [PartSpec("pass_vector", {"hidden_size": cfg.width, "times": times, "index": t, "origin": t > 0},
                            {"step": "loop.step"}) for t in range(times)]
    sizes = {"vocab_size": cfg.vocab, "hidden_size": cfg.width}
    if cfg.pairs is None:
        embedding = PartSpec("token_embedding", sizes, {"weight": "embed"})
    else:
        embedding = PartSpec("bigram_embedding", {**sizes, **cfg.pairs.to_dict()}, {"weight": "embed", "bigram": "bigram"})
    caches = list(part_class("embedding", embedding.kind)(**embedding.args, tensors=embedding.tensors).cache_specs())
    own, order = tuple(range(len(caches))), []
    for i, begins in cfg.run_order():  # every run of a layer has caches of its own
        mixer = layers[i].mixer
        specs = part_class("mixer", mixer.kind)(**mixer.args, tensors=mixer.tensors).cache_specs()
        ids = tuple(range(len(caches), len(caches) + len(specs)))
        caches.extend(specs)
        order.append(RunStep(layer=i, cache=ids[0] if len(ids) == 1 else ids, entry=begins))
    return ModelPlan(
        hidden_size=cfg.width, vocab_size=cfg.vocab, max_positions=cfg.max_positions, embedding=embedding,
        layers=layers, caches=caches, order=order, final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear_head", sizes, {"weight": "head"}), eos_token_id=cfg.eos_token_id, entries=entries,
        embedding_cache=own,
    )


# Small configurations for tests and examples; they differ in every size and option.
PRESETS: dict[str, DekinexConfig] = {
    "dekinex_tiny_a": DekinexConfig(
        vocab=230, width=96, eps=1e-5, residual_mult=0.8, loop=(1, 3, 2), pairs=PairTable(211, 31, 7),
        layers=(
            DekinexLayer("mlstm", MatrixMemorySizes(3, 24, 40, 10.0), ClampedSizes(80, 1.2)),
            DekinexLayer("attention", ConvolvedAttentionSizes(6, 2, 32, 16, 0.2, 21, 3, 12, 5000.0),
                         SharedMixtureSizes(40, 10, 3, 1.5, 56)),
            DekinexLayer("mlstm", MatrixMemorySizes(2, 48, 16, 6.0), SharedMixtureSizes(24, 6, 2, 0.7)),
            DekinexLayer("attention", ConvolvedAttentionSizes(4, 4, 16, 16, 0.3, 13, 4, 16, 300.0), None),
        ),
    ),
    "dekinex_tiny_b": DekinexConfig(
        vocab=170, width=64, eps=1e-6, pairs=PairTable(64, 5, 11),
        layers=(
            DekinexLayer("attention", ConvolvedAttentionSizes(2, 1, 48, 48, 0.15, 9, 2, 20, 50.0), ClampedSizes(48, 2.0)),
            DekinexLayer("mlstm", MatrixMemorySizes(4, 16, 16, 15.0), SharedMixtureSizes(32, 5, 1, 1.0, 24)),
        ),
    ),
}
PRESET_PAGE_SIZE = {"dekinex_tiny_a": 16, "dekinex_tiny_b": 8}


def sized(width: int, layers: int, heads: int, kv_heads: int, dim: int, vocab: int, *, ff: int, expert_ff: int,
          experts: int = 16, top: int = 2, shared_ff: int = 0, window: int = 2048, attention_every: int = 2) -> DekinexConfig:
    """A configuration of the sizes of a real model, for measurements: ``layers`` layer runs, the matrix
    memories and attention in turn; dense feed-forward in the first layer, a mixture in the others; the
    second and third layer run twice."""
    memory = MatrixMemorySizes(heads, dim, dim, 15.0)
    att = ConvolvedAttentionSizes(heads, kv_heads, dim, dim, dim ** -0.5, window, 4, dim // 2, 1e6)
    moe = SharedMixtureSizes(expert_ff, experts, top, 1.0, shared_ff)
    own = layers - 2
    return DekinexConfig(vocab=vocab, width=width, eps=1e-5, loop=(1, 3, 2), pairs=PairTable(65521, 8191, 131), layers=tuple(
        DekinexLayer("attention" if i % attention_every == attention_every - 1 else "mlstm",
                     att if i % attention_every == attention_every - 1 else memory, ClampedSizes(ff, 7.0) if i == 0 else moe)
        for i in range(own)))


register_architecture(DekinexConfig.architecture, DekinexConfig.from_dict, plan_dekinex)
for _name, _cfg in PRESETS.items():
    register_preset(_name, _cfg.to_dict(), PRESET_PAGE_SIZE.get(_name, 16))
# layers of the sizes of the 4B and 8B dense presets, and of a smaller width, with a mixture like
# `sarudra_4b`'s in every layer but the first, for measurements beside it
register_preset("dekinex_4b", sized(2560, 36, 32, 8, 128, 151936, ff=9728, expert_ff=1536, shared_ff=1536).to_dict(), 16)
register_preset("dekinex_8b", sized(4096, 36, 32, 8, 128, 151936, ff=12288, expert_ff=2048, shared_ff=2048).to_dict(), 16)
register_preset("dekinex_2b", sized(2048, 28, 16, 4, 128, 151936, ff=6144, expert_ff=1024, shared_ff=1024).to_dict(), 16)
