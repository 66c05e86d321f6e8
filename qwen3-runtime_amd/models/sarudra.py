"""The Sarudra decoder as a plan of parts.

One residual stream that starts as the embedding times a constant; a sub-layer reads the stream as
it is and its output is normed, in groups of the width, on its way back into it
(``x += norm(f(x))``). A layer's mixer is a state-space mixer (a short convolution, a state per head
that decays by a step size made from the input, a gate and a grouped norm on the read-out) or softmax
attention over a window (queries and keys normed per head and turned over part of it, capped scores,
values that are turned by their own position and turned back by the query's); its feed-forward is
dense with a silu gate, a routed mixture whose weights scale the experts' input, with a shared expert,
or nothing. The head is a matrix of its own and the logits are capped. Tensor names are those of the
model file: ``embed``, ``l<i>.norm1|norm2``, ``l<i>.mix.*``, ``l<i>.mlp.gate|up|down`` or
``l<i>.mlp.router``, ``l<i>.mlp.e<j>.gate|up|down`` and ``l<i>.mlp.shared.gate|up|down``, ``final.norm``,
``head``.
"""

from __future__ import annotations

from ..config.sarudra import (DenseSizes, InputWeightedMixtureSizes, SarudraConfig, SarudraLayer, StateSpaceSizes,
                              TurnedAttentionSizes)
from ..parts.plan import LayerSpec, ModelPlan, PartSpec, RunStep
from ..registry import part_class, register_architecture, register_preset


def _norm(cfg: SarudraConfig, name: str) -> PartSpec:
    return PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.eps, "groups": cfg.norm_groups}, {"weight": name})


def _mixer(cfg: SarudraConfig, layer: SarudraLayer, p: str) -> PartSpec:
    s = layer.mixer
    if layer.kind == "mamba2":
        names = {n: f"{p}.{n}" for n in ("in", "conv", "dt_bias", "A_log", "D", "norm", "o")}
        names["conv_bias"] = f"{p}.conv.b"
        return PartSpec("state_space", {"hidden_size": cfg.width, "num_heads": s.heads, "value_dim": s.vdim,
                                        "state_dim": s.state, "groups": s.groups, "taps": s.conv,
                                        "norm_groups": s.norm_groups, "norm_eps": cfg.eps}, names)
    tensors = {n: f"{p}.{n}" for n in ("q", "k", "v", "o")}
    tensors.update(q_norm=f"{p}.q.norm", k_norm=f"{p}.k.norm")
    position = PartSpec("rope_half", {"head_dim": s.dim, "dims": s.rot_dims, "base": s.rot_base}) if s.rot_dims else None
    return PartSpec("gqa_attention", {"hidden_size": cfg.width, "num_heads": s.heads, "num_kv_heads": s.kv_heads,
                                      "head_dim": s.dim, "value_dim": s.vdim, "scale": s.scale, "window": s.window,
                                      "softcap": s.softcap, "qk_norm_eps": cfg.eps, "position": position,
                                      "value_turn": s.rot_base}, tensors)


def _feed_forward(cfg: SarudraConfig, s, p: str) -> PartSpec | None:
    if s is None:
        return None
    if isinstance(s, DenseSizes):
        return PartSpec("swiglu", {"hidden_size": cfg.width, "intermediate_size": s.ff},
                        {n: f"{p}.mlp.{n}" for n in ("gate", "up", "down")})
    tensors = {n: f"{p}.mlp.e{{e}}.{n}" for n in ("gate", "up", "down")}
    tensors["router"] = f"{p}.mlp.router"
    if s.shared_ff:
        tensors.update({f"shared_{n}": f"{p}.mlp.shared.{n}" for n in ("gate", "up", "down")})
    return PartSpec("routed_experts", {"hidden_size": cfg.width, "intermediate_size": s.ff, "num_experts": s.experts,
                                       "top": s.top, "router_bias": False, "scoring": "sigmoid", "weight_on": "input",
                                       "shared_size": s.shared_ff or None}, tensors)


def plan_sarudra(cfg: SarudraConfig) -> ModelPlan:
    layers, caches, order, unread = [], [], [], []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        mixer, ff = _mixer(cfg, layer, f"{p}.mix"), _feed_forward(cfg, layer.feed_forward, p)
        norms = {"after_mixer": _norm(cfg, f"{p}.norm1")}
        if ff is not None:
            norms["after_ff"] = _norm(cfg, f"{p}.norm2")
        else:
            unread.append(f"{p}.norm2")  # a file may carry the norm of a feed-forward that is not there
        layers.append(LayerSpec(PartSpec("output_norm"), mixer, ff, norms))
        specs = part_class("mixer", mixer.kind)(**mixer.args, tensors=mixer.tensors).cache_specs()
        ids = tuple(range(len(caches), len(caches) + len(specs)))
        caches.extend(specs)
        order.append(RunStep(layer=i, cache=ids[0] if len(ids) == 1 else ids))
    sizes = {"vocab_size": cfg.vocab, "hidden_size": cfg.width}
    return ModelPlan(
        hidden_size=cfg.width, vocab_size=cfg.vocab, max_positions=cfg.max_positions,
        embedding=PartSpec("token_embedding", {**sizes, "scale": cfg.embedding_scale}, {"weight": "embed"}),
        layers=layers, caches=caches, order=order, final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear_head", {**sizes, "softcap": cfg.logit_softcap}, {"weight": "head"}),
        ignorable=tuple(unread), eos_token_id=cfg.eos_token_id,
    )


# Small configurations for tests and examples; they differ in every size and option.
PRESETS: dict[str, SarudraConfig] = {
    "sarudra_tiny_a": SarudraConfig(
        vocab=230, width=96, eps=1e-5, norm_groups=3, embedding_scale=2.0, logit_softcap=12.0,
        layers=(
            SarudraLayer("mamba2", StateSpaceSizes(heads=4, vdim=24, state=16, groups=2, conv=4, norm_groups=3), DenseSizes(80)),
            SarudraLayer("attention", TurnedAttentionSizes(6, 2, 32, 16, 0.2, 24, 5000.0, 21, 20.0),
                         InputWeightedMixtureSizes(ff=40, experts=10, top=3, shared_ff=56)),
            SarudraLayer("mamba2", StateSpaceSizes(heads=3, vdim=40, state=24, groups=1, conv=3), None),
        ),
    ),
    "sarudra_tiny_b": SarudraConfig(
        vocab=170, width=64, eps=1e-6,
        layers=(
            SarudraLayer("attention", TurnedAttentionSizes(4, 4, 16, 16, 0.3, 16, 300.0, 9), DenseSizes(48)),
            SarudraLayer("mamba2", StateSpaceSizes(heads=6, vdim=8, state=40, groups=3, conv=2, norm_groups=2),
                         InputWeightedMixtureSizes(ff=24, experts=5, top=1)),
        ),
    ),
}
PRESET_PAGE_SIZE = {"sarudra_tiny_a": 16, "sarudra_tiny_b": 8}


def sized(width: int, layers: int, heads: int, kv_heads: int, dim: int, vocab: int, *, ff: int, expert_ff: int,
          experts: int = 16, top: int = 2, shared_ff: int = 0, window: int = 2048, state: int = 128, ssm_dim: int = 64,
          ssm_groups: int = 8, attention_every: int = 2) -> SarudraConfig:
    """A configuration of the sizes of a real model, for measurements: state-space layers with twice the
    width's channels, every ``attention_every``-th layer attention; dense feed-forward in the first layer,
    a mixture in the others."""
    ssm_heads = 2 * width // ssm_dim
    ssm = StateSpaceSizes(ssm_heads, ssm_dim, state, ssm_groups, 4, ssm_groups)
    att = TurnedAttentionSizes(heads, kv_heads, dim, dim, dim ** -0.5, dim, 1e6, window, 50.0)
    moe = InputWeightedMixtureSizes(expert_ff, experts, top, shared_ff)
    return SarudraConfig(vocab=vocab, width=width, eps=1e-5, norm_groups=4, embedding_scale=1.0, logit_softcap=30.0, layers=tuple(
        SarudraLayer("attention" if i % attention_every == attention_every - 1 else "mamba2",
                     att if i % attention_every == attention_every - 1 else ssm, DenseSizes(ff) if i == 0 else moe)
        for i in range(layers)))


register_architecture(SarudraConfig.architecture, SarudraConfig.from_dict, plan_sarudra)
for _name, _cfg in PRESETS.items():
    register_preset(_name, _cfg.to_dict(), PRESET_PAGE_SIZE.get(_name, 16))
# layers of the sizes of the 4B and 8B dense presets, and of a smaller width, with a mixture like
# `zisedra_4b`'s in every layer but the first, for measurements beside it
register_preset("sarudra_4b", sized(2560, 36, 32, 8, 128, 151936, ff=9728, expert_ff=1536, shared_ff=1536).to_dict(), 16)
register_preset("sarudra_8b", sized(4096, 36, 32, 8, 128, 151936, ff=12288, expert_ff=2048, shared_ff=2048).to_dict(), 16)
register_preset("sarudra_2b", sized(2048, 28, 16, 4, 128, 151936, ff=6144, expert_ff=1024, shared_ff=1024).to_dict(), 16)
