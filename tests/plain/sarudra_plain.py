"""Plain, slow Sarudra decoder: whole sequences, no cache, one function per mechanism.

It shares no code with the engine: it reads config.json and the safetensors file itself and
works on one whole sequence at a time in ``dtype`` (float64 unless asked otherwise).

The design in short. One residual stream that starts as the embedding times a constant. A
sub-layer reads the stream as it is; only its output is normed before it joins:
``x <- x + norm(f(x))``, RMS norms over equal groups of the width. Two mixers: a state-space mixer
(short convolution, a state per head that decays by a data-dependent step, a skip, a gate in front of
a grouped norm), and softmax attention over a sliding window whose queries and keys are normed per
head and turned over part of the head, whose scores are capped, and whose values are turned by their
own position and turned back by the query's. Feed-forwards are dense with a silu gate, or a routed
mixture whose weights, plain sigmoid scores, scale the experts' input, beside a shared expert. The
head is a matrix of its own and the logits are capped.
"""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch


def silu(x):
    return x * torch.sigmoid(x)


def cap(x, limit):
    """limit * tanh(x / limit); no limit: x."""
    return x if limit is None else limit * torch.tanh(x / limit)


def group_norm(x, weight, eps, groups):
    """Every one of ``groups`` equal parts of the last dimension over its own root mean square, then
    times the weight of the whole dimension (None: no weight)."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    y = (parts / torch.sqrt(parts.pow(2).mean(dim=-1, keepdim=True) + eps)).reshape(x.shape)
    return y if weight is None else y * weight


# ------------------------------------------------------------------ the state-space mixer
def causal_convolution(x, taps, bias):
    """Per channel: y_t = bias + sum_j taps[:, j] x_(t - K + 1 + j), zeros before the start. x [T, C]."""
    k = taps.shape[1]
    padded = torch.cat([x.new_zeros(k - 1, x.shape[1]), x], dim=0)
    y = bias[None, :].expand(x.shape[0], -1).clone()
    for j in range(k):
        y = y + padded[j: j + x.shape[0]] * taps[:, j]
    return y


def state_space_head(x, b, c, dt, a_log, skip):
    """One head, token by token: S <- exp(-exp(a_log) dt) S + dt b x^T; y = S^T c + skip x.
    x [T, P], b and c [T, N], dt [T]."""
    s = x.new_zeros(b.shape[1], x.shape[1])
    rate = math.exp(float(a_log))
    out = []
    for i in range(x.shape[0]):
        s = torch.exp(-rate * dt[i]) * s + dt[i] * torch.outer(b[i], x[i])
        out.append(s.T @ c[i] + skip * x[i])
    return torch.stack(out)


def state_space(h, w, sizes, eps):
    """The mixer 'mamba2'. h [T, width]."""
    t = h.shape[0]
    n, p, state, groups = sizes["heads"], sizes["vdim"], sizes["state"], sizes.get("groups", 1)
    inner = n * p
    z, xbc, dt = (h @ w["in"].T).split([inner, inner + 2 * groups * state, n], dim=-1)
    xbc = silu(causal_convolution(xbc, w["conv"], w["conv.b"]))
    x, b, c = xbc.split([inner, groups * state, groups * state], dim=-1)
    x, b, c = x.view(t, n, p), b.view(t, groups, state), c.view(t, groups, state)
    dt = torch.nn.functional.softplus(dt + w["dt_bias"], threshold=1e9)
    per = n // groups
    y = torch.stack([state_space_head(x[:, j], b[:, j // per], c[:, j // per], dt[:, j], w["A_log"][j], w["D"][j])
                     for j in range(n)], dim=1).reshape(t, inner)
    y = group_norm(y * silu(z), w["norm"], eps, sizes.get("norm_groups", 1))
    return y @ w["o"].T


# ------------------------------------------------------------------ attention
def rotate_half(x, positions, dims, base, sign=1.0):
    """x [T, heads, D]: the first ``dims`` elements of every head turn, element i against element
    i + dims/2, by the angle sign * position * base^(-2i/dims); the rest passes."""
    if dims == 0:
        return x
    half = dims // 2
    i = torch.arange(half, dtype=x.dtype)
    freq = base ** (-2.0 * i / dims)
    ang = sign * torch.as_tensor(positions, dtype=x.dtype)[:, None] * freq[None, :]
    cos, sin = ang.cos()[:, None, :], ang.sin()[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def attention(h, w, sizes, eps):
    """The mixer 'attention'. h [T, width]."""
    t = h.shape[0]
    nq, d = sizes["heads"], sizes["dim"]
    nkv, dv = sizes.get("kv_heads", nq), sizes.get("vdim", d)
    rot = sizes["rot"]
    pos = list(range(t))
    q = group_norm((h @ w["q"].T).view(t, nq, d), w["q.norm"], eps, 1)
    k = group_norm((h @ w["k"].T).view(t, nkv, d), w["k.norm"], eps, 1)
    v = (h @ w["v"].T).view(t, nkv, dv)
    q, k = rotate_half(q, pos, rot["dims"], rot["base"]), rotate_half(k, pos, rot["dims"], rot["base"])
    v = rotate_half(v, pos, dv, rot["base"])
    g = nq // nkv
    k, v = k.repeat_interleave(g, dim=1), v.repeat_interleave(g, dim=1)
    scores = cap(torch.einsum("qhd,khd->hqk", q, k) * sizes["scale"], sizes.get("softcap"))
    i, j = torch.arange(t)[:, None], torch.arange(t)[None, :]
    seen = (j <= i) & (i - j < sizes["mask"]["size"])
    p = torch.softmax(scores.masked_fill(~seen[None], float("-inf")), dim=-1)
    out = torch.einsum("hqk,khd->qhd", p, v)
    out = rotate_half(out, pos, dv, rot["base"], sign=-1.0)
    return out.reshape(t, nq * dv) @ w["o"].T


# ------------------------------------------------------------------ feed-forwards
def gated(h, w, prefix=""):
    """down(silu(gate h) * (up h))."""
    return (silu(h @ w[prefix + "gate"].T) * (h @ w[prefix + "up"].T)) @ w[prefix + "down"].T


def route(h, router, top):
    """(index [T, top], weight [T, top]): the largest sigmoid scores, which are the weights as they are."""
    s = torch.sigmoid(h @ router.T)
    index = torch.topk(s, top, dim=-1).indices
    return index, torch.gather(s, 1, index)


def mixture(h, w, mlp):
    """Sum over the chosen experts of expert(weight * h), and the shared expert on h."""
    index, weight = route(h, w["router"], mlp["router"]["top"])
    rows = []
    for i in range(h.shape[0]):
        rows.append(sum(gated(weight[i, j] * h[i], w, f"e{int(index[i, j])}.") for j in range(index.shape[1])))
    out = torch.stack(rows)
    return out + gated(h, w, "shared.") if mlp.get("shared") else out


def feed_forward(h, w, mlp):
    if mlp["kind"] == "dense":
        return gated(h, w)
    if mlp["kind"] == "moe":
        return mixture(h, w, mlp)
    raise ValueError(mlp["kind"])


MIXERS = {"mamba2": state_space, "attention": attention}


# ------------------------------------------------------------------ the model
def read_safetensors(path, dtype=torch.float64):
    raw = Path(path).read_bytes()
    n = int.from_bytes(raw[:8], "little")
    header = json.loads(raw[8: 8 + n])
    kinds = {"BF16": torch.bfloat16, "F32": torch.float32, "F16": torch.float16, "I32": torch.int32}
    out = {}
    for name, meta in header.items():
        if name == "__metadata__":
            continue
        a, b = meta["data_offsets"]
        t = torch.frombuffer(bytearray(raw[8 + n + a: 8 + n + b]), dtype=kinds[meta["dtype"]]).view(meta["shape"])
        out[name] = t if meta["dtype"] == "I32" else t.to(dtype)
    return out


def sub(weights, prefix):
    return {n[len(prefix):]: x for n, x in weights.items() if n.startswith(prefix)}


def forward(cfg, weights, ids, return_layers=False):
    """Logits [T, vocab] of one whole sequence (and the stream after every layer)."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"].get("groups", 1)
    x = weights["embed"][torch.as_tensor(ids, dtype=torch.long)] * cfg["embedding"]["scale"]
    after = []
    for i, layer in enumerate(cfg["layers"]):
        w = sub(weights, f"l{i}.")
        y = MIXERS[layer["type"]](x, sub(w, "mix."), layer["mixer"], eps)
        x = x + group_norm(y, w["norm1"], eps, groups)
        if layer.get("mlp"):
            x = x + group_norm(feed_forward(x, sub(w, "mlp."), layer["mlp"]), w["norm2"], eps, groups)
        after.append(x)
    logits = cap(group_norm(x, weights["final.norm"], eps, groups) @ weights["head"].T, cfg.get("logit_softcap"))
    return (logits, torch.stack(after)) if return_layers else logits


def load(folder, dtype=torch.float64):
    folder = Path(folder)
    cfg = json.loads((folder / "config.json").read_text())
    return cfg, read_safetensors(folder / "model.safetensors", dtype)
