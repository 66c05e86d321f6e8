"""Plain, slow Dekinex decoder: whole sequences, no cache, no state carried, one function per mechanism.

It shares no code with the engine: it reads config.json and the safetensors file itself and
works on one whole sequence at a time in ``dtype`` (float64 unless asked otherwise).

The design in short. The stream starts as the token's embedding plus a row that the pair (previous
token, token) picks from a second table. A layer has one RMS norm, whose weight is stored around zero;
its mixer and its feed-forward both read the norm's output and their sum joins the stream times a
constant. Two mixers: softmax attention over a sliding window, whose queries, keys and values pass a
short convolution over time straight after their projections, whose queries and keys turn in neighbour
pairs over part of the head and are then divided by their root mean square; and a matrix memory with
exponential gates (mLSTM), held in check by a running maximum. Feed-forwards are dense with a clamped
gate, or a mixture chosen by sigmoid scores plus a correction, beside a shared expert that every token
opens by a sigmoid of its own. A span of layers may run several times in a row; every pass begins with a
vector of its own, and every pass but the first with the embedding added once more.
"""

from __future__ import annotations

import json
from pathlib import Path

import torch


def rms_norm(x, eps, weight=None):
    """x / sqrt(mean(x^2) + eps) over the last dimension, times 1 + weight."""
    y = x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)
    return y if weight is None else y * (1.0 + weight)


# ------------------------------------------------------------------ the embedding
def bigram_rows(ids, mul_prev, mul_cur, buckets):
    """The second table's row of every token; the first token of a sequence has the last row."""
    rows = [buckets]
    for prev, cur in zip(ids[:-1], ids[1:]):
        rows.append((int(prev) * mul_prev + int(cur) * mul_cur) % buckets)
    return rows


def embedding(cfg, weights, ids):
    x = weights["embed"][torch.as_tensor(ids, dtype=torch.long)]
    b = cfg["embedding"]["bigram"]
    return x + weights["bigram"][torch.as_tensor(bigram_rows(ids, b["mul_prev"], b["mul_cur"], b["buckets"]), dtype=torch.long)]


# ------------------------------------------------------------------ attention
def causal_convolution(u, taps):
    """Per channel: y_t = sum_j taps[:, j] u_(t - K + 1 + j), zeros before the start. u [T, C]."""
    k = taps.shape[1]
    padded = torch.cat([u.new_zeros(k - 1, u.shape[1]), u], dim=0)
    y = torch.zeros_like(u)
    for j in range(k):
        y = y + padded[j: j + u.shape[0]] * taps[:, j]
    return y


def rotate_neighbours(x, dims, base):
    """x [T, heads, D]: element 2i of every head turns against element 2i + 1, 2i < dims, by the
    angle position * base^(-2i/dims); the rest passes."""
    y = x.clone()
    p = torch.arange(x.shape[0], dtype=x.dtype)
    for i in range(dims // 2):
        a = p * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i], y[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return y


def attention(h, w, sizes, eps):
    """The mixer 'attention'. h [T, width]."""
    t = h.shape[0]
    nq, d = sizes["heads"], sizes["dim"]
    nkv, dv = sizes.get("kv_heads", nq), sizes.get("vdim", d)
    q, k, v = (causal_convolution(h @ w[n].T, w[n + ".conv"]) for n in ("q", "k", "v"))
    rot = sizes["rot"]
    q = rms_norm(rotate_neighbours(q.view(t, nq, d), rot["dims"], rot["base"]), eps)
    k = rms_norm(rotate_neighbours(k.view(t, nkv, d), rot["dims"], rot["base"]), eps)
    v = v.view(t, nkv, dv)
    g = nq // nkv
    k, v = k.repeat_interleave(g, dim=1), v.repeat_interleave(g, dim=1)
    scores = torch.einsum("qhd,khd->hqk", q, k) * sizes["scale"]
    i, j = torch.arange(t)[:, None], torch.arange(t)[None, :]
    seen = (j <= i) & (i - j < sizes["mask"]["size"])
    p = torch.softmax(scores.masked_fill(~seen[None], float("-inf")), dim=-1)
    return torch.einsum("hqk,khd->qhd", p, v).reshape(t, nq * dv) @ w["o"].T


# ------------------------------------------------------------------ the matrix memory
def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def log_sigmoid(z):
    """log(1 / (1 + exp(-z))) without overflow on either side."""
    return torch.clamp(z, max=0.0) - torch.log1p(torch.exp(-z.abs()))


def matrix_memory(q, k, v, log_in, log_forget):
    """Token by token over all heads. q, k [T, H, D], v [T, H, Dv], gates [T, H]. The memory S, its
    normaliser n and the running maximum m start at zero."""
    heads, d, dv = q.shape[1], q.shape[2], v.shape[2]
    s, n, m = q.new_zeros(heads, d, dv), q.new_zeros(heads, d), q.new_zeros(heads)
    out = []
    for t in range(q.shape[0]):
        top = torch.maximum(log_forget[t] + m, log_in[t])
        keep, write = torch.exp(log_forget[t] + m - top), torch.exp(log_in[t] - top)
        m = top
        s = keep[:, None, None] * s + write[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + write[:, None] * k[t]
        read = torch.einsum("hdv,hd->hv", s, q[t])
        floor = torch.maximum(torch.einsum("hd,hd->h", n, q[t]).abs(), torch.exp(-m))
        out.append(read / (floor + 1e-6)[:, None])
    return torch.stack(out)


def mlstm(h, w, sizes, eps):
    """The mixer 'mlstm'. h [T, width]."""
    t = h.shape[0]
    n, d = sizes["heads"], sizes["dim"]
    dv, cap = sizes.get("vdim", d), sizes["gate_cap"]
    q = (h @ w["q"].T).view(t, n, d) * d ** -0.5
    k, v = (h @ w["k"].T).view(t, n, d), (h @ w["v"].T).view(t, n, dv)
    log_in = soft_cap(h @ w["i"].T + w["i.b"], cap)
    log_forget = log_sigmoid(soft_cap(h @ w["f"].T + w["f.b"], cap))
    o = rms_norm(matrix_memory(q, k, v, log_in, log_forget), eps).reshape(t, n * dv)
    return (o * w["norm"] * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# ------------------------------------------------------------------ feed-forwards
def clamped(h, w, limit):
    """down(g sigmoid(1.702 g) (u + 1)), the gate held from above, the other half from both sides."""
    g, u = torch.clamp(h @ w["gate"].T, max=limit), torch.clamp(h @ w["up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


def silu_gated(h, w, prefix):
    """down(silu(gate h) * (up h))."""
    z = h @ w[prefix + "gate"].T
    return (z * torch.sigmoid(z) * (h @ w[prefix + "up"].T)) @ w[prefix + "down"].T


def route(h, router, correction, top, scale):
    """(index [T, top], weight [T, top]): chosen by sigmoid scores plus the correction, weighed by the
    chosen scores alone over their sum, times ``scale``."""
    s = torch.sigmoid(h @ router.T)
    index = torch.topk(s + correction, top, dim=-1).indices
    weight = torch.gather(s, 1, index)
    return index, weight / (weight.sum(-1, keepdim=True) + 1e-20) * scale


def mixture(h, w, mlp):
    router = mlp["router"]
    index, weight = route(h, w["router"], w["correction"], router["top"], router.get("scale", 1.0))
    rows = []
    for i in range(h.shape[0]):
        rows.append(sum(weight[i, j] * silu_gated(h[i], w, f"e{int(index[i, j])}.") for j in range(index.shape[1])))
    out = torch.stack(rows)
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ w["shared.sg"].T) * silu_gated(h, w, "shared.")
    return out


def feed_forward(h, w, mlp):
    if mlp["kind"] == "dense":
        return clamped(h, w, mlp["limit"])
    if mlp["kind"] == "moe":
        return mixture(h, w, mlp)
    raise ValueError(mlp["kind"])


MIXERS = {"attention": attention, "mlstm": mlstm}


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


def run_order(cfg):
    """(layer, number of the pass that begins with it or None), one entry per layer run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, weights, ids, return_layers=False):
    """Logits [T, vocab] of one whole sequence (and the stream after every layer run)."""
    eps, mult = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
    first = embedding(cfg, weights, ids)
    x, after = first, []
    for i, begins in run_order(cfg):
        if begins is not None:
            if begins > 0:
                x = x + first
            x = x + weights["loop.step"][begins]
        layer, w = cfg["layers"][i], sub(weights, f"l{i}.")
        h = rms_norm(x, eps, w["norm1"])
        y = MIXERS[layer["type"]](h, sub(w, "mix."), layer["mixer"], eps)
        if layer.get("mlp"):
            y = y + feed_forward(h, sub(w, "mlp."), layer["mlp"])
        x = x + mult * y
        after.append(x)
    logits = rms_norm(x, eps, weights["final.norm"]) @ weights["head"].T
    return (logits, torch.stack(after)) if return_layers else logits


def load(folder, dtype=torch.float64):
    folder = Path(folder)
    cfg = json.loads((folder / "config.json").read_text())
    return cfg, read_safetensors(folder / "model.safetensors", dtype)
