"""Dekinex: every mechanism alone against its plain function, and whole models under every cutting.

Each test runs with the plain torch ops on the CPU (which pins the host side: plan, packing,
pages, windows, state slots, the loop) and with the HIP ops on the GPU (marked ``gpu``; float32 and
bfloat16). The oracle is ``plain/dekinex_plain.py``: whole sequences, no cache, no state carried,
float64. Configurations are made here and differ from each other in every size and option, also
in values that a model may happen to make equal or 1. Where random weights would hide a fault (a
key at the edge of a window, a write into a memory hundreds of tokens ago, a pass's own vector), one
token's key, value or write is made to stand out, or the oracle is given the fault and has to differ.
"""

from __future__ import annotations

import math
from types import SimpleNamespace

import pytest
import torch

import traces
from drivers import BACKENDS, DT, DictFetch, MixerDriver, f64, in_steps, make_ops, rnd, rounded
from plain import dekinex_plain as P
from plain.ops_ref import TorchOps


def row_bound(want, dtype):
    """Per row: float32 sums' rounding; in bfloat16 a twentieth of the row's largest element."""
    top = want.abs().amax(1)
    return 2e-4 + 2e-4 * top if dtype == "float32" else 0.05 + 0.05 * top


def assert_rows(got, want, dtype, what=""):
    worst = (got.double() - want).abs().amax(1) / row_bound(want, dtype)
    assert float(worst.max()) <= 1.0, (what, int(worst.argmax()), float(worst.max()))


def close(dtype):
    return dict(atol=3e-5, rtol=3e-5) if dtype == "float32" else dict(atol=3e-2, rtol=2e-2)


def spans(device, lens, slots, starts=None):
    """What embedding and recurrences read of a step's batch."""
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    starts = starts or [0] * len(lens)
    return SimpleNamespace(num_tokens=cu[-1], num_seqs=len(lens), cu_q=i32(cu), state_slots=i32(slots), max_q_len=max(lens),
                           positions=i32([s + i for s, n in zip(starts, lens) for i in range(n)]),
                           seq_of_token=i32([s for s, n in enumerate(lens) for _ in range(n)]), q_lens_host=list(lens), scratch={})


# ------------------------------------------------------------------ embedding
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("vocab,width,buckets,mul_prev,mul_cur", [
    (50, 24, 31, 7, 3), (300, 130, 1, 5, 2), (90, 64, 64, 1, 1), (40, 7, 5, 2147483647, 2000000011), (64, 256, 997, 0, 19), (30, 16, 11, -3, 4)])
def test_pairs_of_tokens_pick_a_second_row(backend, vocab, width, buckets, mul_prev, mul_cur):
    """Two sequences in the same steps, cut down to single tokens: the token before a span comes from the
    request's slot; a sequence's first token has the last row, also in a slot that somebody held before."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    w = {"embed": rnd(vocab, width, seed=1).to(dt).double(), "bigram": rnd(buckets + 1, width, seed=2).to(dt).double()}
    cfg = {"embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}}
    toks = [torch.randint(vocab, (n,), generator=torch.Generator().manual_seed(n)).tolist() for n in (37, 22)]
    want = [P.embedding(cfg, w, t) for t in toks]
    table, pairs = w["embed"].to(dt).to(device), w["bigram"].to(dt).to(device)
    for sizes in ((37,), (1,), (2, 1, 5), (20, 3)):
        last = torch.full((4, 1), 23, dtype=torch.int32, device=device)   # whoever was there before
        steps = [in_steps(len(t), sizes) for t in toks]
        got = [[], []]
        for r in range(max(map(len, steps))):
            live = [i for i in (1, 0) if r < len(steps[i])]
            cuts = [steps[i][r] for i in live]
            ctx = spans(device, [n for _, n in cuts], [(3, 1)[i] for i in live], [p for p, _ in cuts])
            ids = torch.tensor([t for i, (p, n) in zip(live, cuts) for t in toks[i][p: p + n]], dtype=torch.int32, device=device)
            out = ops.embed_pairs(ctx, ids, table, pairs, mul_prev, mul_cur, last)
            assert out.dtype == torch.float32
            for i, piece in zip(live, out.cpu().split([n for _, n in cuts])):
                got[i].append(piece)
        for i in range(2):
            torch.testing.assert_close(torch.cat(got[i]).double(), want[i], atol=1e-6, rtol=1e-6)
        assert last[0, 0] == 23 and last[2, 0] == 23 and last[3, 0] == toks[0][-1] and last[1, 0] == toks[1][-1]


# ------------------------------------------------------------------ the stream between layers
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width", [96, 2560, 70, 4097, 9000, 4])
@pytest.mark.parametrize("terms,planes", [(0, 0), (1, 0), (2, 3), (3, 1), (4, 9), (2, 0)])
def test_outputs_and_a_vector_join_the_stream(backend, width, terms, planes):
    """``x += sum_i s_i y_i + v``, then the norm with its weight stored around zero; all rows, also many of
    them, or chosen ones, which leave the stream alone; matrices and planes side by side."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    eps = 1e-5
    for t in (5, 600) if device != "cpu" and width in (96, 2560, 70) else (5,):
        x0 = rnd(t, width, seed=1)
        ys = [rnd(t, width, seed=2 + i).to(dt) if planes == 0 or i % 2 else rnd(planes, t, width, seed=3 + i) for i in range(terms)]
        scales = [1 + rnd(width, seed=20 + i) for i in range(terms)]
        w, v = rnd(width, seed=30, scale=0.3), rnd(width, seed=31)
        dev = lambda a: None if a is None else a.to(device)  # noqa: E731
        for vector in (v, None) if terms else (v,):
            new = x0.double() + sum(s.double() * (y.double().sum(0) if y.dim() == 3 else y.double()) for y, s in zip(ys, scales))
            new = new if vector is None else new + vector.double()
            want = P.rms_norm(new, eps, w.double())
            for rows in (None, torch.tensor([4, 0, 2], dtype=torch.int32)):
                x = dev(x0.clone())
                got = ops.scaled_add_rmsnorm(x, [(dev(y), dev(s)) for y, s in zip(ys, scales)], dev(1 + w), eps, dt, dev(rows), vector=dev(vector))
                torch.testing.assert_close(got.float().cpu().double(), want if rows is None else want[rows.long()],
                                           **(dict(atol=2e-5, rtol=2e-5) if dtype == "float32" else dict(atol=1e-2, rtol=1e-2)))
                torch.testing.assert_close(x.cpu().double(), new if rows is None else x0.double(), atol=1e-4, rtol=1e-5)


def test_a_norm_weight_stored_around_zero():
    from qwen3_runtime_amd.parts.norm import RMSNorm

    norm = RMSNorm(24, 1e-4, weight_offset=1.0, tensors={"weight": "w"})
    w, x = rnd(24, seed=1, scale=0.4), rnd(5, 24, seed=2)
    norm.load(DictFetch({"w": w}, "cpu", torch.float32))
    got = norm.forward(SimpleNamespace(ops=TorchOps(), dtype=torch.float32), x.clone())
    torch.testing.assert_close(got.double(), P.rms_norm(x.double(), 1e-4, w.double()), atol=1e-5, rtol=1e-5)
    assert norm.tensor_decls()[0].init == "norm_zero"


# ------------------------------------------------------------------ attention behind short convolutions
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("channels,taps", [(200, 4), (64, 2), (330, 3), (130, 1), (37, 6)])
def test_convolution_without_an_activation(backend, channels, taps):
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    lengths, slots = [150, 90], [2, 0]
    x = [rnd(n, channels, seed=3 + i).to(dt) for i, n in enumerate(lengths)]
    w = rnd(channels, taps, seed=9, scale=0.6)
    whole, rest = divmod(channels, 64)
    segments = tuple(s for s in ((whole, 64, 0), (1, rest, 0)) if s[0] * s[1])
    want = [P.causal_convolution(x[i].double(), w.double()) for i in range(2)]
    for sizes in ((150,), (2, 1, 3, 1, 1, 17), (40, 70)):
        tail = torch.zeros(3, channels, max(taps - 1, 1), dtype=torch.float32, device=device)
        tail[1] = float("nan")  # a slot nobody holds
        steps = [in_steps(n, sizes) for n in lengths]
        got = [[], []]
        for r in range(max(map(len, steps))):
            live = [i for i in range(2) if r < len(steps[i])]
            ctx = spans(device, [steps[i][r][1] for i in live], [slots[i] for i in live])
            y = torch.cat([x[i][steps[i][r][0]: sum(steps[i][r])] for i in live]).to(device)
            out = ops.delta_conv(ctx, y, channels, w.to(device), tail, segments, 0.0, activation=None).cpu()
            for i, piece in zip(live, out.split([steps[i][r][1] for i in live])):
                got[i].append(piece)
        for i in range(2):
            torch.testing.assert_close(torch.cat(got[i]).double(), want[i], atol=3e-5, rtol=3e-5)


def attention_sizes(nq, nkv, d, dv, window, conv, dims, base, scale=None):
    return {"heads": nq, "kv_heads": nkv, "dim": d, "vdim": dv, "scale": scale or 2.5 / math.sqrt(d), "mask": {"size": window},
            "conv": conv, "rot": {"dims": dims, "base": base}}


def attention_weights(width, s, seed=0):
    nq, nkv, d, dv = s["heads"], s["kv_heads"], s["dim"], s["vdim"]
    w = {"o": rnd(width, nq * dv, seed=seed + 7, scale=0.3)}
    for i, (n, rows) in enumerate((("q", nq * d), ("k", nkv * d), ("v", nkv * dv))):
        w[n] = rnd(rows, width, seed=seed + 1 + i, scale=0.3)
        w[n + ".conv"] = rnd(rows, s["conv"], seed=seed + 11 + i, scale=0.5)
    return w


def attention_mixer(width, s, eps, w, device, dt):
    from qwen3_runtime_amd.parts.attention import GroupedQueryAttention
    from qwen3_runtime_amd.parts.plan import PartSpec

    names = {n: n for n in ("q", "k", "v", "o")} | {f"{n}_conv": f"{n}.conv" for n in ("q", "k", "v")}
    rot = s["rot"]
    mixer = GroupedQueryAttention(
        width, s["heads"], s["kv_heads"], s["dim"], qk_norm_eps=eps, qk_norm_weight=False, scale=s["scale"], value_dim=s["vdim"],
        window=s["mask"]["size"], conv=s["conv"], neighbour_pairs=True, tensors=names,
        position=PartSpec("rope_half", {"head_dim": s["dim"], "dims": rot["dims"], "base": rot["base"]}) if rot["dims"] else None)
    for child in mixer.children():
        child.load(DictFetch(w, device, dt))
    mixer.load(DictFetch(w, device, dt))
    return mixer


ATTENTION = [
    (4, 2, 32, 32, 40, 4, 32, 1000.0, 16),
    (6, 2, 16, 48, 21, 3, 8, 100.0, 8),       # values wider than keys, on the matrix cores
    (6, 2, 128, 64, 54, 4, 64, 2e5, 16),      # the one-kernel decode form with narrower values
    (4, 2, 64, 64, 65, 2, 64, 1e4, 16),       # ... with values as wide as keys
    (8, 2, 64, 128, 33, 4, 0, 1.0, 32),       # no rotation, wider values
    (3, 1, 128, 64, 45, 3, 48, 3e4, 16),      # too few pairs turn for the one-kernel form
    (3, 1, 48, 48, 9, 1, 20, 50.0, 8),        # one tap, an odd number of 16-wide blocks, a small window
    (5, 5, 8, 6, 1, 5, 2, 10.0, 8),           # a window of the query itself; tiny heads
    (2, 1, 256, 16, 50, 4, 128, 1e5, 16),
    (3, 3, 50, 34, 17, 6, 10, 40.0, 8),       # sizes that are multiples of nothing
    (2, 1, 80, 48, 30, 4, 16, 1e3, 8),
    (16, 1, 64, 16, 64, 3, 64, 1e4, 16),      # as many query heads a key head as a tile has rows
]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("nq,nkv,d,dv,window,conv,dims,base,page", ATTENTION)
def test_attention_behind_convolutions_over_a_window(backend, nq, nkv, d, dv, window, conv, dims, base, page):
    """The mixer (convolutions, neighbour pairs turned, heads over their root mean square) over pages that
    go back to the pool behind the window, its projected values in a slot. One token's value is large, so
    that whether a query sees it shows; queries pass its window's edge one by one and inside a portion."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, eps = 56, 1e-5
    t = 3 * window + 60
    s = attention_sizes(nq, nkv, d, dv, window, conv, dims, base)
    w = rounded(attention_weights(width, s), dt)
    h = rnd(t, width, seed=8)
    marked = t - window - 25
    h[marked] *= 8.0
    h = h.to(dt).float()
    want = P.attention(h.double(), f64(w), s, eps)
    edge = marked + window  # the first query that no longer sees the marked token's key
    pages = -(-(window + 64) // page) + 2
    for cuts in (in_steps(edge - 3, (64, 5)) + [(p, 1) for p in range(edge - 3, edge + 4)] + [(edge + 4, t - edge - 4)],
                 in_steps(edge - 10, (7, 2, 30)) + [(edge - 10, 20)] + in_steps(t, (1,), edge + 10)):
        driver = MixerDriver(attention_mixer(width, s, eps, w, device, dt), device, dt, ops, page, pages)
        for st in driver.cache._state_of_cache.values():
            st.fill_(float("nan"))  # a slot is zeroed when it is taken
        got = driver.run("a", h, cuts)
        assert driver.cache.groups[0].pool.num_free == pages
        assert_rows(got, want, dtype)
    # what would show if it were missing: the window one token off, the turn, the convolutions' order
    limit = 5 * float(row_bound(want, "float32").max())
    if window > 1:
        for other in (window - 1, window + 1):
            off = P.attention(h.double(), f64(w), {**s, "mask": {"size": other}}, eps)
            assert (off - want).abs().amax(1).max() > limit
        if dims:
            off = P.attention(h.double(), f64(w), {**s, "rot": {"dims": dims, "base": base * 1.5}}, eps)
            assert dims == 2 or (off - want).abs().amax(1).max() > limit
    if conv > 1:
        off = P.attention(h.double(), f64({n: x.flip(1) if n.endswith("conv") else x for n, x in w.items()}), s, eps)
        assert (off - want).abs().amax(1).max() > limit


@pytest.mark.parametrize("backend", BACKENDS)
def test_two_requests_share_a_mixer_s_steps(backend):
    """Portions of one beside single tokens of the other; then their slots and pages are taken by a third."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, eps = 40, 1e-5
    s = attention_sizes(4, 2, 64, 32, 23, 4, 64, 500.0)
    w = rounded(attention_weights(width, s, seed=3), dt)
    h = [rnd(n, width, seed=n).to(dt).float() for n in (90, 40, 61)]
    want = [P.attention(x.double(), f64(w), s, eps) for x in h]
    driver = MixerDriver(attention_mixer(width, s, eps, w, device, dt), device, dt, ops, 8, 30)
    driver.admit("a"), driver.admit("b")
    plan = {"a": in_steps(90, (25, 1, 30)), "b": in_steps(40, (1, 2, 20))}
    outs = {"a": [], "b": []}
    for i in range(max(map(len, plan.values()))):
        live = [r for r in ("b", "a") if i < len(plan[r])]
        for r, o in zip(live, driver.step([(r, h["ab".index(r)][plan[r][i][0]: sum(plan[r][i])]) for r in live])):
            outs[r].append(o)
    for j, r in enumerate("ab"):
        assert_rows(torch.cat(outs[r]), want[j], dtype, r)
    driver.release("a"), driver.release("b")
    assert_rows(driver.run("c", h[2], in_steps(61, (1, 1, 9))), want[2], dtype, "a slot taken again")


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("nq,nkv,d,dv,window,dims", [(4, 2, 128, 64, 4000, 64), (2, 1, 32, 80, 4000, 16), (8, 2, 128, 128, 1300, 64), (2, 2, 16, 48, 1100, 16)])
def test_values_of_another_size_over_long_contexts(backend, nq, nkv, d, dv, window, dims):
    """Contexts long enough that keys are cut over blocks whose parts are merged (decoded tokens, few-row
    portions beside long ones), long portions that share keys through LDS, and two requests at once. A token
    a thousand positions back stands out."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, eps, t = 40, 1e-5, 1240
    s = attention_sizes(nq, nkv, d, dv, window, 4, dims, 1e4, scale=1.0 / math.sqrt(d))
    w = rounded(attention_weights(width, s), dt)
    h = rnd(t, width, seed=5)
    h[2] *= 60.0
    h = [h.to(dt).float(), rnd(300, width, seed=6).to(dt).float()]
    want = [P.attention(x.double(), f64(w), s, eps) for x in h]
    driver = MixerDriver(attention_mixer(width, s, eps, w, device, dt), device, dt, ops, 16, 110)
    driver.admit("a"), driver.admit("b")
    got = {"a": [driver.step([("a", h[0][:1216])])[0]], "b": []}
    for i in range(24):  # single tokens over a long context, alone and beside a portion
        spans_ = [("a", h[0][1216 + i: 1217 + i])]
        if i % 2:
            spans_.append(("b", h[1][25 * (i // 2): 25 * (i // 2 + 1)]))
        for (rid, _), out in zip(spans_, driver.step(spans_)):
            got[rid].append(out)
    for j, rid in enumerate("ab"):
        assert_rows(torch.cat(got[rid]), want[j], dtype, rid)


def test_attention_options_that_do_not_go_together():
    from qwen3_runtime_amd.parts.attention import GroupedQueryAttention
    from qwen3_runtime_amd.parts.plan import PartSpec

    names = {n: n for n in ("q", "k", "v", "o", "g", "q_norm", "k_norm")}
    with pytest.raises(ValueError):
        GroupedQueryAttention(32, 2, 1, 16, conv=17, tensors=names)
    with pytest.raises(NotImplementedError):
        GroupedQueryAttention(32, 2, 1, 16, conv=4, bias=True, tensors=names)
    with pytest.raises(ValueError):
        GroupedQueryAttention(32, 2, 1, 16, neighbour_pairs=True, tensors=names,
                              position=PartSpec("rope_pairs", {"head_dim": 16, "dims": 8, "base": 10.0}))


@pytest.mark.parametrize("backend", BACKENDS)
def test_neighbour_pairs_with_norm_weights_and_biases(backend):
    """The order of a head's elements is brought over for everything that is stored per element: biases and
    norm weights too (norm, with weights, in front of the turn)."""
    from qwen3_runtime_amd.parts.attention import GroupedQueryAttention
    from qwen3_runtime_amd.parts.plan import PartSpec

    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, nq, nkv, d, t, dims, base, eps = 48, 4, 2, 32, 40, 12, 100.0, 1e-5
    w = {n: rnd(rows, width, seed=i, scale=0.3) for i, (n, rows) in enumerate((("q", nq * d), ("k", nkv * d), ("v", nkv * d)))}
    w |= {n + "_bias": rnd(w[n].shape[0], seed=7 + i) for i, n in enumerate("qkv")}
    w |= {"o": rnd(width, nq * d, seed=5, scale=0.3), "q_norm": 1 + rnd(d, seed=11, scale=0.4), "k_norm": 1 + rnd(d, seed=12, scale=0.4)}
    w = rounded(w, dt)
    mixer = GroupedQueryAttention(width, nq, nkv, d, qk_norm_eps=eps, bias=True, neighbour_pairs=True, tensors={n: n for n in w},
                                  position=PartSpec("rope_half", {"head_dim": d, "dims": dims, "base": base}))
    mixer.position.load(DictFetch(w, device, dt))
    mixer.load(DictFetch(w, device, dt))
    h = rnd(t, width, seed=20).to(dt).float()
    x, v64 = h.double(), f64(w)
    q, k, v = ((x @ v64[n].T + v64[n + "_bias"]).view(t, -1, d) for n in "qkv")
    q = P.rotate_neighbours(P.rms_norm(q, eps) * v64["q_norm"], dims, base)
    k = P.rotate_neighbours(P.rms_norm(k, eps) * v64["k_norm"], dims, base).repeat_interleave(nq // nkv, 1)
    scores = torch.einsum("qhd,khd->hqk", q, k) / math.sqrt(d)
    scores = scores.masked_fill(torch.arange(t)[None, :] > torch.arange(t)[:, None], float("-inf"))
    want = torch.einsum("hqk,khd->qhd", scores.softmax(-1), v.repeat_interleave(nq // nkv, 1)).reshape(t, -1) @ v64["o"].T
    driver = MixerDriver(mixer, device, dt, ops, 16, 8)
    assert_rows(driver.run("a", h, in_steps(t, (17, 1, 1, 9))), want, dtype)


# ------------------------------------------------------------------ the matrix memory
def gate_logits(t, heads, seed):
    z = rnd(t, 2 * heads, seed=seed, scale=3.0)
    z[:, heads:] += 2.0
    z[t // 3] = 80.0           # far beyond the cap, both gates
    z[t // 2, :heads], z[t // 2, heads:] = -90.0, -70.0
    return z


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,cap", [(4, 15.0), (1, 3.0), (7, 30.0), (32, 0.5)])
def test_gates_and_their_running_maximum(backend, heads, cap):
    """Two sequences in slots 3 and 0: long spans (many tiles of 64 tokens, more than a round of them), single
    tokens, single tokens beside a long span, from the maximum the slot holds. The logarithms are those of the
    rule written out; what a token keeps and writes never exceeds 1."""
    device, _ = backend
    ops = make_ops(device)
    t = 90 if device == "cpu" else 2500
    z, bias = [gate_logits(n, heads, seed=n) for n in (t, t // 2)], rnd(2 * heads, seed=3)
    want = []
    for x in z:
        c = P.soft_cap(x.double() + bias.double(), cap)
        li, lf, m, rows = c[:, :heads], P.log_sigmoid(c[:, heads:]), torch.zeros(heads, dtype=torch.float64), []
        for i in range(x.shape[0]):
            top = torch.maximum(lf[i] + m, li[i])
            rows.append(torch.stack([lf[i] + m - top, li[i] - top, top]))
            m = top
        want.append(torch.stack(rows))
    for sizes in ((t,), (1, 70, 1, 3), (1100, 1, 65, 64), (63, 2)):
        top = torch.full((4, heads), float("nan"), device=device)
        top[3] = top[0] = 0.0
        steps = [in_steps(x.shape[0], sizes if i == 0 else sizes[::-1]) for i, x in enumerate(z)]
        got = [[], []]
        for r in range(max(map(len, steps))):
            live = [i for i in range(2) if r < len(steps[i])]
            ctx = spans(device, [steps[i][r][1] for i in live], [(3, 0)[i] for i in live])
            x = torch.cat([z[i][steps[i][r][0]: sum(steps[i][r])] for i in live]).to(device)
            out = ops.memory_gates(ctx, x, bias.to(device), cap, top, heads).cpu()
            for i, piece in zip(live, out.split([steps[i][r][1] for i in live])):
                got[i].append(piece)
        for i in range(2):
            mine = torch.cat(got[i])
            torch.testing.assert_close(mine.double(), want[i], atol=1e-4, rtol=1e-5)
            assert float(mine[:, :2].max()) < 1e-5
            torch.testing.assert_close(top[(3, 0)[i]].cpu(), mine[-1, 2])
        assert torch.isnan(top[1]).all() and torch.isnan(top[2]).all()


MEMORY = [(4, 16, 24), (3, 56, 40), (2, 128, 128), (1, 1, 1), (5, 20, 7), (2, 100, 3), (8, 64, 16), (1, 256, 64), (1, 512, 8), (2, 40, 200), (4, 32, 8)]


def memory_inputs(t, heads, d, dv, seed):
    return rnd(t, heads, d, seed=seed), rnd(t, heads, d, seed=seed + 1), rnd(t, heads, dv, seed=seed + 2)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,d,dv", MEMORY)
def test_matrix_memory_recurrence_against_the_rule_written_out(backend, heads, d, dv):
    """Gates, memory and read-out together: a whole span, portions down to one token with the state in its
    slot, a second sequence of another length beside the first. With bfloat16 inputs long spans go chunk by
    chunk; the short spans of the same step go token by token beside them. Columns behind q | k | v are the
    output gate's."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    t, cap, eps = (40 if device == "cpu" else 330), 15.0, 1e-5
    q, k, v = (x.to(dt).float() for x in memory_inputs(t, heads, d, dv, seed=heads + d))
    g = rnd(t, heads * dv, seed=50).to(dt).float()
    z, bias, weight = gate_logits(t, heads, seed=9), rnd(2 * heads, seed=4), 1 + rnd(heads * dv, seed=5, scale=0.3)
    c = P.soft_cap(z.double() + bias.double(), cap)
    o = P.matrix_memory(q.double() * d ** -0.5, k.double(), v.double(), c[:, :heads], P.log_sigmoid(c[:, heads:]))
    want = P.rms_norm(o, eps).reshape(t, -1) * weight.double() * torch.sigmoid(g.double())
    rows = torch.cat([x.reshape(t, -1) for x in (q, k, v, g)], 1).to(dt).to(device)
    other = torch.cat([x.reshape(t, -1) for x in memory_inputs(t, heads, d, dv, seed=99)] + [g], 1).to(dt).to(device)
    zd = z.to(device)
    for sizes in ((t,), (37, 2, 1, 1, 16, 5), (130, 3, 64), (64, 65))[: 2 if device == "cpu" else 4]:
        state = torch.full((4, heads, dv + 1, d), float("nan"), device=device)
        top = torch.full((4, heads), float("nan"), device=device)
        state[3], state[1], top[3], top[1] = 0.0, 0.0, 0.0, 0.0
        got = []
        for at, n in in_steps(t, sizes):
            m = 1 + at % min(n, 4) if len(sizes) > 2 else n   # beside a span of another length
            ctx = spans(device, [m, n], [1, 3])
            both = torch.cat([other[at: at + m], rows[at: at + n]]).contiguous()
            gates = ops.memory_gates(ctx, torch.cat([zd[at: at + m], zd[at: at + n]]), bias.to(device), cap, top, heads)
            read, floor = ops.matrix_memory(ctx, both, gates, state, heads, d, dv)
            out = ops.memory_out(read, floor, gates, weight.to(device), both[:, 2 * heads * d + heads * dv:], eps, d ** -0.5, dt)
            got.append(out.float().cpu()[m:])
        got = torch.cat(got)
        if dtype == "float32":
            # a read-out over a sum of keys that happens to cancel is judged against what it is made of
            torch.testing.assert_close(got.double(), want, atol=5e-4, rtol=5e-4)
        else:
            assert_rows(got, want, dtype)
        assert torch.isnan(state[0]).all() and torch.isnan(state[2]).all()  # other slots are left alone


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("d,dv", [(16, 24), (128, 64), (64, 16)])
def test_a_write_from_far_back_is_read_and_a_slot_taken_again_is_empty(backend, d, dv):
    """A head that forgets next to nothing: a marker written along a direction of its own 400 tokens back,
    across many portions, fills the read-out; a second head forgets fast and has nothing of it left. With
    state and maximum zeroed, as when a slot is taken again, only the token's own write is read."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    t, heads, cap = 420, 2, 20.0
    unit = lambda x: x / x.norm(dim=-1, keepdim=True)  # noqa: E731
    v, k = rnd(t, heads, dv, seed=2), unit(rnd(t, heads, d, seed=3))
    direction = unit(rnd(d, seed=77))
    k = k - (k @ direction)[..., None] * direction
    k[5], v[5] = direction, 9.0
    q = torch.zeros(t, heads, d)
    q[-1, 0], q[-1, 1] = direction, k[-1, 1]
    q, k, v = (x.to(dt).float() for x in (q, k, v))
    z = torch.zeros(t, 2 * heads)
    z[:, 2], z[:, 3] = 12.0, -30.0
    bias, ones = torch.zeros(2 * heads), torch.ones(heads * dv)
    c = P.soft_cap(z.double(), cap)
    o = P.matrix_memory(q.double(), k.double(), v.double(), c[:, :2], P.log_sigmoid(c[:, 2:]))
    rows = torch.cat([x.reshape(t, -1) for x in (q, k, v)], 1).to(dt).to(device)
    gate = torch.full((t, heads * dv), 30.0, dtype=dt, device=device)
    state, top = torch.zeros(2, heads, dv + 1, d, device=device), torch.zeros(2, heads, device=device)

    def run(at, n):
        ctx = spans(device, [n], [1])
        gates = ops.memory_gates(ctx, z[at: at + n].to(device), bias.to(device), cap, top, heads)
        read, floor = ops.matrix_memory(ctx, rows[at: at + n].contiguous(), gates, state, heads, d, dv)
        return read.cpu(), ops.memory_out(read, floor, gates, ones.to(device), gate[at: at + n], 1e-12, 1.0, torch.float32 if dtype == "float32" else dt).float().cpu()

    read = [run(at, n) for at, n in in_steps(t, (64, 3, 1, 150, 2))][-1]
    got = read[1][-1].view(heads, dv)
    want = P.rms_norm(o[-1], 1e-12)
    torch.testing.assert_close(got.double(), want, **(dict(atol=1e-3, rtol=1e-3) if dtype == "float32" else dict(atol=2e-2, rtol=2e-2)))
    # the first head reads the marker's value in every channel, the second its own token's value
    assert float((want[0] - 1.0).abs().max()) < 0.1
    own = P.rms_norm(v[-1, 1].double(), 1e-12)
    assert float((want[1] - own).abs().max()) < 0.05
    state[1], top[1] = 0.0, 0.0
    again = run(t - 1, 1)[1][0].view(heads, dv)
    torch.testing.assert_close(again[1].double(), own, atol=2e-2, rtol=2e-2)
    before = read[0][-1, 0].abs().max()
    assert float(run(t - 1, 1)[0][0, 0].abs().max()) < 0.05 * float(before)  # nothing of the marker is left


@pytest.mark.parametrize("backend", BACKENDS)
def test_a_small_read_out_is_held_by_the_maximum(backend):
    """Where the keys' weighted sum nearly cancels against the query, exp(-m) stands in its place: the floor
    decides how far below the norm's eps a read-out falls. Large eps makes that visible."""
    device, dtype = backend
    ops = make_ops(device)
    t, heads, dv = 6, 3, 20
    read, floor = rnd(t, heads, dv, seed=1), rnd(t, heads, seed=2) * torch.tensor([1e-6, 1.0, 40.0])
    gates = torch.stack([torch.zeros(t, heads), torch.zeros(t, heads), rnd(t, heads, seed=3, scale=3.0)], 1)
    weight, g, eps, scale = 1 + rnd(heads * dv, seed=4), rnd(t, heads * dv, seed=5), 0.7, 0.3
    low = torch.maximum((floor.double() * scale).abs(), torch.exp(-gates[:, 2].double())) + 1e-6
    want = P.rms_norm(read.double() * scale / low[..., None], eps).reshape(t, -1) * weight.double() * torch.sigmoid(g.double())
    dev = lambda x: x.to(device)  # noqa: E731
    got = ops.memory_out(dev(read), dev(floor), dev(gates.contiguous()), dev(weight), dev(g), eps, scale, torch.float32)
    torch.testing.assert_close(got.cpu().double(), want, atol=1e-5, rtol=1e-5)


def memory_weights(width, heads, d, dv, seed=0):
    s = width ** -0.5
    w = {"q": rnd(heads * d, width, seed=seed + 1, scale=s), "k": rnd(heads * d, width, seed=seed + 2, scale=s),
         "v": rnd(heads * dv, width, seed=seed + 3, scale=s), "g": rnd(heads * dv, width, seed=seed + 4, scale=s),
         "i": rnd(heads, width, seed=seed + 5, scale=2 * s), "f": rnd(heads, width, seed=seed + 6, scale=2 * s),
         "i.b": rnd(heads, seed=seed + 7), "f.b": 2 + rnd(heads, seed=seed + 8), "norm": 1 + rnd(heads * dv, seed=seed + 9, scale=0.3)}
    return w | {"o": rnd(width, heads * dv, seed=seed + 10, scale=(heads * dv) ** -0.5)}


def memory_mixer(width, heads, d, dv, cap, eps, w, device, dt):
    from qwen3_runtime_amd.parts.memory import MatrixMemory

    names = {n: n for n in ("q", "k", "v", "g", "i", "f", "norm", "o")} | {"i_bias": "i.b", "f_bias": "f.b"}
    mixer = MatrixMemory(width, heads, d, dv, cap, eps, tensors=names)
    mixer.load(DictFetch(w, device, dt))
    return mixer


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,d,dv,cap", [(4, 16, 24, 15.0), (3, 40, 16, 2.0), (2, 128, 64, 15.0), (1, 7, 10, 5.0), (6, 64, 64, 30.0)])
def test_matrix_memory_mixer(backend, heads, d, dv, cap):
    """The whole mixer with its state in a slot: a prompt at once, portions down to one token, two requests in
    the same steps whose slots are then taken again by others."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, eps = 48, 1e-5
    t = 60 if device == "cpu" else 200
    w = memory_weights(width, heads, d, dv)
    if dtype == "bfloat16":
        w["k"] = alike(w["k"], w["q"])
    w = rounded(w, dt)
    sizes = {"heads": heads, "dim": d, "vdim": dv, "gate_cap": cap}
    h = [rnd(n, width, seed=8 + n).to(dt).float() for n in (t, t // 2)]
    want = [P.mlstm(x.double(), f64(w), sizes, eps) for x in h]
    driver = MixerDriver(memory_mixer(width, heads, d, dv, cap, eps, w, device, dt), device, dt, ops, 16, 1, max_requests=3)
    for st in driver.cache._state_of_cache.values():
        st.fill_(float("nan"))  # a slot is zeroed when it is taken
    driver.admit("other")  # slot 0 is somebody else's
    assert_rows(driver.run("a", h[0], [(0, t)]), want[0], dtype, "whole")
    assert_rows(driver.run("a", h[0], in_steps(t, (17, 1, 2, 1, 1, 30, 3))), want[0], dtype, "portions")
    driver.admit("a"), driver.admit("b")
    outs = {"a": [], "b": []}
    plan = {"a": in_steps(t, (25, 1, 64)), "b": in_steps(t // 2, (1, 2, 40))}
    for i in range(max(map(len, plan.values()))):
        live = [r for r in ("b", "a") if i < len(plan[r])]
        res = driver.step([(r, h["ab".index(r)][plan[r][i][0]: sum(plan[r][i])]) for r in live])
        for r, o in zip(live, res):
            outs[r].append(o)
    for j, r in enumerate("ab"):
        assert_rows(torch.cat(outs[r]), want[j], dtype, r)
    driver.release("a"), driver.release("b")
    assert_rows(driver.run("c", h[1], in_steps(t // 2, (5, 1))), want[1], dtype, "a slot taken again")
    # the gates' caps, biases and the order of the two are in what is compared
    limit = 5 * float(row_bound(want[0], "float32").max())
    for fault in ({"gate_cap": cap * 0.5},):
        assert (P.mlstm(h[0].double(), f64(w), {**sizes, **fault}, eps) - want[0]).abs().max() > limit
    swapped = {**w, "i": w["f"], "f": w["i"]}
    assert (P.mlstm(h[0].double(), f64(swapped), sizes, eps) - want[0]).abs().max() > limit


# ------------------------------------------------------------------ feed-forwards
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,ff,activation", [(128, 96, "clamped"), (256, 320, "swiglu"), (96, 40, "clamped"), (50, 33, "swiglu"), (320, 80, "clamped")])
def test_gated_products_with_a_clamp_and_a_factor_per_token(backend, width, ff, activation):
    """Every way the gated product runs (few rows, rows shared through LDS, the library's product and the
    activation behind it), clamped or not, with and without a factor per row."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    limit = 0.8
    w = rnd(2 * ff, width, seed=1, scale=1.5 * width ** -0.5).to(dt)
    for t in (1, 7, 13, 16, 40, 128, 200):
        x, f = rnd(t, width, seed=t).to(dt), torch.rand(t, generator=torch.Generator().manual_seed(t))
        g, u = (x.double() @ w.double().T).split(ff, dim=1)
        if activation == "clamped":
            assert (g > limit).any() and (u.abs() > limit).any()
            g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
            want = g * torch.sigmoid(1.702 * g) * (u + 1)
        else:
            want = g * torch.sigmoid(g) * u
        for scale in (None, f):
            got = ops.gated_linear(x.to(device), w.to(device), activation, limit, row_scale=None if scale is None else scale.to(device))
            torch.testing.assert_close(got.float().cpu().double(), want if scale is None else want * scale.double()[:, None], **close(dtype))


@pytest.mark.parametrize("backend", BACKENDS)
def test_clamped_dense_feed_forward(backend):
    from qwen3_runtime_amd.parts.mlp import SwiGLU

    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, ff, limit = 72, 120, 0.6
    w = rounded({n: rnd(*((width, ff) if n == "down" else (ff, width)), seed=i, scale=0.15) for i, n in enumerate(("gate", "up", "down"))}, dt)
    part = SwiGLU(width, ff, activation="clamped", limit=limit, tensors={n: n for n in w})
    part.load(DictFetch(w, device, dt))
    for t in (1, 9, 70, 300):
        x = rnd(t, width, seed=t, scale=2.0).to(dt)
        got = part.forward(SimpleNamespace(ops=ops, num_tokens=t, dtype=dt), x.to(device))
        got = (got.sum(0) if got.dim() == 3 else got).float().cpu()
        assert_rows(got, P.clamped(x.double(), f64(w), limit), dtype, f"{t} tokens")
    with pytest.raises(ValueError):
        SwiGLU(width, ff, activation="relu2", tensors={})


def mixture_weights(width, ff, experts, shared, seed=0):
    w = {"router": rnd(experts, width, seed=seed + 1, scale=0.3), "correction": rnd(experts, seed=seed + 2, scale=0.3)}
    for e in range(experts):
        for j, n in enumerate(("gate", "up")):
            w[f"e{e}.{n}"] = rnd(ff, width, seed=seed + 10 + 3 * e + j, scale=width ** -0.5)
        w[f"e{e}.down"] = rnd(width, ff, seed=seed + 12 + 3 * e, scale=ff ** -0.5)
    for j, n in enumerate(("gate", "up", "down") if shared else ()):
        w[f"shared.{n}"] = rnd(*((width, shared) if n == "down" else (shared, width)), seed=seed + 5 + j, scale=0.2)
    if shared:
        w["shared.sg"] = rnd(1, width, seed=seed + 9, scale=0.3)
    return w


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,ff,experts,top,scale,shared", [
    (48, 40, 6, 2, 2.0, 56), (64, 24, 10, 3, 1.0, 0), (40, 56, 4, 4, 0.5, 24), (72, 16, 5, 1, 3.0, 32), (50, 18, 3, 2, 1.7, 10),
    (128, 64, 16, 2, 1.0, 128), (160, 72, 40, 3, 2.5, 64)])
def test_mixture_with_a_gated_shared_expert(backend, width, ff, experts, top, scale, shared):
    """Router, experts and shared expert at every step size (one token, a few, tens, hundreds: pair by pair,
    expert by expert on the device, expert by expert through the engine's products). The correction turns
    choices and no weight; the shared expert opens by a number of the token's own."""
    from qwen3_runtime_amd.parts.moe import RoutedSwiGLU

    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    w = rounded(mixture_weights(width, ff, experts, shared), dt)
    names = {"router": "router", "correction": "correction", "gate": "e{e}.gate", "up": "e{e}.up", "down": "e{e}.down"}
    names |= {f"shared_{n}": f"shared.{n}" for n in ("gate", "up", "down", "sg")} if shared else {}
    part = RoutedSwiGLU(width, ff, experts, top, router_bias=False, scoring="sigmoid", correction=True, renormalise=True,
                        weight_scale=scale, shared_size=shared or None, shared_gate=bool(shared), tensors=names)
    part.load(DictFetch(w, device, dt))
    w64, mlp = f64(w), {"router": {"top": top, "scale": scale}, "shared": {"ff": shared} if shared else None}
    for t in (1, 3, 17, 70, 300) if device != "cpu" else (1, 17, 70):
        x = rnd(t, width, seed=t, scale=2.0).to(dt)
        # rows whose choice 8 bits of the scores could turn are not judged
        s = (torch.sigmoid(x.double() @ w64["router"].T) + w64["correction"]).sort(-1, descending=True).values
        clear = torch.ones(t, dtype=torch.bool) if top == experts else (s[:, top - 1] - s[:, top]) > 1e-4
        got = part.forward(SimpleNamespace(ops=ops, num_tokens=t, dtype=dt), x.to(device))
        got = (got.sum(0) if got.dim() == 3 else got).float().cpu()
        want = P.mixture(x.double(), w64, mlp)
        if clear.any():
            assert_rows(got[clear], want[clear], dtype, f"{t} tokens")
    limit = 50 * float(row_bound(want, "float32").max())
    if top < experts:
        assert (P.mixture(x.double(), {**w64, "correction": torch.zeros(experts, dtype=torch.float64)}, mlp) - want).abs().max() > limit
    if shared:
        assert (P.mixture(x.double(), {**w64, "shared.sg": torch.zeros_like(w64["shared.sg"])}, mlp) - want).abs().max() > limit


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,experts", [(64, 5), (2560, 16), (50, 33), (4100, 3)])
def test_the_router_s_gate_row(backend, width, experts):
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    x, w = rnd(9, width, seed=1).to(dt), rnd(experts + 1, width, seed=2, scale=width ** -0.5)
    index, weight, gate = ops.route_top(x.to(device), w.to(device), None, 2, scoring="sigmoid", gate_row=True)
    plain_index, plain_weight = ops.route_top(x.to(device), w[:-1].contiguous().to(device), None, 2, scoring="sigmoid")
    assert torch.equal(index, plain_index) and torch.equal(weight, plain_weight)  # the row is no expert
    torch.testing.assert_close(gate.cpu().double(), torch.sigmoid(x.double() @ w[-1].double()), atol=1e-5, rtol=1e-5)


# ------------------------------------------------------------------ whole models
def memory(heads, d, dv, cap):
    return "mlstm", {"heads": heads, "dim": d, "vdim": dv, "gate_cap": cap}


def attention(nq, nkv, d, dv, scale, window, conv, dims, base):
    return "attention", attention_sizes(nq, nkv, d, dv, window, conv, dims, base, scale)


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff, experts, top, scale, shared):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale},
            **({"shared": {"ff": shared}} if shared else {})}


def model(vocab, width, eps, mult, pairs, loop, layers):
    raw = {"architecture": "Dekinex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
           "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), pairs))},
           "layers": [{"type": kind, "mixer": mixer, "mlp": mlp} for (kind, mixer), mlp in layers]}
    if loop:
        raw["loop"] = dict(zip(("start", "stop", "times"), loop))
    return raw


def config_a():
    """Both mixers, all feed-forwards, a span in the middle run three times; keys and values of different sizes."""
    return model(210, 80, 1e-5, 0.8, (67, 31, 7), (1, 3, 3), [
        (memory(4, 24, 16, 8.0), dense(72, 0.9)),
        (attention(6, 2, 32, 16, 0.3, 13, 4, 24, 500.0), moe(24, 10, 3, 1.5, 40)),
        (memory(3, 40, 24, 15.0), None),
        (attention(4, 4, 16, 16, 0.4, 22, 3, 16, 3000.0), moe(40, 6, 2, 0.6, 0)),
    ]), 16


def config_b():
    """A span at the start run twice; one expert a token; all experts a token; multiplier one."""
    return model(150, 64, 1e-6, 1.0, (8, 1, 3), (0, 2, 2), [
        (attention(2, 1, 48, 48, 0.25, 9, 2, 20, 50.0), moe(32, 5, 1, 1.0, 16)),
        (memory(2, 32, 8, 4.0), dense(40, 2.0)),
        (memory(6, 8, 40, 15.0), moe(48, 4, 4, 2.0, 24)),
    ]), 8


def config_c():
    """Attention alone, windows all round, the last layers looped: nothing grows with the length."""
    return model(97, 48, 1e-5, 0.5, (500, 11, 13), (1, 3, 2), [
        (attention(2, 2, 16, 8, 0.4, 17, 4, 4, 20.0), moe(16, 4, 2, 1.3, 8)),
        (attention(6, 3, 8, 16, 0.5, 6, 2, 8, 100.0), None),
        (attention(3, 1, 16, 16, 0.35, 11, 5, 0, 1.0), dense(24, 1.1)),
    ]), 8


def config_d():
    """Sizes that are multiples of nothing; a loop of one pass."""
    return model(131, 50, 1e-5, 1.3, (19, 5, 2), (0, 3, 1), [
        (memory(3, 7, 10, 6.0), moe(18, 3, 2, 1.0, 11)),
        (attention(3, 1, 10, 14, 0.5, 7, 3, 6, 30.0), dense(33, 0.7)),
        (memory(5, 9, 6, 3.0), moe(10, 5, 2, 2.2, 0)),
    ]), 8


def config_e():
    """Matrix memories alone: no page of cache; no loop."""
    return model(120, 72, 1e-5, 0.9, (1, 4, 9), None, [
        (memory(4, 32, 16, 12.0), dense(64, 1.5)),
        (memory(2, 20, 40, 20.0), moe(24, 7, 2, 1.0, 32)),
    ]), 16


def config_g():
    """Layers of a real model's proportions, narrow: heads of 64 and 128, memories of 128 x 64."""
    return model(500, 256, 1e-6, 0.7, (509, 61, 23), (1, 2, 2), [
        (memory(4, 128, 64, 15.0), dense(512, 3.0)),
        (attention(4, 2, 128, 64, 0.2, 100, 4, 64, 1e4), moe(128, 8, 2, 1.0, 128)),
        (memory(4, 64, 128, 15.0), moe(128, 8, 2, 2.0, 128)),
        (attention(8, 2, 64, 64, 0.25, 150, 4, 64, 1e4), moe(128, 8, 2, 1.0, 128)),
    ]), 16


CONFIGS = {"a": config_a, "b": config_b, "c": config_c, "d": config_d, "e": config_e, "g": config_g}
LENGTHS = {"a": [70, 1, 23], "b": [64, 40, 2], "c": [90, 5], "d": [37, 20], "e": [60, 3, 31], "g": [330, 40]}
NOISE = {name: 0.2 for name in CONFIGS}


def for_dtype(raw, dtype):
    """A model for runs in bfloat16 takes every expert for every token: with fewer, one chosen on a close
    call that 8 bits turn would move that position's logits by a large part of their spread. The choice
    by scores is held to the plain one in float32 here, and in both types in the mixture's own test."""
    if dtype == "bfloat16":
        for layer in raw["layers"]:
            if layer["mlp"] and layer["mlp"]["kind"] == "moe":
                layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return raw


def alike(keys, queries):
    """Keys of a matrix memory that resemble its queries, for runs in bfloat16: with keys and queries that
    have nothing in common the sums over a few of them cancel, a read-out is then the sign of next to
    nothing times a value, and the plain model itself turns it when its activations are rounded to 8 bits."""
    return (0.8 * queries.float() + 0.6 * keys.float()).to(keys.dtype)


@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    """Model folders with random weights, written once per configuration and type."""
    from safetensors.torch import load_file, save_file

    from qwen3_runtime_amd.weights import write_model_folder

    made = {}

    def get(name, dtype="float32"):
        if (name, dtype) not in made:
            raw = for_dtype(CONFIGS[name]()[0], dtype)
            made[(name, dtype)] = write_model_folder(tmp_path_factory.mktemp("dekinex_" + name), raw, seed=60 + sorted(CONFIGS).index(name),
                                                     std=0.06 if name == "g" else 0.12, norm_jitter=0.2)
            if dtype == "bfloat16":
                path = str(made[(name, dtype)] / "model.safetensors")
                w = load_file(path)
                for i, layer in enumerate(raw["layers"]):
                    if layer["type"] == "mlstm":
                        w[f"l{i}.mix.k"] = alike(w[f"l{i}.mix.k"], w[f"l{i}.mix.q"])
                save_file(w, path)
        return made[(name, dtype)]

    return get


def load(folder, page, pages, backend, max_seqs=4, hip_graph=False):
    from qwen3_runtime_amd.config.engine import EngineConfig
    from qwen3_runtime_amd.engine.factory import load as load_model

    device, dtype = backend
    cfg = EngineConfig(page_size=page, num_pages=pages, max_num_seqs=max_seqs, dtype=dtype, device=device,
                       hip_graph=hip_graph)
    return load_model(folder, cfg, ops=TorchOps() if device == "cpu" else None)


def plain_logits(folder, requests):
    cfg, w = P.load(folder)
    out = {}
    for rid, toks in requests.items():
        logits = P.forward(cfg, w, toks).float()
        for p in range(len(toks)):
            out[(rid, p)] = logits[p]
    return out


def check(got, want, dtype, noise=0.2):
    """float32: to rounding of float32 sums, everywhere. bfloat16: as noise relative to the logits'
    own spread: no position over ``noise``, one in a hundred aside (a read-out over a sum that nearly
    cancels), and the root mean square under a quarter of it. A wrong window, cache or portion shows in
    float32, where the bound is rounding."""
    if dtype == "float32":
        traces.compare(got, want, atol=3e-4, rtol=3e-4)
        return
    keys = sorted(want)
    assert set(got) == set(want)
    w = torch.stack([want[k].double() for k in keys])
    err = torch.stack([got[k].double() for k in keys]) - w
    std = float(w.std())
    per_pos = err.abs().amax(dim=1)
    good = per_pos < noise * std
    assert int((~good).sum()) <= len(keys) // 100, \
        f"{int((~good).sum())} of {len(keys)} positions over the bound, the first {keys[int((~good).nonzero()[0])]}"
    rms = float(err[good].pow(2).mean().sqrt())
    assert rms < 0.25 * noise * std, f"rms error {rms:.4f} against a logit deviation of {std:.3f}"


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["a", "b", "c", "d", "e"])
@pytest.mark.parametrize("cut", ["whole", "tail_one_by_one", "portions", "mixed"])
def test_cuttings_match_plain(folder, backend, name, cut):
    """Whole prompts; the last tokens one by one (across window edges); portions down to two tokens;
    up to four live requests mixed in a pool of the peak's size, so that pages are used again
    (freed pages are poisoned first)."""
    raw, page = CONFIGS[name]()
    reqs = traces.make_requests(raw["vocab"], LENGTHS[name] + ([30, 9] if cut == "mixed" else []), seed=5)
    steps = getattr(traces, cut)(reqs)
    loaded = load(folder(name, backend[1]), page, traces.peak_tokens(steps, unit=page) // page, backend)
    got = traces.replay(loaded, steps, poison_freed=True)
    check(got, plain_logits(folder(name, backend[1]), reqs), backend[1], NOISE[name])


@pytest.mark.parametrize("name", ["a", "b", "d"])
def test_the_stream_after_every_layer_run_matches_plain(folder, name):
    """Layer run by layer run (a looped layer counts each time): the engine's residual stream, the pending
    outputs added, against the plain one, for a short prompt."""
    from qwen3_runtime_amd.engine.batch import StepEntry

    raw, page = CONFIGS[name]()
    toks = traces.make_requests(raw["vocab"], [33], seed=3)["r0"]
    cfg, w = P.load(folder(name))
    _, want = P.forward(cfg, w, toks, return_layers=True)
    loaded = load(folder(name), page, 16, ("cpu", "float32"))
    seen = []
    for block in loaded.model.blocks:
        inner = block.forward

        def spy(ctx, residual, delta, cache, inner=inner):
            residual, pending = inner(ctx, residual, delta, cache)
            seen.append(residual.double() + sum(y.double() * s.double() for y, s in pending.parts))
            return residual, pending

        block.forward = spy
    loaded.cache.admit("x")
    loaded.runner.step([StepEntry("x", toks, [len(toks) - 1])])
    loaded.cache.release("x")
    assert len(seen) == len(want)
    for i, (got, ref) in enumerate(zip(seen, want)):
        torch.testing.assert_close(got, ref, atol=2e-4, rtol=2e-4, msg=lambda m, i=i: f"after run {i}: {m}")


def test_faults_in_the_loop_and_the_embedding_would_show(folder):
    """The oracle with a pass's vectors swapped, the embedding not added again, the pair's order turned or the
    first token's row taken for another: each differs from the right one by far more than any bound here."""
    cfg, w = P.load(folder("a"))
    toks = traces.make_requests(cfg["vocab"], [20], seed=3)["r0"]
    right = P.forward(cfg, w, toks)
    off = lambda cfg=cfg, w=w: float((P.forward(cfg, w, toks) - right).abs().max())  # noqa: E731
    assert off(w={**w, "loop.step": w["loop.step"].flip(0)}) > 0.02
    assert off(cfg={**cfg, "loop": {**cfg["loop"], "times": 2}}, w={**w, "loop.step": w["loop.step"][:2]}) > 0.02
    b = cfg["embedding"]["bigram"]
    assert off(cfg={**cfg, "embedding": {"bigram": {**b, "mul_prev": b["mul_cur"], "mul_cur": b["mul_prev"]}}}) > 0.02
    last_row = w["bigram"].clone()
    last_row[-1] = last_row[0]
    assert float((P.forward(cfg, {**w, "bigram": last_row}, toks)[0] - right[0]).abs().max()) > 0.02
    assert off(cfg={**cfg, "residual_mult": 0.9}) > 0.02


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers_of_a_real_model_s_proportions(folder, dtype):
    """A 330-token prompt in one step, then in portions with its last tokens one by one, beside a
    second request: prompt kernels with full tiles, the window passing, experts by expert."""
    raw, page = config_g()
    reqs = traces.make_requests(raw["vocab"], LENGTHS["g"], seed=9)
    want = plain_logits(folder("g", dtype), reqs)
    for steps in (traces.whole(reqs), traces.mixed(reqs, seed=2, decode_tail=12)):
        loaded = load(folder("g", dtype), page, traces.peak_tokens(steps, unit=page) // page, ("cuda:0", dtype))
        check(traces.replay(loaded, steps, poison_freed=True), want, dtype, NOISE["g"])


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decoding_in_a_pool_of_one_window(folder, backend):
    """A request far longer than the pool, decoded token by token: every cache is windowed and gives
    its pages back as the window passes."""
    raw, page = config_c()
    reqs = traces.make_requests(raw["vocab"], [300], seed=8)
    steps = traces.tail_one_by_one(reqs, tail=290)
    loaded = load(folder("c", backend[1]), page, 5, backend)   # a window of 17 touches 3 pages, a step's tokens one more
    assert all(g.window is not None for g in loaded.cache.groups)
    got = traces.replay(loaded, steps, poison_freed=True)
    check(got, plain_logits(folder("c", backend[1]), reqs), backend[1], NOISE["c"])


@pytest.mark.parametrize("backend", BACKENDS)
def test_batches_of_unequal_requests_against_each_alone(folder, backend):
    """A long prompt's portion, a short prompt and two single tokens in one step give what each gives
    alone (float32: to the last bits)."""
    from qwen3_runtime_amd.engine.batch import StepEntry

    raw, page = config_a()
    reqs = traces.make_requests(raw["vocab"], [61, 9, 30, 25], seed=2)
    name = folder("a", backend[1])

    def run(batches):
        loaded = load(name, page, 24, backend)
        out = {}
        for rid in reqs:
            loaded.cache.admit(rid)
        done = {rid: 0 for rid in reqs}
        for batch in batches:
            entries = [StepEntry(rid, reqs[rid][done[rid]: done[rid] + n], [n - 1]) for rid, n in batch]
            logits = loaded.runner.step(entries).float().cpu()
            for (rid, n), row in zip(batch, logits):
                done[rid] += n
                out[(rid, done[rid] - 1)] = row
        return out

    first = [[("r2", 29)], [("r3", 24)]]
    together = run(first + [[("r0", 40), ("r1", 9), ("r2", 1), ("r3", 1)], [("r0", 21)]])
    alone = run(first + [[("r0", 40)], [("r1", 9)], [("r2", 1)], [("r3", 1)], [("r0", 21)]])
    assert set(together) == set(alone)
    if backend[1] == "float32":
        traces.compare(together, alone, atol=3e-5, rtol=3e-5)
    else:
        check(together, alone, "bfloat16", NOISE["a"])


@pytest.mark.parametrize("backend", BACKENDS)
def test_a_restarted_request_computes_the_same_again(folder, backend):
    """Preemption by recompute: pages back, states zeroed (the last token too), the slot kept; the second
    pass over the same tokens gives the first one's logits."""
    from qwen3_runtime_amd.engine.batch import StepEntry

    raw, page = config_a()
    toks = traces.make_requests(raw["vocab"], [70], seed=3)["r0"]
    loaded = load(folder("a"), page, 16, backend)
    loaded.cache.admit("x")
    first = loaded.runner.step([StepEntry("x", toks[:50], [49])]).float().cpu()
    loaded.runner.step([StepEntry("x", toks[50:], [0])])
    loaded.cache.restart("x")
    again = loaded.runner.step([StepEntry("x", toks[:50], [49])]).float().cpu()
    loaded.cache.release("x")
    torch.testing.assert_close(again, first, atol=1e-6 if backend[1] == "float32" else 1e-2, rtol=0)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,graphs", [("float32", False), ("bfloat16", True), ("bfloat16", False)])
@pytest.mark.parametrize("name", ["a", "b", "e"])
def test_greedy_generation_through_the_entry_point(folder, name, dtype, graphs):
    """``LLM.generate`` (scheduler with a small token budget, sampler, graphs where they apply): the
    tokens chosen greedily are, by the plain model given the same context, the best ones or within
    rounding of the best. Requests of unequal lengths, more of them than fit at once; one of them a single
    token long, whose prompt is then a decode step."""
    from qwen3_runtime_amd.llm import LLM

    raw, page = CONFIGS[name]()
    llm = LLM(str(folder(name, dtype)), dtype=dtype, block_size=page, num_kv_blocks=64, max_num_seqs=3,
              max_num_batched_tokens=48, cuda_graph=graphs)
    prompts = list(traces.make_requests(raw["vocab"], [5, 61, 1, 20, 90], seed=4).values())
    outs = llm.generate(prompts, max_tokens=40)
    cfg, w = P.load(folder(name, dtype))
    for prompt, tokens in zip(prompts, outs):
        assert len(tokens) == 40
        logits = P.forward(cfg, w, list(prompt) + list(tokens))[len(prompt) - 1: -1]
        below = logits.max(-1).values - logits[range(40), list(tokens)]
        bound = 1e-3 if dtype == "float32" else 2 * NOISE[name] * float(logits.std())
        assert int((below >= bound).sum()) == 0, (float(below.max()), int(below.argmax()))


@pytest.mark.gpu
def test_decode_steps_from_graphs_equal_eager_ones(folder):
    """Captured steps, replayed many times with eager steps of other batch sizes between them, against the
    same schedule run eagerly: state slots, last tokens and pages move on alike."""
    from qwen3_runtime_amd.engine.batch import StepEntry

    raw, page = config_g()
    reqs = traces.make_requests(raw["vocab"], [90, 41, 64], seed=12)
    name, out = folder("g", "bfloat16"), []
    for graphs in (True, False):
        loaded = load(name, page, 40, ("cuda:0", "bfloat16"), hip_graph=graphs)
        rows, at = [], {}
        for rid, toks in reqs.items():
            loaded.cache.admit(rid)
            loaded.runner.step([StepEntry(rid, toks[:30], [29])])
            at[rid] = 30
        for i in range(20):
            live = list(reqs)[: 3 if at["r1"] < 41 else 1] if i % 5 else ["r0"]
            live = [r for r in live if at[r] < len(reqs[r])]
            logits = loaded.runner.step([StepEntry(r, [reqs[r][at[r]]], [0]) for r in live])
            rows.append(logits.float().cpu().clone())
            for r in live:
                at[r] += 1
        out.append(rows)
    for graph, eager in zip(*out):
        # the same kernels on the same values; a bucket's launch may cut the keys another way
        torch.testing.assert_close(graph, eager, atol=0.03 * float(eager.std()), rtol=0)


def test_greedy_generation_on_the_host(folder):
    """The engine's own scheduler (admission, portions under a small token budget, two requests at
    a time of three) and step function over the plain torch ops; the greedy choice is made here,
    the sampler being a kernel."""
    from qwen3_runtime_amd.config.engine import EngineConfig
    from qwen3_runtime_amd.engine.batch import StepEntry
    from qwen3_runtime_amd.engine.request import Request
    from qwen3_runtime_amd.engine.scheduler import Scheduler

    raw, page = config_d()
    cfg, w = P.load(folder("d"))
    loaded = load(folder("d"), page, 32, ("cpu", "float32"), max_seqs=2)
    prompts = list(traces.make_requests(raw["vocab"], [12, 3, 30], seed=4).values())
    engine = EngineConfig(page_size=page, num_pages=32, max_num_seqs=2, max_num_batched_tokens=10, dtype="float32", device="cpu")
    scheduler = Scheduler(engine, loaded.cache, 100_000)
    lengths = [16, 9, 16]  # the second ends first, and the third one's prompt is read beside the first one's decoding
    requests = [Request(list(p), max_tokens=n) for p, n in zip(prompts, lengths)]
    for r in requests:
        scheduler.add(r)
    sizes = set()
    while not scheduler.is_finished():
        batch = scheduler.schedule()
        entries, caught = [], []
        for r in batch:
            at = loaded.cache.length(r.request_id)
            upto = at + r.grant
            caught.append(upto >= len(r.token_ids))
            entries.append(StepEntry(r.request_id, r.token_ids[at:upto], [r.grant - 1] if caught[-1] else []))
        sizes.add(tuple(sorted(r.grant for r in batch)))
        logits = loaded.runner.step(entries)
        rows = iter(logits if logits is not None else [])
        scheduler.settle(batch, [int(next(rows).argmax()) if c else None for c in caught])
    assert any(len(x) == 2 and x[0] == 1 and x[1] > 1 for x in sizes)  # a decoded token beside a prompt's portion
    for prompt, r, n in zip(prompts, requests, lengths):
        tokens = list(r.output_tokens)
        assert len(tokens) == n
        ref = P.forward(cfg, w, list(prompt) + tokens)[len(prompt) - 1: -1]
        below = ref.max(-1).values - ref[range(n), tokens]
        assert float(below.max()) < 1e-3


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_command_line_and_trace_replay(folder, tmp_path, dtype):
    """As a user runs them: ``python -m qwen3_runtime_amd.cli --model DIR`` generates greedily, and
    ``bin/trace_run`` replays a mixed schedule of seven requests from standard input, four live at
    most, with a pool that only holds what is live."""
    import ast
    import json
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np

    root = Path(__file__).resolve().parents[1]
    raw, page = config_a()
    where = folder("a", dtype)
    cfg, w = P.load(where)
    prompt = [5, 17, 3, 140, 9, 77, 2]
    proc = subprocess.run([sys.executable, "-m", "qwen3_runtime_amd.cli", "--model", str(where), "--dtype", dtype,
                           "--prompt-tokens", *map(str, prompt), "--max-tokens", "8"],
                          capture_output=True, text=True, timeout=600, cwd=str(root))
    assert proc.returncode == 0, proc.stderr[-3000:]
    lines = dict(line.split(" ", 1) for line in proc.stdout.splitlines() if " " in line)
    tokens = ast.literal_eval(lines["runtime"])
    assert len(tokens) == 8
    logits = P.forward(cfg, w, prompt + tokens)[len(prompt) - 1: -1]
    below = logits.max(-1).values - logits[range(8), tokens]
    assert float(below.max()) < (1e-3 if dtype == "float32" else 2 * NOISE["a"] * float(logits.std()))

    reqs = traces.make_requests(raw["vocab"], [70, 9, 41, 100, 35, 1, 66], seed=6)
    steps = traces.mixed(reqs, seed=1)
    out = tmp_path / "logits"
    proc = subprocess.run([str(root / "bin" / "trace_run"), "--model", str(where), "--dtype", dtype, "--out", str(out),
                           "--max-tokens", str(traces.peak_tokens(steps))],
                          input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
                          timeout=600, cwd=str(root))
    assert proc.returncode == 0, proc.stderr[-3000:]
    assert [line for line in proc.stdout.splitlines() if line.startswith("done ")] == [f"done {s['step']}" for s in steps]
    got, pos = {}, {r: 0 for r in reqs}
    for s in steps:
        wanted = sum(len(e["want"]) for e in s["entries"])
        rows = np.fromfile(out / f"{s['step']}.f32", dtype="<f4").reshape(wanted, raw["vocab"]) if wanted else None
        i = 0
        for e in s["entries"]:
            for k in e["want"]:
                got[(e["id"], pos[e["id"]] + k)] = torch.from_numpy(rows[i].copy())
                i += 1
            pos[e["id"]] += len(e["tokens"])
    check(got, plain_logits(where, reqs), dtype, NOISE["a"])


# ------------------------------------------------------------------ configuration and plan
def test_config_reader_and_plan():
    from qwen3_runtime_amd.config.dekinex import DekinexConfig
    from qwen3_runtime_amd.config.model import ConfigError
    from qwen3_runtime_amd.engine.factory import build_model

    raw, _ = config_a()
    cfg = DekinexConfig.from_dict(raw)
    assert DekinexConfig.from_dict(cfg.to_dict()) == cfg
    _, built = build_model(raw)
    plan = built.plan
    # every run of a layer has caches of its own: the embedding's, then two per run of either mixer
    assert [(s.layer, s.entry) for s in plan.order] == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None)]
    assert plan.embedding_cache == (0,) and [s.cache for s in plan.order] == [(1 + 2 * i, 2 + 2 * i) for i in range(8)]
    assert plan.caches[0].dtype == "int32" and plan.caches[1].shape == (4, 17, 24) and plan.caches[2].shape == (4,)
    assert (plan.caches[3].heads, plan.caches[3].head_dim, plan.caches[3].value_dim, plan.caches[3].window) == (2, 32, 16, 13)
    assert plan.caches[4].shape == (8 * 32 + 2 * 16, 3)
    assert [e.origin for e in built.entries] == [False, True, True] and built.blocks[0].mult == 0.8
    shapes = {d.file_name: d.shape for d in built.tensor_decls()}
    assert shapes["bigram"] == (68, 80) and shapes["loop.step"] == (3, 80) and shapes["l1.mix.q.conv"] == (192, 4)
    assert shapes["l0.mix.norm"] == (64,) and shapes["l0.mix.f.b"] == (4,) and shapes["l1.mlp.shared.sg"] == (1, 80)
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.mix.i", "l0.mix.g", "l0.mlp.gate", "l1.mlp.router", "l1.mlp.correction",
            "l1.mlp.e9.down", "l2.mix.i.b", "l3.mlp.e5.gate", "l3.mix.v.conv"} <= set(shapes)
    assert not {"l2.mlp.gate", "l3.mlp.shared.up", "l0.norm2"} & set(shapes)
    # what a file leaves out is not there
    bare = DekinexConfig.from_dict({"architecture": "Dekinex", "vocab": 50, "width": 16, "norm": {"eps": 1e-5}, "layers": [
        {"type": "attention", "mixer": {"heads": 2, "dim": 8, "scale": 0.3}, "mlp": None},
        {"type": "mlstm", "mixer": {"heads": 2, "dim": 8, "gate_cap": 5.0},
         "mlp": {"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 2, "top": 1}, "shared": None}}]})
    s = bare.layers[0].mixer
    assert (s.kv_heads, s.vdim, s.window, s.conv, s.rot_dims) == (2, 8, None, None, 0)
    assert (bare.layers[1].mixer.vdim, bare.layers[1].feed_forward.scale, bare.layers[1].feed_forward.shared_ff) == (8, 1.0, 0)
    assert bare.pairs is None and bare.loop is None and bare.residual_mult == 1.0
    _, built = build_model(bare.to_dict())
    assert built.plan.embedding_cache == () and "bigram" not in {d.file_name for d in built.tensor_decls()}
    ok = attention(2, 2, 8, 8, 0.1, 5, 2, 4, 10.0)
    one = lambda mixer, mlp=None, **more: {**model(50, 16, 1e-5, 1.0, (5, 1, 1), None, [(mixer, mlp)]), **more}  # noqa: E731
    for bad in (one(("delta", {})), one(attention(3, 2, 8, 8, 0.1, 5, 2, 4, 10.0)), one(attention(2, 2, 7, 8, 0.1, 5, 2, 4, 10.0)),
                one(attention(2, 2, 8, 8, 0.1, 5, 2, 10, 10.0)), one(attention(2, 2, 8, 8, 0.1, 5, 2, 3, 10.0)),
                one(attention(2, 2, 8, 8, 0.1, 0, 2, 4, 10.0)), one(attention(2, 2, 8, 8, 0.1, 5, 0, 4, 10.0)),
                one(attention(2, 2, 8, 8, 0.1, 5, 17, 4, 10.0)), one(memory(2, 8, 8, 0.0)), one(memory(0, 8, 8, 1.0)),
                one(ok, moe(8, 2, 3, 1.0, 0)), one(ok, {"kind": "dense", "ff": 8}), one(ok, {"kind": "sparse", "ff": 8}),
                one(ok, norm={"eps": 0.0}), one(ok, layers=[]), one(ok, loop={"start": 0, "stop": 2, "times": 2}),
                one(ok, loop={"start": 0, "stop": 1, "times": 0}), one(ok, embedding={"bigram": {"buckets": 0, "mul_prev": 1, "mul_cur": 1}}),
                one(ok, embedding={"bigram": {"buckets": 5, "mul_prev": 1.5, "mul_cur": 1}}),
                {k: v for k, v in one(ok).items() if k != "norm"}):
        with pytest.raises((ConfigError, ValueError, TypeError)):
            DekinexConfig.from_dict(bad)


def test_a_plan_and_its_embedding_agree_on_caches():
    from dataclasses import replace

    from qwen3_runtime_amd.engine.factory import build_model
    from qwen3_runtime_amd.parts.model import DecoderModel

    plan = build_model(config_b()[0])[1].plan
    with pytest.raises(ValueError):
        DecoderModel(replace(plan, embedding_cache=()))
    with pytest.raises(ValueError):
        replace(plan, embedding_cache=(len(plan.caches),))
    with pytest.raises(ValueError):
        replace(plan, embedding_cache=(plan.order[0].cache_ids()[0],))  # a step of the order writes it


def test_presets_are_registered_and_build():
    from qwen3_runtime_amd.engine.factory import build_model
    from qwen3_runtime_amd.registry import preset_config, preset_names

    assert {"dekinex_tiny_a", "dekinex_tiny_b", "dekinex_2b", "dekinex_4b", "dekinex_8b"} <= set(preset_names())
    for name in ("dekinex_tiny_a", "dekinex_tiny_b"):
        raw = preset_config(name)
        assert raw["architecture"] == "Dekinex"
        build_model(raw)
    assert len(build_model(preset_config("dekinex_4b"))[1].plan.order) == 36
