"""Sarudra: every mechanism alone against its plain function, and whole models under every cutting.

Each test runs with the plain torch ops on the CPU (which pins the host side: plan, packing,
pages, windows, state slots, the loop) and with the HIP ops on the GPU (marked ``gpu``; float32 and
bfloat16). The oracle is ``plain/sarudra_plain.py``: whole sequences, no cache, no state carried,
float64. Configurations are made here and differ from each other in every size and option, also
in values that a model may happen to make equal or 1. Where random weights would hide a fault (a
key far back, the edge of a window, a write into a state hundreds of tokens ago), one token's key,
value or write is made to stand out.
"""

from __future__ import annotations

import math
from types import SimpleNamespace

import pytest
import torch

import traces
from drivers import BACKENDS, DT, DictFetch, MixerDriver, f64, in_steps, make_ops, rnd, rounded
from plain import sarudra_plain as P
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


# ------------------------------------------------------------------ norms in groups
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,groups", [(96, 3), (2560, 4), (70, 7), (2048, 1), (64, 64), (1200, 20), (9000, 1), (9004, 2), (6, 2), (5120, 8)])
@pytest.mark.parametrize("planes", [0, 1, 3, 9])
def test_an_output_joins_the_stream_through_a_norm_in_groups(backend, width, groups, planes):
    """The stream plus a sub-layer's output normed part by part (a matrix, or planes to be summed), read
    as it is or through a norm in groups of its own, all rows or chosen ones, which leave the stream
    alone; also a plain sum, and nothing pending. One part of every output is far larger than the
    others: a root mean square over the whole row would show."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    t, eps, eps2 = 5, 1e-5, 1e-3
    x0 = rnd(t, width, seed=1)
    y = rnd(t, width, seed=2).to(dt) if planes == 0 else rnd(planes, t, width, seed=3)
    y[..., : width // groups] *= 20.0
    total = (y.double() if planes == 0 else y.double().sum(0))
    wa, wn = 1 + rnd(width, seed=4, scale=0.3), 1 + rnd(width, seed=5, scale=0.3)
    dev = lambda a: None if a is None else a.to(device)  # noqa: E731
    for after, update in (((wa, eps), P.group_norm(total, wa.double(), eps, groups)), (None, total)):
        new = x0.double() + update
        for norm in (None, (wn, eps2)):
            want = new if norm is None else P.group_norm(new, wn.double(), eps2, groups)
            for rows in (None, torch.tensor([4, 0, 2], dtype=torch.int32)):
                x = dev(x0.clone())
                got = ops.group_norm_update(x, dev(y), None if after is None else (dev(wa), eps),
                                            None if norm is None else (dev(wn), eps2), groups, dt, dev(rows))
                assert got.dtype == dt
                ref = want if rows is None else want[rows.long()]
                torch.testing.assert_close(got.float().cpu().double(), ref, **(dict(atol=1e-4, rtol=1e-5) if dtype == "float32" else
                                                                              dict(atol=1e-2, rtol=1e-2)))
                torch.testing.assert_close(x.cpu().double(), new if rows is None else x0.double(), atol=1e-4, rtol=1e-5)
    x = dev(x0.clone())
    got = ops.group_norm_update(x, None, None, None, 1, dt)
    assert torch.equal(got.cpu(), x0.to(dt)) and torch.equal(x.cpu(), x0)
    assert got.data_ptr() != x.data_ptr()  # the stream goes on changing under whoever reads this


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,vdim,groups", [(6, 16, 2), (4, 64, 1), (3, 40, 3), (80, 64, 8), (5, 7, 5), (1, 1, 1), (2, 12, 24), (130, 64, 1)])
@pytest.mark.parametrize("tokens", [3, 300])
def test_gate_and_norm_of_the_read_out(backend, heads, vdim, groups, tokens):
    """silu(gate) first, then the norm, part by part; the gate is columns of a wider matrix."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, eps = heads * vdim, 1e-4
    o, z = rnd(tokens, heads, vdim, seed=1), rnd(tokens, width + 12, seed=2, scale=2.0).to(dt)
    w = 1 + rnd(width, seed=3, scale=0.3)
    for first in (0, 5):
        got = ops.gated_group_norm(o.to(device), z.to(device)[:, first: first + width], w.to(device), eps, groups, dt)
        want = P.group_norm(o.double().reshape(tokens, -1) * P.silu(z[:, first: first + width].double()), w.double(), eps, groups)
        torch.testing.assert_close(got.float().cpu().double(), want, **close(dtype))


# ------------------------------------------------------------------ the state-space mixer
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("channels,taps,first", [(200, 4, 24), (64, 2, 0), (330, 3, 7), (130, 1, 130), (37, 6, 3)])
def test_convolution_with_a_bias_carries_its_tail(backend, channels, taps, first):
    """Two sequences in slots 2 and 0, columns ``first ..`` of a wider matrix, in portions down to one token
    and in steps long enough for the kernel that walks eight tokens a wave."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    lengths, slots = [150, 90], [2, 0]
    x = [rnd(n, first + channels + 6, seed=3 + i).to(dt) for i, n in enumerate(lengths)]
    w, b = rnd(channels, taps, seed=9, scale=0.6), rnd(channels, seed=10)
    whole, rest = divmod(channels, 64)
    segments = tuple(s for s in ((whole, 64, 0), (1, rest, 0)) if s[0] * s[1])
    want = [P.silu(P.causal_convolution(x[i][:, first: first + channels].double(), w.double(), b.double())) for i in range(2)]
    for sizes in ((150,), (2, 1, 3, 1, 1, 17), (40, 70)):
        tail = torch.zeros(3, channels, max(taps - 1, 1), dtype=torch.float32, device=device)
        tail[1] = float("nan")  # a slot nobody holds
        steps = [in_steps(n, sizes) for n in lengths]
        got = [[], []]
        for r in range(max(map(len, steps))):
            live = [i for i in range(2) if r < len(steps[i])]
            ctx = spans(device, [steps[i][r][1] for i in live], [slots[i] for i in live])
            y = torch.cat([x[i][steps[i][r][0]: sum(steps[i][r])] for i in live]).to(device)
            out = ops.delta_conv(ctx, y, channels, w.to(device), tail, segments, 0.0, first=first, bias=b.to(device)).cpu()
            for i, piece in zip(live, out.split([steps[i][r][1] for i in live])):
                got[i].append(piece)
        for i in range(2):
            torch.testing.assert_close(torch.cat(got[i]).double(), want[i], atol=3e-5, rtol=3e-5)


def spans(device, lens, slots):
    """What the recurrences read of a step's batch."""
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    return SimpleNamespace(num_tokens=cu[-1], num_seqs=len(lens), cu_q=i32(cu), state_slots=i32(slots), max_q_len=max(lens),
                           seq_of_token=i32([s for s, n in enumerate(lens) for _ in range(n)]), q_lens_host=list(lens), scratch={})


def recurrence_inputs(t, heads, groups, n, p, seed):
    x, b, c = rnd(t, heads, p, seed=seed), rnd(t, groups, n, seed=seed + 1, scale=n ** -0.5), rnd(t, groups, n, seed=seed + 2)
    step, bias = rnd(t, heads, seed=seed + 3, scale=2.0), rnd(heads, seed=seed + 4)
    return x, b, c, step, bias


def plain_recurrence(x, b, c, step, bias, a_log, skip):
    heads, per = x.shape[1], x.shape[1] // b.shape[1]
    dt = torch.nn.functional.softplus(step.double() + bias.double(), threshold=1e9)
    return torch.stack([P.state_space_head(x[:, j].double(), b[:, j // per].double(), c[:, j // per].double(), dt[:, j],
                                           a_log[j].double(), skip[j].double()) for j in range(heads)], 1)


STATE_SIZES = [(6, 2, 16, 24), (4, 4, 32, 16), (3, 1, 40, 7), (2, 1, 128, 64), (8, 2, 64, 64), (5, 5, 1, 1), (2, 2, 100, 3), (4, 1, 256, 16),
               (1, 1, 512, 8), (16, 2, 128, 64), (3, 3, 20, 48), (4, 2, 64, 128), (2, 1, 128, 80)]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,groups,n,p", STATE_SIZES)
def test_state_space_recurrence_against_the_rule_written_out(backend, heads, groups, n, p):
    """The recurrence alone: a whole span, portions down to one token with the state in its slot, a second
    sequence beside the first. Every head's step bias and rate differ, so heads mixed up would show, and
    so would heads that read another group's vectors. Step logits reach from -10 to 25. With bfloat16 inputs
    long spans go chunk by chunk; the short spans of the same step go token by token beside them."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    t = 40 if device == "cpu" else 330
    x, b, c, step, bias = recurrence_inputs(t, heads, groups, n, p, seed=heads + n)
    x, b, c = (v.to(dt).float() for v in (x, b, c))
    step[3], step[9] = -10.0, 25.0
    step = step.to(dt)
    a_log, skip = rnd(heads, seed=20) - 2.0, 1 + rnd(heads, seed=21)
    want = plain_recurrence(x, b, c, step.float(), bias, a_log, skip)
    rows = torch.cat([v.reshape(t, -1) for v in (x, b, c)], 1).to(dt).to(device)
    other = torch.cat([v.reshape(t, -1) for v in recurrence_inputs(t, heads, groups, n, p, seed=99)[:3]], 1).to(dt).to(device)
    wide = torch.cat([rnd(t, 3).to(dt), step], 1).to(device)
    consts = tuple(v.to(device) for v in (bias, a_log, skip))
    for sizes in ((t,), (37, 2, 1, 1, 16, 5), (130, 3, 64), (64, 65))[: 2 if device == "cpu" else 4]:
        state = torch.full((4, heads, p, n), float("nan"), device=device)
        state[3] = state[1] = 0.0
        got = []
        for at, k in in_steps(t, sizes):
            m = 1 + at % min(k, 4) if len(sizes) > 2 else k   # beside a span of another length
            ctx = spans(device, [m, k], [1, 3])
            both = torch.cat([other[at: at + m], rows[at: at + k]]).contiguous()
            steps = torch.cat([wide[at: at + m], wide[at: at + k]])[:, 3:]
            got.append(ops.state_space(ctx, both, steps, *consts, state, heads, groups, n, p).cpu()[m:])
        scale = float(want.abs().max())
        torch.testing.assert_close(torch.cat(got).double(), want, atol=2e-5 * scale, rtol=1e-4)
        assert torch.isnan(state[0]).all() and torch.isnan(state[2]).all()  # other slots are left alone


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("n,p", [(16, 24), (128, 64), (64, 16)])
def test_a_write_from_far_back_is_read_and_a_slot_taken_again_is_empty(backend, n, p):
    """A head that forgets next to nothing: a marker written along a direction of its own 400 tokens back,
    across many portions, is read whole, less the decay since; a second head forgets fast and has nothing
    left. Zeroed as when a slot is taken again, the state gives the skip alone."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    t, heads = 420, 2
    unit = lambda v: v / v.norm(dim=-1, keepdim=True)  # noqa: E731
    x, b = rnd(t, heads, p, seed=2), unit(rnd(t, 1, n, seed=3))
    direction = unit(rnd(n, seed=77))
    b = b - (b @ direction)[..., None] * direction
    b[5, 0], x[5] = direction, 9.0
    b, x, direction = (v.to(dt).float() for v in (b, x, direction))
    c = torch.zeros(t, 1, n)
    c[-1, 0] = direction
    step, bias = torch.zeros(t, heads), torch.tensor([0.3, -0.2])
    a_log, skip = torch.tensor([-12.0, 0.0]), torch.tensor([0.5, 2.0])
    want = plain_recurrence(x, b, c, step, bias, a_log, skip)
    assert (want[-1, 0] - 0.5 * x[-1, 0]).abs().min() > 5.0 and (want[-1, 1] - 2.0 * x[-1, 1]).abs().max() < (1e-4 if dtype == "float32" else 0.1)
    rows = torch.cat([v.reshape(t, -1) for v in (x, b, c)], 1).to(dt).to(device)
    consts = tuple(v.to(device) for v in (bias, a_log, skip))
    state = torch.zeros(2, heads, p, n, device=device)
    got = [ops.state_space(spans(device, [k], [1]), rows[at: at + k].contiguous(), step[:k].to(device), *consts, state, heads, 1, n, p).cpu()
           for at, k in in_steps(t, (64, 3, 1, 150, 2))]
    torch.testing.assert_close(torch.cat(got).double(), want, atol=2e-4, rtol=2e-4)
    state[1].zero_()
    again = ops.state_space(spans(device, [1], [1]), rows[-1:].contiguous(), step[:1].to(device), *consts, state, heads, 1, n, p).cpu()
    want = skip[:, None] * x[-1] + torch.nn.functional.softplus(bias)[:, None] * x[-1] * (b[-1, 0] @ c[-1, 0])
    torch.testing.assert_close(again[0], want, atol=1e-5, rtol=1e-5)


def space_weights(width, s, seed=0):
    inner, state = s["heads"] * s["vdim"], s["groups"] * s["state"]
    ch = inner + 2 * state
    return {"in": rnd(inner + ch + s["heads"], width, seed=seed + 1, scale=width ** -0.5), "conv": rnd(ch, s["conv"], seed=seed + 2, scale=0.5),
            "conv.b": rnd(ch, seed=seed + 3, scale=0.3), "dt_bias": rnd(s["heads"], seed=seed + 4), "A_log": rnd(s["heads"], seed=seed + 5) - 2.0,
            "D": 1 + rnd(s["heads"], seed=seed + 6), "norm": 1 + rnd(inner, seed=seed + 7, scale=0.2), "o": rnd(width, inner, seed=seed + 8, scale=inner ** -0.5)}


def space_mixer(width, s, eps, w, device, dt):
    from qwen3_runtime_amd.parts.statespace import StateSpace

    names = {n: n for n in ("in", "conv", "dt_bias", "A_log", "D", "norm", "o")} | {"conv_bias": "conv.b"}
    mixer = StateSpace(width, s["heads"], s["vdim"], s["state"], s["groups"], s["conv"], s["norm_groups"], eps, tensors=names)
    mixer.load(DictFetch(w, device, dt))
    return mixer


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,vdim,state,groups,conv,norm_groups", [
    (4, 24, 16, 2, 4, 3), (3, 40, 24, 1, 3, 1), (6, 8, 40, 3, 2, 2), (2, 64, 128, 1, 4, 2), (8, 16, 64, 8, 5, 4), (1, 10, 7, 1, 1, 1),
    (4, 64, 64, 2, 4, 8)])
def test_state_space_mixer(backend, heads, vdim, state, groups, conv, norm_groups):
    """The whole mixer with its state and the convolution's inputs in a slot: a prompt at once, portions
    down to one token, two requests in the same steps whose slots are then taken again by others."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, eps = 48, 1e-5
    t = 60 if device == "cpu" else 200
    s = {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}
    w = rounded(space_weights(width, s), dt)
    h = [rnd(t, width, seed=8).to(dt).float(), rnd(t // 2, width, seed=9).to(dt).float()]
    want = [P.state_space(x.double(), f64(w), s, eps) for x in h]
    driver = MixerDriver(space_mixer(width, s, eps, w, device, dt), device, dt, ops, 16, 1, max_requests=3)
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


# ------------------------------------------------------------------ attention with turned values
def turned_weights(width, nq, nkv, d, dv, seed=0):
    s = 0.3
    return {"q": rnd(nq * d, width, seed=seed + 1, scale=s), "k": rnd(nkv * d, width, seed=seed + 2, scale=s),
            "v": rnd(nkv * dv, width, seed=seed + 3, scale=s), "q.norm": 1 + rnd(d, seed=seed + 5, scale=0.2),
            "k.norm": 1 + rnd(d, seed=seed + 6, scale=0.2), "o": rnd(width, nq * dv, seed=seed + 7, scale=s)}


def turned_mixer(width, s, eps, w, device, dt):
    from qwen3_runtime_amd.parts.attention import GroupedQueryAttention
    from qwen3_runtime_amd.parts.plan import PartSpec

    names = {n: n for n in ("q", "k", "v", "o")} | {"q_norm": "q.norm", "k_norm": "k.norm"}
    rot = s["rot"]
    mixer = GroupedQueryAttention(
        width, s["heads"], s["kv_heads"], s["dim"], qk_norm_eps=eps, scale=s["scale"], value_dim=s["vdim"], window=s["mask"]["size"],
        softcap=s.get("softcap"), value_turn=rot["base"], tensors=names,
        position=PartSpec("rope_half", {"head_dim": s["dim"], "dims": rot["dims"], "base": rot["base"]}) if rot["dims"] else None)
    for child in mixer.children():
        child.load(DictFetch(w, device, dt))
    mixer.load(DictFetch(w, device, dt))
    return mixer


def turned_sizes(nq, nkv, d, dv, window, dims, base, softcap):
    return {"heads": nq, "kv_heads": nkv, "dim": d, "vdim": dv, "scale": 1.5 / math.sqrt(d), "mask": {"size": window},
            "rot": {"dims": dims, "base": base}, **({"softcap": softcap} if softcap else {})}


TURNED = [
    (4, 2, 32, 32, 40, 32, 1000.0, 8.0, 16),
    (6, 2, 16, 24, 21, 8, 100.0, 5.0, 8),      # values wider than keys; half of each key turns
    (2, 2, 64, 64, 70, 64, 1e4, None, 16),     # a key head per query head, no cap
    (3, 1, 48, 48, 9, 20, 50.0, 3.0, 8),       # an odd number of 16-wide blocks, a small window
    (2, 1, 128, 128, 130, 64, 1e5, 30.0, 16),  # half of a wide head turns
    (5, 5, 8, 6, 1, 2, 10.0, 20.0, 8),         # a window of the query itself; tiny heads
    (8, 2, 96, 96, 33, 96, 3e4, 15.0, 32),
    (4, 1, 128, 128, 65, 128, 1e6, 20.0, 16),  # every element turns, as the one-kernel decode form has it
    (4, 4, 80, 80, 50, 16, 500.0, 9.0, 16),
    (2, 1, 64, 64, 24, 0, 700.0, 12.0, 16),    # keys do not turn, values do
    (16, 1, 64, 64, 64, 64, 1e4, 10.0, 16),    # as many query heads a key head as a tile has rows
    (4, 2, 256, 256, 40, 128, 1e4, 10.0, 16),
    (2, 1, 16, 16, 30, 16, 100.0, 6.0, 8),
    (3, 3, 50, 34, 17, 10, 40.0, 7.0, 8),      # sizes that are multiples of nothing
]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("nq,nkv,d,dv,window,dims,base,softcap,page", TURNED)
def test_turned_values_over_a_window(backend, nq, nkv, d, dv, window, dims, base, softcap, page):
    """The attention mixer (normed queries and keys, part of them turned, capped scores, values turned by
    their positions and outputs turned back) over pages that go back to the pool behind the window. One
    token's input lies along another's query direction and its value is large, so that it takes nearly
    all the weight while it is seen; queries pass its window's edge one by one and inside a portion."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, eps = 56, 1e-5
    t = 3 * window + 60
    s = turned_sizes(nq, nkv, d, dv, window, dims, base, softcap)
    w = rounded(turned_weights(width, nq, nkv, d, dv), dt)
    h = rnd(t, width, seed=8)
    marked = t - window - 25
    h[marked] *= 8.0  # its key is normed and stays, its value grows
    h = h.to(dt).float()
    want = P.attention(h.double(), f64(w), s, eps)
    edge = marked + window  # the first query that no longer sees the marked token
    pages = -(-(window + 64) // page) + 2
    for cuts in (in_steps(edge - 3, (64, 5)) + [(p, 1) for p in range(edge - 3, edge + 4)] + [(edge + 4, t - edge - 4)],
                 in_steps(edge - 10, (7, 2, 30)) + [(edge - 10, 20)] + in_steps(t, (1,), edge + 10)):
        driver = MixerDriver(turned_mixer(width, s, eps, w, device, dt), device, dt, ops, page, pages)
        got = driver.run("a", h, cuts)
        assert driver.cache.groups[0].pool.num_free == pages
        assert_rows(got, want, dtype)
    # what would show if it were missing: the window one token off, the values' turn and the way back
    if window > 1:
        assert (want[edge - 1] - want[edge]).abs().max() > 5 * float(row_bound(want, "float32")[edge - 1])
        for other in (window - 1, window + 1):
            off = P.attention(h.double(), f64(w), {**s, "mask": {"size": other}}, eps)
            assert (off - want).abs().amax(1).max() > 5 * float(row_bound(want, "float32").max())
        off = P.attention(h.double(), f64(w), {**s, "rot": {"dims": dims, "base": base * 1.5}}, eps)
        assert (off - want).abs().amax(1).max() > 5 * float(row_bound(want, "float32").max())


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("nq,nkv,d,dv,window,dims", [(4, 2, 64, 64, 4000, 64), (2, 1, 48, 48, 4000, 16), (8, 2, 128, 128, 1300, 64), (2, 2, 16, 16, 1100, 16)])
def test_turned_values_over_long_contexts(backend, nq, nkv, d, dv, window, dims):
    """Contexts long enough that keys are cut over blocks whose parts are merged (decoded tokens, few-row
    portions beside long ones), long portions that share keys through LDS, and two requests at once. The
    first token's value is large and lies a thousand positions back. The mixer's rows depend on the
    distance of query and key alone, so that positions of thousands give what small ones give."""
    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    width, eps, t = 40, 1e-5, 1240
    s = turned_sizes(nq, nkv, d, dv, window, dims, 1e4, 25.0)
    w = rounded(turned_weights(width, nq, nkv, d, dv), dt)
    h = rnd(t, width, seed=5)
    h[2] *= 60.0
    h = [h.to(dt).float(), rnd(300, width, seed=6).to(dt).float()]
    want = [P.attention(x.double(), f64(w), s, eps) for x in h]
    driver = MixerDriver(turned_mixer(width, s, eps, w, device, dt), device, dt, ops, 16, 110)
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
        GroupedQueryAttention(32, 2, 1, 16, value_dim=15, value_turn=10.0, tensors=names)
    with pytest.raises(ValueError):
        GroupedQueryAttention(32, 2, 1, 16, output_gate=True, value_turn=10.0, tensors=names)
    with pytest.raises(ValueError):
        GroupedQueryAttention(32, 2, 1, 16, qk_norm_eps=1e-5, qk_norm_scope="projection", value_turn=10.0, tensors=names)
    with pytest.raises(ValueError):
        GroupedQueryAttention(32, 2, 1, 16, position=PartSpec("rope_half", {"head_dim": 16, "dims": 18, "base": 10.0}), tensors=names)


# ------------------------------------------------------------------ the mixture weighted on its input
def mixture_weights(width, ff, experts, shared, seed=0):
    w = {"router": rnd(experts, width, seed=seed + 1, scale=0.3)}
    for e in range(experts):
        for j, n in enumerate(("gate", "up")):
            w[f"e{e}.{n}"] = rnd(ff, width, seed=seed + 10 + 3 * e + j, scale=width ** -0.5)
        w[f"e{e}.down"] = rnd(width, ff, seed=seed + 12 + 3 * e, scale=ff ** -0.5)
    for j, n in enumerate(("gate", "up", "down") if shared else ()):
        w[f"shared.{n}"] = rnd(*((width, shared) if n == "down" else (shared, width)), seed=seed + 5 + j, scale=0.15)
    return w


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,ff,experts,top,shared,activation", [
    (48, 40, 6, 2, 56, "swiglu"), (64, 24, 10, 3, 0, "swiglu"), (40, 56, 4, 4, 24, "swiglu"), (72, 16, 5, 1, 32, "swiglu"),
    (50, 18, 3, 2, 10, "swiglu"), (64, 32, 4, 2, 0, "clamped"), (128, 64, 8, 2, 128, "swiglu")])
def test_weights_scale_the_experts_input(backend, width, ff, experts, top, shared, activation):
    """Router, experts and shared expert at every step size (one token, a few, tens, hundreds: pair by pair,
    expert by expert on the device, expert by expert through the engine's products). A weight on the
    output instead gives something else by far."""
    from qwen3_runtime_amd.parts.moe import RoutedSwiGLU

    device, dtype = backend
    ops, dt = make_ops(device), DT[dtype]
    w = rounded(mixture_weights(width, ff, experts, shared), dt)
    names = {"router": "router", "gate": "e{e}.gate", "up": "e{e}.up", "down": "e{e}.down"}
    names |= {f"shared_{n}": f"shared.{n}" for n in ("gate", "up", "down")} if shared else {}
    part = RoutedSwiGLU(width, ff, experts, top, router_bias=False, scoring="sigmoid", weight_on="input", activation=activation,
                        limit=0.7, shared_size=shared or None, shared_limit=0.7, tensors=names)
    part.load(DictFetch(w, device, dt))
    w64 = f64(w)

    def plain(x):
        if activation == "swiglu":
            return P.mixture(x, w64, {"router": {"top": top}, "shared": shared or None})
        index, weight = P.route(x, w64["router"], top)
        out = torch.zeros_like(x)
        for i in range(x.shape[0]):
            for j in range(top):
                e, xi = int(index[i, j]), weight[i, j] * x[i]
                g, u = torch.clamp(w64[f"e{e}.gate"] @ xi, max=0.7), torch.clamp(w64[f"e{e}.up"] @ xi, -0.7, 0.7)
                out[i] += w64[f"e{e}.down"] @ (g * torch.sigmoid(1.702 * g) * (u + 1))
        return out

    for t in (1, 3, 17, 70, 300) if device != "cpu" else (1, 17, 70):
        x = rnd(t, width, seed=t, scale=2.0).to(dt)
        # rows whose choice 8 bits of the scores could turn are not judged
        s = torch.sigmoid(x.double() @ w64["router"].T).sort(-1, descending=True).values
        clear = torch.ones(t, dtype=torch.bool) if top == experts else (s[:, top - 1] - s[:, top]) > 1e-4
        holder = SimpleNamespace(ops=ops, num_tokens=t, dtype=dt)
        got = part.forward(holder, x.to(device))
        got = (got.sum(0) if got.dim() == 3 else got).float().cpu()
        want = plain(x.double())
        if clear.any():
            assert_rows(got[clear], want[clear], dtype, f"{t} tokens")
    index, weight = P.route(x.double(), w64["router"], top)
    if activation == "swiglu":
        elsewhere = torch.stack([sum(weight[i, j] * P.gated(x[i].double(), w64, f"e{int(index[i, j])}.") for j in range(top)) for i in range(t)])
        here = want - (P.gated(x.double(), w64, "shared.") if shared else 0.0)
        assert ((elsewhere - here).abs().amax(1) / row_bound(want, "float32")).max() > 50


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("limit", [3.0, 30.0])
def test_capped_logits(backend, limit):
    device, _ = backend
    x = rnd(7, 301, seed=1, scale=20.0)
    x[0, :4] = torch.tensor([1e4, -1e4, 0.0, 1e-3])
    got = make_ops(device).softcap(x.clone().to(device), limit).cpu()
    torch.testing.assert_close(got.double(), P.cap(x.double(), limit), atol=2e-5, rtol=2e-5)


# ------------------------------------------------------------------ whole models
def space(heads, vdim, state, groups, conv, norm_groups):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def attention(nq, nkv, d, dv, scale, window, dims, base, softcap):
    return "attention", {"heads": nq, "kv_heads": nkv, "dim": d, "vdim": dv, "scale": scale, "mask": {"size": window},
                         "rot": {"dims": dims, "base": base}, "softcap": softcap}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, shared):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, **({"shared": {"ff": shared}} if shared else {})}


def model(vocab, width, eps, groups, scale, softcap, layers):
    return {"architecture": "Sarudra", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups}, "embedding": {"scale": scale},
            "logit_softcap": softcap, "layers": [{"type": kind, "mixer": mixer, "mlp": mlp} for (kind, mixer), mlp in layers]}


def config_a():
    """Both mixers, all three feed-forwards; keys and values of different sizes; part of the keys turns."""
    return model(210, 80, 1e-5, 5, 2.5, 20.0, [
        (attention(6, 2, 32, 16, 0.2, 13, 24, 500.0, 11.0), dense(72)),
        (space(4, 24, 16, 2, 4, 3), moe(24, 10, 3, 40)),
        (space(3, 40, 24, 1, 3, 1), None),
        (attention(4, 4, 16, 16, 0.3, 22, 16, 3000.0, 30.0), moe(40, 6, 2, 0)),
    ]), 16


def config_b():
    """One group everywhere, scale one; one expert a token; all experts a token."""
    return model(150, 64, 1e-6, 1, 1.0, 12.0, [
        (space(6, 8, 40, 3, 2, 2), moe(32, 5, 1, 16)),
        (attention(2, 1, 48, 48, 0.15, 9, 20, 50.0, 5.0), moe(48, 4, 4, 24)),
        (space(2, 32, 8, 2, 5, 1), dense(40)),
    ]), 8


def config_c():
    """Attention alone, windows all round: nothing grows with the length."""
    return model(97, 48, 1e-5, 4, 0.5, 30.0, [
        (attention(2, 2, 16, 8, 0.3, 17, 4, 20.0, 4.0), moe(16, 4, 2, 8)),
        (attention(6, 3, 8, 16, 0.4, 6, 8, 100.0, 9.0), None),
        (attention(3, 1, 16, 16, 0.25, 11, 0, 70.0, 50.0), dense(24)),
    ]), 8


def config_d():
    """Sizes that are multiples of nothing."""
    return model(131, 50, 1e-5, 2, 1.7, 9.0, [
        (space(3, 10, 7, 1, 3, 5), moe(18, 3, 2, 11)),
        (attention(3, 1, 10, 14, 0.4, 7, 6, 30.0, 6.0), dense(33)),
        (space(5, 6, 9, 5, 1, 3), moe(10, 5, 2, 0)),
    ]), 8


def config_e():
    """State-space layers alone: no page of cache."""
    return model(120, 72, 1e-5, 3, 3.0, 15.0, [
        (space(4, 16, 32, 4, 4, 4), dense(64)),
        (space(2, 40, 20, 1, 6, 2), moe(24, 7, 2, 32)),
    ]), 16


def config_g():
    """Layers of a real model's proportions, narrow: heads of 64 and 128, a state of 128."""
    return model(500, 256, 1e-6, 4, 1.0, 30.0, [
        (space(8, 64, 128, 2, 4, 2), dense(512)),
        (attention(4, 2, 128, 128, 0.09, 100, 128, 1e4, 50.0), moe(128, 8, 2, 128)),
        (space(8, 64, 128, 1, 4, 8), moe(128, 8, 2, 128)),
        (attention(8, 2, 64, 64, 0.12, 150, 32, 1e4, 50.0), moe(128, 8, 2, 128)),
    ]), 16


CONFIGS = {"a": config_a, "b": config_b, "c": config_c, "d": config_d, "e": config_e, "g": config_g}
LENGTHS = {"a": [70, 1, 23], "b": [64, 40, 2], "c": [90, 5], "d": [37, 20], "e": [60, 3, 31], "g": [330, 40]}
NOISE = {"a": 0.2, "b": 0.2, "c": 0.2, "d": 0.2, "e": 0.2, "g": 0.2}


def for_dtype(raw, dtype):
    """A model for runs in bfloat16 takes every expert for every token: with fewer, one chosen on a close
    call that 8 bits turn would move that position's logits by a large part of their spread. The choice
    by scores is held to the plain one in float32 here, and in both types in the mixture's own test."""
    if dtype == "bfloat16":
        for layer in raw["layers"]:
            if layer["mlp"] and layer["mlp"]["kind"] == "moe":
                layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return raw


@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    """Model folders with random weights, written once per configuration and type."""
    from qwen3_runtime_amd.weights import write_model_folder

    made = {}

    def get(name, dtype="float32"):
        if (name, dtype) not in made:
            raw = for_dtype(CONFIGS[name]()[0], dtype)
            made[(name, dtype)] = write_model_folder(tmp_path_factory.mktemp("sarudra_" + name), raw, seed=60 + sorted(CONFIGS).index(name),
                                                     std=0.03 if name == "g" else 0.08, norm_jitter=0.2)
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
    own spread: no position over ``noise``, one in a hundred aside (an expert chosen on a close call),
    and the root mean square under a quarter of it. A wrong window, cache or portion shows in
    float32, where the bound is rounding."""
    if dtype == "float32":
        traces.compare(got, want, atol=2e-4, rtol=2e-4)
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


def test_the_stream_after_every_layer_matches_plain(folder):
    """Layer by layer: the engine's residual stream after each layer (the pending output normed and
    added) against the plain one, for a short prompt."""
    from qwen3_runtime_amd.engine.batch import StepEntry

    raw, page = config_a()
    toks = traces.make_requests(raw["vocab"], [33], seed=3)["r0"]
    cfg, w = P.load(folder("a"))
    _, want = P.forward(cfg, w, toks, return_layers=True)
    loaded = load(folder("a"), page, 8, ("cpu", "float32"))
    seen = []
    for block in loaded.model.blocks:
        inner = block.forward

        def spy(ctx, residual, delta, cache, inner=inner):
            residual, pending = inner(ctx, residual, delta, cache)
            y = pending.y.double().sum(0) if pending.y.dim() == 3 else pending.y.double()
            seen.append(residual.double() + P.group_norm(y, pending.weight.double(), pending.eps, pending.groups))
            return residual, pending

        block.forward = spy
    loaded.cache.admit("x")
    loaded.runner.step([StepEntry("x", toks, [len(toks) - 1])])
    loaded.cache.release("x")
    assert len(seen) == len(raw["layers"])
    for i, (got, ref) in enumerate(zip(seen, want)):
        torch.testing.assert_close(got, ref, atol=2e-4, rtol=2e-4, msg=lambda m, i=i: f"after layer {i}: {m}")


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
        traces.compare(together, alone, atol=2e-5, rtol=2e-5)
    else:
        check(together, alone, "bfloat16", NOISE["a"])


@pytest.mark.parametrize("backend", BACKENDS)
def test_a_restarted_request_computes_the_same_again(folder, backend):
    """Preemption by recompute: pages back, states zeroed, the slot kept; the second pass over the
    same tokens gives the first one's logits."""
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
    rounding of the best. Requests of unequal lengths, more of them than fit at once."""
    from qwen3_runtime_amd.llm import LLM

    raw, page = CONFIGS[name]()
    llm = LLM(str(folder(name, dtype)), dtype=dtype, block_size=page, num_kv_blocks=64, max_num_seqs=3,
              max_num_batched_tokens=48, cuda_graph=graphs)
    prompts = list(traces.make_requests(raw["vocab"], [5, 61, 20, 90], seed=4).values())
    outs = llm.generate(prompts, max_tokens=40)
    cfg, w = P.load(folder(name, dtype))
    for prompt, tokens in zip(prompts, outs):
        assert len(tokens) == 40
        logits = P.forward(cfg, w, list(prompt) + list(tokens))[len(prompt) - 1: -1]
        below = logits.max(-1).values - logits[range(40), list(tokens)]
        bound = 1e-3 if dtype == "float32" else 2 * NOISE[name] * float(logits.std())
        assert int((below >= bound).sum()) == 0, (float(below.max()), int(below.argmax()))


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
    from qwen3_runtime_amd.config.model import ConfigError
    from qwen3_runtime_amd.config.sarudra import SarudraConfig
    from qwen3_runtime_amd.engine.factory import build_model

    raw, _ = config_a()
    cfg = SarudraConfig.from_dict(raw)
    assert SarudraConfig.from_dict(cfg.to_dict()) == cfg
    _, built = build_model(raw)
    plan = built.plan
    # pages for the attention layers, a state and the convolution's inputs for the others
    assert [s.cache for s in plan.order] == [0, (1, 2), (3, 4), 5]
    assert (plan.caches[0].heads, plan.caches[0].head_dim, plan.caches[0].value_dim, plan.caches[0].window) == (2, 32, 16, 13)
    assert plan.caches[1].shape == (4, 24, 16) and plan.caches[2].shape == (4 * 24 + 2 * 2 * 16, 3)
    assert all(c.dtype == "float32" for c in plan.caches if c.kind == "state")
    assert built.blocks[0].after_mixer.groups == 5 and built.head.softcap == 20.0 and built.embedding.scale == 2.5
    shapes = {d.file_name: d.shape for d in built.tensor_decls()}
    assert shapes["l1.mix.in"] == (2 * 96 + 64 + 4, 80) and shapes["l1.mix.conv"] == (160, 4) and shapes["l1.mix.conv.b"] == (160,)
    assert shapes["l0.mix.q.norm"] == (32,) and shapes["l0.mix.v"] == (32, 80) and shapes["l0.mix.o"] == (80, 96)
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.norm2", "l1.mlp.router", "l1.mlp.e9.down", "l1.mlp.shared.up", "l0.mlp.gate",
            "l2.mix.A_log", "l2.mix.D", "l2.mix.dt_bias", "l2.mix.norm", "l3.mlp.e5.gate"} <= set(shapes)
    assert not {"l2.norm2", "l3.mlp.shared.up", "l0.mlp.router"} & set(shapes) and "l2.norm2" in plan.ignorable
    # what a file leaves out is not there
    bare = SarudraConfig.from_dict(model(50, 16, 1e-5, 1, 1.0, None, [
        (("attention", {"heads": 2, "dim": 8, "scale": 0.3, "mask": {"size": 5}, "rot": {"dims": 4, "base": 10.0}}), None),
        (("mamba2", {"heads": 2, "vdim": 8, "state": 4, "conv": 2}), {"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 2, "top": 1},
                                                                     "shared": None})]))
    s = bare.layers[0].mixer
    assert (s.kv_heads, s.vdim, s.softcap, bare.logit_softcap) == (2, 8, None, None)
    assert (bare.layers[1].mixer.groups, bare.layers[1].mixer.norm_groups, bare.layers[1].feed_forward.shared_ff) == (1, 1, 0)
    ok = attention(2, 2, 8, 8, 0.1, 5, 4, 10.0, 5.0)
    one = lambda mixer, mlp=None, **more: {**model(50, 16, 1e-5, 1, 1.0, None, [(mixer, mlp)]), **more}  # noqa: E731
    for bad in (one(("retention", {})), one(attention(3, 2, 8, 8, 0.1, 5, 4, 10.0, 5.0)), one(attention(2, 2, 8, 7, 0.1, 5, 4, 10.0, 5.0)),
                one(attention(2, 2, 8, 8, 0.1, 5, 10, 10.0, 5.0)), one(attention(2, 2, 8, 8, 0.1, 5, 3, 10.0, 5.0)),
                one(attention(2, 2, 8, 8, 0.1, 0, 4, 10.0, 5.0)), one(attention(2, 2, 8, 8, 0.1, 5, 4, 10.0, -5.0)),
                one(space(4, 8, 8, 3, 4, 1)), one(space(4, 8, 8, 2, 4, 5)), one(space(4, 8, 0, 2, 4, 1)), one(ok, moe(8, 2, 3, 0)),
                one(ok, {"kind": "sparse", "ff": 8}), one(ok, norm={"eps": 1e-5, "groups": 3}), one(ok, norm={"eps": 0.0}), one(ok, layers=[]),
                {k: v for k, v in one(ok).items() if k != "norm"}):
        with pytest.raises((ConfigError, ValueError, TypeError)):
            SarudraConfig.from_dict(bad)


def test_presets_are_registered_and_build():
    from qwen3_runtime_amd.engine.factory import build_model
    from qwen3_runtime_amd.registry import preset_config, preset_names

    assert {"sarudra_tiny_a", "sarudra_tiny_b", "sarudra_2b", "sarudra_4b", "sarudra_8b"} <= set(preset_names())
    for name in ("sarudra_tiny_a", "sarudra_tiny_b"):
        raw = preset_config(name)
        assert raw["architecture"] == "Sarudra"
        build_model(raw)
