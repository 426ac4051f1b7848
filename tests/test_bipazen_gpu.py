"""Bipazen on the GPU against the plain implementation (``tests/plain/bipazen_plain.py``): every mechanism alone on inputs
made so that a fault shows, then whole models with random weights under every kind of schedule: whole prompts,
token-by-token decoding, portions down to two tokens, batches of unequal requests, pages and slots that are given back and
used again, long decoding, greedy generation through the engine and its scheduler, and the trace replay tool."""

from __future__ import annotations

import copy

import numpy as np
import pytest
import torch

from bipazen_models import BIPAZEN, make_folder, tokens_for
from gpu_util import DEV, PAGE, close, dev, in_steps, make_runner, ops, portions, rounded, run_schedule, step_batch
from plain import bipazen_plain as B
from plain.model_folder import read_model_folder
from tolerances import check_logits, check_logits_against_rounding

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]

# five sequences side by side: whole; one after the other in portions; many short rows in one step; token by token
LENS = [170, 1, 47, 9, 66]
STEPS = {
    "whole": [[170, 1, 47, 9, 66]],
    "portions": [[2, 0, 3, 0, 1], [3, 1, 1, 2, 2], [64, 0, 2, 1, 1], [1, 0, 1, 1, 17], [5, 0, 17, 5, 45], [31, 0, 1, 0, 0], [1, 0, 22, 0, 0], [63, 0, 0, 0, 0]],
    "one by one": [[1, 1, 1, 1, 1]] * 66 + [[104, 0, 0, 0, 0]],
    "twos and threes": [[2, 0, 3, 1, 2], [3, 1, 2, 2, 1]] * 40 + [[70, 0, 0, 0, 0]],
}
SLOTS = [3, 0, 5, 1, 4]  # of six: slot 2 belongs to nobody


# ---------------------------------------------------------------- mechanisms alone


@pytest.mark.parametrize("channels,taps,col,more,act,in_bias", [
    (64, 4, 8, 4, "silu", False), (60, 3, 0, 0, None, True), (45, 5, 7, 2, "silu", True), (10, 1, 3, 1, None, True), (36, 2, 4, 0, "silu", False),
    (300, 8, 0, 4, None, True), (17, 9, 2, 3, "silu", True), (1, 2, 0, 1, None, False), (2048, 4, 16, 0, "silu", True), (72, 12, 0, 0, None, False),
    (40, 6, 0, 0, None, True), (40, 7, 4, 0, "silu", False)])
def test_short_convolution_over_time(channels, taps, col, more, act, in_bias):
    """Every cut of five sequences gives the convolution of the whole: the inputs before a step come from the slot, in a step of
    many short rows too; nothing of what a slot held before reaches a new request, and slots of others stay as they are. The
    bias in front of the convolution belongs to the inputs: before the start there are zeros, not biases."""
    o = ops()
    rng = np.random.default_rng(channels * taps)
    w, b = rng.normal(size=(channels, taps)), rng.normal(size=channels)
    ib = rng.normal(size=channels) * 2 if in_bias else np.zeros(channels)
    seqs = [rng.normal(size=(n, channels)) for n in LENS]
    f = B.silu if act else (lambda y: y)
    want = [f(B.causal_conv(u + ib, w, b)) for u in seqs]
    wd, bd, ibd = dev(w.T), dev(b), dev(ib) if in_bias else None
    for name, steps in STEPS.items():
        state = torch.full((6, taps - 1, channels), 9.0, dtype=torch.float32, device=DEV) if taps > 1 else None

        def run(batch, parts):
            x = np.full((batch.num_tokens, col + channels + more), 1e3)
            x[:, col : col + channels] = np.concatenate([seqs[i][s : s + c] for i, s, c in parts])
            return o.time_conv(dev(x), col, wd, bd, state, batch, act, ibd)

        for i, got in enumerate(in_steps(LENS, steps, SLOTS, run)):
            close(got, want[i], torch.float32, f"{name}: sequence {i}", 5e-6)
        if taps > 1:
            assert (state[2] == 9).all(), "a slot nobody uses was written"
            close(state[3], (seqs[0] + ib)[-(taps - 1) :], torch.float32, f"{name}: what is kept", 1e-6)
    with pytest.raises(ValueError):
        o.time_conv(dev(np.zeros((3, channels))), 1, wd, bd, state, step_batch([3], [0]), act, ibd)


@pytest.mark.parametrize("heads,groups,dim,value_dim", [(4, 2, 24, 16), (3, 1, 7, 10), (8, 1, 64, 32), (4, 4, 128, 64), (2, 2, 200, 136), (1, 1, 1, 1),
                                                        (6, 3, 33, 5), (16, 2, 128, 64), (2, 1, 256, 256), (5, 5, 16, 100)])
def test_recurrence_with_a_step_size(heads, groups, dim, value_dim):
    """Five sequences in cuts of every kind against the loop over tokens. The first head hardly forgets and an early token is
    large there, so a token far back is most of a late output; the last head's steps are now and then so large that it forgets
    everything at once (its log decays reach the hundreds); slots that held another request's state start from zero."""
    o = ops()
    rng = np.random.default_rng(heads * dim)
    decay = -np.exp(rng.normal(size=heads))
    decay[0] = -2e-4
    skip, bias = rng.normal(size=heads), rng.normal(size=heads) * 0.5
    seqs = []
    for n in LENS:
        q, k = rng.normal(size=(n, groups, dim)) / np.sqrt(dim), rng.normal(size=(n, groups, dim))
        v, raw = rng.normal(size=(n, heads, value_dim)), rng.normal(size=(n, heads)) * 2 - 1
        if heads > 1:
            raw[4::7, -1] = 300.0
        if n > 2:
            k[2, 0] = q[-1, 0] / (q[-1, 0] @ q[-1, 0]) * 60.0  # what the last token looks for
            raw[2, 0] = 2.0
        seqs.append((q, k, v, raw))
    of_head = np.arange(heads) // (heads // groups)

    def loop(q, k, v, raw):
        step = B.softplus(raw + bias)
        return B.scalar_decay_recurrence(q[:, of_head], k[:, of_head], v, decay * step, step, skip)

    want = [loop(*s) for s in seqs]
    q, k, v, raw = seqs[0]
    lost = loop(q, np.where((np.arange(len(q)) == 2)[:, None, None], 0.0, k), v, raw)[0]
    assert np.abs(lost - want[0][0])[-1, 0].max() > 0.3 * np.abs(want[0][0][-1, 0]).max(), "the far token matters at the end"
    g, h = groups * dim, heads * value_dim
    cols = {"v": 4, "k": 4 + h, "q": 4 + h + g}
    for name, steps in STEPS.items():
        S = torch.full((6, heads, dim, value_dim), 7.0, dtype=torch.float32, device=DEV)

        def run(batch, parts):
            rows = [np.concatenate([a[s : s + c].reshape(c, -1) for a in (seqs[i][2], seqs[i][1], seqs[i][0])], axis=1) for i, s, c in parts]
            x = np.pad(np.concatenate(rows), ((0, 0), (4, 3 if dim % 4 else 0)))
            d = np.pad(np.concatenate([seqs[i][3][s : s + c] for i, s, c in parts]), ((0, 0), (5, 1)))
            return o.step_recurrence(dev(x), cols, heads, dim, value_dim, groups, dev(d), 5, dev(bias), dev(decay), dev(skip), batch, S)

        for i, got in enumerate(in_steps(LENS, steps, SLOTS, run)):
            close(got.view(LENS[i], heads, value_dim)[:, 0], want[i][0][:, 0], torch.float32, f"{name}: sequence {i}, the slow head", 3e-5)
            close(got.view(LENS[i], heads, value_dim), want[i][0], torch.float32, f"{name}: sequence {i}", 3e-5)
        close(S[3], want[0][1], torch.float32, f"{name}: the state that is kept", 3e-5)
        assert (S[2] == 7).all(), "a slot nobody uses was written"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,blocks", [(60, 3), (45, 5), (72, 72), (36, 1), (256, 2), (8, 8), (1, 1), (512, 2), (320, 1), (200, 25)])
def test_gated_recurrence_per_channel(width, blocks, dtype):
    """Five sequences in cuts of every kind against the loop over tokens, gates and all. Every third channel hardly forgets and
    takes in a large early input, which is most of its late outputs; the weights' storage type changes nothing: products of
    bfloat16 weights are held to float32's bound too."""
    o = ops()
    rng = np.random.default_rng(width + blocks)
    bs = width // blocks
    R, I = (rounded(rng.normal(size=(blocks, bs, bs)) * bs ** -0.5, dtype) for _ in range(2))
    rb, ib, yb = (rng.normal(size=width) * 0.5 for _ in range(3))
    coef = -np.exp(rng.normal(size=width) * 1.5)
    coef[::3] = -1e-3
    seqs = [(rng.normal(size=(n, width)), rng.normal(size=(n, width))) for n in LENS]
    for u, _ in seqs:
        if len(u) > 2:
            u[2, ::3] = 300.0 * np.sign(np.concatenate([np.diag(M) for M in I])[::3])  # (its own share in its input gate opens it)

    def loop(u, y):
        parts = u.reshape(len(u), blocks, bs)
        r, i = (B.sigmoid(np.concatenate([parts[:, b] @ M[b].T for b in range(blocks)], axis=1) + c) for M, c in ((R, rb), (I, ib)))
        return B.channel_recurrence(coef * r, i * u)

    states = [loop(*s) for s in seqs]
    want = [S * B.gelu_tanh(y + yb) for S, (_, y) in zip(states, seqs)]
    u, y = seqs[0]
    lost = loop(np.where((np.arange(len(u)) == 2)[:, None], 0.0, u), y)
    if width > 1:  # (a lone channel may well close its own gates to a large input)
        assert np.abs(lost - states[0])[-1, ::3].max() > 0.3 * np.abs(states[0][-1, ::3]).max()
    scale = max(np.abs(w).max() for w in want)
    for name, steps in STEPS.items():
        S = torch.full((6, width), 7.0, dtype=torch.float32, device=DEV)

        def run(batch, parts):
            us = np.concatenate([seqs[i][0][s : s + c] for i, s, c in parts])
            ys = np.pad(np.concatenate([seqs[i][1][s : s + c] for i, s, c in parts]), ((0, 0), (3, 2)))
            return o.rglru(dev(us), blocks, dev(R, dtype), dev(I, dtype), dev(rb), dev(ib), dev(coef), dev(ys), 3, dev(yb), batch, S, torch.float32)

        for i, got in enumerate(in_steps(LENS, steps, SLOTS, run)):
            close(got / scale, want[i] / scale, torch.float32, f"{name}: sequence {i}", 1e-5 * scale / np.abs(want[i]).max() if i == 1 else 3e-5)
        close(S[3], states[0][-1], torch.float32, f"{name}: the state that is kept", 3e-5)
        assert (S[2] == 7).all(), "a slot nobody uses was written"


@pytest.mark.parametrize("width,group", [(64, 32), (30, 30), (30, 5), (1, 1), (6000, 6000), (4096, 512), (5000, 2500), (300, 1)])
def test_a_gate_in_front_of_the_norm(width, group):
    o = ops()
    rng = np.random.default_rng(width + group)
    x, z, w = rng.normal(size=(9, width)), rng.normal(size=(9, width + 8)) * 2, rng.normal(size=width) + 1
    x[2, :group] *= 1e-3  # eps under the root shows
    gz = z[:, 4 : 4 + width]
    norm = lambda a: B.unit_rms(a.reshape(9, -1, group), 1e-4).reshape(9, width) * w
    zd = dev(z)
    for act, f in (("silu", B.silu), ("sigmoid", B.sigmoid)):
        first = o.group_rmsnorm_gate(dev(x), group, dev(w), zd[:, 4 : 4 + width], 1e-4, torch.float32, act, gate_first=True)
        close(first, norm(x * f(gz)), torch.float32, f"{act} in front", 1e-5)
        behind = o.group_rmsnorm_gate(dev(x), group, dev(w), zd[:, 4 : 4 + width], 1e-4, torch.float32, act)
        close(behind, norm(x) * f(gz), torch.float32, f"{act} behind", 1e-5)
    with pytest.raises(ValueError):
        o.group_rmsnorm_gate(dev(x), group, dev(w), None, 1e-4, torch.float32, gate_first=True)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 9, 70, 300])
def test_a_scale_on_what_a_product_adds_to_the_stream(rows, dtype):
    """Products that leave one partial sum or several, taken along by a norm (with and without a row list) or added at once."""
    o = ops()
    rng = np.random.default_rng(rows)
    for width, k in ((64, 48), (90, 200), (2500, 96), (128, 4096)):
        x, w = rng.normal(size=(rows, k)), rng.normal(size=(width, k)) / np.sqrt(k)
        s, g, stream = rng.normal(size=width), rng.normal(size=width) + 1, rng.normal(size=(rows, width))
        want = stream + (rounded(x, dtype) @ rounded(w, dtype).T) * s
        res = dev(stream)
        pending = o.linear(dev(x, dtype), dev(w, dtype), accumulate_into=res, defer=True, scale=dev(s))
        at = dev([rows - 1, 0, rows - 1], torch.int32)
        listed = o.rmsnorm(res, dev(g, dtype), 1e-5, torch.float32, at, pending)
        normed = B.weighted_norm(want, rounded(g, dtype), 1e-5)
        close(listed, normed[[rows - 1, 0, rows - 1]], torch.float32, "rows by a list", 3e-5)
        assert torch.equal(res, dev(stream)), "a row list leaves the stream as it is"
        close(o.rmsnorm(res, dev(g, dtype), 1e-5, dtype, None, pending), normed, dtype, "norm", 3e-5 if dtype == torch.float32 else 8e-3)
        close(res, want, torch.float32, "the stream", 2e-5)
        res = dev(stream)
        assert o.linear(dev(x, dtype), dev(w, dtype), accumulate_into=res, scale=dev(s)) is None
        close(res, want, torch.float32, "added at once", 2e-5)
        with pytest.raises(NotImplementedError):
            o.normed_add(res, None, dev(g), 1e-5, pending)  # a norm of the sublayer's output takes no scale


@pytest.mark.parametrize("experts,top", [(1, 1), (4, 1), (8, 3), (70, 8), (300, 5), (64, 64)])
def test_routing_by_sigmoid_scores(experts, top):
    o = ops()
    rng = np.random.default_rng(experts)
    z = (rng.normal(size=(133, experts)) * 4).astype(np.float32)
    if experts > 3:
        z[5] = 0.25                        # every score equal: ties go to the lower number
        z[6] = 60.0 + np.arange(experts)   # scores that float32 rounds to one: the order is still the logits'
    chosen = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    ids, w = o.moe_route(dev(z), None, top, "sigmoid")
    assert np.array_equal(ids.cpu().numpy(), chosen)
    close(w, B.sigmoid(np.take_along_axis(z.astype(np.float64), chosen, axis=-1)), torch.float32, "weights", 1e-6)
    parts = rng.normal(size=(5, 133, experts)).astype(np.float32)
    total = np.zeros((133, experts), np.float32)
    for p in parts:
        total = total + p
    got, want = o.moe_route(o.SplitSum(dev(parts)), None, top, "sigmoid"), o.moe_route(dev(total), None, top, "sigmoid")
    assert torch.equal(got[0], want[0]) and torch.equal(got[1], want[1])
    if experts == 8:  # a correction moves the choice and not the weights; groups go by the corrected scores
        corr = np.zeros(8)
        corr[7] = 2.0
        ids, w = o.moe_route(dev(z), dev(corr), 1, "sigmoid")
        assert (ids == 7).all()
        close(w[:, 0], B.sigmoid(z[:, 7].astype(np.float64)), torch.float32, "weights", 1e-6)
        ids, _ = o.moe_route(dev(z), dev(corr), 2, "sigmoid", 4, 1)
        assert ids.cpu().numpy().tolist() == [[7, 6]] * 133


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff,experts,top,gated", [(24, 10, 3, 3, True), (90, 50, 6, 2, True), (64, 32, 1, 1, True), (128, 64, 20, 4, True),
                                                        (136, 72, 4, 1, False), (128, 192, 2, 1, True), (512, 520, 6, 2, False), (512, 512, 4, 1, True)])
def test_experts_that_read_their_input_times_the_weight(width, ff, experts, top, gated, dtype):
    """Weights far from one, so that one in the wrong place shows: an expert is not linear in its input. Steps of one token to
    several tiles an expert (one expert gets every token of one of them), with a scale on what joins the stream."""
    o = ops()
    rng = np.random.default_rng(width + experts)
    gate, up = (rng.normal(size=(experts, ff, width)) * 2 / np.sqrt(width) for _ in range(2))
    down = rng.normal(size=(experts, width, ff)) / np.sqrt(ff)
    gr, ur, dr = (rounded(a, dtype) for a in (gate, up, down))
    scale = rng.normal(size=width)
    for T in (1, 5, 150, 700):
        x, start = rng.normal(size=(T, width)), rng.normal(size=(T, width))
        ids = np.stack([rng.permutation(experts)[:top] for _ in range(T)])
        if T == 150:
            ids[:] = ids[0]
        wts = rng.random(size=(T, top)) * 2 + 0.1
        xr = rounded(x, dtype)
        add = np.zeros((T, width))
        for t in range(T):
            for e, p in zip(ids[t], wts[t].astype(np.float32)):
                v = float(p) * xr[t]
                h = B.silu(gr[e] @ v) * (ur[e] @ v) if gated else np.maximum(ur[e] @ v, 0.0) ** 2
                add[t] += dr[e] @ (rounded(h, dtype) if dtype == torch.bfloat16 else h)
        stream = dev(start)
        o.moe_experts(dev(x, dtype), dev(ids, torch.int32), dev(wts), dev(gate, dtype) if gated else None, dev(up, dtype), dev(down, dtype),
                      "silu" if gated else "relu_squared", stream, True, dev(scale))
        close(stream, start + add * scale, dtype, f"{T} tokens", tol=3e-5 if dtype == torch.float32 else 8e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,rot_dim,dims,value_dim,rank", [(3, 16, 8, 8, 12, 40), (5, 6, 6, 4, 14, 22), (8, 64, 32, 32, 64, 96), (4, 32, 32, 16, 48, 288),
                                                                   (1, 8, 2, 2, 8, 8), (16, 24, 16, 16, 32, 112), (2, 128, 64, 64, 128, 512)])
def test_latent_attention_with_a_gate_per_element(heads, dim, rot_dim, dims, value_dim, rank, dtype):
    """Projection rows through norm, rotation and store, the products into the latent's space, attention over every earlier
    token, the products out of it and the gates, in cuts of every kind through scattered pages. A key far back is made to meet
    the last query of the first head (its latent is planted), so a lost page, a wrong place or a key too few shows."""
    o = ops()
    rng = np.random.default_rng(heads * dim + rank)
    T, eps, scale = 330, 1e-4, 4.0 / np.sqrt(dim + rot_dim)
    rot = {"base": 1000.0, "dims": dims}
    nq, nk, ng = heads * (dim + rot_dim), rank + rot_dim, heads * value_dim
    x = rng.normal(size=(T, nq + nk + ng))
    wn = rounded(rng.uniform(0.7, 1.4, size=rank), dtype)
    uk, uv = (rounded(rng.normal(size=(heads * d, rank)) / np.sqrt(rank), dtype) for d in (dim, value_dim))
    far = 5  # the latent of this token lies along the last query of head 0, mapped into the latent's space
    x[far, nq : nq + rank] = (uk[:dim].T @ x[T - 1, :dim]) / wn * 50
    q = x[:, :nq].reshape(T, heads, dim + rot_dim)
    c = rounded(B.weighted_norm(x[:, nq : nq + rank], wn, eps), dtype)
    pos = np.arange(T, dtype=np.float64)
    shared = rounded(B.rotate_halves(x[:, None, nq + rank : nq + nk], pos, rot)[:, 0], dtype)
    qp, qt = rounded(q[..., :dim], dtype), rounded(B.rotate_halves(q[..., dim:], pos, rot), dtype)
    k, v = (c @ uk.T).reshape(T, heads, dim), (c @ uv.T).reshape(T, heads, value_dim)
    gate = B.sigmoid(x[:, nq + nk :])

    def attend(k, v, shared):
        out = np.zeros((T, heads, value_dim))
        for a in range(heads):
            out[:, a] = B.causal_softmax((qp[:, a] @ k[:, a].T + qt[:, a] @ shared.T) * scale) @ v[:, a]
        return out.reshape(T, ng) * gate

    want = attend(k, v, shared)
    lost = attend(np.where((np.arange(T) == far)[:, None, None], 0.0, k), v, shared)
    if rank > 8:  # (in eight dimensions some of the other keys lie along the query too)
        assert np.abs(lost - want)[T - 1, :value_dim].max() > 0.1 * np.abs(want[T - 1, :value_dim]).max()
    ukt = dev(uk, dtype).view(heads, dim, rank).transpose(1, 2).contiguous()
    uvd = dev(uv, dtype).view(heads, value_dim, rank).contiguous()
    pages = [int(p) for p in rng.permutation(30)[: -(-T // PAGE)]]
    table = dev([pages + [0] * (-len(pages) % 4)], torch.int32)
    f = (rot["base"] ** (-2.0 * np.arange(dims // 2) / dims)).astype(np.float32)
    for cuts in ([T], [130] + [1] * 200, portions(T, [2, 3, 64, 5, 2, 31, 1, 1, 90])):
        kc = torch.zeros((31, 1, PAGE, rank + rot_dim), dtype=dtype, device=DEV)
        vc = torch.zeros((31, 1, rank, PAGE), dtype=dtype, device=DEV)
        got, at = [], 0
        for n in cuts:
            b = step_batch([n], [at])
            xs = dev(x[at : at + n])
            slots = dev([pages[p // PAGE] * PAGE + p % PAGE for p in range(at, at + n)], torch.int32)
            rope = o.rope_table(b.positions, dev(f))
            plain, full = o.latent_prepare(xs, 0, nq, rope, dims, "halves", dev(wn, dtype), eps, slots, kc, vc, heads, dim, rot_dim, rank, dtype)
            o.head_linear(plain, ukt, full, 0)
            a = o.paged_attention(full, kc, vc, table, b, heads, 1, rank + rot_dim, scale, 0, rank, wide_heads=True)
            out = torch.empty((n, ng), dtype=dtype, device=DEV)
            got.append(o.head_linear(a, uvd, out, 0, gate=(xs, nq + nk), gate_each=True))
            at += n
        close(torch.cat(got), want, dtype, f"cuts {cuts[:3]}", 3e-5 if dtype == torch.float32 else 2e-2)


# ---------------------------------------------------------------- whole models


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("bipazen")
    return {name: make_folder(root, name) for name in BIPAZEN}


@pytest.fixture(scope="module")
def plain(folders):
    """``(exact logits, logits with what a 16-bit engine rounds rounded)`` of a model and a list of tokens."""
    memo = {}

    def get(name, tokens):
        key = (name, tuple(tokens))
        if key not in memo:
            cfg, w = read_model_folder(folders[name])
            memo[key] = B.forward(cfg, w, tokens), B.forward(cfg, w, tokens, rounding=B.to_bfloat16)
        return memo[key]

    return get


def check(got, want, dtype, what):
    exact, rounding = want
    if dtype == "float32":
        check_logits(got, exact, dtype, what)
    elif len(got) > 1:
        check_logits_against_rounding(got, exact, rounding, what)
    else:
        check_logits(got, exact, dtype, what)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(BIPAZEN))
def test_schedules_agree_with_plain(name, dtype, folders, plain):
    """One sequence whole, decoded token by token behind a short prefix, and in portions of changing sizes down to two tokens
    and one, through a pool hardly larger than the request."""
    toks = tokens_for(folders[name], 150, 1)
    want = plain(name, toks)
    runner = make_runner(folders[name], dtype, 160, 2)
    seen = {}
    for label, cuts in (("whole", [150]), ("decode", [20] + [1] * 130), ("first token alone", [1, 149]), ("two, then one by one", [2] + [1] * 148),
                        ("portions", portions(150, [2, 3, 17, 64, 5, 2, 31, 1, 1]))):
        got = run_schedule(runner, {"a": toks}, [[("a", n)] for n in cuts])["a"]
        check(got, want, dtype, f"{name} {label}")
        seen[label] = got
        assert runner.cache.idle
    if dtype == "float32":  # cuts change nothing beyond rounding
        for label, got in seen.items():
            assert np.abs(got - seen["whole"]).max() <= 3e-5 * np.abs(want[0]).max(), label


@pytest.mark.parametrize("name", sorted(set(BIPAZEN) - {"bpE"}))  # (bpE's ones leave some options without effect, on purpose)
def test_the_models_show_what_is_left_out(name, folders, plain):
    """What the comparisons are worth: with these weights a missing bias, skip, gate, layer scale or norm weight, a convolution
    one tap short, one norm where there are several, another base, a state that is not carried, one choice fewer or a layer
    that shares another's state moves the logits by far more than the tolerance."""
    cfg, w = read_model_folder(folders[name])
    toks = tokens_for(folders[name], 150, 1)
    want = plain(name, toks)[0]
    floor = 20 * 1e-4 * np.abs(want).max()

    def moved(c=cfg, weights=w):
        return np.abs(B.forward(c, weights, toks) - want).max()

    def other(i, change):
        """The configuration with ``change`` applied to its layer ``i`` and to the layers that run its weights."""
        off = copy.deepcopy(cfg)
        for j, layer in enumerate(off["layers"]):
            if j == i or layer.get("weights_of") == i:
                change(layer)
        return off

    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        m, mlp, p = layer["mixer"], layer.get("mlp"), f"l{i}."
        keys = {"mamba2": ["conv.b", "dt_bias", "A_log", "D"], "rglru": ["y.b", "x.b", "conv.b", "ra.b", "ri.b", "ra", "ri", "lam"],
                "latent_attention": ["g"]}[layer["type"]]
        for key in keys:
            assert moved(weights={**w, p + "mix." + key: w[p + "mix." + key] * 0.0}) > floor, (name, i, key)
        for key in ["ls1", "mix.norm" if layer["type"] == "mamba2" else "norm1"] + (["ls2"] if mlp else []):
            assert moved(weights={**w, p + key: np.where(w[p + key] != 0, 1.0, 0.0)}) > floor, (name, i, key)
        if layer["type"] != "latent_attention" and m["conv"] > 1:
            short = w[p + "mix.conv"].copy()
            short[:, 0] = 0.0
            assert moved(weights={**w, p + "mix.conv": short}) > floor, (name, i, "taps")
        if layer["type"] == "mamba2" and m["norm_groups"] > 1:
            assert moved(other(i, lambda l: l["mixer"].update(norm_groups=1))) > floor, (name, i, "norm groups")
        if layer["type"] == "latent_attention":
            assert moved(other(i, lambda l: l["mixer"]["rot"].update(base=7.0))) > floor, (name, i, "base")
        if mlp and mlp["router"]["top"] > 1:
            assert moved(other(i, lambda l: l["mlp"]["router"].update(top=l["mlp"]["router"]["top"] - 1))) > floor, (name, i, "choices")
    # tokens far back matter to the last one
    other_start = [t for t in toks]
    other_start[:3] = tokens_for(folders[name], 3, 77)
    assert np.abs(B.forward(cfg, w, other_start)[-1] - want[-1]).max() > 3 * 1e-4 * np.abs(want).max()


def random_config(seed):
    """A configuration drawn at random: any order of the mixers, any sizes (odd ones among them), layers that run an earlier
    layer's weights, with and without a feed-forward."""
    from bipazen_models import again, latent, mamba2, model, moe, rglru

    rng = np.random.default_rng(seed)
    pick = lambda *a: a[int(rng.integers(0, len(a)))]
    layers = []
    for _ in range(int(rng.integers(2, 7))):
        if layers and rng.random() < 0.25:
            layers.append(again(layers, int(pick(*[j for j, l in enumerate(layers) if l.get("weights_of") is None]))))
            continue
        experts = int(pick(1, 2, 5, 8, 17))
        mlp = pick(None, moe(experts, int(rng.integers(1, min(experts, 4) + 1)), int(pick(16, 40, 72))), moe(experts, 1, int(pick(9, 64))))
        kind = pick("mamba2", "rglru", "latent")
        if kind == "mamba2":
            groups, per, vdim = int(pick(1, 2, 3)), int(pick(1, 2, 4)), int(pick(4, 9, 16, 32, 64))
            inner = groups * per * vdim
            layers.append(mamba2(groups * per, vdim, int(pick(3, 16, 40, 64, 130)), groups, int(pick(1, 2, 3, 4, 6)),
                                 int(pick(*[n for n in (1, 2, 3, groups, groups * per) if inner % n == 0])), mlp))
        elif kind == "rglru":
            blocks = int(pick(1, 2, 5, 8))
            layers.append(rglru(blocks * int(pick(1, 7, 16, 40, 64)), blocks, int(pick(1, 2, 4, 5)), mlp))
        else:
            rot = int(pick(2, 8, 16, 32))
            layers.append(latent(int(pick(1, 3, 8, 16)), int(pick(4, 16, 20, 64)), rot, int(pick(8, 12, 64)), int(pick(16, 48, 100, 224, 300)),
                                 float(pick(0.1, 0.25)), float(pick(50.0, 5e5)), int(pick(2, rot)), mlp))
    return model(int(pick(50, 131, 300)), int(pick(48, 72, 100, 136, 200)), float(pick(1e-6, 1e-5, 1e-3)), layers)


@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random(seed, tmp_path):
    """Random sizes and orders in float32, where a router's choice needs no help: whole, in portions, decoded, and two
    requests side by side, against the plain implementation; in bfloat16 where the model has no choice to make."""
    from bipazen_models import make_telling
    from miniserve_amd.weights.random_init import Init, write_model_folder

    cfg = random_config(seed)
    folder = write_model_folder(tmp_path / "m", cfg, seed, Init(0.15, (0.6, 1.4)))
    make_telling(folder, cfg, seed)
    cfg, w = read_model_folder(folder)
    rng = np.random.default_rng(seed)
    reqs = {"a": rng.integers(0, cfg["vocab"], size=90).tolist(), "b": rng.integers(0, cfg["vocab"], size=41).tolist()}
    want = {r: B.forward(cfg, w, t) for r, t in reqs.items()}
    mixed = [[("a", 37), ("b", 2)], [("a", 1), ("b", 20)], [("a", 2), ("b", 1)]] + [[("a", 1), ("b", 1)]] * 18 + [[("a", 32)]]
    runner = make_runner(folder, "float32", 16 * 10, 2)
    for steps in ([[("a", 90)], [("b", 41)]], mixed):
        got = run_schedule(runner, reqs, steps)
        assert runner.cache.idle
        for r in reqs:
            check_logits(got[r], want[r], "float32", f"seed {seed} request {r}: {[l['type'] for l in cfg['layers']]}")
    runner = make_runner(folder, "bfloat16", 16 * 10, 2)
    got = run_schedule(runner, reqs, mixed)
    chooses = any(layer.get("mlp") and layer["mlp"]["router"]["top"] < layer["mlp"]["router"]["experts"] for layer in cfg["layers"])
    for r in reqs:
        assert np.isfinite(got[r]).all()
        if not chooses:
            check_logits_against_rounding(got[r], want[r], B.forward(cfg, w, reqs[r], rounding=B.to_bfloat16), f"seed {seed} request {r} in bfloat16")


def test_a_router_that_reads_the_whole_stream(tmp_path, folders):
    """The test models' routers read channels that hold the embedding alone. Here the router's weights are random over the whole
    width and the layer scales reach every channel; in float32 the choice is still the plain implementation's."""
    from safetensors.torch import load_file, save_file

    name = "bpA"
    src = load_file(str(folders[name] / "model.safetensors"))
    gen = torch.Generator().manual_seed(3)
    for k in list(src):
        if k.endswith(".router"):
            src[k] = (torch.randn(src[k].shape, generator=gen) * 0.3).to(torch.bfloat16)
        if k.endswith((".ls1", ".ls2")):
            src[k] = (torch.rand(src[k].shape, generator=gen) + 0.3).to(torch.bfloat16)
    folder = tmp_path / "free"
    folder.mkdir()
    (folder / "config.json").write_text((folders[name] / "config.json").read_text())
    save_file(src, str(folder / "model.safetensors"))
    cfg, w = read_model_folder(folder)
    toks = np.random.default_rng(2).integers(0, cfg["vocab"], size=120).tolist()
    runner = make_runner(folder, "float32", 128, 1)
    got = run_schedule(runner, {"a": toks}, [[("a", n)] for n in portions(120, [33, 1, 2, 50])])["a"]
    check_logits(got, B.forward(cfg, w, toks), "float32", "a router over the whole stream")


def test_weights_of_a_later_layer_and_through_another(tmp_path):
    """The first layer runs the last layer's weights, the third runs the first's (and so the last's): three states, one set of
    tensors."""
    from miniserve_amd.weights.random_init import Init, write_model_folder

    cfg = copy.deepcopy(BIPAZEN["bpC"][0])
    first = cfg["layers"][0]
    cfg["layers"] = [dict(copy.deepcopy(first), weights_of=3), cfg["layers"][1], dict(copy.deepcopy(first), weights_of=0), first]
    folder = write_model_folder(tmp_path / "m", cfg, 3, Init(0.15, (0.6, 1.4)))
    cfg, w = read_model_folder(folder)
    assert not any(k.startswith(("l0.", "l2.")) for k in w)
    toks = np.random.default_rng(0).integers(0, cfg["vocab"], size=70).tolist()
    runner = make_runner(folder, "float32", 128, 1)
    got = run_schedule(runner, {"a": toks}, [[("a", n)] for n in portions(70, [20, 1, 1, 2, 30])])["a"]
    check_logits(got, B.forward(cfg, w, toks), "float32", "weights of a later layer")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(BIPAZEN))
def test_unequal_requests_in_one_batch_with_pages_and_slots_used_again(name, dtype, folders, plain):
    """Five requests through three slots and a pool that never holds them all: portions of some beside single tokens of
    others, a request of one token, requests admitted into slots and pages that others gave back, steps that leave a live
    request out."""
    lens = {"a": 150, "b": 37, "c": 1, "d": 70, "e": 33}
    reqs = {r: tokens_for(folders[name], n, 10 + i) for i, (r, n) in enumerate(lens.items())}
    steps = [
        [("a", 29)], [("a", 2), ("b", 3)], [("a", 16), ("b", 30), ("c", 1)], [("a", 1), ("b", 1), ("d", 33)],
        [("a", 64), ("b", 1), ("d", 1)], [("b", 1), ("d", 2), ("a", 1)], [("b", 1), ("d", 30), ("a", 7)], [("a", 1), ("d", 1), ("e", 2)],
    ] + [[("a", 1), ("d", 1), ("e", 1)] for _ in range(3)] + [[("a", 26), ("e", 28)]]
    runner = make_runner(folders[name], dtype, 16 * 18, 3)
    got = run_schedule(runner, reqs, steps)
    assert runner.cache.idle
    for r in reqs:
        check(got[r], plain(name, reqs[r]), dtype, f"{name} request {r}")
    with pytest.raises(Exception):
        for _ in range(4):
            runner.acquire()


@pytest.mark.parametrize("name", ["bpA", "bpC"])
def test_long_decoding_through_a_pool_of_its_size(name, folders, plain):
    """300 tokens one by one: the states run long, the cache fills to its last page."""
    toks = tokens_for(folders[name], 300, 7)
    runner = make_runner(folders[name], "float32", 16 * 19, 1)
    got = run_schedule(runner, {"a": toks}, [[("a", 1)] for _ in toks])["a"]
    check(got, plain(name, toks), "float32", "long decoding")
    assert runner.cache.idle


@pytest.mark.parametrize("name", sorted(BIPAZEN))
@pytest.mark.parametrize("chunk,graph", [(0, True), (16, True), (16, False)])
def test_greedy_generation_through_the_engine(name, chunk, graph, folders):
    from miniserve_amd.engine.engine import Engine
    from miniserve_amd.engine.request import SamplingParams
    from miniserve_amd.loading import load_model

    cfg, w = read_model_folder(folders[name])
    prompts = [tokens_for(folders[name], n, 20 + n) for n in (1, 9, 40, 17, 26)]
    want = [B.greedy(cfg, w, p, 12) for p in prompts]
    eng = Engine(load_model(folders[name], "float32", DEV), kv_pool_tokens=16 * 14, max_running=3, chunked_prefill_size=chunk,
                 decode_graph=graph)
    assert eng.generate(prompts, SamplingParams(max_new_tokens=12)) == want
    assert eng.runner.cache.idle


def test_captured_decode_steps_replay_in_bfloat16(folders, plain):
    """Decode steps of a batch as captured graphs, several replays with other tokens, other experts and states that move."""
    name = "bpD"
    reqs = {r: tokens_for(folders[name], 90, 40 + i) for i, r in enumerate("abc")}
    steps = [[(r, 30) for r in reqs]] + [[(r, 1) for r in reqs] for _ in range(60)]
    runner = make_runner(folders[name], "bfloat16", 16 * 20, 3, decode_graph=True)
    got = run_schedule(runner, reqs, steps)
    assert runner.graph_steps >= 50
    for r in reqs:
        check(got[r], plain(name, reqs[r]), "bfloat16", f"request {r}")


def test_trace_replay(folders, plain, tmp_path):
    from replay_util import Replay

    name = "bpA"
    a, b = tokens_for(folders[name], 70, 31), tokens_for(folders[name], 21, 32)
    with Replay(folders[name], "float32", tmp_path / "out", 128) as run:
        got = [run.step([("a", a[:33], [0, 32])]),
               run.step([("a", a[33:35], [1]), ("b", b, [20])], end=["b"]),
               run.step([("a", a[35:], [34])], end=["a"]),
               run.step([("c", b, [3, 20])], end=["c"])]
        assert run.close() == 0
    wa, wb = plain(name, a)[0], plain(name, b)[0]
    check_logits(np.concatenate(got), np.stack([wa[0], wa[32], wa[34], wb[20], wa[69], wb[3], wb[20]]), "float32", "trace replay")


def test_command_line_random_weights_generate_and_stress(tmp_path):
    """The command line serves the architecture like any other: a folder of random weights from the named preset, greedy
    generation from it against the plain implementation, and a sampled load that returns every page and slot."""
    import json
    import subprocess
    import sys

    from replay_util import ROOT

    folder = tmp_path / "m"
    run = lambda *a: subprocess.run([sys.executable, "-m", "miniserve_amd", *a], capture_output=True, text=True, cwd=str(ROOT), timeout=110)
    res = run("random-weights", "--preset", "bipazen-tiny", "--seed", "5", "--std", "0.1", "--norm-range", "0.6", "1.4", "--out", str(folder))
    assert res.returncode == 0, res.stderr[-2000:]
    cfg, w = read_model_folder(folder)
    prompt = np.random.default_rng(8).integers(0, cfg["vocab"], size=30).tolist()
    res = run("generate", "--model", str(folder), "--dtype", "float32", "--prompt-ids", ",".join(map(str, prompt)),
              "--max-new-tokens", "8", "--kv-pool-tokens", "256")
    assert res.returncode == 0, res.stderr[-2000:]
    assert json.loads(res.stdout.strip().splitlines()[-1])["outputs"] == [B.greedy(cfg, w, prompt, 8)]
    res = run("stress", "--model", str(folder), "--num-requests", "12", "--prompt-len", "4", "90", "--max-new-tokens", "1", "20",
              "--kv-pool-tokens", "640", "--max-running", "4", "--chunked-prefill-size", "64", "--temperature", "0.7", "--top-p", "0.9")
    assert res.returncode == 0, res.stdout[-1000:] + res.stderr[-2000:]
    report = json.loads(res.stdout.strip().splitlines()[-1])
    assert report["finished"] == 12 and report["idle"] and report["engine"]["architecture"] == "Bipazen"
