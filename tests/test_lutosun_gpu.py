"""Lutosun on the GPU against the plain implementation (``tests/plain/lutosun_plain.py``): every mechanism alone on inputs
made so that a fault shows, then whole models with random weights under every kind of schedule: whole prompts,
token-by-token decoding, portions down to two tokens, batches of unequal requests, pages and slots that are given back and
used again, long decoding, greedy generation through the engine and its scheduler, and the trace replay tool."""

from __future__ import annotations

import numpy as np
import pytest
import torch

from gpu_util import DEV, PAGE, close, dev, in_steps, make_runner, ops, portions, rounded, run_schedule, step_batch
from lutosun_models import LUTOSUN, latent, make_folder, make_telling, model, moe, tokens_for
from plain import lutosun_plain as L
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


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("vocab,width,buckets,mul_prev,mul_cur,scale", [
    (50, 64, 31, 13, 5, 0.5), (300, 90, 1009, 2 ** 40 + 1, 10 ** 12, 2.0), (7, 1, 1, 1, 1, 1.0), (1000, 2500, 97, 0, 3, 1.5), (40, 300, 65521, 8191, 131, 0.25)])
def test_a_row_per_pair_of_tokens(vocab, width, buckets, mul_prev, mul_cur, scale, dtype):
    """Every cut of five sequences gives the rows of the whole, exactly: the token before a portion comes from the slot, nothing
    of what a slot held before reaches a new request, and slots of others stay as they are."""
    o = ops()
    rng = np.random.default_rng(vocab + width)
    table, pairs = (rounded(rng.normal(size=(n, width)), dtype) for n in (vocab, buckets + 1))
    pair = {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}
    seqs = [rng.integers(0, vocab, size=n) for n in LENS]
    want = [L.embed(s, {"embed": table, "bigram": pairs}, {"scale": scale, "bigram": pair}) for s in seqs]
    td, pd = dev(table, dtype), dev(pairs, dtype)
    for name, steps in STEPS.items():
        last = torch.full((6, 1), vocab - 1, dtype=torch.int32, device=DEV)

        def run(batch, parts):
            ids = dev(np.concatenate([seqs[i][s : s + c] for i, s, c in parts]), torch.int32)
            x, copy = o.embed_pairs(ids, td, scale, pd, mul_prev, mul_cur, batch, last, keep=True)
            assert torch.equal(x, copy) and x.data_ptr() != copy.data_ptr()
            return x

        for i, got in enumerate(in_steps(LENS, steps, SLOTS, run)):
            close(got, want[i], torch.float32, f"{name}: sequence {i}", 2e-7)
        assert last[[3, 0, 5, 1, 4], 0].tolist() == [int(s[-1]) for s in seqs] and int(last[2, 0]) == vocab - 1
    ids = dev(seqs[0], torch.int32)
    close(o.embed_pairs(ids, td, scale), table[seqs[0]] * scale, torch.float32, "without pairs", 1e-7)
    with pytest.raises(ValueError):
        o.embed_pairs(ids, td, scale, pd[:, : width // 2].contiguous() if width > 1 else pd[:1], mul_prev, mul_cur, step_batch([len(ids)], [0]), last)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,k", [(1, 64, 48), (9, 90, 200), (70, 2500, 96), (300, 128, 4096), (5, 9000, 64), (40, 1028, 512)])
def test_sums_that_join_the_stream(rows, width, k, dtype):
    """What a product over few or many rows leaves pending (one partial sum or several, with a factor per channel or without),
    taken along by a layer norm (with and without a row list) or added together with a start and a step."""
    o = ops()
    rng = np.random.default_rng(rows + width)
    x, w = rng.normal(size=(rows, k)), rng.normal(size=(width, k)) / np.sqrt(k)
    scale, start, step = rng.normal(size=width), rng.normal(size=(rows, width)), rng.normal(size=width)
    g, b = rng.normal(size=width) + 1, rng.normal(size=width)
    stream = rng.normal(size=(rows, width)) + rng.normal(size=(rows, 1)) * 5  # far from a mean of zero
    gr, br = rounded(g, dtype), rounded(b, dtype)
    xd, wd, gd, bd = dev(x, dtype), dev(w, dtype), dev(g, dtype), dev(b, dtype)
    prod = rounded(x, dtype) @ rounded(w, dtype).T
    for factor in (None, scale):
        res = dev(stream)
        pending = o.linear_sum(xd, wd)
        pending = o.SplitSum(pending.parts, None if factor is None else dev(factor))
        want = stream + (prod if factor is None else prod * factor)
        normed = L.layer_norm(want, gr, br, 1e-5)
        tol = 3e-5 if dtype == torch.float32 else 8e-3
        at = dev([rows - 1, 0, rows - 1], torch.int32)
        close(o.layernorm(res, gd, bd, 1e-5, torch.float32, at, pending), normed[[rows - 1, 0, rows - 1]], torch.float32, "rows by a list", 3e-5)
        assert torch.equal(res, dev(stream)), "a row list leaves the stream as it is"
        close(o.layernorm(res, gd, bd, 1e-5, dtype, None, pending), normed, dtype, "norm", tol)
        close(res, want, torch.float32, "the stream", 2e-5)
        close(o.layernorm(res, gd, None, 1e-5, torch.float32), L.layer_norm(want, gr, 0.0, 1e-5), torch.float32, "without a bias", 3e-5)
        for s in (None, start):
            res = dev(stream)
            o.stream_inject(res, dev(step), None if s is None else dev(s), pending)
            close(res, want + step + (0 if s is None else s), torch.float32, "start and step", 2e-5)
    res = dev(stream)
    o.stream_inject(res, dev(step), dev(start))
    close(res, stream + start + step, torch.float32, "nothing pending", 1e-6)
    with pytest.raises(ValueError):
        o.stream_inject(res, dev(np.ones(width + 1)))


def test_a_layer_norm_of_a_row_far_from_zero():
    """The variance is the mean of the squared deviations: a mean a thousand times the spread costs no more than the mean's own rounding."""
    o = ops()
    rng = np.random.default_rng(1)
    for width in (48, 91, 2048, 8192, 8200):
        x = np.float32(rng.normal(size=(4, width)) + 1000.0).astype(np.float64)
        x[1] *= 1e-3
        w, b = rng.normal(size=width), rng.normal(size=width)
        close(o.layernorm(dev(x), dev(w), dev(b), 1e-4, torch.float32), L.layer_norm(x, np.float32(w), np.float32(b), 1e-4), torch.float32, f"width {width}", 3e-4)


def test_bounded_logits():
    o = ops()
    x = np.random.default_rng(0).normal(size=(7, 333)) * 20
    x[0, :3] = [0.0, 1e4, -1e4]
    for cap in (0.5, 15.0, 1e6):
        got = o.softcap_(dev(x), cap)
        close(got, cap * np.tanh(np.float32(x).astype(np.float64) / cap), torch.float32, f"cap {cap}", 1e-6)


@pytest.mark.parametrize("experts,top", [(1, 1), (4, 1), (8, 3), (70, 8), (300, 5), (64, 64), (130, 2)])
def test_routing_by_a_corrected_softmax_brought_to_one(experts, top):
    """Choice by score plus correction, weights by score alone, brought to the sum one and scaled; the logits may lie in wider
    rows and come as partial sums."""
    o = ops()
    rng = np.random.default_rng(experts)
    T = 133
    z = (rng.normal(size=(T, experts)) * 2).astype(np.float32)
    corr = np.float32(rng.normal(size=experts) * 0.3)
    if experts > 3:
        z[5] = 0.25            # every score equal: ties go by the correction, equal ones to the lower number
        corr[:2] = corr[2]
        z[6, 1:] -= 200.0      # scores of nothing but one: the others' weights are next to nothing, and no division by zero
    if experts == 8:
        corr[7] = 5.0          # taken always, whatever its score
        z[9, 7] = -300.0
    ids, w = L.route(z.astype(np.float64), np.eye(experts), corr.astype(np.float64), {"top": top, "scale": 2.5})
    s = np.exp(z - z.max(axis=-1, keepdims=True).astype(np.float64))
    c = np.sort(s / s.sum(axis=-1, keepdims=True) + corr, axis=-1)[:, ::-1]
    clear = np.ones(T, bool) if top == experts else (c[:, top - 1] - c[:, top] > 1e-6)
    wide = np.concatenate([z, rng.normal(size=(T, 3)) * 50], axis=1)
    for rows, outputs in ((z, None), (wide, experts)):
        got_ids, got = o.moe_route(dev(rows), dev(corr), top, "softmax", outputs=outputs, renormalise=True, factor=2.5)
        got_ids, got = got_ids.cpu().numpy(), got.cpu().numpy()
        assert clear.sum() > 100
        for t in np.flatnonzero(clear):
            assert set(got_ids[t]) == set(ids[t])
            order = {e: k for k, e in enumerate(got_ids[t])}
            assert np.abs(got[t][[order[e] for e in ids[t]]] - w[t]).max() < 1e-5
        if experts > 3 and top < experts:
            assert list(got_ids[5]) == list(np.argsort(-corr, kind="stable")[:top])
    parts = rng.normal(size=(5, T, experts + 2)).astype(np.float32)
    total = np.zeros((T, experts + 2), np.float32)
    for p in parts:
        total = total + p
    more = dict(outputs=experts, renormalise=True, factor=0.5)
    got, want = o.moe_route(o.SplitSum(dev(parts)), dev(corr), top, "softmax", **more), o.moe_route(dev(total), dev(corr), top, "softmax", **more)
    assert torch.equal(got[0], want[0]) and torch.equal(got[1], want[1])
    a, b = o.moe_route(dev(total), dev(corr), top, "sigmoid", outputs=experts), o.moe_route(dev(total), dev(corr), top, "sigmoid", outputs=experts, factor=4.0)
    assert torch.equal(a[0], b[0]) and torch.equal(a[1] * 4.0, b[1])
    for bad in (dict(outputs=experts + 1), dict(renormalise=True, scoring="chosen_softmax")):
        with pytest.raises((ValueError, NotImplementedError)):
            o.moe_route(dev(z), dev(corr), top, **{"scoring": "softmax", **bad})


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff,shared,experts,top", [(24, 10, 7, 3, 3), (90, 50, 33, 6, 2), (64, 32, 64, 1, 1), (128, 64, 48, 20, 4), (136, 72, 16, 4, 1),
                                                         (512, 520, 1024, 6, 2), (512, 512, 256, 4, 1), (1024, 128, 512, 8, 2)])
def test_bounded_experts_beside_a_gated_shared_one(width, ff, shared, experts, top, dtype):
    """The part as the model runs it: the router's product with the shared expert's gate as one more row, bounded experts, the
    gated shared expert added by the kernel that adds the chosen ones, a factor on all of it. A third of the gate and up values
    lie beyond the limits. Steps of one token to several tiles an expert."""
    from miniserve_amd.config.spec import PartSpec
    from miniserve_amd.loading import runtime
    from miniserve_amd.parts.registry import part_class

    rng = np.random.default_rng(width + experts)
    mlp = moe(experts, top, ff, shared, 0.9, 1.4, 1.7)
    w = {"router": rng.normal(size=(experts, width)) * 2 / np.sqrt(width), "correction": rng.normal(size=experts) * 0.1,
         "shared.sg": rng.normal(size=(1, width)) * 2 / np.sqrt(width)}
    for e, f in [(f"e{j}", ff) for j in range(experts)] + [("shared", shared)]:
        w.update({f"{e}.gate": rng.normal(size=(f, width)) * 1.5 / np.sqrt(width), f"{e}.up": rng.normal(size=(f, width)) * 1.5 / np.sqrt(width),
                  f"{e}.down": rng.normal(size=(width, f)) / np.sqrt(f)})
    w = {k: rounded(v, torch.bfloat16) for k, v in w.items()}
    names = {"gate": "gate", "up": "up", "down": "down"}
    spec = PartSpec("moe_mlp", {
        "hidden_size": width, "intermediate_size": ff, "num_experts": experts, "top": top, "activation": "swiglu_clamped", "limit": 0.9, "gated": True,
        "scoring": "softmax", "router_bias": True, "renormalise": True, "factor": 1.7, "shared_gate": True,
        "shared": PartSpec("gated_mlp", {"prefix": "shared.", "hidden_size": width, "intermediate_size": shared, "activation": "swiglu_clamped",
                                         "limit": 1.4, "names": names}),
        "names": {"router": "router", "router_bias": "correction", "expert": "e{}.", "shared_gate": "shared.sg", **names}})
    part = part_class("feed_forward", spec)(spec, runtime(dtype, DEV))
    assert set(type(part).tensors(spec)) == set(w)
    part.bind({k: dev(v, dtype) for k, v in w.items()})
    scale = rng.normal(size=width) + 1
    part.scale_output(dev(scale))
    for T in (1, 5, 40, 150, 700):
        x = rounded(rng.normal(size=(T, width)), torch.bfloat16)
        start = rng.normal(size=(T, width))
        stream = dev(start)
        assert part.forward(dev(x, dtype), stream) is None, "nothing is left pending"
        # tokens whose choice is close may go either way
        z = x @ w["router"].T
        s = np.exp(z - z.max(axis=-1, keepdims=True))
        c = np.sort(s / s.sum(axis=-1, keepdims=True) + w["correction"], axis=-1)[:, ::-1]
        clear = np.ones(T, bool) if top == experts else (c[:, top - 1] - c[:, top] > 1e-5)
        assert clear.sum() >= 0.9 * T
        want = start + L.mixture_ff(x, w, mlp) * scale
        close(stream[torch.tensor(clear)], want[clear], dtype, f"{T} tokens", tol=3e-5 if dtype == torch.float32 else 8e-3)


LATENTS = [(3, 16, 8, 8, 12, 24, 40), (5, 6, 6, 4, 14, 23, 22), (8, 64, 32, 32, 64, 64, 96), (4, 32, 32, 16, 48, 1100, 288), (1, 8, 2, 2, 8, 1, 8),
           (16, 24, 16, 16, 32, 100, 112), (2, 128, 64, 64, 128, 384, 512), (7, 40, 16, 16, 24, 64, 48)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,rot_dim,dims,value_dim,q_rank,rank,far", [(*s, far) for s in LATENTS for far in (0, 16)] + [
    (*s, far) for s in (LATENTS[0], LATENTS[2]) for far in (15, 170)])  # two places for every shape, four for two of them
def test_latent_attention_with_queries_from_a_latent(heads, dim, rot_dim, dims, value_dim, q_rank, rank, far, dtype):
    """The mixer over scattered pages in cuts of every kind: both norms, the second query product, rotation, store, attention over
    every earlier token. The latent of one token (the first, the last of a page, the first of a page, one in the middle) is made
    to meet the last query of the first head, so a lost page, a wrong place or a key too few shows."""
    from types import SimpleNamespace

    from miniserve_amd.config.spec import PartSpec
    from miniserve_amd.loading import runtime
    from miniserve_amd.parts.registry import part_class

    rng = np.random.default_rng(heads * dim + rank)
    T, W, eps, scale = 330, 64, 1e-4, 4.0 / np.sqrt(dim + rot_dim)
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": value_dim, "q_rank": q_rank, "kv_rank": rank, "scale": scale,
         "rot": {"base": 1000.0, "dims": dims}}
    nq = heads * (dim + rot_dim)
    w = {"dq": rng.normal(size=(q_rank, W)) / 8, "dq.norm": rng.uniform(0.7, 1.4, size=q_rank), "uq": rng.normal(size=(nq, q_rank)) / np.sqrt(q_rank),
         "dkv": rng.normal(size=(rank + rot_dim, W)) / 8, "dkv.norm": rng.uniform(0.7, 1.4, size=rank),
         "uk": rng.normal(size=(heads * dim, rank)) / np.sqrt(rank), "uv": rng.normal(size=(heads * value_dim, rank)) / np.sqrt(rank),
         "o": rng.normal(size=(W, heads * value_dim)) / np.sqrt(heads * value_dim)}
    w = {k: rounded(v, torch.bfloat16) for k, v in w.items()}
    x = rng.normal(size=(T, W))
    # token `far`: its latent lies along the last query of head 0, mapped into the latent's space
    aim = (w["uk"][:dim].T @ L.latent_queries(x[T - 1 :], w, m, eps)[0, 0, :dim]) / w["dkv.norm"]
    x[far] = np.linalg.pinv(w["dkv"]) @ np.concatenate((aim / np.linalg.norm(aim) * 30, np.zeros(rot_dim)))
    x = rounded(x, torch.bfloat16)
    want = L.latent_attention(x, w, m, eps, np.arange(float(T)))
    gone = x.copy()
    gone[far] = -x[far]
    floor = 0.1 if rank >= 40 else 5e-3  # (in few dimensions some of the other keys lie along the query too)
    assert np.abs(L.latent_attention(gone, w, m, eps, np.arange(float(T))) - want)[-1].max() > floor * np.abs(want[-1]).max(), "the planted key matters"
    rt = runtime(dtype, DEV)
    spec = PartSpec("latent_attention", {
        "hidden_size": W, "num_heads": heads, "head_dim": dim, "rot_dim": rot_dim, "value_dim": value_dim, "latent_dim": rank, "query_rank": q_rank,
        "scale": scale, "eps": eps, "position": PartSpec("rotary", {"dim": dims, "theta": 1000.0, "pairing": "adjacent"})})
    mixer = part_class("mixer", spec)(spec, rt)
    assert set(type(mixer).tensors(spec)) == set(w)
    mixer.bind({k: dev(v, dtype) for k, v in w.items()})
    pages = [int(p) for p in rng.permutation(30)[: -(-T // PAGE)]]
    table = dev([pages + [0] * (-len(pages) % 4)], torch.int32)
    for cuts in ([T], [130] + [1] * 200, portions(T, [2, 3, 64, 5, 2, 31, 1, 1, 90])):
        kc = torch.zeros((31, 1, PAGE, rank + rot_dim), dtype=dtype, device=DEV)
        vc = torch.zeros((31, 1, rank, PAGE), dtype=dtype, device=DEV)
        got, at = [], 0
        for n in cuts:
            b = step_batch([n], [at])
            slots = dev([pages[p // PAGE] * PAGE + p % PAGE for p in range(at, at + n)], torch.int32)
            cache = SimpleNamespace(writes=True, slots=slots, k=kc, v=vc, block_table=table)
            out = torch.zeros((n, W), dtype=torch.float32, device=DEV)
            pending = mixer.forward(dev(x[at : at + n], dtype), b, cache, None, out)
            rt.ops.add_pending(out, pending)
            got.append(out)
            at += n
        close(torch.cat(got), want, dtype, f"cuts {cuts[:3]}", 3e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_preparation_adds_partial_sums(dtype):
    """Rows that come as partial sums give, bit for bit, what their sum in ascending order gives."""
    o = ops()
    rng = np.random.default_rng(4)
    for T, q_rank, rank, heads, dim, rot in ((3, 40, 24, 3, 10, 6), (300, 1100, 64, 2, 16, 16)):
        ld = q_rank + rank + rot + 5
        parts, qparts = (rng.normal(size=(n, T, k)).astype(np.float32) for n, k in ((7, ld), (12, heads * (dim + rot))))
        total, qtotal = np.zeros((T, ld), np.float32), np.zeros((T, heads * (dim + rot)), np.float32)
        for p in parts:
            total = total + p
        for p in qparts:
            qtotal = qtotal + p
        slots = dev(rng.permutation(20 * PAGE)[:T], torch.int32)
        rope = o.rope_table(dev(np.arange(T), torch.int32), dev(np.full(rot // 2, 0.3)))
        wq, wc = dev(rng.normal(size=q_rank), dtype), dev(rng.normal(size=rank), dtype)
        seen = []
        for rows, q in ((o.SplitSum(dev(parts)), o.SplitSum(dev(qparts))), (dev(total), dev(qtotal))):
            kc = torch.zeros((20, 1, PAGE, rank + rot), dtype=dtype, device=DEV)
            vc = torch.zeros((20, 1, rank, PAGE), dtype=dtype, device=DEV)
            common = (rope, rot, "adjacent", wc, 1e-5, slots, kc, vc, heads, dim, rot, rank, dtype)
            none, _, c = o.latent_prepare(rows, None, q_rank, *common, query_latent=(0, wq))
            assert none is None
            plain, full = o.latent_prepare(q, 0, None, *common)
            full = full.view(T, heads, rank + rot)[:, :, rank:].contiguous()
            seen.append((c, plain, full, kc, vc))
        for a, b in zip(*seen):
            assert torch.equal(a, b)
        close(seen[0][0], L.rms_norm(total[:, :q_rank].astype(np.float64), wq.double().cpu().numpy(), 1e-5), dtype, "the queries' latent", None)


# ---------------------------------------------------------------- whole models


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("lutosun")
    return {name: make_folder(root, name) for name in LUTOSUN}


@pytest.fixture(scope="module")
def plain(folders):
    """``(exact logits, logits with what a 16-bit engine rounds rounded)`` of a model and a list of tokens."""
    memo = {}

    def get(name, tokens):
        key = (name, tuple(tokens))
        if key not in memo:
            cfg, w = read_model_folder(folders[name])
            memo[key] = L.forward(cfg, w, tokens), L.forward(cfg, w, tokens, rounding=L.to_bfloat16)
        return memo[key]

    return get


def check(got, want, dtype, what):
    exact, rounding = want
    if dtype == "float32":
        check_logits(got, exact, dtype, what)
    elif len(got) > 1 and not what.startswith("luE"):  # (latents of a few elements: one draw of the rounding says little about another)
        check_logits_against_rounding(got, exact, rounding, what)
    else:
        check_logits(got, exact, dtype, what)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(LUTOSUN))
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


@pytest.mark.parametrize("name", ["luA", "luB"])
def test_the_stream_after_every_layer_run(name, folders):
    """Where a pass begins, what joins it there and which weights it runs, run by run."""
    from miniserve_amd.engine.batch import StepRow

    cfg, w = read_model_folder(folders[name])
    toks = tokens_for(folders[name], 37, 9)
    _, want = L.forward(cfg, w, toks, return_layers=True)
    runner = make_runner(folders[name], "float32", 64, 1)
    seen = []

    def watched(block):
        forward = block.forward

        def run(residual, *args):
            pending = forward(residual, *args)
            now = residual.clone()
            runner.model.rt.ops.add_pending(now, pending)
            seen.append(now.cpu().numpy())
            return pending

        return run

    for block in runner.model.blocks:
        block.forward = watched(block)
    runner.step([StepRow(runner.acquire(), toks, [])])
    assert len(seen) == len(want)
    for n, (got, exact) in enumerate(zip(seen, want)):
        assert np.abs(got - exact).max() <= 2e-5 * np.abs(exact).max(), (name, n)


def random_config(seed):
    """A configuration drawn at random: any sizes (odd ones among them), any run of layers run any number of times, with and
    without feed-forwards."""
    rng = np.random.default_rng(seed)
    pick = lambda *a: a[int(rng.integers(0, len(a)))]
    layers = []
    for _ in range(int(rng.integers(1, 5))):
        experts = int(pick(1, 2, 5, 8, 17))
        mlp = None if rng.random() < 0.2 else moe(experts, int(rng.integers(1, min(experts, 4) + 1)), int(pick(9, 16, 40, 72)), int(pick(1, 24, 64, 100)),
                                                   float(pick(0.4, 1.0, 5.0)), float(pick(0.4, 1.0, 5.0)), float(pick(0.5, 1.0, 2.5)))
        rot = int(pick(2, 8, 16, 32))
        layers.append(latent(int(pick(1, 3, 8, 16)), int(pick(4, 16, 20, 64)), rot, int(pick(8, 12, 64)), int(pick(1, 16, 48, 130)), int(pick(16, 48, 100, 224, 300)),
                             float(pick(0.1, 0.25)), float(pick(50.0, 5e5)), int(pick(2, rot)), mlp))
    start = int(rng.integers(0, len(layers)))
    loop = pick(None, (start, int(rng.integers(start + 1, len(layers) + 1)), int(rng.integers(1, 4))))
    return model(int(pick(50, 131, 300)), int(pick(48, 72, 100, 136, 200)), float(pick(1e-6, 1e-5, 1e-3)), layers, loop,
                 (int(pick(1, 7, 251)), int(pick(0, 31, 10 ** 9)), int(pick(1, 17, 10 ** 10))), float(pick(0.3, 1.0, 2.0)), float(pick(0.3, 1.0, 1.4)),
                 float(pick(2.0, 30.0)))


@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random(seed, tmp_path):
    """Random sizes and orders in float32, where a router's choice needs no help (its weights reach over the whole width here):
    whole, in portions, decoded, and two requests side by side, against the plain implementation; in bfloat16 where the model
    has no choice to make."""
    from miniserve_amd.weights.random_init import Init, write_model_folder

    cfg = random_config(seed)
    folder = write_model_folder(tmp_path / "m", cfg, seed, Init(0.15, (0.6, 1.4)))
    make_telling(folder, cfg, seed, router=False)
    cfg, w = read_model_folder(folder)
    rng = np.random.default_rng(seed)
    reqs = {"a": rng.integers(0, cfg["vocab"], size=90).tolist(), "b": rng.integers(0, cfg["vocab"], size=41).tolist()}
    want = {r: L.forward(cfg, w, t) for r, t in reqs.items()}
    mixed = [[("a", 37), ("b", 2)], [("a", 1), ("b", 20)], [("a", 2), ("b", 1)]] + [[("a", 1), ("b", 1)]] * 18 + [[("a", 32)]]
    runner = make_runner(folder, "float32", 16 * 10, 2)
    for steps in ([[("a", 90)], [("b", 41)]], mixed):
        got = run_schedule(runner, reqs, steps)
        assert runner.cache.idle
        for r in reqs:
            check_logits(got[r], want[r], "float32", f"seed {seed} request {r}")
    runner = make_runner(folder, "bfloat16", 16 * 10, 2)
    got = run_schedule(runner, reqs, mixed)
    chooses = any(layer.get("mlp") and layer["mlp"]["router"]["top"] < layer["mlp"]["router"]["experts"] for layer in cfg["layers"])
    for r in reqs:
        assert np.isfinite(got[r]).all()
        if not chooses:
            check_logits_against_rounding(got[r], want[r], L.forward(cfg, w, reqs[r], rounding=L.to_bfloat16), f"seed {seed} request {r} in bfloat16")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(LUTOSUN))
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


@pytest.mark.parametrize("name,dtype", [("luA", "float32"), ("luD", "bfloat16")])
def test_long_decoding_through_a_pool_of_its_size(name, dtype, folders, plain):
    """300 tokens one by one: the cache fills to its last page."""
    toks = tokens_for(folders[name], 300, 7)
    runner = make_runner(folders[name], dtype, 16 * 19, 1)
    got = run_schedule(runner, {"a": toks}, [[("a", 1)] for _ in toks])["a"]
    check(got, plain(name, toks), dtype, "long decoding")
    assert runner.cache.idle


@pytest.mark.parametrize("name", sorted(LUTOSUN))
@pytest.mark.parametrize("chunk,graph", [(0, True), (16, True), (16, False)])
def test_greedy_generation_through_the_engine(name, chunk, graph, folders):
    from miniserve_amd.engine.engine import Engine
    from miniserve_amd.engine.request import SamplingParams
    from miniserve_amd.loading import load_model

    cfg, w = read_model_folder(folders[name])
    prompts = [tokens_for(folders[name], n, 20 + n) for n in (1, 9, 40, 17, 26)]
    want = [L.greedy(cfg, w, p, 12) for p in prompts]
    eng = Engine(load_model(folders[name], "float32", DEV), kv_pool_tokens=16 * 14, max_running=3, chunked_prefill_size=chunk,
                 decode_graph=graph)
    assert eng.generate(prompts, SamplingParams(max_new_tokens=12)) == want
    assert eng.runner.cache.idle


def test_captured_decode_steps_replay_in_bfloat16(folders, plain):
    """Decode steps of a batch as captured graphs, several replays with other tokens and experts; the previous token moves along in
    the slots."""
    name = "luD"
    reqs = {r: tokens_for(folders[name], 90, 40 + i) for i, r in enumerate("abc")}
    steps = [[(r, 30) for r in reqs]] + [[(r, 1) for r in reqs] for _ in range(60)]
    runner = make_runner(folders[name], "bfloat16", 16 * 20, 3, decode_graph=True)
    got = run_schedule(runner, reqs, steps)
    assert runner.graph_steps >= 50
    for r in reqs:
        check(got[r], plain(name, reqs[r]), "bfloat16", f"request {r}")


def test_trace_replay(folders, plain, tmp_path):
    from replay_util import Replay

    name = "luA"
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
    res = run("random-weights", "--preset", "lutosun-tiny", "--seed", "5", "--std", "0.1", "--norm-range", "0.6", "1.4", "--out", str(folder))
    assert res.returncode == 0, res.stderr[-2000:]
    cfg, w = read_model_folder(folder)
    prompt = np.random.default_rng(8).integers(0, cfg["vocab"], size=30).tolist()
    res = run("generate", "--model", str(folder), "--dtype", "float32", "--prompt-ids", ",".join(map(str, prompt)),
              "--max-new-tokens", "8", "--kv-pool-tokens", "256")
    assert res.returncode == 0, res.stderr[-2000:]
    assert json.loads(res.stdout.strip().splitlines()[-1])["outputs"] == [L.greedy(cfg, w, prompt, 8)]
    res = run("stress", "--model", str(folder), "--num-requests", "12", "--prompt-len", "4", "90", "--max-new-tokens", "1", "20",
              "--kv-pool-tokens", "640", "--max-running", "4", "--chunked-prefill-size", "64", "--temperature", "0.7", "--top-p", "0.9")
    assert res.returncode == 0, res.stdout[-1000:] + res.stderr[-2000:]
    report = json.loads(res.stdout.strip().splitlines()[-1])
    assert report["finished"] == 12 and report["idle"] and report["engine"]["architecture"] == "Lutosun"
