"""Lutosun on the CPU: its configuration and lowering (runs of layers that are run several times over caches of their own, what
joins the stream in front of them, what the embedding keeps per request), and the plain implementation held against forms that
do not share its loops."""

from __future__ import annotations

import copy
import math

import numpy as np
import pytest
import torch

from lutosun_models import LUTOSUN, ROUTER_CHANNELS, decisive_tokens, make_folder, tokens_for
from miniserve_amd.cache import CacheLayout
from miniserve_amd.config import config_from_dict
from miniserve_amd.config.presets import preset
from miniserve_amd.config.spec import PartSpec
from miniserve_amd.parts.model import CacheSlotNeed, expected_tensors
from miniserve_amd.parts.registry import part_class
from plain import lutosun_plain as L
from plain.model_folder import read_model_folder


# ---------------------------------------------------------------- configuration


@pytest.mark.parametrize("name", sorted(LUTOSUN))
def test_config_reads_back_and_names_its_tensors(name):
    cfg = LUTOSUN[name][0]
    c = config_from_dict(cfg)
    assert config_from_dict(c.to_dict()).to_dict() == c.to_dict()
    names = expected_tensors(c.to_spec())
    w = cfg["width"]
    assert names["embed"].shape == names["head"].shape == (cfg["vocab"], w) and names["final.norm"].shape == names["final.norm.b"].shape == (w,)
    pair = cfg["embedding"]["bigram"]
    assert ("bigram" in names) == bool(pair) and (not pair or names["bigram"].shape == (pair["buckets"] + 1, w))
    assert ("loop.step" in names) == bool(cfg["loop"]) and (not cfg["loop"] or names["loop.step"].shape == (cfg["loop"]["times"], w))
    for i, layer in enumerate(cfg["layers"]):
        m, mlp, p = layer["mixer"], layer["mlp"], f"l{i}."
        assert names[p + "norm1"].shape == names[p + "norm1.b"].shape == (w,)
        assert names[p + "norm2"].optional == names[p + "norm2.b"].optional == (not mlp)
        h, d, r, e, q, c_ = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
        assert names[p + "mix.dq"].shape == (q, w) and names[p + "mix.dq.norm"].shape == (q,) and names[p + "mix.uq"].shape == (h * (d + r), q)
        assert names[p + "mix.dkv"].shape == (c_ + r, w) and names[p + "mix.dkv.norm"].shape == (c_,)
        assert names[p + "mix.uk"].shape == (h * d, c_) and names[p + "mix.uv"].shape == (h * e, c_) and names[p + "mix.o"].shape == (w, h * e)
        assert not {p + "mix." + k for k in ("q", "g", "sink")} & set(names)
        if not mlp:
            assert not any(k.startswith(p + "mlp.") for k in names)
        else:
            n, f, s = mlp["router"]["experts"], mlp["expert"]["ff"], mlp["shared"]["ff"]
            assert names[p + "mlp.router"].shape == (n, w) and names[p + "mlp.correction"].shape == (n,)
            assert names[p + f"mlp.e{n - 1}.gate"].shape == (f, w) and names[p + "mlp.e0.down"].shape == (w, f) and p + f"mlp.e{n}.up" not in names
            assert names[p + "mlp.shared.up"].shape == (s, w) and names[p + "mlp.shared.down"].shape == (w, s) and names[p + "mlp.shared.sg"].shape == (1, w)


def runs(name):
    spec = config_from_dict(LUTOSUN[name][0]).to_spec()
    return [(e.layer, e.cache, None if e.before is None else (e.before["row"], e.before["restart"])) for e in spec.run_order]


def test_passes_have_caches_of_their_own_and_begin_with_their_step():
    assert runs("luA") == [(0, 0, None), (1, 1, (0, False)), (2, 2, None), (1, 3, (1, True)), (2, 4, None), (3, 5, None)]
    assert runs("luB") == [(0, 0, (0, False)), (1, 1, None), (0, 2, (1, True)), (1, 3, None), (0, 4, (2, True)), (1, 5, None)]
    assert runs("luC") == [(0, 0, None), (1, 1, None)]
    assert runs("luE") == [(0, 0, None), (1, 1, (0, False))]
    for name in LUTOSUN:  # the plain implementation's order is the same
        cfg = LUTOSUN[name][0]
        assert [(i, t) for i, t in L.run_plan(cfg)] == [(layer, None if b is None else b[0]) for layer, _, b in runs(name)]


def test_cache_groups_and_what_the_embedding_keeps():
    spec = config_from_dict(LUTOSUN["luA"][0]).to_spec()
    needs = []
    for e in spec.run_order:
        layer = spec.layers[e.layer]
        mixer = part_class("mixer", layer.mixer)(layer.mixer, None)
        needs.append(CacheSlotNeed(e.cache, mixer.kv_need(), mixer.state_need()))
    assert [(p.heads, p.width) for p in needs[0].kv.planes] == [(1, 48), (1, 40)] and needs[0].kv == needs[5].kv
    layout = CacheLayout.from_needs(needs)
    assert sorted(g.slots for g in layout.groups) == [(0, 5), (1, 3), (2, 4)]
    emb = part_class("embedding", spec.embedding)(spec.embedding, None)
    state = emb.state_need()
    assert [(t.name, t.shape, t.dtype) for t in state.tensors] == [("last", (1,), "int32")]
    layout = CacheLayout.from_needs(needs + [CacheSlotNeed(spec.num_cache_slots, None, state)])
    assert [s.slot for s in layout.states] == [6] and len(layout.groups) == 3
    without = config_from_dict(LUTOSUN["luC"][0]).to_spec().embedding
    assert part_class("embedding", without)(without, None).state_need() is None


def test_config_refusals():
    base = LUTOSUN["luA"][0]

    def broken(change):
        cfg = copy.deepcopy(base)
        change(cfg)
        return cfg

    for change, error in [
        (lambda c: c["layers"][1].update(type="attention"), NotImplementedError),
        (lambda c: c["layers"][0]["mixer"].pop("q_rank"), KeyError),
        (lambda c: c["layers"][0]["mixer"].update(q_rank=0), ValueError),
        (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=18), ValueError),
        (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3), ValueError),
        (lambda c: c["layers"][1]["mixer"].update(scale=0.0), ValueError),
        (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), ValueError),
        (lambda c: c["layers"][1]["mlp"]["router"].pop("scale"), KeyError),
        (lambda c: c["layers"][1]["mlp"]["expert"].update(limit=0.0), ValueError),
        (lambda c: c["layers"][1]["mlp"]["shared"].pop("limit"), KeyError),
        (lambda c: c["layers"][1]["mlp"].update(kind="dense"), NotImplementedError),
        (lambda c: c["loop"].update(stop=5), ValueError),
        (lambda c: c["loop"].update(start=3), ValueError),
        (lambda c: c["loop"].update(times=0), ValueError),
        (lambda c: c["embedding"]["bigram"].update(buckets=0), ValueError),
        (lambda c: c["embedding"]["bigram"].pop("mul_cur"), KeyError),
        (lambda c: c["embedding"].pop("scale"), KeyError),
        (lambda c: c.update(logit_softcap=0.0), ValueError),
        (lambda c: c.pop("residual_mult"), KeyError),
        (lambda c: c.pop("norm"), KeyError),
    ]:
        with pytest.raises(error):
            config_from_dict(broken(change))


def test_the_preset_and_the_measured_shapes_are_valid_configurations():
    from miniserve_amd.measurement.designs import SHAPES, lutosun_config

    for cfg in [preset("lutosun-tiny")] + [lutosun_config(s) for s in SHAPES.values()]:
        assert config_from_dict(cfg).to_spec().architecture == "Lutosun"
    for s in SHAPES.values():
        assert len(config_from_dict(lutosun_config(s)).to_spec().run_order) == s["layers"]


# ---------------------------------------------------------------- parts


def test_one_factor_for_what_a_layer_adds():
    norm = lambda t: PartSpec("rmsnorm", {"width": 4, "eps": 1e-5, "tensor": t})
    one = torch.ones(4)

    def scales(**more):
        from miniserve_amd.parts.base import FeedForward, Mixer

        class M(Mixer):
            scales_output = True

        class F(FeedForward):
            scales_output = True

        spec = PartSpec("prenorm", {"mixer_norm": norm("n1"), "ffn_norm": norm("n2"), **more})
        block = part_class("block", spec)(spec, None, M(PartSpec("m"), None), F(PartSpec("f"), None))
        block.bind({"n1": one, "n2": one, "s": torch.arange(4.0)})
        return [None if p.out_scale is None else p.out_scale.tolist() for p in (block.mixer, block.feed_forward)]

    assert scales(residual_scale=0.25) == [[0.25] * 4, [0.25] * 4]
    assert scales(residual_scale=0.5, mixer_scale="s") == [[0.0, 0.5, 1.0, 1.5], [0.5] * 4]
    assert scales(residual_scale=1.0) == scales() == [None, None]


def test_mixture_options_that_do_not_go_together():
    base = {"hidden_size": 4, "intermediate_size": 8, "num_experts": 3, "top": 2, "gated": True, "activation": "swiglu_clamped", "limit": 1.0}
    cls = part_class("feed_forward", PartSpec("moe_mlp", base))
    for more, error in (({"renormalise": True}, NotImplementedError), ({"factor": 2.0}, NotImplementedError), ({"shared_gate": True, "scoring": "softmax"}, ValueError)):
        with pytest.raises(error):
            cls(PartSpec("moe_mlp", dict(base, **more)), None)
    shared = PartSpec("dense_mlp", {"prefix": "s.", "hidden_size": 4, "intermediate_size": 8})
    spec = PartSpec("moe_mlp", dict(base, shared=shared, shared_gate=True, scoring="softmax", renormalise=True, factor=2.0,
                                    names={"shared_gate": "s.g"}))
    assert cls.tensors(spec)["s.g"].shape == (1, 4)


def test_two_parts_may_declare_one_table_and_only_with_one_shape():
    spec = config_from_dict(LUTOSUN["luB"][0]).to_spec()
    assert len(spec.injections) == 3 and {p["tensor"] for p in spec.injections} == {"loop.step"}
    step = part_class("injection", spec.injections[0])
    assert step(spec.injections[1], None).needs_start and not step(spec.injections[0], None).needs_start
    with pytest.raises(ValueError):
        step(PartSpec("step_vector", {"tensor": "t", "rows": 2, "row": 2, "width": 4}), None)


# ---------------------------------------------------------------- the plain implementation against other forms


def test_rows_of_pairs_by_hand():
    b = {"buckets": 10, "mul_prev": 3, "mul_cur": 7}
    assert L.bigram_rows([4, 5, 9, 0], b).tolist() == [10, (12 + 35) % 10, (15 + 63) % 10, 27 % 10]
    big = {"buckets": 1009, "mul_prev": 2 ** 40 + 1, "mul_cur": 10 ** 12}
    assert L.bigram_rows([7, 8], big).tolist() == [1009, (7 * (2 ** 40 + 1) + 8 * 10 ** 12) % 1009]
    w = {"embed": np.arange(20.0).reshape(10, 2), "bigram": 100.0 * np.arange(22.0).reshape(11, 2)}
    x = L.embed([4, 5], w, {"scale": 0.5, "bigram": b})
    assert x.tolist() == [[4.0 + 2000.0, 4.5 + 2100.0], [5.0 + 1400.0, 5.5 + 1500.0]]


def test_layer_norm_sees_neither_shift_nor_scale():
    rng = np.random.default_rng(0)
    x, w, b = rng.normal(size=(5, 12)), rng.normal(size=12), rng.normal(size=12)
    y = L.layer_norm(x, w, b, 0.0)
    assert np.allclose(L.layer_norm(3.0 * x + 7.0, w, b, 0.0), y)
    assert np.allclose(((y - b) / w).mean(axis=-1), 0) and np.allclose((((y - b) / w) ** 2).mean(axis=-1), 1)


def test_latent_attention_of_one_token_returns_its_value():
    rng = np.random.default_rng(2)
    W = 12
    m = {"heads": 2, "dim": 3, "rot_dim": 4, "vdim": 5, "q_rank": 7, "kv_rank": 6, "scale": 0.7, "rot": {"base": 10.0, "dims": 4}}
    w = {"dq": rng.normal(size=(7, W)), "dq.norm": rng.normal(size=7), "uq": rng.normal(size=(14, 7)), "dkv": rng.normal(size=(10, W)),
         "dkv.norm": rng.normal(size=6), "uk": rng.normal(size=(6, 6)), "uv": rng.normal(size=(10, 6)), "o": np.eye(10)}
    h = rng.normal(size=(1, W))
    c = (h @ w["dkv"].T)[:, :6]
    c = c / np.sqrt((c * c).mean() + 1e-5) * w["dkv.norm"]
    assert np.allclose(L.latent_attention(h, w, m, 1e-5, np.arange(1.0)), c @ w["uv"].T)


def test_attention_with_the_keys_products_on_the_querys_side():
    """Two heads over six tokens, head by head and pair by pair, with ``q . (uk c) = (uk^T q) . c``."""
    rng = np.random.default_rng(6)
    W, T = 8, 6
    m = {"heads": 2, "dim": 3, "rot_dim": 2, "vdim": 4, "q_rank": 5, "kv_rank": 6, "scale": 0.4, "rot": {"base": 10.0, "dims": 2}}
    w = {"dq": rng.normal(size=(5, W)), "dq.norm": rng.normal(size=5), "uq": rng.normal(size=(10, 5)), "dkv": rng.normal(size=(8, W)),
         "dkv.norm": rng.normal(size=6), "uk": rng.normal(size=(6, 6)), "uv": rng.normal(size=(8, 6)), "o": rng.normal(size=(W, 8))}
    h = rng.normal(size=(T, W))
    unit = lambda v: v / math.sqrt((v * v).mean() + 1e-5)
    turn = lambda v, p: np.array([v[0] * math.cos(p) - v[1] * math.sin(p), v[1] * math.cos(p) + v[0] * math.sin(p)])
    want = np.zeros((T, W))
    for t in range(T):
        q = (w["uq"] @ (unit(w["dq"] @ h[t]) * w["dq.norm"])).reshape(2, 5)
        out = []
        for a in range(2):
            folded = w["uk"][3 * a : 3 * a + 3].T @ q[a, :3]
            scores, values = [], []
            for j in range(t + 1):
                d = w["dkv"] @ h[j]
                c = unit(d[:6]) * w["dkv.norm"]
                scores.append(0.4 * (folded @ c + turn(q[a, 3:], t) @ turn(d[6:], j)))
                values.append(w["uv"][4 * a : 4 * a + 4] @ c)
            p = np.exp(np.array(scores) - max(scores))
            out.append((p / p.sum()) @ np.array(values))
        want[t] = w["o"] @ np.concatenate(out)
    assert np.allclose(L.latent_attention(h, w, m, 1e-5, np.arange(float(T))), want)


def test_rotation_turns_neighbours_by_the_distance():
    """Scores of turned vectors depend on the distance of their places alone, and what lies behind the turned part passes."""
    rng = np.random.default_rng(3)
    a, b = rng.normal(size=(1, 1, 10)), rng.normal(size=(1, 1, 10))
    rot = {"base": 50.0, "dims": 6}
    at = lambda x, p: L.rotate_neighbours(x, np.array([float(p)]), rot)[0, 0]
    assert np.isclose(at(a, 3) @ at(b, 10), at(a, 33) @ at(b, 40)) and not np.isclose(at(a, 3) @ at(b, 10), at(a, 3) @ at(b, 11))
    assert np.array_equal(at(a, 9)[6:], a[0, 0, 6:]) and np.allclose(at(a, 0), a[0, 0])
    z = (a[0, 0, 2] + 1j * a[0, 0, 3]) * np.exp(1j * 7 * 50.0 ** (-2 / 6))
    assert np.allclose([at(a, 7)[2], at(a, 7)[3]], [z.real, z.imag])


def test_routing_by_hand():
    """Logits whose softmax is (1, 2, 3, 4) / 10: the correction moves the choice, the weights are the softmax values brought to
    one, times the scale."""
    h, router = np.ones((1, 1)), np.log([[1.0], [2.0], [3.0], [4.0]])
    for corr, chosen in (([0, 0, 0, 0], [3, 2]), ([0.35, 0, 0, 0], [0, 3]), ([0.2, 0.1, 0, 0], [3, 0]), ([0, 0, 0, -1.0], [2, 1])):
        ids, w = L.route(h, router, np.array(corr), {"top": 2, "scale": 2.5})
        assert ids[0].tolist() == chosen, corr
        picked = np.array([chosen[0] + 1.0, chosen[1] + 1.0])
        assert np.allclose(w[0], 2.5 * picked / picked.sum())


def test_bounded_gate_and_up():
    f = lambda g, u: float(L.bounded_swiglu(np.array(g), np.array(u), 2.0))
    s = lambda z: 1 / (1 + math.exp(-z))
    assert math.isclose(f(1.0, 0.5), s(1.702) * 1.5)
    assert math.isclose(f(5.0, 7.0), 2 * s(3.404) * 3) and math.isclose(f(5.0, -7.0), 2 * s(3.404) * -1)
    assert math.isclose(f(-5.0, 1.0), -5 * s(-8.51) * 2), "gates are bounded from above only"


def test_a_one_layer_model_in_closed_form():
    """One layer run twice without a feed-forward, one token: attention returns the token's value."""
    cfg = LUTOSUN["luA"][0] | {"vocab": 7, "width": 6, "loop": {"start": 0, "stop": 1, "times": 2}, "residual_mult": 0.3, "logit_softcap": 2.0,
                               "layers": [{"type": "latent_attention", "mlp": None,
                                           "mixer": {"heads": 1, "dim": 2, "rot_dim": 2, "vdim": 3, "q_rank": 2, "kv_rank": 4, "scale": 1.0,
                                                     "rot": {"base": 10.0, "dims": 2}}}]}
    rng = np.random.default_rng(5)
    shapes = {"dq": (2, 6), "dq.norm": (2,), "uq": (4, 2), "dkv": (6, 6), "dkv.norm": (4,), "uk": (2, 4), "uv": (3, 4), "o": (6, 3)}
    w = {f"l0.mix.{k}": rng.normal(size=s) for k, s in shapes.items()}
    w.update({"embed": rng.normal(size=(7, 6)), "bigram": rng.normal(size=(98, 6)), "loop.step": rng.normal(size=(2, 6)), "head": rng.normal(size=(7, 6))})
    w.update({k: rng.normal(size=6) for k in ("final.norm", "final.norm.b", "l0.norm1", "l0.norm1.b")})
    ln = lambda x, k: (x - x.mean()) / np.sqrt(((x - x.mean()) ** 2).mean() + 1e-5) * w[k] + w[k + ".b"]

    def sub(x):
        c = (w["l0.mix.dkv"] @ ln(x, "l0.norm1"))[:4]
        c = c / np.sqrt((c * c).mean() + 1e-5) * w["l0.mix.dkv.norm"]
        return x + 0.3 * (w["l0.mix.o"] @ (w["l0.mix.uv"] @ c))

    e = 1.5 * w["embed"][2] + w["bigram"][97]
    x = sub(sub(e + w["loop.step"][0]) + e + w["loop.step"][1])
    assert np.allclose(L.forward(cfg, w, [2])[0], 2.0 * np.tanh(w["head"] @ ln(x, "final.norm") / 2.0))


@pytest.mark.parametrize("name", ["luA", "luB"])
def test_the_test_models_route_by_the_tokens_embedding_alone(name, tmp_path):
    """What ``make_folder`` promises: the router's channels hold a positive multiple of the token's embedding in every pass, so a
    token chooses the same experts wherever it stands."""
    folder = make_folder(tmp_path, name)
    cfg, w = read_model_folder(folder)
    toks = tokens_for(folder, 60, 3)
    assert set(toks) <= set(decisive_tokens(folder).tolist())
    seen = {}
    L.forward(cfg, w, toks, watch=lambda run, i, x: seen.setdefault((run, i), x))
    r = ROUTER_CHANNELS
    e = w["embed"][toks][:, -r:] * cfg["embedding"]["scale"]
    by_token = {}
    for (run, i), x in seen.items():
        k = x[:, -r:] / e
        assert np.allclose(k, k[0, 0]) and k[0, 0] >= 1 - 1e-9
        p = f"l{i}."
        h = L.layer_norm(x, w[p + "norm2"], w[p + "norm2.b"], cfg["norm"]["eps"])
        assert np.abs(x.mean(axis=-1)).max() < 2.0 * k[0, 0], "the allowance of decisive_tokens for the norm's mean"
        chosen, _ = L.route(h, w[p + "mlp.router"], w[p + "mlp.correction"], cfg["layers"][i]["mlp"]["router"])
        for t, c in zip(toks, chosen):
            assert by_token.setdefault((i, t), set(c)) == set(c)


@pytest.mark.parametrize("name", sorted(set(LUTOSUN) - {"luE"}))  # (luE's ones leave some options without effect, on purpose)
def test_the_models_show_what_is_left_out(name, tmp_path, monkeypatch):
    """What the comparisons are worth: with these weights a missing bias, norm weight, correction, gate, pair row, step vector or
    restart, another limit, scale, base, bound or order of the turned pairs, one choice fewer or a pass that shares another's
    input moves the logits by far more than the tolerance."""
    folder = make_folder(tmp_path, name)
    cfg, w = read_model_folder(folder)
    toks = tokens_for(folder, 150, 1)
    want = L.forward(cfg, w, toks)
    floor = 20 * 1e-4 * np.abs(want).max()

    def moved(c=cfg, weights=w):
        return np.abs(L.forward(c, weights, toks) - want).max()

    def other(change):
        off = copy.deepcopy(cfg)
        change(off)
        return off

    changes = {"the embedding's scale": lambda c: c["embedding"].update(scale=1.1 * c["embedding"]["scale"]),
               "the residual's factor": lambda c: c.update(residual_mult=0.9 * c["residual_mult"]),
               "the bound": lambda c: c.update(logit_softcap=1.2 * c["logit_softcap"] if c["logit_softcap"] else 30.0)}
    zeros, ones = ["final.norm.b"], ["final.norm"]
    if cfg["embedding"]["bigram"]:
        zeros.append("bigram")
        if cfg["embedding"]["bigram"]["mul_prev"]:
            changes["the previous token"] = lambda c: c["embedding"]["bigram"].update(mul_prev=0)
        first = dict(w, bigram=w["bigram"].copy())
        first["bigram"][-1] = 0.0
        assert np.abs(L.forward(cfg, first, toks) - want)[0].max() > floor, "the first token's row"
    if cfg["loop"]:
        zeros.append("loop.step")
    for i, layer in enumerate(cfg["layers"]):
        m, mlp, p = layer["mixer"], layer.get("mlp"), f"l{i}."
        zeros += [p + "norm1.b", p + "mix.uq"]
        ones += [p + "norm1", p + "mix.dq.norm", p + "mix.dkv.norm"]
        if m["rot"]["dims"] > 2:  # (one pair turns by the position itself, whatever the base)
            changes[f"base {i}"] = lambda c, i=i: c["layers"][i]["mixer"]["rot"].update(base=7.0)
        changes[f"attention scale {i}"] = lambda c, i=i: c["layers"][i]["mixer"].update(scale=1.2 * c["layers"][i]["mixer"]["scale"])
        if not mlp:
            continue
        zeros += [p + "norm2.b", p + "mlp.shared.sg"]
        changes[f"router scale {i}"] = lambda c, i=i: c["layers"][i]["mlp"]["router"].update(scale=1.0)
        for key in ("expert", "shared"):
            changes[f"{key} limit {i}"] = lambda c, i=i, key=key: c["layers"][i]["mlp"][key].update(limit=1.3 * c["layers"][i]["mlp"][key]["limit"])
        if mlp["router"]["experts"] > mlp["router"]["top"] + 1:
            zeros.append(p + "mlp.correction")
        if mlp["router"]["top"] > 1:
            changes[f"choices {i}"] = lambda c, i=i: c["layers"][i]["mlp"]["router"].update(top=c["layers"][i]["mlp"]["router"]["top"] - 1)
    for key in zeros:
        assert moved(weights={**w, key: w[key] * 0.0}) > floor, (name, key)
    for key in ones:
        assert moved(weights={**w, key: np.ones_like(w[key])}) > floor, (name, key)
    for what, change in changes.items():
        assert moved(other(change)) > floor, (name, what)
    with monkeypatch.context() as patch:
        if cfg["loop"] and cfg["loop"]["times"] > 1:
            patch.setattr(L, "begin_pass", lambda x, start, steps, t: x + steps[t])
            assert moved() > floor, (name, "the restart")
    with monkeypatch.context() as patch:
        swapped = lambda x, pos, rot: L_rotate(x[..., ::-1], pos, rot)[..., ::-1]
        L_rotate = L.rotate_neighbours
        patch.setattr(L, "rotate_neighbours", swapped)
        assert moved() > floor, (name, "the direction of the turn")
    # tokens far back matter to the last one
    other_start = list(toks)
    other_start[:3] = tokens_for(folder, 3, 77)
    assert np.abs(L.forward(cfg, w, other_start)[-1] - want[-1]).max() > 3 * 1e-4 * np.abs(want).max()
