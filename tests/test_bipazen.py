"""Bipazen on the CPU: its configuration and lowering (layers that run another layer's weights over a state of their own,
what the cache manager makes of latents and states), the layer scale's place in the parts, and the plain implementation
held against forms that do not share its loops."""

from __future__ import annotations

import copy
import math

import numpy as np
import pytest
import torch

from bipazen_models import BIPAZEN, ROUTER_CHANNELS, decisive_tokens, make_folder, tokens_for
from miniserve_amd.cache import CacheLayout
from miniserve_amd.config import config_from_dict
from miniserve_amd.config.presets import preset
from miniserve_amd.config.spec import PartSpec
from miniserve_amd.parts.base import FeedForward, Mixer
from miniserve_amd.parts.model import CacheSlotNeed, expected_tensors
from miniserve_amd.parts.registry import part_class
from plain import bipazen_plain as B
from plain.model_folder import read_model_folder


# ---------------------------------------------------------------- configuration


@pytest.mark.parametrize("name", sorted(BIPAZEN))
def test_config_reads_back_and_names_its_tensors(name):
    cfg = BIPAZEN[name][0]
    c = config_from_dict(cfg)
    assert config_from_dict(c.to_dict()).to_dict() == c.to_dict()
    names = expected_tensors(c.to_spec())
    w = cfg["width"]
    assert names["embed"].shape == (cfg["vocab"], w) and names["final.norm"].shape == (w,) and "head" not in names
    for i, layer in enumerate(cfg["layers"]):
        m, mlp, p = layer["mixer"], layer["mlp"], f"l{i}."
        if layer.get("weights_of") is not None:
            assert not any(k.startswith(p) for k in names), "a layer that runs another's weights has no tensors"
            continue
        assert names[p + "norm1"].shape == names[p + "ls1"].shape == (w,)
        assert names[p + "norm2"].optional == names[p + "ls2"].optional == (not mlp)
        if layer["type"] == "mamba2":
            inner, keys = m["heads"] * m["vdim"], m["groups"] * m["state"]
            assert names[p + "mix.in"].shape == (2 * inner + 2 * keys + m["heads"], w)
            assert names[p + "mix.conv"].shape == (inner + 2 * keys, m["conv"]) and names[p + "mix.conv.b"].shape == (inner + 2 * keys,)
            assert names[p + "mix.A_log"].shape == names[p + "mix.D"].shape == names[p + "mix.dt_bias"].shape == (m["heads"],)
            assert names[p + "mix.norm"].shape == (inner,) and names[p + "mix.o"].shape == (w, inner)
        elif layer["type"] == "rglru":
            n, bs = m["width"], m["width"] // m["blocks"]
            assert names[p + "mix.y"].shape == names[p + "mix.x"].shape == (n, w) and names[p + "mix.o"].shape == (w, n)
            assert names[p + "mix.ra"].shape == names[p + "mix.ri"].shape == (m["blocks"], bs, bs)
            assert names[p + "mix.ra.b"].shape == names[p + "mix.ri.b"].shape == (m["blocks"], bs)
            assert names[p + "mix.conv"].shape == (n, m["conv"])
            assert {names[p + "mix." + k].shape for k in ("y.b", "x.b", "conv.b", "lam")} == {(n,)}
        else:
            h, d, r, e, c_ = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
            assert names[p + "mix.q"].shape == (h * (d + r), w) and names[p + "mix.dkv"].shape == (c_ + r, w)
            assert names[p + "mix.uk"].shape == (h * d, c_) and names[p + "mix.uv"].shape == (h * e, c_)
            assert names[p + "mix.g"].shape == (h * e, w) and names[p + "mix.o"].shape == (w, h * e) and p + "mix.sink" not in names
        if not mlp:
            assert not any(k.startswith(p + "mlp.") for k in names)
        else:
            e, f = mlp["router"]["experts"], mlp["expert"]["ff"]
            assert names[p + "mlp.router"].shape == (e, w) and names[p + f"mlp.e{e - 1}.gate"].shape == (f, w)
            assert names[p + "mlp.e0.down"].shape == (w, f) and p + f"mlp.e{e}.up" not in names


def test_layers_that_run_anothers_weights_have_a_state_of_their_own():
    spec = config_from_dict(BIPAZEN["bpA"][0]).to_spec()
    assert [(e.layer, e.cache, e.writes_cache) for e in spec.run_order] == [
        (0, 0, True), (1, 1, True), (2, 2, True), (1, 3, True), (0, 4, True), (3, 5, True), (2, 6, True)]
    assert [layer.prefix for layer in spec.layers] == ["l0.", "l1.", "l2.", "l5."]
    cfg = copy.deepcopy(BIPAZEN["bpC"][0])
    first = cfg["layers"][0]
    cfg["layers"] = [dict(copy.deepcopy(first), weights_of=3), cfg["layers"][1], dict(copy.deepcopy(first), weights_of=0), first]
    spec = config_from_dict(cfg).to_spec()
    assert [layer.prefix for layer in spec.layers] == ["l1.", "l3."]
    assert [(e.layer, e.cache) for e in spec.run_order] == [(1, 0), (0, 1), (1, 2), (1, 3)]


def needs(name):
    spec = config_from_dict(BIPAZEN[name][0]).to_spec()
    out = []
    for e in spec.run_order:
        layer = spec.layers[e.layer]
        mixer = part_class("mixer", layer.mixer)(layer.mixer, None)
        out.append(CacheSlotNeed(e.cache, mixer.kv_need(), mixer.state_need()))
    return out


def test_cache_groups_and_states():
    a = needs("bpA")
    assert [n.kv is not None for n in a] == [False, True, False, True, False, False, False]
    assert a[1].kv.window == 0 and [(p.heads, p.width) for p in a[1].kv.planes] == [(1, 48), (1, 40)] and a[1].kv == a[3].kv
    assert {t.name: t.shape for t in a[0].state.tensors} == {"S": (4, 24, 16), "conv": (3, 64 + 2 * 2 * 24)}
    assert {t.name: t.shape for t in a[2].state.tensors} == {"S": (60,), "conv": (2, 60)}
    layout = CacheLayout.from_needs(a)
    assert len(layout.groups) == 1 and layout.groups[0].slots == (1, 3)
    assert len(CacheLayout.from_needs(needs("bpC")).groups) == 0
    assert {t.name for t in needs("bpB")[1].state.tensors} == {"S"}, "a convolution of one tap keeps no inputs"


def test_config_refusals():
    base = BIPAZEN["bpA"][0]

    def broken(change):
        cfg = copy.deepcopy(base)
        change(cfg)
        return cfg

    for change, error in [
        (lambda c: c["layers"][1].update(type="attention"), NotImplementedError),
        (lambda c: c["layers"][0]["mixer"].update(groups=3), ValueError),
        (lambda c: c["layers"][0]["mixer"].update(norm_groups=5), ValueError),
        (lambda c: c["layers"][0]["mixer"].update(conv=0), ValueError),
        (lambda c: c["layers"][0]["mixer"].pop("state"), KeyError),
        (lambda c: c["layers"][2]["mixer"].update(blocks=7), ValueError),
        (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10), ValueError),
        (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3), ValueError),
        (lambda c: c["layers"][1]["mixer"].update(scale=0.0), ValueError),
        (lambda c: c["layers"][3].update(weights_of=9), ValueError),
        (lambda c: c["layers"][3].update(weights_of=0), ValueError),               # a layer of another kind
        (lambda c: c["layers"][1].update(weights_of=3), ValueError),               # a ring: nobody has the tensors
        (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), ValueError),
        (lambda c: c["layers"][1]["mlp"].update(kind="dense"), NotImplementedError),
        (lambda c: c.pop("norm"), KeyError),
    ]:
        with pytest.raises(error):
            config_from_dict(broken(change))


def test_the_preset_and_the_measured_shapes_are_valid_configurations():
    from miniserve_amd.measurement.designs import SHAPES, bipazen_config

    for cfg in [preset("bipazen-tiny")] + [bipazen_config(s) for s in SHAPES.values()]:
        spec = config_from_dict(cfg).to_spec()
        assert spec.architecture == "Bipazen" and len(spec.run_order) == len(cfg["layers"])
        assert {layer["type"] for layer in cfg["layers"]} == {"mamba2", "rglru", "latent_attention"}


# ---------------------------------------------------------------- parts


class _Norm:
    def __init__(self):
        self.tensors_seen = None

    def bind(self, tensors):
        self.tensors_seen = set(tensors)


def test_a_layer_scale_goes_to_the_sublayers_and_only_to_those_that_take_one():
    class Takes(Mixer):
        scales_output = True

    class TakesToo(FeedForward):
        scales_output = True

    norm = lambda t: PartSpec("rmsnorm", {"width": 4, "eps": 1e-5, "tensor": t})
    spec = PartSpec("prenorm", {"mixer_norm": norm("n1"), "ffn_norm": norm("n2"), "mixer_scale": "s1", "ffn_scale": "s2"})
    cls = part_class("block", spec)
    assert set(cls.tensors(spec)) == {"n1", "n2", "s1", "s2"}
    block = cls(spec, None, Takes(PartSpec("m"), None), TakesToo(PartSpec("f"), None))
    s1, s2 = torch.arange(4.0).to(torch.bfloat16), torch.ones(4).to(torch.bfloat16)
    block.bind({"n1": s2, "n2": s2, "s1": s1, "s2": s2})
    assert block.mixer.out_scale.dtype == torch.float32 and block.mixer.out_scale.tolist() == [0.0, 1.0, 2.0, 3.0]
    assert block.feed_forward.out_scale.tolist() == [1.0] * 4

    class Plain(Mixer):
        kind = "plain"

    block = cls(spec, None, Plain(PartSpec("m"), None), TakesToo(PartSpec("f"), None))
    with pytest.raises(NotImplementedError):
        block.bind({"n1": s2, "n2": s2, "s1": s1, "s2": s2})
    without = PartSpec("prenorm", {"mixer_norm": norm("n1"), "ffn_norm": None, "mixer_scale": "s1", "spare": {"n2": 4, "s2": 4}})
    got = cls.tensors(without)
    assert not got["s1"].optional and got["n2"].optional and got["s2"].optional


def test_a_mixture_hands_its_scale_to_the_shared_expert():
    shared = PartSpec("dense_mlp", {"prefix": "s.", "hidden_size": 4, "intermediate_size": 8})
    spec = PartSpec("moe_mlp", {"hidden_size": 4, "intermediate_size": 8, "num_experts": 2, "top": 1, "scoring": "sigmoid", "weigh": "input",
                                "shared": shared})
    part = part_class("feed_forward", spec)(spec, None)
    part.scale_output(torch.full((4,), 2.0))
    assert part.shared.out_scale.tolist() == part.out_scale.tolist() == [2.0] * 4
    with pytest.raises(ValueError):
        part_class("feed_forward", spec)(PartSpec("moe_mlp", dict(spec.params, weigh="both")), None)


# ---------------------------------------------------------------- the plain implementation against other forms


def test_convolution_by_hand():
    u = np.array([[1.0], [10.0], [100.0], [1000.0]])
    y = B.causal_conv(u, np.array([[2.0, 3.0, 5.0]]), np.array([7.0]))
    assert y[:, 0].tolist() == [7 + 5, 7 + 50 + 3, 7 + 500 + 30 + 2, 7 + 5000 + 300 + 20]
    assert np.array_equal(B.causal_conv(u[:1], np.array([[2.0, 3.0, 5.0]]), np.array([0.0])), [[5.0]])


def test_step_recurrence_as_a_sum_over_earlier_tokens():
    """``o_t = sum_(j <= t) exp(sum_(j < i <= t) log_decay_i) step_j (q_t . k_j) v_j + skip v_t``: the recurrence written out."""
    rng = np.random.default_rng(0)
    T, H, N, E = 25, 3, 5, 4
    q, k = rng.normal(size=(T, H, N)), rng.normal(size=(T, H, N))
    v = rng.normal(size=(T, H, E))
    step = B.softplus(rng.normal(size=(T, H)))
    la = -np.exp(rng.normal(size=H)) * step
    skip = rng.normal(size=H)
    out, S = B.scalar_decay_recurrence(q, k, v, la, step, skip)
    cum = np.cumsum(la, axis=0)
    for t in range(T):
        for h in range(H):
            want = sum(np.exp(cum[t, h] - cum[j, h]) * step[j, h] * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1)) + skip[h] * v[t, h]
            assert np.allclose(out[t, h], want)
    assert np.allclose(S[1], sum(np.exp(cum[-1, 1] - cum[j, 1]) * step[j, 1] * np.outer(k[j, 1], v[j, 1]) for j in range(T)))


def test_channel_recurrence_as_a_sum_over_earlier_tokens():
    rng = np.random.default_rng(1)
    T, W = 30, 6
    la, x = -np.exp(rng.normal(size=(T, W)) * 2 - 2), rng.normal(size=(T, W))
    got = B.channel_recurrence(la, x)
    cum = np.cumsum(la, axis=0)
    for t in (0, 1, 13, T - 1):
        want = sum(np.exp(cum[t] - cum[j]) * np.sqrt(1 - np.exp(la[j]) ** 2) * x[j] for j in range(t + 1))
        assert np.allclose(got[t], want)


def test_latent_attention_of_one_token_returns_its_gated_value():
    rng = np.random.default_rng(2)
    W = 12
    m = {"heads": 2, "dim": 3, "rot_dim": 4, "vdim": 5, "kv_rank": 6, "scale": 0.7, "rot": {"base": 10.0, "dims": 4}}
    w = {"q": rng.normal(size=(14, W)), "dkv": rng.normal(size=(10, W)), "dkv.norm": rng.normal(size=6), "uk": rng.normal(size=(6, 6)),
         "uv": rng.normal(size=(10, 6)), "g": rng.normal(size=(10, W)), "o": np.eye(10)}
    h = rng.normal(size=(1, W))
    c = (h @ w["dkv"].T)[:, :6]
    c = c / np.sqrt((c * c).mean() + 1e-5) * w["dkv.norm"]
    want = (c @ w["uv"].T) / (1 + np.exp(-(h @ w["g"].T)))
    assert np.allclose(B.latent_attention(h, w, m, 1e-5, np.arange(1.0)), want)


def test_rotation_turns_halves_by_the_distance():
    """Scores of turned vectors depend on the distance of their places alone, and what lies behind the turned part passes."""
    rng = np.random.default_rng(3)
    a, b = rng.normal(size=(1, 1, 10)), rng.normal(size=(1, 1, 10))
    rot = {"base": 50.0, "dims": 6}
    at = lambda x, p: B.rotate_halves(x, np.array([float(p)]), rot)[0, 0]
    assert np.isclose(at(a, 3) @ at(b, 10), at(a, 33) @ at(b, 40)) and not np.isclose(at(a, 3) @ at(b, 10), at(a, 3) @ at(b, 11))
    assert np.array_equal(at(a, 9)[6:], a[0, 0, 6:]) and np.allclose(at(a, 0), a[0, 0])
    z = (a[0, 0, 1] + 1j * a[0, 0, 4]) * np.exp(1j * 7 * 50.0 ** (-2 / 6))
    assert np.allclose([at(a, 7)[1], at(a, 7)[4]], [z.real, z.imag])


def test_the_weight_multiplies_what_an_expert_reads():
    rng = np.random.default_rng(4)
    h = rng.normal(size=(5, 6))
    w = {"router": rng.normal(size=(3, 6)), **{f"e{j}.{k}": rng.normal(size=s) for j in range(3) for k, s in (("gate", (4, 6)), ("up", (4, 6)), ("down", (6, 4)))}}
    got = B.mixture_ff(h, w, {"router": {"experts": 3, "top": 1}})
    for t in range(5):
        z = w["router"] @ h[t]
        e = int(np.argmax(z))
        x = h[t] / (1 + math.exp(-z[e]))
        g = w[f"e{e}.gate"] @ x
        assert np.allclose(got[t], w[f"e{e}.down"] @ (g / (1 + np.exp(-g)) * (w[f"e{e}.up"] @ x)))


def test_a_one_layer_model_in_closed_form():
    """One rglru layer without a feed-forward, one token: no state yet, so the branch is sqrt(1 - a^2) i u."""
    cfg = {"architecture": "Bipazen", "vocab": 7, "width": 4, "norm": {"eps": 1e-6},
           "layers": [{"type": "rglru", "mixer": {"width": 4, "blocks": 2, "conv": 3}, "mlp": None}]}
    rng = np.random.default_rng(5)
    shapes = {"y": (4, 4), "y.b": (4,), "x": (4, 4), "x.b": (4,), "conv": (4, 3), "conv.b": (4,), "ra": (2, 2, 2), "ra.b": (2, 2), "ri": (2, 2, 2),
              "ri.b": (2, 2), "lam": (4,), "o": (4, 4)}
    w = {f"l0.mix.{k}": rng.normal(size=s) for k, s in shapes.items()}
    w.update({"embed": rng.normal(size=(7, 4)), "final.norm": rng.normal(size=4), "l0.norm1": rng.normal(size=4), "l0.ls1": rng.normal(size=4)})
    m = {k[7:]: v for k, v in w.items() if k.startswith("l0.mix.")}
    norm = lambda y, g: y / np.sqrt((y * y).mean() + 1e-6) * g
    x = w["embed"][2]
    h = norm(x, w["l0.norm1"])
    u = (m["x"] @ h + m["x.b"]) * m["conv"][:, 2] + m["conv.b"]
    gate = lambda k: 1 / (1 + np.exp(-np.concatenate([m[k][b] @ u[2 * b : 2 * b + 2] + m[k + ".b"][b] for b in range(2)])))
    a = np.exp(-8 * gate("ra") * np.log1p(np.exp(m["lam"])))
    x = x + w["l0.ls1"] * (m["o"] @ (np.sqrt(1 - a * a) * gate("ri") * u * B.gelu_tanh(m["y"] @ h + m["y.b"])))
    assert np.allclose(B.forward(cfg, w, [2])[0], w["embed"] @ norm(x, w["final.norm"]))


def test_the_test_models_route_by_the_tokens_embedding_alone(tmp_path):
    """What ``make_folder`` promises: no sublayer writes the stream's last channels, so a token chooses the same experts
    wherever it stands."""
    name = "bpA"
    folder = make_folder(tmp_path, name)
    cfg, w = read_model_folder(folder)
    toks = tokens_for(folder, 60, 3)
    assert set(toks) <= set(decisive_tokens(folder).tolist())
    seen = {}
    _, layers = B.forward(cfg, w, toks, return_layers=True, watch=lambda i, x: seen.setdefault(i, x))
    r = ROUTER_CHANNELS
    for after in layers:
        assert np.array_equal(after[:, -r:], w["embed"][toks][:, -r:])
    for i, x in seen.items():
        p = f"l{B.weights_layer(cfg, i)}."
        chosen, _ = B.route(B.weighted_norm(x, w[p + "norm2"], cfg["norm"]["eps"]), w[p + "mlp.router"], cfg["layers"][i]["mlp"]["router"]["top"])
        by_token = {}
        for t, c in zip(toks, chosen):
            assert by_token.setdefault(t, tuple(c)) == tuple(c)
