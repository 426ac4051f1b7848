"""Small Bipazen configurations for the tests. They differ from one another in every size and option: the order of the
three mixers, layers that run another layer's weights (an earlier or a later one's), one to eight heads to a group of keys
and queries, norms in one part, in a part per group and in a part per head, convolutions of one tap to nine, blocks of one
channel and one block of all, sizes that are multiples of nothing, sizes that the matrix-core kernels take, latents wider
than 256, partly turned key parts, one expert, one chosen, every expert chosen, layers without a feed-forward, and a model
that keeps no keys at all.

``make_folder`` draws random weights and then makes them telling: biases, steps, decays (some of them next to one), layer
scales and gates large enough to matter, and a router whose choice is exact in every number format. It reads only the
stream's last channels, which the layer scales keep out of every sublayer's reach (they are zero there), so they hold the
token's embedding, bit for bit; the norm in front of the feed-forward multiplies all of them by one positive factor, which
leaves the order of the scores alone, and ``decisive_tokens`` keeps the tokens whose choice no rounding of those channels to
bfloat16 could change. In bfloat16 a router fed by a rounded stream would otherwise now and then choose another expert than
the plain implementation, and the comparison would say nothing about the kernels."""

from __future__ import annotations

import copy
from pathlib import Path

import numpy as np
import torch
from safetensors.torch import load_file, save_file

from miniserve_amd.weights.random_init import Init, write_model_folder
from plain import bipazen_plain as B
from plain.model_folder import read_model_folder

ROUTER_CHANNELS = 8  # the stream's last channels: no sublayer writes them, the routers read nothing else


def mamba2(heads, vdim, state, groups, conv, norm_groups, mlp=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": norm_groups}, "mlp": mlp}


def rglru(width, blocks, conv, mlp=None):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": mlp}


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, base=100.0, dims=None, mlp=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                                                  "scale": scale, "rot": {"base": base, "dims": rot_dim if dims is None else dims}}, "mlp": mlp}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def again(layers, j):
    """Layer ``j`` of ``layers`` once more: its weights, a cache and state of its own."""
    return dict(copy.deepcopy(layers[j]), weights_of=j)


def model(vocab, width, eps, layers):
    return {"architecture": "Bipazen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def _bpa():
    layers = [mamba2(4, 16, 24, 2, 4, 2, moe(5, 2, 24)), latent(3, 16, 8, 12, 40, 0.2, mlp=moe(4, 1, 40)), rglru(60, 3, 3, moe(6, 3, 16))]
    layers += [again(layers, 1), again(layers, 0), rglru(48, 4, 2, None), again(layers, 2)]
    return model(101, 64, 1e-5, layers)


def _bpb():
    # sizes that are multiples of nothing; convolutions of five taps, of one and of nine; every expert chosen
    layers = [rglru(45, 5, 5, moe(3, 3, 50)), mamba2(3, 10, 7, 1, 1, 1, moe(6, 2, 10)), latent(5, 6, 6, 14, 22, 0.3, 30.0, 4, moe(7, 1, 18)),
              mamba2(6, 5, 33, 6, 9, 6, None)]
    return model(77, 90, 1e-6, layers + [again(layers, 0), again(layers, 2)])


def _bpc():
    # no keys kept anywhere
    layers = [mamba2(2, 24, 48, 1, 3, 1, moe(4, 2, 16)), rglru(72, 72, 4, moe(2, 1, 32)), rglru(36, 1, 8, moe(3, 1, 24))]
    return model(64, 72, 1e-5, layers + [again(layers, 0), again(layers, 1)])


def _bpd():
    # sizes that the matrix-core kernels take; more experts than a tile has rows; a latent of more than 256 elements
    return model(400, 128, 1e-5, [
        latent(8, 64, 32, 64, 96, 0.1, 1000.0, mlp=moe(20, 4, 64)), mamba2(8, 32, 64, 1, 4, 2, moe(6, 2, 128)), rglru(256, 2, 4, moe(24, 1, 64)),
        mamba2(4, 64, 128, 2, 4, 4, moe(4, 4, 64)), latent(4, 32, 32, 48, 288, 0.12, 1000.0, 16, moe(9, 3, 32)), mamba2(2, 136, 200, 2, 2, 2, None)])


def _bpe():
    # values that are one: one head, one group, one tap, one block, blocks of one channel, one expert, one channel a head
    return model(53, 40, 1e-4, [
        mamba2(1, 1, 1, 1, 1, 1, moe(1, 1, 8)), rglru(8, 8, 1, moe(2, 2, 8)), latent(1, 8, 2, 8, 8, 1.0, 20.0, mlp=moe(3, 1, 1)),
        rglru(1, 1, 2, None), mamba2(2, 4, 1, 2, 2, 1, moe(2, 1, 8)), latent(2, 1, 4, 1, 12, 0.5, 50.0, 2, None)])


BIPAZEN = {
    # name: (config, seed, init)
    "bpA": (_bpa(), 51, Init(0.12, (0.6, 1.4))),
    "bpB": (_bpb(), 52, Init(0.12, (0.5, 1.5))),
    "bpC": (_bpc(), 53, Init(0.12, (0.6, 1.4))),
    "bpD": (_bpd(), 54, Init(0.1, (0.6, 1.4))),
    "bpE": (_bpe(), 55, Init(0.15, (0.6, 1.4))),
}


def make_telling(folder: Path, cfg: dict, seed: int) -> None:
    gen = torch.Generator().manual_seed(seed + 1000)
    file = folder / "model.safetensors"
    t = load_file(str(file))
    r = ROUTER_CHANNELS

    def redraw(name, mean, spread):
        t[name] = (torch.randn(t[name].shape, generator=gen) * spread + mean).to(torch.bfloat16)

    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p = f"l{i}."
        for name in ("ls1", "ls2"):
            if p + name in t:
                t[p + name][-r:] = 0.0  # the sublayers add nothing to the router's channels
        if layer["type"] == "mamba2":
            redraw(p + "mix.dt_bias", -1.0, 1.0)
            redraw(p + "mix.A_log", -1.5, 1.5)  # decays from next to one to nearly nothing
            redraw(p + "mix.D", 0.8, 0.4)
            redraw(p + "mix.conv", 0.0, 0.5)
            redraw(p + "mix.conv.b", 0.0, 0.3)
        elif layer["type"] == "rglru":
            redraw(p + "mix.lam", -3.0, 2.0)
            redraw(p + "mix.conv", 0.0, 0.6)
            for name in ("y.b", "x.b", "conv.b", "ra.b", "ri.b"):
                redraw(p + "mix." + name, 0.0, 0.4)
            for name in ("ra", "ri"):
                redraw(p + "mix." + name, 0.0, 0.8 * t[p + "mix." + name].shape[-1] ** -0.5)
        else:
            redraw(p + "mix.g", 0.0, 0.3)
        if layer.get("mlp"):
            router = torch.zeros_like(t[p + "mlp.router"])
            router[:, -r:] = (torch.randn((router.shape[0], r), generator=gen) * 0.4).to(torch.bfloat16)
            t[p + "mlp.router"] = router
    t["embed"][:, -r:] = torch.randn((t["embed"].shape[0], r), generator=gen).to(torch.bfloat16)
    save_file({k: v.contiguous() for k, v in t.items()}, str(file))


def make_folder(tmp: Path, name: str) -> Path:
    cfg, seed, init = BIPAZEN[name]
    folder = write_model_folder(Path(tmp) / name, cfg, seed, init)
    make_telling(folder, cfg, seed)
    return folder


def decisive_tokens(folder, margin=0.012):
    """The token ids whose choice of experts is beyond rounding in every mixture of the model: the gap between the last score
    that is chosen and the first that is not is at least ``margin`` of the sum of the terms' sizes. (A channel rounded to
    bfloat16 moves by a 2^-9 part of itself, so a logit by at most that part of the sum.)"""
    cfg, w = read_model_folder(folder)
    r = ROUTER_CHANNELS
    ok = np.ones(cfg["vocab"], dtype=bool)
    for i, layer in enumerate(cfg["layers"]):
        mlp = layer.get("mlp")
        if not mlp or mlp["router"]["top"] == mlp["router"]["experts"]:
            continue
        p = f"l{B.weights_layer(cfg, i)}."
        h = w["embed"][:, -r:] * w[p + "norm2"][-r:]
        router = w[p + "mlp.router"][:, -r:]
        z = np.sort(h @ router.T, axis=-1)[:, ::-1]
        top = mlp["router"]["top"]
        ok &= z[:, top - 1] - z[:, top] > margin * (np.abs(h) @ np.abs(router).T).max(axis=-1)
    return np.flatnonzero(ok)


def tokens_for(folder, n, seed):
    pool = decisive_tokens(folder)
    assert len(pool) >= 12, f"only {len(pool)} tokens choose their experts clearly"
    return pool[np.random.default_rng(seed).integers(0, len(pool), size=n)].tolist()
