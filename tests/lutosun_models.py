"""Small Lutosun configurations for the tests. They differ from one another in every size and option: runs of layers that are
run once, twice and three times, at the start, in the middle and at the end of the model or not at all, with and without a row
per pair of tokens, sizes that are multiples of nothing, sizes that the matrix-core kernels take, latents wider than 256, partly
turned key parts, one expert, one chosen, every expert chosen, layers without a feed-forward, limits that bite and limits that
do not.

``make_folder`` draws random weights and then makes them telling: biases, step vectors, corrections and gates large enough to
matter, and a router whose choice is exact in every number format. It reads only the stream's last channels, which no sublayer
and nothing that joins the stream later writes, so they hold the token's embedding times the number of passes begun, and it
reads differences of neighbours among them, from which a layer norm's mean drops out; the norm's factor is positive and leaves
the order of the scores alone. The corrections take one expert in always and one never, and are zero otherwise.
``decisive_tokens`` keeps the tokens whose choice no rounding of those channels to bfloat16 could change. In bfloat16 a router fed
by a rounded stream would otherwise now and then choose another expert than the plain implementation, and the comparison would
say nothing about the kernels."""

from __future__ import annotations

from pathlib import Path

import numpy as np
import torch
from safetensors.torch import load_file, save_file

from miniserve_amd.weights.random_init import Init, write_model_folder
from plain.model_folder import read_model_folder

ROUTER_CHANNELS = 8  # the stream's last channels: the routers read nothing else


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base=100.0, dims=None, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
                      "rot": {"base": base, "dims": rot_dim if dims is None else dims}}}


def moe(experts, top, ff, shared, limit=1.0, shared_limit=0.8, scale=1.7):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff, "limit": limit},
            "shared": {"ff": shared, "limit": shared_limit}}


def model(vocab, width, eps, layers, loop=None, bigram=(97, 13, 5), scale=1.5, mult=0.8, cap=12.0):
    return {"architecture": "Lutosun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "logit_softcap": cap,
            "embedding": {"scale": scale, "bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram)) if bigram else None},
            "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None, "layers": layers}


LUTOSUN = {
    # name: (config, seed, init)
    "luA": (model(101, 64, 1e-5, [
        latent(4, 16, 8, 12, 24, 40, 0.2, mlp=moe(5, 2, 24, 40)), latent(3, 8, 16, 20, 32, 24, 0.25, 50.0, mlp=moe(4, 1, 40, 16, 0.5)),
        latent(2, 24, 8, 16, 20, 32, 0.2, mlp=None), latent(5, 16, 8, 8, 24, 40, 0.2, 300.0, mlp=moe(6, 3, 16, 24))], loop=(1, 3, 2)), 61,
        Init(0.12, (0.6, 1.4))),
    # sizes that are multiples of nothing, a loop over the last layers, every expert chosen, partly turned key parts
    "luB": (model(77, 90, 1e-6, [
        latent(5, 6, 6, 14, 23, 22, 0.3, 30.0, 4, moe(3, 3, 50, 30, 2.0)), latent(3, 10, 4, 7, 17, 33, 0.3, 60.0, 2, moe(7, 2, 18, 9, 0.7, 0.5))],
        loop=(0, 2, 3), bigram=(31, 1000003, 2 ** 40 + 1), scale=0.7, mult=1.0, cap=5.0), 62, Init(0.12, (0.5, 1.5))),
    # no loop, no row per pair, no bound on the logits
    "luC": (model(64, 72, 1e-5, [latent(2, 16, 8, 24, 16, 48, 0.2, mlp=moe(4, 2, 16, 20)), latent(6, 12, 4, 10, 28, 36, 0.25, mlp=moe(2, 1, 32, 8))],
                  bigram=None, scale=1.0, mult=0.6, cap=None), 63, Init(0.12, (0.6, 1.4))),
    # sizes that the matrix-core kernels take; more experts than a tile has rows; a latent of more than 256 elements
    "luD": (model(400, 128, 1e-5, [
        latent(8, 64, 32, 64, 64, 96, 0.1, 1000.0, mlp=moe(20, 4, 64, 64)), latent(4, 32, 32, 48, 96, 288, 0.12, 1000.0, 16, moe(9, 3, 32, 128)),
        latent(16, 32, 32, 32, 80, 128, 0.12, 1000.0, mlp=moe(24, 1, 64, 48))], loop=(0, 1, 2), bigram=(509, 211, 7)), 64, Init(0.1, (0.6, 1.4))),
    # values that are one: one head, one expert, one pass, one bucket, one channel a head
    "luE": (model(53, 40, 1e-4, [
        latent(1, 8, 2, 8, 8, 8, 0.3, 20.0, mlp=moe(1, 1, 8, 1, 1.0, 1.0, 1.0)), latent(2, 1, 4, 1, 6, 12, 0.3, 50.0, 2, moe(3, 1, 1, 8))],
        loop=(1, 2, 1), bigram=(1, 1, 1), scale=1.0, mult=1.0, cap=6.0), 65, Init(0.15, (0.6, 1.4))),
}


def make_telling(folder: Path, cfg: dict, seed: int, router: bool = True) -> None:
    """``router=False`` leaves the routers as drawn, over the whole width (in float32 their choice needs no help)."""
    gen = torch.Generator().manual_seed(seed + 1000)
    file = folder / "model.safetensors"
    t = load_file(str(file))
    r = ROUTER_CHANNELS

    def redraw(name, mean, spread):
        t[name] = (torch.randn(t[name].shape, generator=gen) * spread + mean).to(torch.bfloat16)

    redraw("embed", 0.0, 0.6)
    if "bigram" in t:
        redraw("bigram", 0.0, 0.6)
    if "loop.step" in t:
        redraw("loop.step", 0.0, 0.5)
    redraw("final.norm.b", 0.0, 0.3)
    redraw("head", 0.0, 3.0 * cfg["width"] ** -0.5)
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        redraw(p + "norm1.b", 0.0, 0.4)
        for name, size in (("dq", cfg["width"]), ("dkv", cfg["width"]), ("uq", m["q_rank"]), ("uk", m["kv_rank"]), ("uv", m["kv_rank"])):
            redraw(p + "mix." + name, 0.0, 1.4 * size ** -0.5)
        redraw(p + "mix.o", 0.0, 1.5 * (m["heads"] * m["vdim"]) ** -0.5)
        if not mlp:
            continue
        redraw(p + "norm2.b", 0.0, 0.4)
        n = mlp["router"]["experts"]
        corr = torch.zeros(n)
        if n > mlp["router"]["top"] + 1:
            corr[n // 2], corr[0] = 2.0, -2.0  # one is always taken, one never
        t[p + "mlp.correction"] = corr.to(torch.bfloat16)
        redraw(p + "mlp.shared.sg", 0.0, 1.0 * cfg["width"] ** -0.5)
        for e in [f"e{j}" for j in range(n)] + ["shared"]:
            ff = mlp["shared" if e == "shared" else "expert"]["ff"]
            for name, size in (("gate", cfg["width"]), ("up", cfg["width"]), ("down", ff)):
                redraw(p + f"mlp.{e}.{name}", 0.0, 1.2 * size ** -0.5)
    if router:
        for name in ("bigram", "loop.step"):
            if name in t:
                t[name][:, -r:] = 0.0
        t["embed"][:, -r:] = (torch.randn((t["embed"].shape[0], r), generator=gen) * 2).to(torch.bfloat16)
        for i, layer in enumerate(cfg["layers"]):
            p, mlp = f"l{i}.", layer.get("mlp")
            for name in [k for k in t if k == p + "mix.o" or (k.startswith(p + "mlp.") and k.endswith(".down"))]:
                t[name][-r:] = 0.0
            if mlp:
                t[p + "norm2"][-r:] = 1.0
                t[p + "norm2.b"][-r:] = 0.0
                n = mlp["router"]["experts"]
                half = (torch.randn((n, r // 2), generator=gen) * 0.5).to(torch.bfloat16)
                t[p + "mlp.router"] = torch.zeros_like(t[p + "mlp.router"])
                t[p + "mlp.router"][:, -r:] = torch.stack((half, -half), dim=-1).reshape(n, r)
    save_file({k: v.contiguous() for k, v in t.items()}, str(file))


def make_folder(tmp: Path, name: str) -> Path:
    cfg, seed, init = LUTOSUN[name]
    folder = write_model_folder(Path(tmp) / name, cfg, seed, init)
    make_telling(folder, cfg, seed)
    return folder


def decisive_tokens(folder, mean_allowance=2.0):
    """The token ids whose choice of experts is beyond rounding in every mixture of the model: the gap between the last score
    that is chosen and the first that is not is at least twice what rounding the router's channels could move a logit by (a
    2^-9 part of each term, the norm's mean allowed for in its size)."""
    cfg, w = read_model_folder(folder)
    r = ROUTER_CHANNELS
    ok = np.ones(cfg["vocab"], dtype=bool)
    e = w["embed"][:, -r:] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        mlp = layer.get("mlp")
        if not mlp or mlp["router"]["top"] == mlp["router"]["experts"]:
            continue
        p, top = f"l{i}.mlp.", mlp["router"]["top"]
        router = w[p + "router"][:, -r:]
        z = e @ router.T + 1e3 * w[p + "correction"]
        z = np.sort(z, axis=-1)[:, ::-1]
        ok &= z[:, top - 1] - z[:, top] > 4 * 2.0 ** -9 * ((np.abs(e) + mean_allowance) @ np.abs(router).T).max(axis=-1)
    return np.flatnonzero(ok)


def tokens_for(folder, n, seed):
    pool = decisive_tokens(folder)
    assert len(pool) >= 12, f"only {len(pool)} tokens choose their experts clearly"
    return pool[np.random.default_rng(seed).integers(0, len(pool), size=n)].tolist()
