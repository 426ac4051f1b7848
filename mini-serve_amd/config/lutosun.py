"""Typed configuration of the Lutosun decoder, read from its own ``config.json`` keys. The reference has no such
architecture.

``config.json``: ``architecture`` (the name), ``vocab``, ``width``, ``norm.eps``, ``embedding``, ``residual_mult``,
``logit_softcap`` and ``layers``, a list in which every entry names its mixer (``type``), the mixer's sizes and constants
(``mixer``) and its feed-forward (``mlp``, or null for none). Layer ``i``'s tensors start with ``l<i>.``.

* ``embedding``: the token's row of ``embed`` times ``scale``; with ``bigram`` (``buckets``, ``mul_prev``, ``mul_cur``) plus row
  ``(previous token * mul_prev + token * mul_cur) mod buckets`` of ``bigram [buckets + 1, width]``, the last row for a
  sequence's first token.
* ``loop`` (optional; ``start``, ``stop``, ``times``): layers ``start .. stop - 1`` run ``times`` times in a row with the same
  weights, every pass over a cache of its own. In front of pass ``t`` row ``t`` of ``loop.step [times, width]`` joins the stream,
  and in front of every pass but the first the embedding's output as well.
* A layer is ``x += m mixer(N1(x))``, then ``x += m ff(N2(x))`` with ``m`` = ``residual_mult`` and layer norms (tensors ``norm1 norm2``,
  biases ``norm1.b norm2.b``).
* ``latent_attention`` (``heads``, ``dim``, ``rot_dim``, ``vdim``, ``q_rank``, ``kv_rank``, ``scale``, ``rot``; tensors ``mix.dq dq.norm uq
  dkv dkv.norm uk uv o``): queries ``uq N(dq h)`` with an RMS norm over the ``q_rank`` elements of their latent; ``dkv`` projects to
  ``kv_rank`` latent elements (RMS-normed, weight ``dkv.norm``) and ``rot_dim`` elements of a key part shared by all heads; ``uk``
  / ``uv`` make each head's plain key part (``dim``) and value (``vdim``) from the latent; query heads are ``[dim plain, rot_dim
  rotated]``. The rotation turns the first ``rot.dims`` rotated elements, neighbours paired, by ``position * rot.base ** (-2i /
  rot.dims)``. Every earlier token is visible.
* Feed-forward (``kind: moe``; ``router.experts``, ``router.top``, ``router.scale``, ``expert.ff``, ``expert.limit``, ``shared.ff``,
  ``shared.limit``; tensors ``mlp.router correction``, ``mlp.e<j>.gate up down``, ``mlp.shared.gate up down sg``): scores ``s`` =
  ``softmax(router h)`` over all experts; the ``top`` largest ``s + correction`` are chosen; weights are the chosen ``s`` divided by their
  sum, times ``router.scale``. An expert is ``down(g sigmoid(1.702 g) (u + 1))`` with ``g = min(gate h, limit)``, ``u = clamp(up h,
  -limit, limit)``. A shared expert of the same form runs for every token and is added, times ``sigmoid(sg h)``.

The final norm is ``final.norm`` / ``final.norm.b``, the head ``head``; logits are ``cap * tanh(logits / cap)``.
"""

from __future__ import annotations

import copy
from dataclasses import dataclass

from .registry import register_architecture
from .spec import LayerSpec, ModelSpec, PartSpec, RunEntry

MIXER_TYPES = ("latent_attention",)
MIXER_SIZES = ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")


def _need(d, keys, where: str) -> None:
    if not isinstance(d, dict):
        raise ValueError(f"{where} must be an object, got {d!r}")
    missing = [k for k in keys if k not in d]
    if missing:
        raise KeyError(f"config.json lacks {missing} in {where}")


def _int(d: dict, key: str, where: str, least: int = 1) -> int:
    v = d[key]
    if not isinstance(v, int) or isinstance(v, bool) or v < least:
        raise ValueError(f"{where}.{key} must be an integer of at least {least}, got {v!r}")
    return v


def _positive(d: dict, key: str, where: str) -> float:
    v = d[key]
    if not isinstance(v, (int, float)) or isinstance(v, bool) or not v > 0:
        raise ValueError(f"{where}.{key} must be a positive number, got {v!r}")
    return float(v)


@register_architecture("Lutosun")
@dataclass(frozen=True)
class LutosunConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    bigram: dict | None   # {"buckets", "mul_prev", "mul_cur"}
    residual_mult: float
    logit_softcap: float | None
    loop: dict | None     # {"start", "stop", "times"}
    layers: tuple         # of dicts as in config.json: {"type", "mixer", "mlp"}

    @classmethod
    def from_dict(cls, cfg: dict) -> "LutosunConfig":
        _need(cfg, ("vocab", "width", "norm", "embedding", "residual_mult", "layers"), "config.json")
        _need(cfg["norm"], ("eps",), "norm")
        _need(cfg["embedding"], ("scale",), "embedding")
        if not isinstance(cfg["layers"], (list, tuple)) or not cfg["layers"]:
            raise ValueError("layers must be a non-empty list")
        cap = cfg.get("logit_softcap")
        out = cls(
            vocab=_int(cfg, "vocab", "config.json"),
            width=_int(cfg, "width", "config.json"),
            eps=float(cfg["norm"]["eps"]),
            embedding_scale=float(cfg["embedding"]["scale"]),
            bigram=copy.deepcopy(cfg["embedding"].get("bigram")) or None,
            residual_mult=float(cfg["residual_mult"]),
            logit_softcap=None if cap is None else _positive(cfg, "logit_softcap", "config.json"),
            loop=copy.deepcopy(cfg.get("loop")) or None,
            layers=tuple(copy.deepcopy(layer) for layer in cfg["layers"]),
        )
        out.validate()
        return out

    def validate(self) -> None:
        if not self.eps >= 0:
            raise ValueError(f"norm.eps must not be negative, got {self.eps}")
        if self.bigram is not None:
            _need(self.bigram, ("buckets", "mul_prev", "mul_cur"), "embedding.bigram")
            _int(self.bigram, "buckets", "embedding.bigram")
            for k in ("mul_prev", "mul_cur"):
                _int(self.bigram, k, "embedding.bigram", 0)
        if self.loop is not None:
            _need(self.loop, ("start", "stop", "times"), "loop")
            start, stop = (_int(self.loop, k, "loop", 0) for k in ("start", "stop"))
            _int(self.loop, "times", "loop")
            if not start < stop <= len(self.layers):
                raise ValueError(f"loop runs layers {start} .. {stop - 1}, the model has {len(self.layers)}")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            _need(layer, ("type", "mixer"), where)
            if layer["type"] not in MIXER_TYPES:
                raise NotImplementedError(f"{where}.type {layer['type']!r} is not supported, expected one of {MIXER_TYPES}")
            m, mw = layer["mixer"], f"{where}.mixer"
            _need(m, MIXER_SIZES + ("scale", "rot"), mw)
            for k in MIXER_SIZES:
                _int(m, k, mw)
            _positive(m, "scale", mw)
            _need(m["rot"], ("base", "dims"), f"{mw}.rot")
            dims = _int(m["rot"], "dims", f"{mw}.rot", 2)
            if dims % 2 or dims > m["rot_dim"]:
                raise ValueError(f"{mw}.rot.dims must be even and at most rot_dim, got {dims}")
            _positive(m["rot"], "base", f"{mw}.rot")
            if layer.get("mlp"):
                self._validate_mlp(layer["mlp"], f"{where}.mlp")

    @staticmethod
    def _validate_mlp(mlp: dict, where: str) -> None:
        _need(mlp, ("router", "expert"), where)
        if mlp.get("kind", "moe") != "moe":
            raise NotImplementedError(f"{where}.kind {mlp['kind']!r} is not supported, expected 'moe'")
        _need(mlp["router"], ("experts", "top", "scale"), f"{where}.router")
        n, top = (_int(mlp["router"], k, f"{where}.router") for k in ("experts", "top"))
        if top > n:
            raise ValueError(f"{where}.router: top {top} of {n} experts")
        for key in ("expert",) + (("shared",) if mlp.get("shared") else ()):
            _need(mlp[key], ("ff", "limit"), f"{where}.{key}")
            _int(mlp[key], "ff", f"{where}.{key}")
            _positive(mlp[key], "limit", f"{where}.{key}")

    def to_dict(self) -> dict:
        """The ``config.json`` that reads back as this configuration."""
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
                "embedding": {"scale": self.embedding_scale, "bigram": copy.deepcopy(self.bigram)}, "residual_mult": self.residual_mult,
                "logit_softcap": self.logit_softcap, "loop": copy.deepcopy(self.loop),
                "layers": [copy.deepcopy(layer) for layer in self.layers]}

    # ------------------------------------------------------------------ lowering

    def _norm(self, tensor: str) -> PartSpec:
        return PartSpec("layernorm", {"width": self.width, "eps": self.eps, "tensor": tensor, "bias_tensor": tensor + ".b"})

    def _mixer(self, m: dict) -> PartSpec:
        rot = m["rot"]
        position = PartSpec("rotary", {"dim": int(rot["dims"]), "theta": float(rot["base"]), "pairing": "adjacent"})
        return PartSpec("latent_attention", {
            "prefix": "mix.", "hidden_size": self.width, "num_heads": m["heads"], "head_dim": m["dim"], "rot_dim": m["rot_dim"],
            "value_dim": m["vdim"], "latent_dim": m["kv_rank"], "query_rank": m["q_rank"], "scale": float(m["scale"]), "eps": self.eps,
            "position": position})

    def _feed_forward(self, mlp: dict | None) -> PartSpec:
        if not mlp:
            return PartSpec("none")
        shared = mlp.get("shared")
        parts = {"gate": "gate", "up": "up", "down": "down"}
        return PartSpec("moe_mlp", {
            "prefix": "mlp.", "hidden_size": self.width, "intermediate_size": int(mlp["expert"]["ff"]),
            "num_experts": int(mlp["router"]["experts"]), "top": int(mlp["router"]["top"]), "activation": "swiglu_clamped",
            "limit": float(mlp["expert"]["limit"]), "gated": True, "scoring": "softmax", "router_bias": True, "renormalise": True,
            "factor": float(mlp["router"]["scale"]),
            "shared": PartSpec("gated_mlp", {
                "prefix": "mlp.shared.", "hidden_size": self.width, "intermediate_size": int(shared["ff"]), "activation": "swiglu_clamped",
                "limit": float(shared["limit"]), "names": parts}) if shared else None,
            "shared_gate": bool(shared),
            "names": {"router": "router", "router_bias": "correction", "expert": "e{}.", "shared_gate": "shared.sg", **parts}})

    def _layer(self, i: int) -> LayerSpec:
        layer = self.layers[i]
        mlp = layer.get("mlp")
        block = PartSpec("prenorm", {
            "mixer_norm": self._norm("norm1"), "ffn_norm": self._norm("norm2") if mlp else None, "residual_scale": self.residual_mult,
            "spare": None if mlp else {"norm2": self.width, "norm2.b": self.width}})
        return LayerSpec(f"l{i}.", block, self._mixer(layer["mixer"]), self._feed_forward(mlp))

    def _run_order(self) -> tuple[RunEntry, ...]:
        """Every run of a layer over a cache of its own; the passes of the loop begin with what joins the stream there."""
        n, loop = len(self.layers), self.loop
        if loop is None:
            return tuple(RunEntry(i, i) for i in range(n))
        start, stop, times = loop["start"], loop["stop"], loop["times"]
        runs = [(i, None) for i in range(start)]
        for t in range(times):
            step = PartSpec("step_vector", {"tensor": "loop.step", "rows": times, "row": t, "width": self.width, "restart": t > 0})
            runs += [(i, step if i == start else None) for i in range(start, stop)]
        runs += [(i, None) for i in range(stop, n)]
        return tuple(RunEntry(i, slot, True, before) for slot, (i, before) in enumerate(runs))

    def to_spec(self) -> ModelSpec:
        w = self.width
        return ModelSpec(
            architecture=self.architecture,
            vocab_size=self.vocab,
            hidden_size=w,
            embedding=PartSpec("token_embedding", {
                "vocab_size": self.vocab, "width": w, "tensor": "embed", "scale": self.embedding_scale,
                "pairs": dict(self.bigram, tensor="bigram") if self.bigram is not None else None}),
            layers=tuple(self._layer(i) for i in range(len(self.layers))),
            run_order=self._run_order(),
            final_norm=self._norm("final.norm"),
            head=PartSpec("linear_head", {"vocab_size": self.vocab, "width": w, "tensor": "head", "softcap": self.logit_softcap}),
            max_position=None,
        )
