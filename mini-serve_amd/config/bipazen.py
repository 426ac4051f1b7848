"""Typed configuration of the Bipazen decoder, read from its own ``config.json`` keys. The reference has no such
architecture.

``config.json``: ``architecture`` (the name), ``vocab``, ``width``, ``norm.eps`` and ``layers``, a list in which every
entry names its mixer (``type``), the mixer's sizes and constants (``mixer``) and its feed-forward (``mlp``, or null for
none). Layer ``i``'s tensors start with ``l<i>.``. An entry with ``weights_of: j`` has no tensors: it runs layer ``j``'s
weights (mixer, feed-forward, norms and layer scales) over a cache and state of its own, and the rest of its entry equals
layer ``j``'s (``j`` may come before or after it; where ``j`` runs another layer's weights in turn, that layer's are meant).

A layer is ``x += ls1 * mixer(N1(x))``, then ``x += ls2 * ff(N2(x))``: RMS norms with plain weights (tensors ``norm1
norm2``) and a learned factor per channel behind each sublayer (``ls1 ls2``). The mixers:

* ``mamba2`` (``heads``, ``vdim``, ``state``, ``groups``, ``conv``, ``norm_groups``; tensors ``mix.in conv conv.b dt_bias A_log D
  norm o``): ``in`` projects to [gate: heads vdim | values: heads vdim | keys: groups state | queries: groups state | step:
  heads]; values, keys and queries pass a causal convolution of ``conv`` taps per channel with a bias, and a SiLU; ``d =
  softplus(step + dt_bias)``; head ``h`` reads the keys and queries of group ``h // (heads / groups)``: ``S_t = exp(-exp(A_log_h)
  d) S_(t-1) + d k_t v_t^T`` (``S: [state, vdim]``), ``y_t = S_t^T q_t + D_h v_t``; ``y silu(gate)`` is RMS-normed in
  ``norm_groups`` equal parts, times ``norm``, projected by ``o``.
* ``rglru`` (``width``, ``blocks``, ``conv``; tensors ``mix.y y.b x x.b conv conv.b ra ra.b ri ri.b lam o``): ``y = gelu_tanh(W_y h +
  b)``, ``u = conv(W_x h + b)`` (causal, per channel, with a bias, no activation); in each of ``blocks`` equal parts ``r =
  sigmoid(ra u + b)``, ``i = sigmoid(ri u + b)`` (square matrices per part); ``log a = -8 r softplus(lam)``, ``S_t = a S_(t-1) +
  sqrt(1 - a^2) i u`` per channel from zero; output ``o (S y)``.
* ``latent_attention`` (``heads``, ``dim``, ``rot_dim``, ``vdim``, ``kv_rank``, ``scale``, ``rot``; tensors ``mix.q dkv dkv.norm uk uv
  g o``): ``dkv`` projects to ``kv_rank`` latent elements (RMS-normed, weight ``dkv.norm``) and ``rot_dim`` elements of a key part
  shared by all heads; ``uk`` / ``uv`` make each head's plain key part (``dim``) and value (``vdim``) from the latent; query heads
  are ``[dim plain, rot_dim rotated]``. The rotation turns the first ``rot.dims`` rotated elements, halves paired, by
  ``position * rot.base ** (-2i / rot.dims)``. Every earlier token is visible; the concatenated heads are multiplied by
  ``sigmoid(g h)`` element by element.

Feed-forward (``kind: moe``; ``router.experts``, ``router.top``, ``expert.ff``; tensors ``mlp.router``, ``mlp.e<j>.gate up down``):
scores ``sigmoid(router h)``; the ``top`` experts with the largest scores run; a chosen expert's input is ``h`` times its score,
and the outputs (``down(silu(gate z) * up z)``) are added as they stand. The final norm is ``final.norm``; the head is the
embedding table ``embed``.
"""

from __future__ import annotations

import copy
from dataclasses import dataclass

from .registry import register_architecture
from .spec import LayerSpec, ModelSpec, PartSpec, RunEntry

DECAY_FACTOR = 8.0  # what the log decay of an rglru channel is at most, in units of softplus(lam)

MIXER_KEYS = {
    "mamba2": ("heads", "vdim", "state", "groups", "conv", "norm_groups"),
    "rglru": ("width", "blocks", "conv"),
    "latent_attention": ("heads", "dim", "rot_dim", "vdim", "kv_rank"),
}


def _need(d, keys, where: str) -> None:
    if not isinstance(d, dict):
        raise ValueError(f"{where} must be an object, got {d!r}")
    missing = [k for k in keys if k not in d]
    if missing:
        raise KeyError(f"config.json lacks {missing} in {where}")


def _positive_int(d: dict, key: str, where: str) -> int:
    v = d[key]
    if not isinstance(v, int) or isinstance(v, bool) or v < 1:
        raise ValueError(f"{where}.{key} must be a positive integer, got {v!r}")
    return v


@register_architecture("Bipazen")
@dataclass(frozen=True)
class BipazenConfig:
    vocab: int
    width: int
    eps: float
    layers: tuple  # of dicts as in config.json: {"type", "mixer", "mlp"[, "weights_of"]}

    @classmethod
    def from_dict(cls, cfg: dict) -> "BipazenConfig":
        _need(cfg, ("vocab", "width", "norm", "layers"), "config.json")
        _need(cfg["norm"], ("eps",), "norm")
        if not isinstance(cfg["layers"], (list, tuple)) or not cfg["layers"]:
            raise ValueError("layers must be a non-empty list")
        out = cls(
            vocab=_positive_int(cfg, "vocab", "config.json"),
            width=_positive_int(cfg, "width", "config.json"),
            eps=float(cfg["norm"]["eps"]),
            layers=tuple(copy.deepcopy(layer) for layer in cfg["layers"]),
        )
        out.validate()
        return out

    def validate(self) -> None:
        if not self.eps >= 0:
            raise ValueError(f"norm.eps must not be negative, got {self.eps}")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            _need(layer, ("type", "mixer"), where)
            kind, m = layer["type"], layer["mixer"]
            if kind not in MIXER_KEYS:
                raise NotImplementedError(f"{where}.type {kind!r} is not supported, expected one of {tuple(MIXER_KEYS)}")
            mw = f"{where}.mixer"
            _need(m, MIXER_KEYS[kind], mw)
            for k in MIXER_KEYS[kind]:
                _positive_int(m, k, mw)
            if kind == "mamba2":
                if m["heads"] % m["groups"]:
                    raise ValueError(f"{mw}: {m['heads']} heads are no multiple of {m['groups']} groups")
                if (m["heads"] * m["vdim"]) % m["norm_groups"]:
                    raise ValueError(f"{mw}: {m['heads'] * m['vdim']} channels cannot be normed in {m['norm_groups']} equal parts")
            elif kind == "rglru":
                if m["width"] % m["blocks"]:
                    raise ValueError(f"{mw}: a width of {m['width']} cannot be cut into {m['blocks']} equal blocks")
            else:
                _need(m, ("scale", "rot"), mw)
                if not float(m["scale"]) > 0:
                    raise ValueError(f"{mw}.scale must be positive")
                rot = m["rot"]
                _need(rot, ("base", "dims"), f"{mw}.rot")
                dims = rot["dims"]
                if not isinstance(dims, int) or isinstance(dims, bool) or dims % 2 or not 2 <= dims <= m["rot_dim"]:
                    raise ValueError(f"{mw}.rot.dims must be even and at most rot_dim, got {dims!r}")
                if not float(rot["base"]) > 0:
                    raise ValueError(f"{mw}.rot.base must be positive")
            if layer.get("weights_of") is not None:
                root = self.source(i)
                if self.layers[root]["type"] != kind:
                    raise ValueError(f"{where} is a {kind!r} layer but runs the weights of layer {root}, a {self.layers[root]['type']!r} layer")
            mlp = layer.get("mlp")
            if mlp:
                fw = f"{where}.mlp"
                _need(mlp, ("router", "expert"), fw)
                if mlp.get("kind", "moe") != "moe":
                    raise NotImplementedError(f"{fw}.kind {mlp['kind']!r} is not supported, expected 'moe'")
                _need(mlp["router"], ("experts", "top"), f"{fw}.router")
                _need(mlp["expert"], ("ff",), f"{fw}.expert")
                _positive_int(mlp["expert"], "ff", f"{fw}.expert")
                n, top = (_positive_int(mlp["router"], k, f"{fw}.router") for k in ("experts", "top"))
                if top > n:
                    raise ValueError(f"{fw}.router: top {top} of {n} experts")

    def source(self, i: int) -> int:
        """The layer whose tensors layer ``i`` runs: itself, or what its ``weights_of`` leads to."""
        seen = {i}
        while self.layers[i].get("weights_of") is not None:
            j = self.layers[i]["weights_of"]
            if not isinstance(j, int) or isinstance(j, bool) or not 0 <= j < len(self.layers):
                raise ValueError(f"layers[{i}].weights_of must be the number of a layer, got {j!r}")
            if j in seen:
                raise ValueError(f"layers[{i}].weights_of leads back to layer {j}: no layer of the chain has tensors")
            seen.add(j)
            i = j
        return i

    def to_dict(self) -> dict:
        """The ``config.json`` that reads back as this configuration."""
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
                "layers": [copy.deepcopy(layer) for layer in self.layers]}

    # ------------------------------------------------------------------ lowering

    def _norm(self, tensor: str) -> PartSpec:
        return PartSpec("rmsnorm", {"width": self.width, "eps": self.eps, "tensor": tensor})

    def _mixer(self, kind: str, m: dict) -> PartSpec:
        w, eps = self.width, self.eps
        if kind == "mamba2":
            return PartSpec("mamba2", {
                "prefix": "mix.", "hidden_size": w, "num_heads": m["heads"], "head_dim": m["state"], "value_dim": m["vdim"],
                "groups": m["groups"], "conv_taps": m["conv"], "norm_groups": m["norm_groups"], "eps": eps})
        if kind == "rglru":
            return PartSpec("rglru", {
                "prefix": "mix.", "hidden_size": w, "width": m["width"], "blocks": m["blocks"], "conv_taps": m["conv"],
                "decay_factor": DECAY_FACTOR})
        rot = m["rot"]
        position = PartSpec("rotary", {"dim": int(rot["dims"]), "theta": float(rot["base"]), "pairing": "halves"})
        return PartSpec("latent_attention", {
            "prefix": "mix.", "hidden_size": w, "num_heads": m["heads"], "head_dim": m["dim"], "rot_dim": m["rot_dim"],
            "value_dim": m["vdim"], "latent_dim": m["kv_rank"], "scale": float(m["scale"]), "eps": eps, "gate": "element",
            "position": position})

    def _feed_forward(self, mlp: dict | None) -> PartSpec:
        if not mlp:
            return PartSpec("none")
        return PartSpec("moe_mlp", {
            "prefix": "mlp.", "hidden_size": self.width, "intermediate_size": int(mlp["expert"]["ff"]),
            "num_experts": int(mlp["router"]["experts"]), "top": int(mlp["router"]["top"]), "activation": "silu", "gated": True,
            "scoring": "sigmoid", "weigh": "input",
            "names": {"router": "router", "expert": "e{}.", "gate": "gate", "up": "up", "down": "down"}})

    def to_spec(self) -> ModelSpec:
        w = self.width
        layers, index = [], {}
        for i, layer in enumerate(self.layers):
            if layer.get("weights_of") is not None:
                continue
            mlp = layer.get("mlp")
            block = PartSpec("prenorm", {
                "mixer_norm": self._norm("norm1"), "ffn_norm": self._norm("norm2") if mlp else None,
                "mixer_scale": "ls1", "ffn_scale": "ls2" if mlp else None, "spare": None if mlp else {"norm2": w, "ls2": w}})
            index[i] = len(layers)
            layers.append(LayerSpec(f"l{i}.", block, self._mixer(layer["type"], layer["mixer"]), self._feed_forward(mlp)))
        # every entry runs over a cache and state of its own, whosever weights it runs
        order = [RunEntry(index[self.source(i)], i) for i in range(len(self.layers))]
        return ModelSpec(
            architecture=self.architecture,
            vocab_size=self.vocab,
            hidden_size=w,
            embedding=PartSpec("token_embedding", {"vocab_size": self.vocab, "width": w, "tensor": "embed"}),
            layers=tuple(layers),
            run_order=tuple(order),
            final_norm=self._norm("final.norm"),
            head=PartSpec("linear_head", {"vocab_size": self.vocab, "width": w, "tensor": "head", "tied_to": "embed"}),
            max_position=None,
        )
