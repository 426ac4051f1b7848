"""Token embedding, what may join the stream later on, and output head.

Embedding: ``h = E[token_ids]`` without scaling (miniserve/model/qwen3.py:211), widened to the
float32 residual stream. Head: ``logits = x W^T`` without bias, scaling or soft-cap
(miniserve/model/qwen3.py:152,186,195), returned in float32; a tied head reads the embedding's
tensor itself, no copy (miniserve/model/weights.py:116-119,135-136). ``logit_scale`` (optional, no
counterpart in the reference) multiplies the float32 logits.

Further parameters, none of which the reference has. Embedding: ``scale`` multiplies the token's row; ``pairs`` (``{"tensor",
"buckets", "mul_prev", "mul_cur"}``) names a second table ``[buckets + 1, width]`` of which every token adds the row
``(previous token * mul_prev + token * mul_cur) mod buckets``, a sequence's first token the last row; the previous token is
kept per request, so that a sequence may be cut anywhere. Head: ``softcap`` bounds the logits (after ``logit_scale``) to
``softcap * tanh(logits / softcap)``. ``step_vector`` is an injection: row ``row`` of a table ``[rows, width]`` joins the stream of
every token, and with ``restart`` the embedding's output once more: what a run of layers that is run several times with the
same weights is told about the pass it is in."""

from __future__ import annotations

import torch

from ..config.spec import PartSpec
from .base import Embedding, Head, Injection, StateNeed, TensorSpec
from .registry import register


@register("embedding", "token_embedding")
class TokenEmbedding(Embedding):
    def __init__(self, spec: PartSpec, rt):
        super().__init__(spec, rt)
        self.vocab = int(spec["vocab_size"])
        self.width = int(spec["width"])
        self.scale = 1.0 if spec.get("scale") is None else float(spec["scale"])
        self.pairs = dict(spec["pairs"]) if spec.get("pairs") else None
        self.table = self.pair_table = None

    @classmethod
    def tensors(cls, spec: PartSpec) -> dict[str, TensorSpec]:
        out = {spec["tensor"]: TensorSpec((int(spec["vocab_size"]), int(spec["width"])))}
        if spec.get("pairs"):
            out[spec["pairs"]["tensor"]] = TensorSpec((int(spec["pairs"]["buckets"]) + 1, int(spec["width"])))
        return out

    def bind(self, tensors) -> None:
        self.table = tensors[self.spec["tensor"]]
        if self.pairs is not None:
            self.pair_table = tensors[self.pairs["tensor"]]
            if self.pair_table.dtype != self.table.dtype:
                raise ValueError(f"{self.pairs['tensor']} and {self.spec['tensor']} are stored in different dtypes")

    def state_need(self) -> StateNeed | None:
        return StateNeed.single((1,), "int32", "last") if self.pairs is not None else None

    def forward(self, token_ids, batch=None, state=None, keep=False):
        ops = self.rt.ops
        if self.pairs is None and self.scale == 1.0 and not keep:
            return ops.embed(token_ids, self.table)
        if self.pairs is None:
            return ops.embed_pairs(token_ids, self.table, self.scale, keep=keep)
        return ops.embed_pairs(token_ids, self.table, self.scale, self.pair_table, self.pairs["mul_prev"], self.pairs["mul_cur"],
                               batch, state["last"], keep)

    def parameters_bytes(self) -> int:
        return 0  # a decode step gathers single rows


@register("injection", "step_vector")
class StepVector(Injection):
    def __init__(self, spec: PartSpec, rt):
        super().__init__(spec, rt)
        self.row = int(spec["row"])
        self.needs_start = bool(spec.get("restart", False))
        if not 0 <= self.row < int(spec["rows"]):
            raise ValueError(f"row {self.row} of a table of {spec['rows']}")
        self.vector = None

    @classmethod
    def tensors(cls, spec: PartSpec) -> dict[str, TensorSpec]:
        return {spec["tensor"]: TensorSpec((int(spec["rows"]), int(spec["width"])))}

    def bind(self, tensors) -> None:
        self.vector = tensors[self.spec["tensor"]][self.row].to(torch.float32).contiguous()

    def forward(self, residual, start, pending=None) -> None:
        self.rt.ops.stream_inject(residual, self.vector, start if self.needs_start else None, pending)

    def parameters_bytes(self) -> int:
        return self.vector.numel() * self.vector.element_size()


@register("head", "linear_head")
class LinearHead(Head):
    def __init__(self, spec: PartSpec, rt):
        super().__init__(spec, rt)
        self.vocab = int(spec["vocab_size"])
        self.width = int(spec["width"])
        self.tied_to = spec.get("tied_to")
        self.logit_scale = 1.0 if spec.get("logit_scale") is None else float(spec["logit_scale"])
        self.softcap = float(spec.get("softcap") or 0.0)
        self.weight = None

    @classmethod
    def tensors(cls, spec: PartSpec) -> dict[str, TensorSpec]:
        if spec.get("tied_to"):
            return {}
        return {spec["tensor"]: TensorSpec((int(spec["vocab_size"]), int(spec["width"])))}

    @classmethod
    def aliases(cls, spec: PartSpec) -> dict[str, str]:
        return {spec["tensor"]: spec["tied_to"]} if spec.get("tied_to") else {}

    def bind(self, tensors) -> None:
        self.weight = tensors[self.spec["tensor"]]

    def forward(self, x):
        logits = self.rt.ops.linear(x, self.weight, out_dtype=torch.float32)
        if self.logit_scale != 1.0:
            self.rt.ops.scale_(logits, self.logit_scale)
        return self.rt.ops.softcap_(logits, self.softcap) if self.softcap else logits

    def parameters_bytes(self) -> int:
        return self.weight.numel() * self.weight.element_size()

    def flops(self, rows) -> int:
        return 2 * len(rows) * self.vocab * self.width  # one wanted position per request
