"""The generic decoder: parts assembled from a ``ModelSpec`` and run in the order it lists.

One class serves every registered architecture; an architecture is its typed configuration's
``to_spec``. The model owns no cache: the step function hands it a batch and the pool's views.
"""

from __future__ import annotations

from dataclasses import dataclass

from ..config.spec import ModelSpec
from .base import ROUNDED_RESIDUAL, KVNeed, Runtime, StateNeed, TensorSpec
from .registry import part_class


def expected_tensors(spec: ModelSpec) -> dict[str, TensorSpec]:
    """Every checkpoint tensor of the model with its shape, collected from the parts' own
    declarations (the reference lists them in one flat function, miniserve/model/weights.py:60-91)."""
    out: dict[str, TensorSpec] = {}

    def add(tensors: dict[str, TensorSpec], prefix: str = "") -> None:
        for name, ts in tensors.items():
            full = prefix + name
            if full in out and out[full] != ts:
                raise ValueError(f"tensor {full} is declared twice with different shapes")
            out[full] = ts

    add(part_class("embedding", spec.embedding).tensors(spec.embedding))
    for p in spec.injections:  # (several may read rows of one table)
        add(part_class("injection", p).tensors(p))
    for layer in spec.layers:
        add(part_class("block", layer.block).tensors(layer.block), layer.prefix)
        add(part_class("mixer", layer.mixer).tensors(layer.mixer), layer.prefix)
        add(part_class("feed_forward", layer.feed_forward).tensors(layer.feed_forward), layer.prefix)
    add(part_class("norm", spec.final_norm).tensors(spec.final_norm))
    add(part_class("head", spec.head).tensors(spec.head))
    return out


def expected_aliases(spec: ModelSpec) -> dict[str, str]:
    """Every tensor name a part reads under which nothing is stored, with the full name of the tensor
    that stands for it, collected from the parts' own ``aliases``. A source must be a declared tensor."""
    out: dict[str, str] = {}

    def add(aliases: dict[str, str], prefix: str = "") -> None:
        for name, source in aliases.items():
            out[prefix + name] = source

    add(part_class("embedding", spec.embedding).aliases(spec.embedding))
    for layer in spec.layers:
        for category, part in (("block", layer.block), ("mixer", layer.mixer), ("feed_forward", layer.feed_forward)):
            add(part_class(category, part).aliases(part), layer.prefix)
    add(part_class("norm", spec.final_norm).aliases(spec.final_norm))
    add(part_class("head", spec.head).aliases(spec.head))
    declared = expected_tensors(spec)
    for name, source in out.items():
        if name in declared:
            raise ValueError(f"tensor {name} is declared as stored and as an alias of {source}")
        if source not in declared:
            raise ValueError(f"tensor {name} is an alias of {source}, which no part declares")
    return out


@dataclass(frozen=True)
class CacheSlotNeed:
    """What one cache slot of the run order holds: paged keys/values and/or fixed-size state."""

    slot: int
    kv: KVNeed | None
    state: StateNeed | None


class DecoderModel:
    def __init__(self, spec: ModelSpec, weights: dict, rt: Runtime):
        self.spec = spec
        self.rt = rt
        self.dtype = rt.dtype
        self.device = rt.device
        self.vocab_size = spec.vocab_size

        weights = dict(weights)
        for name, source in expected_aliases(spec).items():
            weights[name] = weights[source]  # the same tensor under its second name

        def local(prefix: str, part_type, part_spec) -> dict:
            declared = part_type.tensors(part_spec)
            names = [n for n, ts in declared.items() if not ts.optional] + list(part_type.aliases(part_spec))
            return {n: weights[prefix + n] for n in names}

        self.embedding = part_class("embedding", spec.embedding)(spec.embedding, rt)
        self.embedding.bind(weights)
        self.blocks = []
        for layer in spec.layers:
            mixer = part_class("mixer", layer.mixer)(layer.mixer, rt)
            mixer.bind(local(layer.prefix, type(mixer), layer.mixer))
            ffn = part_class("feed_forward", layer.feed_forward)(layer.feed_forward, rt)
            ffn.bind(local(layer.prefix, type(ffn), layer.feed_forward))
            block = part_class("block", layer.block)(layer.block, rt, mixer, ffn)
            block.bind(local(layer.prefix, type(block), layer.block))
            self.blocks.append(block)
        self.injections = []  # per run-order entry: what joins the stream before it, or None
        for e in spec.run_order:
            part = part_class("injection", e.before)(e.before, rt) if e.before is not None else None
            if part is not None:
                part.bind(weights)
            self.injections.append(part)
        self.keeps_start = any(p is not None and p.needs_start for p in self.injections)
        # what the embedding keeps per request lies in a slot of its own, behind the run order's
        self.embedding_slot = spec.num_cache_slots if self.embedding.state_need() is not None else None
        self.final_norm = part_class("norm", spec.final_norm)(spec.final_norm, rt)
        self.final_norm.bind(weights)
        self.head = part_class("head", spec.head)(spec.head, rt)
        self.head.bind(weights)

    # ------------------------------------------------------------------ cache needs

    def cache_slots(self) -> list[CacheSlotNeed]:
        """One entry per cache slot of the run order, from the mixer that writes it (and one for what the embedding keeps). An entry that reads a slot
        another entry wrote must keep the same planes and state; its window may differ, and the slot then keeps
        the widest of them (every token, if one of its readers sees every token)."""
        needs: dict[int, CacheSlotNeed] = {}
        for e in self.spec.run_order:
            if e.cache is None:
                continue
            mixer = self.blocks[e.layer].mixer
            need = CacheSlotNeed(e.cache, mixer.kv_need(), mixer.state_need())
            if e.writes_cache:
                needs[e.cache] = need
                continue
            held = needs[e.cache]
            same = (held.kv is None) == (need.kv is None) and (held.kv is None or held.kv.planes == need.kv.planes)
            if not same or held.state != need.state:
                raise ValueError(
                    f"layer {e.layer} reads cache slot {e.cache} but needs {need}, the slot holds {held}"
                )
            if held.kv is not None and (held.kv.window, held.kv.keep_first) != (need.kv.window, need.kv.keep_first):
                window = 0 if 0 in (held.kv.window, need.kv.window) else max(held.kv.window, need.kv.window)
                keep = max(held.kv.keep_first, need.kv.keep_first) if window else 0
                needs[e.cache] = CacheSlotNeed(e.cache, KVNeed(held.kv.planes, window, keep), held.state)
        if self.embedding_slot is not None:
            needs[self.embedding_slot] = CacheSlotNeed(self.embedding_slot, None, self.embedding.state_need())
        return [needs[s] for s in sorted(needs)]

    # ------------------------------------------------------------------ forward

    def forward(self, batch, pool):
        """Run the batch's tokens through every run-order entry and return float32 logits
        ``[len(batch.want_rows), vocab]`` at the wanted flat token indices."""
        with self.rt.ops.stream_scope():
            return self._forward(batch, pool)

    def _forward(self, batch, pool):
        batch.memo = {}  # what parts share between layers is made anew in every pass (a captured pass records it)
        kept = pool.state_view(self.embedding_slot, batch) if self.embedding_slot is not None else None
        residual = self.embedding.forward(batch.token_ids, batch, kept, self.keeps_start)
        residual, start = residual if self.keeps_start else (residual, None)
        pending = None  # a sum a layer left to be added to the residual stream by its next reader
        for e, injection in zip(self.spec.run_order, self.injections):
            if injection is not None:
                injection.forward(residual, start, pending)
                pending = None
                batch.memo.pop(ROUNDED_RESIDUAL, None)
            cache = pool.view(e.cache, batch, e.writes_cache) if e.cache is not None else None
            state = pool.state_view(e.cache, batch) if e.cache is not None else None
            left = batch.memo.get(ROUNDED_RESIDUAL)
            pending = self.blocks[e.layer].forward(residual, batch, cache, state, pending)
            if left is not None and batch.memo.get(ROUNDED_RESIDUAL) is left:
                del batch.memo[ROUNDED_RESIDUAL]  # an earlier block's copy: the stream has moved on since
        if batch.num_wanted == 0:
            return None
        x = self.final_norm.forward(residual, rows=batch.want_rows, add=pending)
        return self.head.forward(x)

    def step_flops(self, rows) -> int:
        """Floating-point operations of one step over ``rows`` (``(new tokens, cached tokens)`` per request),
        logits at one position per request: the sum of what the parts say of themselves."""
        total = self.final_norm.flops(rows) + self.head.flops(rows)
        for e in self.spec.run_order:
            b = self.blocks[e.layer]
            total += b.flops(rows) + b.mixer.flops(rows) + b.feed_forward.flops(rows)
        return total

    def decode_read_bytes(self, tokens: int = 1) -> int:
        """Bytes of weights one decode step of ``tokens`` requests reads: every run-order entry's layer once, the final
        norm and the head (embedding rows are only gathered). Only parts that route tokens to some of their weights read
        more for more tokens."""
        total = self.final_norm.parameters_bytes() + self.head.parameters_bytes()
        total += sum(p.parameters_bytes() for p in self.injections if p is not None)
        for e in self.spec.run_order:
            b = self.blocks[e.layer]
            total += b.parameters_bytes() + b.mixer.step_read_bytes(tokens) + b.feed_forward.step_read_bytes(tokens)
        return total
