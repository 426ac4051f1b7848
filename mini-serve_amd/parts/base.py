"""Interfaces of the parts a layer is put together from.

A part is built from a ``PartSpec`` (its sizes and constants) and a ``Runtime`` (compute dtype,
device, kernels); it declares the tensors it needs under its own prefix and receives exactly
those. No part knows which model it is in. The kinds:

* ``Norm``            ``forward(x_f32, rows=None, add=None) -> y``  (residual stream in, compute dtype out)
* ``PositionEncoding`` ``rotation(batch) -> Rotation | None``       (what a mixer's q/k are turned by in this step)
* ``Mixer``           ``forward(x, batch, cache, state, residual) -> pending`` (``state``: name -> tensor)
* ``FeedForward``     ``forward(x, residual) -> pending``
* ``Block``           ``forward(residual, batch, cache, state, pending) -> pending`` (where norms and sums sit)
* ``Embedding``       ``forward(token_ids, batch, state, keep) -> residual``  (float32 ``[T, width]``)
* ``Injection``       ``forward(residual, start, pending)``        (what joins the stream ahead of a run-order entry)
* ``Head``            ``forward(x) -> logits``                      (float32 ``[rows, vocab]``)

The residual stream is float32 in every compute dtype: sums of layer outputs are never rounded
to bfloat16. Mixers and feed-forwards do not return their output: they either add it into
``residual`` themselves (a matrix product can do that in its epilogue) and return None, or return a
*pending* sum (``ops.SplitSum``: partial sums that still have to be added to ``residual``). Whoever
reads the residual stream next takes the pending sum along: a norm adds it while it normalises
(``add=``), anything else calls ``ops.add_pending`` first.

A block may hang a factor per channel behind a sublayer (``Sublayer.scale_output``: a layer scale); what the sublayer adds or
leaves pending is then already multiplied by it (a ``SplitSum`` carries the factors to the kernel that adds it).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import TYPE_CHECKING, Any, Mapping

from ..config.spec import PartSpec

if TYPE_CHECKING:  # pragma: no cover
    import torch


@dataclass(frozen=True)
class TensorSpec:
    """A tensor a part expects in the checkpoint. ``kind``: ``"float"`` tensors follow the compute
    dtype (a tensor stored in 32-bit stays 32-bit); ``"int"`` tables are kept as int32.

    ``init`` says how the random-weights mode draws it: ``"normal"`` N(0, std) (matrices, embeddings),
    ``"ones"`` a scale around one (norm weights: all one, or uniform in the range the caller gives),
    ``"uniform"`` U(-std, std), ``"zeros"`` (a bias that starts switched off); integer tables are
    drawn uniformly from ``[0, high)``. ``optional``: a checkpoint may hold the tensor or not; nothing reads it
    (the loader accepts it, the random-weights mode does not draw it, the part is not handed it).

    A dimension of ``None`` is free: the checkpoint's size is taken as it comes and the part reads it off the tensor it
    is bound to (a size that no configuration key states); the random-weights mode draws ``free`` there."""

    shape: tuple
    kind: str = "float"
    init: str = "normal"
    high: int | None = None
    optional: bool = False
    free: int | None = None

    def fits(self, shape) -> bool:
        return len(shape) == len(self.shape) and all(w is None or w == g for w, g in zip(self.shape, shape))

    def drawn_shape(self) -> tuple[int, ...]:
        return tuple(self.free if d is None else d for d in self.shape)

    def __post_init__(self):
        if any(d is None for d in self.shape) and (self.free is None or self.free < 1):
            raise ValueError("a tensor with a free dimension needs ``free``: the size the random-weights mode draws")
        if self.kind not in ("float", "int"):
            raise ValueError(f"unknown tensor kind {self.kind!r}")
        if self.kind == "float" and self.init not in ("normal", "ones", "uniform", "zeros"):
            raise ValueError(f"unknown init {self.init!r}")
        if self.kind == "int" and (self.high is None or self.high < 1):
            raise ValueError("an integer table needs ``high``: its entries are drawn from [0, high)")


@dataclass(frozen=True)
class CachePlane:
    """One thing a mixer keeps per token in the paged cache: ``heads`` vectors of ``width`` elements.
    Within a page a plane lies ``[page_size, width]`` per head, or, ``token_minor``, ``[width,
    page_size]`` (the tokens of one element side by side: what a product over tokens reads)."""

    name: str
    heads: int
    width: int
    token_minor: bool = False


@dataclass(frozen=True)
class KVNeed:
    """What a mixer keeps per token, as a list of planes (keys and values of equal or different
    widths, one latent vector, ...). ``window == 0`` keeps every token, ``window > 0`` only the last
    ``window`` (older pages may be given back) and, with ``keep_first > 0``, the sequence's first
    ``keep_first`` tokens as well (their pages never go back while the request lives)."""

    planes: tuple[CachePlane, ...]
    window: int = 0
    keep_first: int = 0

    def __post_init__(self):
        names = [p.name for p in self.planes]
        if not names or len(set(names)) != len(names):
            raise ValueError(f"cache planes need distinct names, got {names}")

    @classmethod
    def keys_values(cls, num_kv_heads: int, head_dim: int, window: int = 0, value_dim: int | None = None,
                    keep_first: int = 0) -> "KVNeed":
        """Keys ``[page_size, head_dim]`` and values ``[value_dim, page_size]`` per KV head (``value_dim``
        defaults to ``head_dim``): what the attention kernels read."""
        return cls((CachePlane("k", num_kv_heads, head_dim),
                    CachePlane("v", num_kv_heads, head_dim if value_dim is None else value_dim, token_minor=True)),
                   window, keep_first if window else 0)

    @property
    def elements_per_token(self) -> int:
        return sum(p.heads * p.width for p in self.planes)


@dataclass(frozen=True)
class StateTensor:
    """One tensor of a mixer's per-request state: shape per request and torch dtype name."""

    name: str
    shape: tuple[int, ...]
    dtype: str = "float32"


@dataclass(frozen=True)
class StateNeed:
    """Per-request state of fixed size a mixer keeps: one or several named tensors."""

    tensors: tuple[StateTensor, ...]

    def __post_init__(self):
        names = [t.name for t in self.tensors]
        if not names or len(set(names)) != len(names):
            raise ValueError(f"state tensors need distinct names, got {names}")

    @classmethod
    def single(cls, shape, dtype: str = "float32", name: str = "state") -> "StateNeed":
        return cls((StateTensor(name, tuple(shape), dtype),))


@dataclass(frozen=True)
class Rotation:
    """Rotary position encoding as a mixer's kernels need it: the first ``dim`` elements of each
    head are turned in pairs by the step's angles, whose cosines and sines are the two halves of a row
    of ``table`` (pair ``j`` by angle ``j``). ``pairing`` says which elements make pair ``j``:
    ``"halves"`` (j, j + dim/2), ``"adjacent"`` (2j, 2j + 1); the kernels name the pairings they know
    (``ops.ROTATION_PAIRINGS``) and refuse any other."""

    dim: int
    table: Any  # float32 device tensor [tokens of the step, dim]: cosines, then sines
    pairing: str = "halves"


class Runtime:
    """What every part is built with: the compute dtype, the device and the kernel library."""

    def __init__(self, dtype, device, ops):
        self.dtype = dtype  # torch.float32 or torch.bfloat16
        self.device = device
        self.ops = ops


class Part:
    """Base of all parts. Subclasses override ``tensors`` (static: needs no device) and ``bind``."""

    kind: str = ""

    def __init__(self, spec: PartSpec, rt: Runtime | None):
        self.spec = spec
        self.rt = rt

    @classmethod
    def tensors(cls, spec: PartSpec) -> dict[str, TensorSpec]:
        """Checkpoint tensors of this part, named relative to the layer prefix (or absolutely
        for parts outside layers)."""
        return {}

    @classmethod
    def aliases(cls, spec: PartSpec) -> dict[str, str]:
        """Tensors this part reads that are stored under another name: ``{name: source}``, ``name``
        relative like the names of ``tensors`` (and never among them), ``source`` the full name of a
        tensor some part declares. The part receives the source's tensor under ``name`` (the same memory,
        no copy); a tensor stored under ``name`` itself is a duplicate and is dropped."""
        return {}

    def bind(self, tensors: Mapping[str, "torch.Tensor"]) -> None:
        """Receive the tensors declared by ``tensors`` and ``aliases`` (same names), already on the device."""

    def parameters_bytes(self) -> int:
        """Bytes of weights a decode step reads from this part (for the bandwidth model)."""
        return 0

    def step_read_bytes(self, tokens: int) -> int:
        """Bytes of weights a step of ``tokens`` single tokens reads from this part: ``parameters_bytes()`` unless what
        is read depends on the tokens (a part that routes them to some of its weights)."""
        return self.parameters_bytes()

    def flops(self, rows) -> int:
        """Floating-point operations of one pass over ``rows``: a list of ``(new tokens, tokens already in
        the cache)`` per request; a multiply-add counts two. What a measurement divides by its time."""
        return 0


# ``batch.memo`` key under which a block may leave the residual stream as it stands after the block, in the compute dtype,
# for the block that runs next (which would otherwise cast it). The model drops what the block that just ran did not
# leave itself, so an entry is never older than one block.
ROUNDED_RESIDUAL = "residual_in_compute_dtype"


class Norm(Part):
    def forward(self, x, rows=None, add=None):
        """Normalise rows of the float32 ``x`` plus ``add`` (a pending sum). Without ``rows``, ``x`` is
        also brought up to date in place; with ``rows`` the stream is not read again and stays as it is."""
        raise NotImplementedError

    def add_normed(self, residual, stream, pending=None, next_out=None, clear=False) -> None:
        """``residual += norm(stream + pending)`` row by row, both float32 and of one shape (``pending``: a sum the
        sublayer left to be added to its stream): the norm of a layer that norms what a sublayer puts out instead of
        what it reads. ``next_out`` (the compute dtype, same shape; None: not wanted) receives the new residual, and
        with ``clear`` the stream is zero afterwards."""
        raise NotImplementedError(f"norm {self.kind!r} cannot norm a sublayer's output into the residual stream")


class PositionEncoding(Part):
    def rotation(self, batch) -> Rotation | None:
        """What the mixer turns q and k by in this step. Anything computed from the step's positions
        alone belongs in ``batch.memo`` (a dict that lives as long as the step), under a key that names
        the encoding's constants, so that layers with equal constants compute it once."""
        return None


class Sublayer(Part):
    """What adds to the residual stream: a mixer or a feed-forward. ``scales_output``: the part multiplies what it adds by
    ``out_scale`` (float32 ``[width]``; None: by nothing)."""

    scales_output = False
    out_scale = None

    def scale_output(self, scale) -> None:
        """Multiply what this part adds to the stream by ``scale [width]``, element by element."""
        if not self.scales_output:
            raise NotImplementedError(f"{self.kind!r} cannot scale what it adds to the residual stream")
        self.out_scale = scale.float().contiguous()


class Mixer(Sublayer):
    def kv_need(self) -> KVNeed | None:
        return None

    def state_need(self) -> StateNeed | None:
        return None

    def forward(self, x, batch, cache, state, residual):
        """Add the mixer's output to ``residual``, or return it as a pending sum."""
        raise NotImplementedError


class FeedForward(Sublayer):
    def forward(self, x, residual):
        """Add the feed-forward's output to ``residual``, or return it as a pending sum."""
        raise NotImplementedError


class Block(Part):
    def __init__(self, spec: PartSpec, rt, mixer: Mixer, feed_forward: FeedForward):
        super().__init__(spec, rt)
        self.mixer = mixer
        self.feed_forward = feed_forward

    def forward(self, residual, batch, cache, state, pending=None):
        """Run the layer on ``residual`` (to which ``pending`` still has to be added); returns what is
        pending afterwards."""
        raise NotImplementedError


class Embedding(Part):
    """``state_need``: what it keeps per request (a token's vector may depend on tokens of earlier steps)."""

    def state_need(self) -> StateNeed | None:
        return None

    def forward(self, token_ids, batch=None, state=None, keep=False):
        """The residual stream of the step's tokens; ``keep``: the pair (stream, a copy that nobody adds to)."""
        raise NotImplementedError


class Injection(Part):
    """What joins the residual stream right before a run-order entry. ``needs_start``: it reads what the embedding put out."""

    needs_start = False

    def forward(self, residual, start, pending=None) -> None:
        """Add to ``residual`` in place, together with ``pending``. ``start``: the embedding's output (None unless an
        injection of the model needs it)."""
        raise NotImplementedError


class Head(Part):
    def forward(self, x):
        raise NotImplementedError
