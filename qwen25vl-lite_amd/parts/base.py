"""What a layer is made of: the interfaces of the parts and the data a step hands them.

A part is built from a dictionary of its own sizes and constants and never learns which
model it sits in.  It declares the tensors it needs (by local name and shape), receives
them once, and then transforms activations of a flat batch of tokens.

Kinds of parts and what each must provide:

* ``Norm``: ``forward(stream) -> x``.  Folds the stream's pending addend into the float32
  residual and returns the normalised activations in the run dtype.
* ``Mixer``: ``forward(x, step, slot) -> y`` for ``x`` of ``[N, hidden]``; it may keep keys and
  values in pages (``cache_need()``) and/or a state of fixed size per request
  (``state_need()``), both handed to it through ``slot``.
* ``FeedForward``: ``forward(x, step) -> y``.
  A mixer or feed-forward may add ``y`` into ``step.residual`` (the float32 residual, if the block
  offers it) itself and return None; one that sets ``takes_lazy_norm`` may be handed
  :class:`~qwen25vl_lite_amd.ops.linear.NormedRows` instead of a tensor and passes it to its first
  product, which then computes the norm on the way.
* ``PositionEncoding``: ``rotary_tables(head_dim, device)`` gives the per-frequency inverse
  frequencies and the row of the position tensor each frequency reads.
* ``Block``: ``forward(stream, step, slot)`` arranges two norms, a mixer and a feed-forward.
* ``Filter``: ``forward(h, step, slot) -> x``: what a sublayer reads, made from float32 rows (a short
  convolution over time, a step towards the token before); it may keep a per-request state like a mixer.
* ``Embedding``: ``forward(token_ids, step) -> h``; one with a ``state_need()`` of its own is called with its
  slot as a third argument.

New kinds are added with :func:`register_part` and named in a model's layer specs.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Callable, Dict, List, Optional, Sequence, Tuple

import torch

__all__ = [
    "ParamSpec", "PartSpec", "CacheNeed", "StateNeed", "LayerSlot", "GroupStep", "StepContext", "ResidualStream",
    "NormedMean", "SumTerm", "ScaledSum",
    "Part", "Norm", "Mixer", "FeedForward", "Filter", "PositionEncoding", "Block", "register_part", "build_part",
    "known_parts", "Embedding", "Head",
]


@dataclass(frozen=True)
class ParamSpec:
    """A tensor a part needs.  ``role`` decides how it is kept on the device:
    ``"matrix"`` and ``"table"`` in the run dtype (bfloat16 or float32), ``"vector"`` in
    float32 (norm weights, biases: they enter float32 arithmetic), ``"int"`` as int32.
    ``init`` says how the random-weights mode draws it: ``"normal"`` N(0, std),
    ``"around_one"`` 1 + N(0, std) (a gain), ``"zeros"``, ``"ones"``, ``"unit_interval"`` uniform on [0, 1)
    (a floor of a gate), ``"identity"`` a square matrix of N(0, std) plus the identity.  ``free``: the axes
    whose size the checkpoint decides (the part takes whatever comes and checks that its tensors fit each
    other); ``shape`` then holds the size the random-weights mode draws."""

    shape: Tuple[int, ...]
    role: str = "matrix"
    init: str = "normal"
    free: Tuple[int, ...] = ()

    def takes(self, shape) -> bool:
        """Whether a stored tensor of this shape fits."""
        shape = tuple(shape)
        return len(shape) == len(self.shape) and all(
            got > 0 if axis in self.free else got == want for axis, (got, want) in enumerate(zip(shape, self.shape)))


@dataclass(frozen=True)
class PartSpec:
    """A part named by its registered kind, with its sizes and constants."""

    kind: str
    params: Dict[str, Any] = field(default_factory=dict)


@dataclass(frozen=True)
class CacheNeed:
    """Keys and values a mixer keeps per token.  ``window`` None: all keys stay; a number:
    only the last ``window`` keys are read, older pages may be given back, except the pages of
    the first ``keep_first`` tokens, which every later token still reads.  ``value_dim`` None:
    values are as wide as keys (``head_dim``).  ``chunk`` a number: positions are cut into chunks of
    that many from the sequence's start on and only keys of a token's own chunk are read."""

    num_kv_heads: int
    head_dim: int
    window: Optional[int] = None
    keep_first: int = 0
    value_dim: Optional[int] = None
    chunk: Optional[int] = None

    @property
    def v_dim(self) -> int:
        return self.head_dim if self.value_dim is None else self.value_dim

    def first_visible(self, position: int) -> int:
        """The first key that a token at ``position``, and with it any later one, sees (kept first keys aside)."""
        first = 0
        if self.window is not None:
            first = max(first, position - self.window + 1)
        if self.chunk is not None:
            first = max(first, position - position % self.chunk)
        return first


@dataclass(frozen=True)
class StateNeed:
    """A state of fixed size a mixer keeps per request (zeroed when a request starts)."""

    shape: Tuple[int, ...]
    dtype: torch.dtype = torch.float32


@dataclass
class LayerSlot:
    """What one entry of the run list owns in the cache: its group and cache layer, whether
    it writes keys and values (an entry that reads another's cache does not), and its state."""

    group: Optional[int] = None
    k_cache: Optional[torch.Tensor] = None  # [pages, nkv, page_size, hd]
    v_cache: Optional[torch.Tensor] = None  # [pages, nkv, vd, page_size]
    writes: bool = True
    state: Optional[torch.Tensor] = None    # [max_num_seqs, *StateNeed.shape]
    # the slot of a run entry: every part's that owns anything under its dotted name in the block (this
    # slot stands for the first of them); the slot of a part: its own sub-parts' under their names in it
    by_part: Dict[str, "LayerSlot"] = field(default_factory=dict)

    def of(self, name: str) -> "LayerSlot":
        """The named part's slot, or this one where none is kept under that name."""
        return self.by_part.get(name, self)


@dataclass
class GroupStep:
    """A cache group's view of a step: where each token's keys and values go, and the pages
    of each request of the batch (row r, entry i = page of tokens i*page_size ...; -1 = none)."""

    slot_mapping: torch.Tensor  # int32 [N]
    block_table: torch.Tensor   # int32 [R, width]
    page_size: int


@dataclass
class StepContext:
    """One step's batch on the device: N tokens of R requests, each request a contiguous run."""

    num_tokens: int
    num_reqs: int
    token_ids: torch.Tensor     # int32 [N]
    positions: torch.Tensor     # int32 [rows, N]
    token_req: torch.Tensor     # int32 [N]   row of the request in this batch
    token_seqpos: torch.Tensor  # int32 [N]   index of the token in its sequence
    cu_q: torch.Tensor          # int32 [R+1] where each request's run starts
    ctx_len: torch.Tensor       # int32 [R]   tokens of the request in the cache after this step
    req_slots: torch.Tensor     # int32 [R]   the request's state slot
    groups: List[GroupStep]
    logit_rows: torch.Tensor    # int32 [M]
    cu_q_host: Sequence[int] = ()
    ctx_len_host: Sequence[int] = ()
    req_slots_host: Sequence[int] = ()
    max_q_len: int = 0
    max_ctx_len: int = 0
    dtype: torch.dtype = torch.float32
    residual: Optional[torch.Tensor] = None   # set by a block while a part may add its result in place
    # the model's second table of token rows [vocab, columns], where it has one: layers read columns of their own
    token_side: Optional[torch.Tensor] = None
    derived: Dict[Any, Any] = field(default_factory=dict)   # per-step arrays kernels derive once (tile lists)
    # tensors computed from the step's values once per forward pass (rotation tables): a context
    # that is run again with new values (a captured step) starts each pass with this empty
    per_pass: Dict[Any, Any] = field(default_factory=dict)


@dataclass
class ResidualStream:
    """The residual sum in float32 and an addend that has not been folded in yet.  The next
    norm adds ``pending`` to ``h`` in float32 in the same kernel that normalises."""

    h: torch.Tensor                          # float32 [N, hidden]
    pending: Optional[torch.Tensor] = None   # float32 or run dtype [N, hidden]
    # (gain float32 [hidden], eps, factor): the pending addend enters the sum as
    # factor * rmsnorm(pending) * gain instead of as it is (a sublayer with a norm behind it)
    pending_norm: Optional[Tuple[torch.Tensor, float, float]] = None
    # a vector float32 [hidden] that the next norm adds to every row of the sum
    row_addend: Optional[torch.Tensor] = None
    # several copies of the sum, mixed anew by every sublayer (hyper-connections): float32 [N, copies, hidden].
    # None while every copy still equals ``h`` (the embedding's output)
    copies: Optional[torch.Tensor] = None
    # (mix [copies, copies], out [copies]) float32: how the pending addend joins the copies
    pending_join: Optional[Tuple[torch.Tensor, torch.Tensor]] = None
    # ``h`` rounded to the run dtype, where the kernel that wrote ``h`` last wrote that too (a block that leaves it
    # says so: ``Block.leaves_rounded``)
    rounded: Optional[torch.Tensor] = None


@dataclass
class NormedMean:
    """A sublayer's result that is ``factor * (rmsnorm(first) gain_first + rmsnorm(second) gain_second)`` and
    has not been computed yet: the kernel that adds it to the sum forms it on the way.  The addends are ``[N, hidden]``
    (float32 or run dtype) or float32 slabs ``[slabs, N, hidden]`` that are added in order."""

    first: torch.Tensor
    second: torch.Tensor
    gain_first: torch.Tensor
    gain_second: torch.Tensor
    eps: float
    factor: float


@dataclass
class ScaledSum:
    """A sublayer's result ``factor_first * first + factor_second * second`` that has not been computed yet (addends as
    in :class:`NormedMean`)."""

    first: torch.Tensor
    second: torch.Tensor
    factor_first: float
    factor_second: float


@dataclass
class SumTerm:
    """One term of a residual sum: ``factor * value``, or with a gain ``factor * rmsnorm(value) * gain``.  ``value`` is
    ``[N, hidden]`` (float32 or bfloat16) or float32 slabs ``[slabs, N, hidden]`` that are added in order."""

    value: torch.Tensor
    factor: float = 1.0
    gain: Optional[torch.Tensor] = None
    eps: float = 0.0

    @staticmethod
    def of(result) -> List["SumTerm"]:
        """The terms of what a sublayer returned."""
        if isinstance(result, NormedMean):
            return [SumTerm(result.first, result.factor, result.gain_first, result.eps),
                    SumTerm(result.second, result.factor, result.gain_second, result.eps)]
        if isinstance(result, ScaledSum):
            return [SumTerm(result.first, result.factor_first), SumTerm(result.second, result.factor_second)]
        return [SumTerm(result)]


class Part:
    """Base of all parts.  ``graph_safe`` says that ``forward`` only launches device work whose
    shape depends on the step's shape alone (no host reads of device data, no host loops over
    the step's values: requests, positions, state rows and pages are found through the step's
    device tensors), so a decode step through it may be captured in a HIP graph and replayed
    with other values in the same buffers.  It promises nothing about running a step twice: a
    mixer may advance its per-request state on every pass (the engine puts the state rows back
    after the passes it runs to warm a new graph up)."""

    graph_safe: bool = False
    takes_lazy_norm: bool = False   # forward accepts NormedRows in place of the normalised tensor

    def __init__(self, dtype: torch.dtype, device: torch.device):
        self.dtype = dtype
        self.device = device

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {}

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        """Receive the tensors of :meth:`param_specs`, already on the device in their kept dtype."""

    def sub_parts(self) -> Dict[str, "Part"]:
        return {}

    def cache_need(self) -> Optional[CacheNeed]:
        """Keys and values this part keeps per token in pages, or None."""
        return None

    def state_need(self) -> Optional[StateNeed]:
        """A state of fixed size this part keeps per request, or None.  A part with either need gets a
        :class:`LayerSlot` of its own for every entry of the run list that names its layer."""
        return None


class Norm(Part):
    def forward(self, stream: ResidualStream, rows: Optional[torch.Tensor] = None, lazy: bool = False):
        """Fold ``stream.pending`` into ``stream.h`` and return the normalised rows; with ``lazy`` it
        may return :class:`~qwen25vl_lite_amd.ops.linear.NormedRows` instead of computing them."""
        raise NotImplementedError


class Mixer(Part):
    # a mixer that reads several mixes of a token's input with the one's before it names the sub-part that
    # holds their weights (a TokenMixes part): a block may then hand it the mixes instead of the input
    token_mixes: Optional[Part] = None

    def forward(self, x: torch.Tensor, step: StepContext, slot: LayerSlot) -> torch.Tensor:
        raise NotImplementedError


class FeedForward(Part):
    def forward(self, x: torch.Tensor, step: StepContext) -> torch.Tensor:
        raise NotImplementedError


class Filter(Part):
    """A transform of float32 rows (the residual's, or a norm's) on their way into a sublayer (a short
    convolution over time, a step towards the token before); it may keep a state per request."""

    def forward(self, h: torch.Tensor, step: StepContext, slot: LayerSlot) -> torch.Tensor:
        """float32 ``[N, hidden]`` -> ``[N, hidden]`` in the run dtype."""
        raise NotImplementedError


class PositionEncoding(Part):
    num_rows: int = 1

    def rotary_tables(self, head_dim: int) -> Tuple[torch.Tensor, torch.Tensor]:
        """``(inv_freq float32 [rot/2], freq_row int32 [rot/2])`` on the device."""
        raise NotImplementedError

    def table_key(self, head_dim: int):
        """A hashable value that is equal for encodings with equal tables: layers whose encodings
        agree share what a step derives from the tables.  Default: this instance only."""
        return (id(self), head_dim)


class Block(Part):
    leaves_rounded: bool = False    # forward leaves ``stream.rounded`` equal to the ``stream.h`` it leaves

    def forward(self, stream: ResidualStream, step: StepContext, slot: LayerSlot) -> ResidualStream:
        raise NotImplementedError


class Embedding(Part):
    """Token ids to the start of the residual sum.  ``table`` is the tensor a tied head shares.  An
    embedding may keep a state per request (``state_need``); ``forward`` then gets its slot too."""

    table: Optional[torch.Tensor] = None

    def forward(self, token_ids: torch.Tensor, step: StepContext, slot: Optional[LayerSlot] = None) -> torch.Tensor:
        """int32 ``[N]`` -> float32 ``[N, hidden]``."""
        raise NotImplementedError


class Head(Part):
    """Normalised rows to logits."""

    def forward(self, x, step: StepContext) -> torch.Tensor:
        """``[rows, hidden]`` -> float32 ``[rows, vocab]``."""
        raise NotImplementedError

    def tie(self, embedding: Embedding) -> None:
        """Use the embedding's table instead of a tensor of its own (a model that ties the two)."""
        raise NotImplementedError


_REGISTRY: Dict[str, Dict[str, Callable[..., Part]]] = {
    "norm": {}, "mixer": {}, "ffn": {}, "position": {}, "block": {}, "embedding": {}, "head": {}, "filter": {},
}


def register_part(category: str, kind: str, factory: Callable[..., Part], *, replace: bool = False) -> None:
    """Register ``factory(params, dtype, device) -> Part`` under ``category``/``kind``."""
    if category not in _REGISTRY:
        raise KeyError(f"unknown part category {category!r}; known: {sorted(_REGISTRY)}")
    if kind in _REGISTRY[category] and not replace:
        raise ValueError(f"{category} part {kind!r} is already registered")
    _REGISTRY[category][kind] = factory


def known_parts(category: str) -> List[str]:
    return sorted(_REGISTRY[category])


def build_part(category: str, spec: PartSpec, dtype: torch.dtype, device: torch.device) -> Part:
    try:
        factory = _REGISTRY[category][spec.kind]
    except KeyError:
        raise KeyError(f"no {category} part of kind {spec.kind!r}; known: {known_parts(category)}") from None
    return factory(dict(spec.params), dtype, device)
