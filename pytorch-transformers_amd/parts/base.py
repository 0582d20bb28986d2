"""Interfaces of the parts a model is put together from, and the table of part kinds.

A part is built from sizes and constants only; it never sees a model
configuration and does not know which model it is in.  Every part

* lists the tensors it needs (``tensor_specs``) under the names the weight file
  uses, and takes them from a dict by those names (``load``);
* works on activations ``[tokens, features]`` of all sequences of a step laid
  end to end; which token belongs to which sequence, and where it stands, is in
  the :class:`StepContext`.

Kinds and their ``forward``:

=============  ==================================================================
mixer          ``forward(x, ctx, call, residual=None) -> [tokens, hidden]``; reads
               and writes the cache layer that ``call`` names (keys and values, or
               a state table); ``residual`` is added to the result if given
feed_forward   ``forward(x, ctx, add1=None, add2=None) -> [tokens, hidden]``
norm           ``forward(x, rows=None) -> [tokens, hidden]`` (``rows``: int32
               indices of the rows to take); ``forward_pair(x, other)`` may fuse
               two norms of the same input
positions      ``rotation() -> (inv_freq or None, scale)`` for queries and keys,
               ``score_bias() -> per-head slopes or None`` for attention scores;
               optionally ``rotation_for(ctx) -> (table, scale)`` where the table may
               have a row per sequence of the step (frequencies that follow a length)
block          ``forward(x, ctx, call) -> x``: the arrangement of the above
stream         what a block does to the residual stream between layers (a weighted
               sum of the streams that earlier layers left: ``parts.depth``)
=============  ==================================================================

Optional: a mixer may offer to be one half of a ``SideBySideMixer``: ``input_parts()`` (the products of its input, as
loaded ``Linear`` layers, which the two halves' mixer runs as one), ``result_columns`` and ``result_into(proj, out, mult,
ctx, call)`` (from those products' columns to what its last product ``out`` would read, times ``mult``, written into the
given columns).

Optional: a mixer or feed-forward that sets ``can_defer = True`` and is called with
``defer=True`` returns its last product not run, as a ``PendingProjection`` (the
``Linear`` and its input; residual and additions are then the caller's), and one
with ``input_projection()`` lets the block run its first product and hand the result
in as ``projected``.  A block may so run two branches' products in one launch, and
leave the last ones as 32-bit partial sums (:class:`PartialProduct`) in a
:class:`ResidualSum` that it returns in place of a tensor.  A norm with
``forward_sum(sum, rows=None, other=None, want_x=True) -> (x, normed, normed_other)``
forms such a sum while it normalises it; a block with ``accepts_sum = True`` takes one
as its input.  Everything else receives plain tensors.
"""
from __future__ import annotations

import dataclasses
from typing import Any, Dict, List, Optional, Sequence

import torch

from ..engine.spec import TensorSpec

_KINDS = ("mixer", "feed_forward", "norm", "positions", "block", "stream")
_TABLE: Dict[str, Dict[str, type]] = {k: {} for k in _KINDS}


def register_part(kind: str, name: str, cls: type, *, exist_ok: bool = False) -> type:
    if kind not in _TABLE:
        raise ValueError(f"unknown part kind {kind!r}; kinds: {_KINDS}")
    if not exist_ok and name in _TABLE[kind]:
        raise ValueError(f"{kind} {name!r} is already registered")
    _TABLE[kind][name] = cls
    return cls


def make_part(kind: str, name: str, **params):
    try:
        cls = _TABLE[kind][name]
    except KeyError:
        raise ValueError(f"no {kind} named {name!r}; registered: {sorted(_TABLE.get(kind, {}))}") from None
    return cls(**params)


def registered_parts(kind: str) -> List[str]:
    return sorted(_TABLE[kind])


class Part:
    """Base of all parts: tensors by name."""

    def tensor_specs(self) -> List[TensorSpec]:
        return []

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        """Take this part's tensors out of ``tensors`` (already on the device, in device types)."""

    def children(self) -> Sequence["Part"]:
        return ()

    def all_tensor_specs(self) -> List[TensorSpec]:
        out = list(self.tensor_specs())
        for c in self.children():
            out.extend(c.all_tensor_specs())
        return out

    def load_all(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.load(tensors)
        for c in self.children():
            c.load_all(tensors)

    def check_sizes(self) -> None:
        """Raise ``ValueError`` if no kernel takes this part's sizes; called before a weight is read or drawn."""

    def check_all_sizes(self) -> None:
        self.check_sizes()
        for c in self.children():
            c.check_all_sizes()


@dataclasses.dataclass
class PartialProduct:
    """A matrix product that its kernel left as 32-bit partial sums over ranges of K, ``[ranges, tokens,
    features]``, with the bias still to be added.  Whoever reads it adds the ranges in order, rounds, and adds
    the bias: the value the product's own epilogue would have stored."""

    parts: torch.Tensor
    bias: Optional[torch.Tensor] = None

    def term(self):
        return (self.parts, self.bias)


class ResidualSum:
    """The residual stream as a sum that is not formed yet: products first, then tensors, added in that
    order and rounded once.  A block may return it in place of a tensor; the norm that reads it next forms
    the sum in the same pass (``forward_sum``), and ``tensor()`` forms it for anyone else."""

    def __init__(self, terms: Sequence[Any]):
        self.terms = [t for t in terms if t is not None]
        first = self.terms[0]
        self.features = (first.parts if isinstance(first, PartialProduct) else first).shape[-1]

    def kernel_terms(self):
        return [t.term() if isinstance(t, PartialProduct) else t for t in self.terms]

    def tensor(self) -> torch.Tensor:
        from .. import ops

        if len(self.terms) == 1 and not isinstance(self.terms[0], PartialProduct):
            return self.terms[0]
        return ops.layernorm_sum(self.kernel_terms(), self.features)[0]


class WideResidual:
    """The residual stream held in 32-bit (``wide``) beside the same values in the model's compute type
    (``narrow``), which is what the next matrix product reads; in a 32-bit model the two are one tensor.
    ``history``: what a block that mixes the streams of earlier layers keeps for the step (see
    ``parts.depth.DepthMix``), handed on from block to block."""

    def __init__(self, wide: torch.Tensor, narrow: torch.Tensor, history=None):
        self.wide, self.narrow, self.history = wide, narrow, history


class WideSum(WideResidual):
    """A 32-bit stream as a sum that is not formed yet: ``base`` (32-bit) plus the ``terms`` (up to two tensors of
    the compute type) that a block's branches left.  The block that runs next forms the sum in the launch that norms
    it (``ops.shift_norm``); anyone else who asks for ``wide`` (the final norm, a hook) has it formed then."""

    def __init__(self, base: torch.Tensor, terms: Sequence[torch.Tensor], dtype: torch.dtype):
        self.base, self.terms, self.dtype = base, [t for t in terms if t is not None], dtype
        self.history = None
        self._wide = None

    @property
    def wide(self) -> torch.Tensor:
        if self._wide is None:
            from .. import ops

            self._wide = ops.wide_sum(self.base, self.terms)
        return self._wide

    @property
    def narrow(self) -> torch.Tensor:
        return self.wide if self.dtype == torch.float32 else self.wide.to(self.dtype)


class PendingNormSum(WideResidual):
    """A 32-bit stream whose last sublayer is not added yet: ``x + mult * LN(y) * weight + bias`` with ``x`` the stream
    before the sublayer, ``y`` the sublayer's output in the compute type and ``post = (weight, bias)`` the norm that
    stands on it (``eps`` inside its root; ``rms``: an RMS norm, whose bias is None).  The launch that reads the stream next (the next block's first norm, the
    final norm) forms it on its way (``launch_terms`` are its arguments for ``ops.layernorm_stream``); anyone else who
    asks for ``wide`` has it formed then."""

    def __init__(self, x: torch.Tensor, y: torch.Tensor, post, mult: float, eps: float, dtype: torch.dtype, rms: bool = False):
        self.x, self.y, self.post, self.mult, self.eps, self.dtype = x, y, post, float(mult), float(eps), dtype
        self.rms = bool(rms)
        self.history = None
        self._wide = None

    @property
    def formed(self) -> bool:
        return self._wide is not None

    def launch_terms(self) -> Dict[str, Any]:
        if self._wide is not None:
            return {"x": self._wide}
        return {"x": self.x, "y": self.y, "post": self.post, "mult": self.mult}

    @property
    def wide(self) -> torch.Tensor:
        if self._wide is None:
            from .. import ops

            self._wide = ops.layernorm_stream(self.dtype, eps=self.eps, rms=self.rms, **self.launch_terms())[1]
        return self._wide

    @property
    def narrow(self) -> torch.Tensor:
        return self.wide if self.dtype == torch.float32 else self.wide.to(self.dtype)


class HyperStreams(WideResidual):
    """``count`` residual streams per token in 32-bit: ``x`` ``[tokens, count, features]``, or ``[tokens, features]`` where
    all of them are still that one.  A sublayer's result ``y`` (compute type) may be not yet taken in: the streams are then
    ``sum_s mix[s, t] x_s + out[t] y``, formed by the launch that reads them next (``parts.blocks.HyperBlock``; the final
    norm, for the wanted rows alone).  As one stream (``wide``) they are their sum."""

    def __init__(self, x: torch.Tensor, count: int, dtype: torch.dtype, y: Optional[torch.Tensor] = None, mix=None, out=None):
        self.x, self.count, self.dtype = x, int(count), dtype
        self.y, self.mix, self.out = y, mix, out
        self.history = None
        self._wide = None

    def launch(self, **how):
        """``ops.hyper_norm`` on these streams."""
        from .. import ops

        return ops.hyper_norm(self.x, self.count, self.dtype, y=self.y, mix=self.mix, out=self.out, **how)

    @property
    def wide(self) -> torch.Tensor:
        if self._wide is None:
            self._wide = self.launch(want_u=True)[2]
        return self._wide

    @property
    def narrow(self) -> torch.Tensor:
        return self.wide if self.dtype == torch.float32 else self.wide.to(self.dtype)


def as_tensor(x):
    """A tensor from what a part may hand on: a tensor, a ``PartialProduct``, a ``ResidualSum`` or a
    ``WideResidual`` (its 32-bit side)."""
    if isinstance(x, WideResidual):
        return x.wide
    if isinstance(x, PartialProduct):
        return ResidualSum([x]).tensor()
    if isinstance(x, ResidualSum):
        return x.tensor()
    return x


@dataclasses.dataclass
class StepContext:
    """What one step's tokens are: built once per step by the engine, read by every part."""

    dtype: torch.dtype
    device: torch.device
    n_seqs: int
    n_tokens: int
    #: per token: index of its sequence in this step, and its position in that sequence
    token_seq: torch.Tensor
    token_pos: torch.Tensor
    #: per sequence: first token's offset in the step (n_seqs + 1 entries), cached length before the step
    cu_tokens: torch.Tensor
    seq_start: torch.Tensor
    #: per sequence: its slot (row of state tables)
    seq_slot: torch.Tensor
    #: per paged cache group: [n_seqs, pages] page ids
    block_tables: Dict[str, torch.Tensor]
    cache: Any
    #: host copies, for launch geometry
    slots: List[int]
    new_tokens: List[int]
    starts: List[int]
    #: True if every sequence brings exactly one token
    is_decode: bool = False
    #: upper bound of any sequence's length after this step, used to size launches
    max_len: int = 0
    #: upper bound of the sequences' mean length after this step (0: not known, take ``max_len``); launches
    #: may be shaped by it, but no result depends on it
    mean_len: int = 0
    extras: Dict[str, Any] = dataclasses.field(default_factory=dict)
