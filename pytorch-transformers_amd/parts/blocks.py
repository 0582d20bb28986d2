"""How norm, mixer and feed-forward stand in a block, and how the residual is summed.

The two arrangements of ``FalconDecoderLayer.forward``
(src/transformers/models/falcon/modeling_falcon.py:614-683):

parallel    ``x + (ffn(norm_ffn(x)) + mixer(norm_mixer(x)))``; with one norm both branches read
            the same normed input (:630-634, :648-676).  The sum is formed in that order:
            feed-forward plus mixer first (:673-674), then the residual (:676).
sequential  ``r = x + mixer(norm_in(x))``; ``r + ffn(norm_post(r))`` (:652-659, :676).

The additions ride in the last matrix product's epilogue of each branch, or, in steps of few tokens,
the products stay unreduced and the next norm forms the sum while it reads it (``ResidualSum``).
"""
from __future__ import annotations

from typing import Optional, Sequence

import torch

from ..engine.spec import INIT_EYE_NOISE, INIT_NORMAL, INIT_ONE_NOISE, INIT_ZERO_NOISE, VECTOR, TensorSpec
from .base import HyperStreams, Part, PendingNormSum, ResidualSum, StepContext, WideResidual, WideSum, as_tensor, register_part
from .linear import Linear, PendingProjection


def _can_defer(part: Part) -> bool:
    return bool(getattr(part, "can_defer", False))


def _normed(x, norm: Part, other: Optional[Part] = None):
    """``(x as a tensor, norm(x), other(x) or None)`` for a block input that may be a sum not formed yet."""
    if isinstance(x, ResidualSum):
        if hasattr(norm, "forward_sum"):
            return norm.forward_sum(x, other=other)
        x = x.tensor()
    if other is None:
        return x, norm.forward(x), None
    if hasattr(norm, "forward_pair"):  # two norms of one input in one pass, where the norm offers it
        a, m = norm.forward_pair(x, other)
    else:
        a, m = norm.forward(x), other.forward(x)
    return x, a, m


def _sum_parallel(ffn_out: PendingProjection, mixer_out: PendingProjection, x: torch.Tensor):
    """feed-forward + mixer + residual, in that order, formed now or left to the next norm."""
    both = PendingProjection.partial_pair(ffn_out, mixer_out)
    if both is not None:
        return ResidualSum([both[0], both[1], x])
    p = ffn_out.partial()
    if p is not None:
        return ResidualSum([p, mixer_out.partial() or mixer_out.run(), x])
    if ffn_out.additions_cost_a_pass():  # prompts: the next norm adds the three while it reads them
        return ResidualSum([ffn_out.run(), mixer_out.run(), x])
    return ffn_out.run(add1=mixer_out.run(), add2=x)


def _sum_sequential(out: PendingProjection, residual: torch.Tensor):
    p = out.partial()
    if p is not None:
        return ResidualSum([p, residual])
    if out.additions_cost_a_pass():
        return ResidualSum([out.run(), residual])
    return out.run(add1=residual)


class ParallelBlock(Part):
    accepts_sum = True

    def __init__(self, mixer: Part, feed_forward: Part, norm_mixer: Part, norm_ffn: Optional[Part] = None):
        self.mixer = mixer
        self.feed_forward = feed_forward
        self.norm_mixer = norm_mixer
        self.norm_ffn = norm_ffn

    def children(self) -> Sequence[Part]:
        return tuple(p for p in (self.norm_mixer, self.norm_ffn, self.mixer, self.feed_forward) if p is not None)

    def after_load(self) -> None:
        """With one norm both branches start from the same input: their first matrices are laid out side by
        side, so that prompts can run them as one product."""
        if self.norm_ffn is None and hasattr(self.mixer, "input_projection") and hasattr(self.feed_forward, "input_projection"):
            Linear.join(self.mixer.input_projection()[0], self.feed_forward.input_projection()[0])

    def forward(self, x, ctx: StepContext, call):
        x, a, m = _normed(x, self.norm_mixer, self.norm_ffn)
        if m is None:
            m = a
        kw_mixer, kw_ffn = {}, {}
        # both branches start with a product of the norm's output: one launch for the two in small steps
        if hasattr(self.mixer, "input_projection") and hasattr(self.feed_forward, "input_projection"):
            (lin_a, kw_a), (lin_m, kw_m) = self.mixer.input_projection(), self.feed_forward.input_projection()
            tail = self.mixer.projection_tail(ctx, call) if hasattr(self.mixer, "projection_tail") else None
            both = Linear.pair(lin_a, a, kw_a, lin_m, m, kw_m, tail=tail)
            if both is not None:
                kw_mixer["projected"], kw_ffn["projected"] = both
        if _can_defer(self.feed_forward) and _can_defer(self.mixer):
            # the branches' last products: one launch of partial sums where that pays, which the
            # next norm adds to the residual while it reads them
            out_a = self.mixer.forward(a, ctx, call, defer=True, **kw_mixer)
            out_m = self.feed_forward.forward(m, ctx, defer=True, **kw_ffn)
            return _sum_parallel(out_m, out_a, x)
        mixed = self.mixer.forward(a, ctx, call, **kw_mixer)
        return self.feed_forward.forward(m, ctx, add1=mixed, add2=x, **kw_ffn)


class SequentialBlock(Part):
    accepts_sum = True

    def __init__(self, mixer: Part, feed_forward: Part, norm_in: Part, norm_post: Part):
        self.mixer = mixer
        self.feed_forward = feed_forward
        self.norm_in = norm_in
        self.norm_post = norm_post

    def children(self) -> Sequence[Part]:
        return (self.norm_in, self.norm_post, self.mixer, self.feed_forward)

    def forward(self, x, ctx: StepContext, call):
        x, a, _ = _normed(x, self.norm_in)
        if _can_defer(self.mixer):
            r = _sum_sequential(self.mixer.forward(a, ctx, call, defer=True), x)
        else:
            r = self.mixer.forward(a, ctx, call, residual=x)
        r, m, _ = _normed(r, self.norm_post)
        if _can_defer(self.feed_forward):
            return _sum_sequential(self.feed_forward.forward(m, ctx, defer=True), r)
        return self.feed_forward.forward(m, ctx, add1=r)


class PostNormBlock(Part):
    """``x <- x + m * norm_mixer(mixer(x))``, then ``x <- x + m * norm_ffn(ffn(x))``: the sublayers read the stream
    itself and the norm stands on each sublayer's output; ``m`` is a constant.  The stream is kept in 32-bit
    whatever the compute type (``WideResidual``): a sublayer reads its copy in the compute type, the norm, the
    scaling and the addition are one 32-bit launch that also writes that copy for the next sublayer.
    ``feed_forward`` may be None (a layer of the mixer alone).  With ``depth_mix`` (``parts.depth.DepthMix``) the
    block's result is kept as the next of the step's streams and what goes on is their weighted sum.  ``hand_on_unformed``
    (for a model's last block, with LayerNorms): the last sublayer's output goes on not yet normed and added
    (``PendingNormSum``), and the final norm's launch does both on its way, for the rows whose logits are wanted alone."""

    accepts_sum = False
    accepts_wide = True

    def __init__(self, mixer: Part, feed_forward: Optional[Part], norm_mixer: Part, norm_ffn: Optional[Part],
                 residual_mult: float = 1.0, depth_mix: Optional[Part] = None, hand_on_unformed: bool = False):
        if (feed_forward is None) != (norm_ffn is None):
            raise ValueError("a feed-forward and its norm come together or not at all")
        self.mixer, self.feed_forward, self.norm_mixer, self.norm_ffn = mixer, feed_forward, norm_mixer, norm_ffn
        self.residual_mult = float(residual_mult)
        self.depth_mix = depth_mix
        last_norm = norm_mixer if norm_ffn is None else norm_ffn
        self.hand_on_unformed = bool(hand_on_unformed) and depth_mix is None and hasattr(last_norm, "affine")

    def children(self) -> Sequence[Part]:
        return tuple(p for p in (self.norm_mixer, self.norm_ffn, self.mixer, self.feed_forward, self.depth_mix)
                     if p is not None)

    def after_load(self) -> None:
        for part in (self.mixer, self.feed_forward):
            if part is not None and hasattr(part, "after_load"):
                part.after_load()

    def _enter(self, x, ctx: StepContext) -> WideResidual:
        """The stream as this block wants it; the first block of a model is given the embedding's plain tensor."""
        from .. import ops

        if isinstance(x, WideResidual):
            return x
        x = as_tensor(x)
        history = None
        if self.depth_mix is not None:
            history = self.depth_mix.new_history(x.shape[0], x.shape[1], x.device)
            wide = ops.widen(x, history.next_plane())
        else:
            wide = x if x.dtype == torch.float32 else ops.widen(x)
        return WideResidual(wide, x if x.dtype == ctx.dtype else wide, history)

    def forward(self, x, ctx: StepContext, call):
        x = self._enter(x, ctx)
        last = self.feed_forward is None
        history = x.history
        keep = history.next_plane() if (history is not None and self.depth_mix is not None) else None
        # the launch that forms the block's result also keeps it as a stream and goes on to the streams' weighted sum
        mix = self.depth_mix.fused(history) if keep is not None else None
        mixed = self.mixer.forward(x.narrow, ctx, call)
        if last and self.hand_on_unformed:
            return PendingNormSum(x.wide, mixed, self.norm_mixer.affine(), self.residual_mult, self.norm_mixer.eps, ctx.dtype)
        narrow, wide = self.norm_mixer.apply(mixed, ctx.dtype, residual=x.wide, mult=self.residual_mult, want_wide=True,
                                             out_wide=keep if last else None, mix=mix if last else None)
        if not last:
            out = self.feed_forward.forward(narrow, ctx)
            if self.hand_on_unformed:
                return PendingNormSum(wide, out, self.norm_ffn.affine(), self.residual_mult, self.norm_ffn.eps, ctx.dtype)
            narrow, wide = self.norm_ffn.apply(out, ctx.dtype, residual=wide, mult=self.residual_mult, want_wide=True,
                                               out_wide=keep, mix=mix)
        return WideResidual(wide, narrow, history)


class ShiftedParallelBlock(Part):
    """``x <- x + (mixer(shift(norm_mixer(x))) + ffn(norm_ffn(x)))`` over a stream kept in 32-bit: both branches read
    norms of the same x.  ``shift``: what the mixer reads, ``h = norm_mixer(x)``, is replaced by ``h + (h' - h) * mu``
    with h' the h of the token before (zeros at a sequence's first token) and ``mu`` a learned vector (``shift_name``
    in the file).  The h of a sequence's last token is part of its state: a row of the state table that the run
    order's entry names as ``also("shift")``.  ``feed_forward`` may be None (a layer of the mixer alone).

    The block hands on ``x`` and its branches' results as a sum that is not formed (``WideSum``); the next block's
    first launch forms it, norms it twice and shifts (``ops.shift_norm``)."""

    accepts_sum = False
    accepts_wide = True

    def __init__(self, mixer: Part, feed_forward: Optional[Part], norm_mixer: Part, norm_ffn: Optional[Part],
                 shift_name: str, hidden_size: int):
        if (feed_forward is None) != (norm_ffn is None):
            raise ValueError("a feed-forward and its norm come together or not at all")
        if getattr(norm_mixer, "offset", 0.0) or getattr(norm_mixer, "groups", 1) != 1 or (
                norm_ffn is not None and (norm_ffn.offset or norm_ffn.groups != 1 or norm_ffn.eps != norm_mixer.eps)):
            raise ValueError("the shifted block's launch takes plain RMS norms with one eps")
        self.mixer, self.feed_forward, self.norm_mixer, self.norm_ffn = mixer, feed_forward, norm_mixer, norm_ffn
        self.shift_name, self.hidden_size = shift_name, int(hidden_size)
        self.mu: Optional[torch.Tensor] = None

    def children(self) -> Sequence[Part]:
        return tuple(p for p in (self.norm_mixer, self.norm_ffn, self.mixer, self.feed_forward) if p is not None)

    def tensor_specs(self):
        return [TensorSpec(self.shift_name, (self.hidden_size,), VECTOR, INIT_ZERO_NOISE)]

    def load(self, tensors) -> None:
        self.mu = tensors[self.shift_name]

    def after_load(self) -> None:
        for part in (self.mixer, self.feed_forward):
            if part is not None and hasattr(part, "after_load"):
                part.after_load()

    def forward(self, x, ctx: StepContext, call):
        from .. import ops

        if isinstance(x, WideSum):
            base, terms = x.base, x.terms
        elif isinstance(x, WideResidual):
            base, terms = x.wide, []
        else:
            x = as_tensor(x)
            base, terms = (x if x.dtype == torch.float32 else ops.widen(x)), []
        group, layer = call.also("shift")
        state = ctx.cache.state_layer(group, layer)
        stream, a, m = ops.shift_norm(base, terms, self.norm_mixer.weight, None if self.norm_ffn is None else self.norm_ffn.weight,
                                      self.mu, self.norm_mixer.eps, state, ctx, ctx.dtype)
        kw_mixer, kw_ffn = {}, {}
        # both branches start with a product of a norm of x: one launch for the two in small steps
        if hasattr(self.mixer, "input_projection") and hasattr(self.feed_forward, "input_projection"):
            (lin_a, kw_a), (lin_m, kw_m) = self.mixer.input_projection(), self.feed_forward.input_projection()
            both = Linear.pair(lin_a, a, kw_a, lin_m, m, kw_m) if lin_a is not None and lin_m is not None else None
            if both is not None:
                kw_mixer["projected"], kw_ffn["projected"] = both
        mixed = self.mixer.forward(a, ctx, call, **kw_mixer)
        ff = self.feed_forward.forward(m, ctx, **kw_ffn) if self.feed_forward is not None else None
        return WideSum(stream, [mixed, ff], ctx.dtype)


class SandwichBlock(Part):
    """A norm in front of and behind each sublayer, over a stream kept in 32-bit:

        x <- x + m * norm_mixer_out(mixer(norm_mixer(x)));   x <- x + m * norm_ffn_out(ffn(norm_ffn(x)))

    with ``m`` a constant and the four norms LayerNorms with weight and bias, or RMS norms, with one eps (``ops.layernorm_stream``: the
    norm behind a sublayer, the addition and the norm in front of the next sublayer are one launch, across the
    block's end too: the block hands its last sublayer on not yet added, ``PendingNormSum``).  ``feed_forward`` may be
    None (a layer of the mixer alone).  ``loop_entry`` (``parts.depth.LoopEntry``): where the run order's entry says
    that a pass of a loop starts with this block (``call.loop_pass``), the terms that the loop adds to the stream in
    front of the pass ride in the block's first launch."""

    accepts_sum = False
    accepts_wide = True

    def __init__(self, mixer: Part, feed_forward: Optional[Part], norm_mixer: Part, norm_mixer_out: Part,
                 norm_ffn: Optional[Part], norm_ffn_out: Optional[Part], residual_mult: float = 1.0,
                 loop_entry: Optional[Part] = None):
        if not ((feed_forward is None) == (norm_ffn is None) == (norm_ffn_out is None)):
            raise ValueError("a feed-forward and its two norms come together or not at all")
        norms = [n for n in (norm_mixer, norm_mixer_out, norm_ffn, norm_ffn_out) if n is not None]
        if any(not hasattr(n, "affine") for n in norms) or len({(n.eps, n.rms) for n in norms}) != 1:
            raise ValueError("the block's launches take norms of one kind (LayerNorms with weight and bias, or RMS norms) and one eps")
        self.mixer, self.feed_forward = mixer, feed_forward
        self.norm_mixer, self.norm_mixer_out, self.norm_ffn, self.norm_ffn_out = norm_mixer, norm_mixer_out, norm_ffn, norm_ffn_out
        self.residual_mult, self.eps, self.rms = float(residual_mult), norm_mixer.eps, norm_mixer.rms
        self.loop_entry = loop_entry

    def children(self) -> Sequence[Part]:
        return tuple(p for p in (self.norm_mixer, self.norm_mixer_out, self.norm_ffn, self.norm_ffn_out, self.mixer,
                                 self.feed_forward, self.loop_entry) if p is not None)

    def after_load(self) -> None:
        for part in (self.mixer, self.feed_forward):
            if part is not None and hasattr(part, "after_load"):
                part.after_load()

    def forward(self, x, ctx: StepContext, call):
        from .. import ops

        dtype, eps, m = ctx.dtype, self.eps, self.residual_mult
        if isinstance(x, PendingNormSum) and not x.formed and x.eps == eps and x.rms == self.rms:
            terms = x.launch_terms()
        elif isinstance(x, WideResidual):
            terms = {"x": x.wide}
        else:
            x = as_tensor(x)
            terms = {"x": x if x.dtype == torch.float32 else ops.widen(x)}
        if self.loop_entry is not None and getattr(call, "loop_pass", None) is not None:
            add, vec = self.loop_entry.terms(call.loop_pass, ctx)
            terms.update(add=add, vec=vec)
        changed = len(terms) > 1  # the launch forms a stream that is not in memory yet
        h, wide = ops.layernorm_stream(dtype, pre=self.norm_mixer.affine(), eps=eps, want_wide=changed, rms=self.rms, **terms)
        if not changed:
            wide = terms["x"]
        mixed = self.mixer.forward(h, ctx, call)
        if self.feed_forward is None:
            return PendingNormSum(wide, mixed, self.norm_mixer_out.affine(), m, eps, dtype, self.rms)
        h, wide = ops.layernorm_stream(dtype, x=wide, y=mixed, post=self.norm_mixer_out.affine(), mult=m,
                                       pre=self.norm_ffn.affine(), eps=eps, rms=self.rms)
        out = self.feed_forward.forward(h, ctx)
        return PendingNormSum(wide, out, self.norm_ffn_out.affine(), m, eps, dtype, self.rms)


class HyperBlock(Part):
    """Several residual streams (hyper-connections) with a norm in front of each sublayer.  For sublayer q (1: the mixer, 2:
    the feed-forward), over the streams x_1 .. x_S held in 32-bit:

        u = sum_s in_q[s] x_s;   y = sublayer(norm_q(u));   x_t <- sum_s mix_q[s, t] x_s + out_q[t] y  (all at once)

    Between norm and mixer stands a causal convolution per channel that adds to what it reads, ``h + conv(h)`` (``taps``
    inputs, the last column of ``conv_name`` ``[width, taps]`` being the token's own; 0: none), whose last ``taps - 1``
    inputs are part of a sequence's state: a row of the state table that the run order's entry names as ``also("conv")``.
    ``feed_forward`` may be None (a layer of the mixer alone).  The file holds ``name.hc<q>.in``, ``.out`` ``[S]`` and
    ``.mix`` ``[S, S]`` (from, to).

    Everything between two sublayers is one launch (``ops.hyper_norm``), across the block's end too: the block hands its
    last sublayer's result on not yet taken in (``HyperStreams``).  In steps of one token per sequence the convolution
    rides in that launch as well."""

    accepts_sum = False
    accepts_wide = True

    def __init__(self, name: str, mixer: Part, feed_forward: Optional[Part], norm_mixer: Part, norm_ffn: Optional[Part],
                 streams: int, hidden_size: int, taps: int = 0, conv_name: Optional[str] = None):
        if (feed_forward is None) != (norm_ffn is None):
            raise ValueError("a feed-forward and its norm come together or not at all")
        if any(n is not None and (not hasattr(n, "launch_terms") or n.groups != 1) for n in (norm_mixer, norm_ffn)):
            raise ValueError("the block's launches take RMS norms over whole rows")
        if taps and conv_name is None:
            raise ValueError("a convolution needs its tensor's name")
        self.name, self.streams, self.hidden_size, self.taps, self.conv_name = name, int(streams), int(hidden_size), int(taps), conv_name
        self.mixer, self.feed_forward, self.norm_mixer, self.norm_ffn = mixer, feed_forward, norm_mixer, norm_ffn
        self.links = {}  # sublayer -> (in, mix, out)
        self.conv_w: Optional[torch.Tensor] = None

    @property
    def conv_state(self) -> int:
        """Elements of a sequence's state that the convolution keeps."""
        return max(self.taps - 1, 0) * self.hidden_size

    def children(self) -> Sequence[Part]:
        return tuple(p for p in (self.norm_mixer, self.norm_ffn, self.mixer, self.feed_forward) if p is not None)

    def _sublayers(self):
        return (1,) if self.feed_forward is None else (1, 2)

    def tensor_specs(self):
        S, specs = self.streams, []
        for q in self._sublayers():
            specs += [TensorSpec(f"{self.name}.hc{q}.in", (S,), VECTOR, INIT_ONE_NOISE),
                      TensorSpec(f"{self.name}.hc{q}.out", (S,), VECTOR, INIT_ONE_NOISE),
                      TensorSpec(f"{self.name}.hc{q}.mix", (S, S), VECTOR, INIT_EYE_NOISE)]
        if self.taps:
            specs.append(TensorSpec(self.conv_name, (self.hidden_size, self.taps), VECTOR, INIT_NORMAL))
        return specs

    def load(self, tensors) -> None:
        for q in self._sublayers():
            self.links[q] = tuple(tensors[f"{self.name}.hc{q}.{t}"] for t in ("in", "mix", "out"))
        if self.taps:
            self.conv_w = tensors[self.conv_name].t().contiguous()  # tap by tap, so that neighbouring channels lie side by side

    def after_load(self) -> None:
        for part in (self.mixer, self.feed_forward):
            if part is not None and hasattr(part, "after_load"):
                part.after_load()

    def check_sizes(self) -> None:
        from .. import ops

        if not (1 <= self.streams <= ops.HYPER_MAX_STREAMS):
            raise ValueError(f"{self.name}: {self.streams} streams are outside the 1..{ops.HYPER_MAX_STREAMS} that the kernel takes")
        if self.taps > 16:
            raise ValueError(f"{self.name}: a convolution of {self.taps} taps is more than the kernel's 16")
        if self.hidden_size > 16384:
            raise ValueError(f"{self.name}: rows of {self.hidden_size} features are more than the kernel's 16384")

    def _head(self, x: HyperStreams, q: int, norm: Part, ctx: StepContext, conv=None):
        """``(h, the streams with nothing left to take in)``: what sublayer q reads."""
        from .. import ops

        one_each = conv is None or ctx.n_tokens == ctx.n_seqs  # (the convolution rides along: its inputs are in the tails)
        h, n, _, new = x.launch(weights=self.links[q][0], norm=norm.launch_terms(), want_x=x.y is not None, want_h=one_each,
                                want_n=not one_each, conv=conv if one_each else None, ctx=ctx)
        if not one_each:
            h = ops.conv_add(n, conv[0], conv[1], ctx, ctx.dtype)
        return h, (x.x if new is None else new)

    def forward(self, x, ctx: StepContext, call):
        from .. import ops

        if not isinstance(x, HyperStreams):
            x = as_tensor(x)
            x = HyperStreams(x if x.dtype == torch.float32 else ops.widen(x), self.streams, ctx.dtype)
        conv = None
        if self.taps:
            tail = ctx.cache.state_layer(*call.also("conv")) if self.taps > 1 else None
            conv = (self.conv_w, tail)
        h, streams = self._head(x, 1, self.norm_mixer, ctx, conv)
        _, mix, out = self.links[1]
        x = HyperStreams(streams, self.streams, ctx.dtype, self.mixer.forward(h, ctx, call), mix, out)
        if self.feed_forward is None:
            return x
        h, streams = self._head(x, 2, self.norm_ffn, ctx)
        _, mix, out = self.links[2]
        return HyperStreams(streams, self.streams, ctx.dtype, self.feed_forward.forward(h, ctx), mix, out)


register_part("block", "hyper", HyperBlock)
register_part("block", "sandwich", SandwichBlock)
register_part("block", "shifted_parallel", ShiftedParallelBlock)
register_part("block", "post_norm", PostNormBlock)
register_part("block", "parallel", ParallelBlock)
register_part("block", "sequential", SequentialBlock)
