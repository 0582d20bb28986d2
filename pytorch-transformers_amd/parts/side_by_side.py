"""Two mixers side by side that read the same input: ``left_scale * left(h) + right_scale * right(h)``.

The products of h of both halves run as one.  Each half leaves what its own last product would read, times its scale (in
32-bit, before the one rounding), in its columns of one matrix, and the two last products are one product of that matrix:
``[left_scale * l | right_scale * r] . [W_left | W_right]^T``, so that the sum of the halves is formed in its accumulators.

The left half's storage is the run order's entry's own, the right half's is its further storage ``"right"``.  A half is a mixer
that offers ``input_parts``, ``result_columns``, ``result_into`` and ``out`` (see ``parts.base``).
"""
from __future__ import annotations

from typing import Optional, Sequence

import torch

from .base import Part, StepContext, register_part
from .linear import Linear


class SideBySideMixer(Part):
    def __init__(self, name: str, left: Part, right: Part, left_scale: float = 1.0, right_scale: float = 1.0):
        for half in (left, right):
            if not all(hasattr(half, a) for a in ("input_parts", "result_columns", "result_into", "out")):
                raise ValueError(f"{name}: a {type(half).__name__} cannot be one half of a mixer")
        self.name, self.left, self.right = name, left, right
        self.left_scale, self.right_scale = float(left_scale), float(right_scale)
        self.inp: Optional[Linear] = None
        self.out: Optional[Linear] = None

    def children(self) -> Sequence[Part]:
        return (self.left, self.right)

    def after_load(self) -> None:
        self.inp = Linear.stacked(f"{self.name}.in", self.left.input_parts() + self.right.input_parts(), pad_to=8)
        self.left_in = sum(p.out_features for p in self.left.input_parts())
        self.right_in = sum(p.out_features for p in self.right.input_parts())
        a, b = self.left.out.weight, self.right.out.weight
        # the halves' columns start at multiples of eight, as does what follows them
        self.right_at = -(-a.shape[1] // 8) * 8
        self.columns = -(-(self.right_at + b.shape[1]) // 8) * 8
        self.gaps = self.columns != a.shape[1] + b.shape[1]
        both = torch.zeros((a.shape[0], self.columns), dtype=a.dtype, device=a.device)
        both[:, :a.shape[1]].copy_(a)
        both[:, self.right_at:self.right_at + b.shape[1]].copy_(b)
        self.out = Linear(f"{self.name}.o", self.columns, a.shape[0], False)
        self.out.weight, self.out.bias, self.out.joined = both, None, None
        self.left.out.weight, self.right.out.weight = both[:, :a.shape[1]], both[:, self.right_at:self.right_at + b.shape[1]]

    def forward(self, x: torch.Tensor, ctx: StepContext, call, residual: Optional[torch.Tensor] = None):
        proj = self.inp(x)
        both = (torch.zeros if self.gaps else torch.empty)((x.shape[0], self.columns), dtype=x.dtype, device=x.device)
        self.left.result_into(proj[:, :self.left_in], both[:, :self.left.result_columns], self.left_scale, ctx, call)
        self.right.result_into(proj[:, self.left_in:self.left_in + self.right_in],
                               both[:, self.right_at:self.right_at + self.right.result_columns], self.right_scale, ctx, call.on("right"))
        return self.out(both, add1=residual)


register_part("mixer", "side_by_side", SideBySideMixer)
