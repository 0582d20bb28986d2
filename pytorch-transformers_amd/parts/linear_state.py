"""Linear attention whose state decays, as a mixer with a state of fixed size.

With h the mixer's input and H heads of ``key_dim`` (queries, keys) and ``value_dim`` (values) elements:

    q = W_q h, k = W_k h, v = W_v h                        (no biases)
    q <- rotate(q) * q_scale, k <- rotate(k) * k_scale     by position (``positions``: any rotation, or none)
    S_t = diag(a_t) S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t  per head, S: [key_dim, value_dim], zero at the start
    out = W_o (every head's o / sqrt(mean(o^2) + eps) * w  *  silu(W_g h))

The decay a is a constant per head (``decay``), or one number per head and key channel from the token (``tau`` and
``decay_rank``): ``sigmoid(W_a2 (W_a1 h) + b)^(1 / tau)`` with the inner vector of ``decay_rank`` numbers.  w is a learned weight
``[value_dim]`` for all heads, ``name.norm``, or absent (``gain=False``).

The products of h run as one; the state is a row of a state table of the cache.  Everything between the products and the
gated heads is 32-bit and one launch in decode steps (``ops.linear_state``).
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple

import torch

from .. import ops
from ..engine.spec import INIT_ONE_NOISE, VECTOR, TensorSpec
from .base import Part, StepContext, register_part
from .linear import Linear
from .positions import as_rotation


class LinearStateMixer(Part):
    def __init__(self, name: str, hidden_size: int, heads: int, key_dim: int, value_dim: int, eps: float, positions: Part,
                 q_scale: float = 1.0, k_scale: float = 1.0, decay: Optional[Sequence[float]] = None, tau: float = 0.0,
                 decay_rank: int = 0, gain: bool = True):
        if (decay is None) != (tau > 0 and decay_rank > 0):
            raise ValueError(f"{name}: a decay is a list of constants, or comes from the token (tau and decay_rank above 0)")
        if decay is not None and len(decay) != heads:
            raise ValueError(f"{name}: {len(decay)} decays for {heads} heads")
        self.name, self.hidden_size = name, int(hidden_size)
        self.heads, self.key_dim, self.value_dim = int(heads), int(key_dim), int(value_dim)
        self.eps, self.positions, self.q_scale, self.k_scale, self.gain = float(eps), positions, float(q_scale), float(k_scale), bool(gain)
        self.decay = None if decay is None else torch.tensor([float(d) for d in decay], dtype=torch.float32)
        self.tau, self.decay_rank = float(tau), int(decay_rank)
        bare = lambda short, i, o, b=False: Linear(f"{name}.{short}", i, o, b, weight_name=f"{name}.{short}", bias_name=f"{name}.{short}.b")
        self.q = bare("q", hidden_size, self.heads * self.key_dim)
        self.k = bare("k", hidden_size, self.heads * self.key_dim)
        self.v = bare("v", hidden_size, self.heads * self.value_dim)
        self.g = bare("g", hidden_size, self.heads * self.value_dim)
        self.a1 = bare("a1", hidden_size, self.decay_rank) if decay is None else None
        self.a2 = bare("a2", self.decay_rank, self.heads * self.key_dim, True) if decay is None else None
        self.out = bare("o", self.heads * self.value_dim, hidden_size)
        self.norm_w: Optional[torch.Tensor] = None
        self.inp: Optional[Linear] = None

    @property
    def state_shape(self) -> Tuple[int, ...]:
        return (self.heads * self.key_dim * self.value_dim,)

    def children(self) -> Sequence[Part]:
        return tuple(p for p in (self.q, self.k, self.v, self.g, self.a1, self.a2, self.out, self.positions) if p is not None)

    def to(self, device) -> None:
        if self.decay is not None:
            self.decay = self.decay.to(device)

    def tensor_specs(self) -> List[TensorSpec]:
        return [TensorSpec(f"{self.name}.norm", (self.value_dim,), VECTOR, INIT_ONE_NOISE)] if self.gain else []

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        if self.gain:
            self.norm_w = tensors[f"{self.name}.norm"]

    def check_sizes(self) -> None:
        problem = None
        if max(self.key_dim, self.value_dim) > 256:
            problem = f"keys of {self.key_dim} and values of {self.value_dim} elements are more than the 256 the kernels hold"
        rot = as_rotation(self.positions.rotation())
        if problem is None and rot is not None:
            problem = ops.rotation_problem(self.key_dim, rot.rotary_dim, rot.pairing)
        if problem is not None:
            raise ValueError(f"{self.name}: {problem}")

    def input_parts(self) -> List[Linear]:
        return [p for p in (self.q, self.k, self.v, self.g, self.a1) if p is not None]

    def after_load(self) -> None:
        self.inp = Linear.stacked(f"{self.name}.qkvg", self.input_parts(), pad_to=8)

    @property
    def result_columns(self) -> int:
        return self.heads * self.value_dim

    def result_into(self, proj: torch.Tensor, out: Optional[torch.Tensor], mult: float, ctx: StepContext, call) -> torch.Tensor:
        """The normed and gated heads side by side, times ``mult``, into ``out`` (None: a new matrix)."""
        state = ctx.cache.state_layer(call.cache_group, call.cache_layer)
        H, dk, dv = self.heads, self.key_dim, self.value_dim
        a, b, c, d = H * dk, 2 * H * dk, 2 * H * dk + H * dv, 2 * (H * dk + H * dv)
        channel = None
        if self.decay is None:
            channel = (proj[:, d:d + self.decay_rank], self.a2.weight, self.a2.bias, self.tau)
        return ops.linear_state(proj[:, :a], proj[:, a:b], proj[:, b:c], proj[:, c:d], state, ctx, H, dk, dv,
                                rotation=as_rotation(self.positions.rotation()), q_scale=self.q_scale, k_scale=self.k_scale, decay=self.decay,
                                channel_decay=channel, w=self.norm_w, eps=self.eps, mult=mult, out=out)

    def forward(self, x: torch.Tensor, ctx: StepContext, call, residual: Optional[torch.Tensor] = None):
        return self.out(self.result_into(self.inp(x), None, 1.0, ctx, call), add1=residual)


register_part("mixer", "linear_state", LinearStateMixer)
