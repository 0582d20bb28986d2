"""The gated delta rule with a decay per key channel, as a mixer with a state of fixed size.

With x the mixer's input, H heads with values of ``value_dim`` and G <= H heads of queries and keys of ``key_dim``:

    q, k, v = silu(conv(W_q x)), silu(conv(W_k x)), silu(conv(W_v x))   short causal convolutions per channel, no bias
    q, k    <- head / sqrt(sum(head^2) + 1e-6);  q <- q * key_dim^(-1/2)
    beta    = sigmoid(W_b x)                                            one a head
    g       = exp(-exp(A_log) * softplus(W_a2 W_a1 x + dt_bias))        one a head and key channel
    S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q  per head, S: [key_dim, value_dim], zero at the start
    out = W_o (every head's o / sqrt(mean(o^2) + eps) * w  *  sigmoid(W_g2 W_g1 x))

head h reads q / k head h // (H / G).  The state and the convolutions' last inputs are a row of a state table of the cache,
32-bit, as is everything between the projections and the output gate.  q, k, v and b are one product of x; the two inner
vectors W_a1 x and W_g1 x are another (one launch with the first in small steps), and the two products of those run as
one, with the two matrices side by side on the diagonal.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple

import torch

from .. import ops
from ..engine.spec import INIT_NORMAL, INIT_ONE_NOISE, INIT_ZERO_NOISE, VECTOR, TensorSpec
from .base import Part, StepContext, register_part
from .linear import Linear

UNIT_EPS = 1e-6  # in the root of a query's and a key's length


class ChannelDeltaMixer(Part):
    def __init__(self, name: str, hidden_size: int, heads: int, kv_heads: int, key_dim: int, value_dim: int, taps: int,
                 decay_rank: int, gate_rank: int, eps: float):
        """``decay_rank``, ``gate_rank``: the sizes of W_a1 x and W_g1 x; ``taps``: the convolutions' inputs."""
        if heads % kv_heads:
            raise ValueError(f"{name}: heads ({heads}) must be a multiple of kv heads ({kv_heads})")
        self.name, self.hidden_size = name, int(hidden_size)
        self.heads, self.kv_heads, self.key_dim, self.value_dim = int(heads), int(kv_heads), int(key_dim), int(value_dim)
        self.taps, self.decay_rank, self.gate_rank, self.eps = int(taps), int(decay_rank), int(gate_rank), float(eps)
        self.q_cols, self.v_cols, self.a_cols = self.kv_heads * self.key_dim, self.heads * self.value_dim, self.heads * self.key_dim
        self.channels = 2 * self.q_cols + self.v_cols  # what the convolutions run over
        bare = lambda short, i, o: Linear(f"{name}.{short}", i, o, False, weight_name=f"{name}.{short}")
        self.q, self.k, self.v = bare("q", hidden_size, self.q_cols), bare("k", hidden_size, self.q_cols), bare("v", hidden_size, self.v_cols)
        self.b = bare("b", hidden_size, self.heads)
        self.a1, self.a2 = bare("a1", hidden_size, self.decay_rank), bare("a2", self.decay_rank, self.a_cols)
        self.g1, self.g2 = bare("g1", hidden_size, self.gate_rank), bare("g2", self.gate_rank, self.v_cols)
        self.out = bare("o", self.v_cols, hidden_size)
        self.inp: Optional[Linear] = None
        self.inner: Optional[Linear] = None
        self.outer: Optional[Linear] = None
        self.conv_w = self.a_log = self.dt_bias = self.norm_w = None

    @property
    def state_shape(self) -> Tuple[int, ...]:
        """The recurrence's state ``[heads, key_dim, value_dim]``, then the convolutions' last ``taps - 1`` inputs."""
        return (self.heads * self.key_dim * self.value_dim + (self.taps - 1) * self.channels,)

    def children(self) -> Sequence[Part]:
        return (self.q, self.k, self.v, self.b, self.a1, self.a2, self.g1, self.g2, self.out)

    def check_sizes(self) -> None:
        if not (1 <= self.taps <= 16):
            raise ValueError(f"{self.name}: a convolution of {self.taps} taps is outside the 1..16 that the kernel takes")
        if self.key_dim > 256:
            raise ValueError(f"{self.name}: keys of {self.key_dim} elements are more than the 256 the kernel holds")

    def tensor_specs(self) -> List[TensorSpec]:
        n = self.name
        return [TensorSpec(f"{n}.q.conv", (self.q_cols, self.taps), VECTOR, INIT_NORMAL),
                TensorSpec(f"{n}.k.conv", (self.q_cols, self.taps), VECTOR, INIT_NORMAL),
                TensorSpec(f"{n}.v.conv", (self.v_cols, self.taps), VECTOR, INIT_NORMAL),
                TensorSpec(f"{n}.A_log", (self.heads,), VECTOR, INIT_ZERO_NOISE),
                TensorSpec(f"{n}.dt_bias", (self.a_cols,), VECTOR, INIT_ZERO_NOISE),
                TensorSpec(f"{n}.norm", (self.value_dim,), VECTOR, INIT_ONE_NOISE)]

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        n = self.name
        # tap by tap, the channels of q, k and v side by side
        self.conv_w = torch.cat([tensors[f"{n}.{t}.conv"] for t in ("q", "k", "v")], dim=0).t().contiguous()
        self.a_log, self.dt_bias, self.norm_w = tensors[f"{n}.A_log"], tensors[f"{n}.dt_bias"], tensors[f"{n}.norm"]

    def after_load(self) -> None:
        self.inp = Linear.stacked(f"{self.name}.qkvb", [self.q, self.k, self.v, self.b], pad_to=8)
        self.inner = Linear.stacked(f"{self.name}.a1_g1", [self.a1, self.g1], pad_to=8)
        ra, rg, rows = self.decay_rank, self.gate_rank, self.a_cols + self.v_cols
        both = torch.zeros((rows + -rows % 8, self.inner.out_features), dtype=self.a2.weight.dtype, device=self.a2.weight.device)
        both[:self.a_cols, :ra].copy_(self.a2.weight)
        both[self.a_cols:rows, ra:ra + rg].copy_(self.g2.weight)
        self.outer = Linear(f"{self.name}.a2_g2", both.shape[1], both.shape[0], False)
        self.outer.weight, self.outer.bias, self.outer.joined = both, None, None
        self.a2.weight, self.g2.weight = both[:self.a_cols, :ra], both[self.a_cols:rows, ra:ra + rg]

    def forward(self, x: torch.Tensor, ctx: StepContext, call, residual: Optional[torch.Tensor] = None):
        row = ctx.cache.state_layer(call.cache_group, call.cache_layer)
        cut = self.heads * self.key_dim * self.value_dim
        sizes = (self.heads, self.kv_heads, self.key_dim, self.value_dim)
        both = Linear.pair(self.inp, x, {}, self.inner, x, {})
        proj, low = both if both is not None else (self.inp(x), self.inner(x))
        high = self.outer(low)
        qkv, g, beta = ops.delta_prep(proj[:, :self.channels], self.conv_w, high[:, :self.a_cols],
                                      proj[:, self.channels:self.channels + self.heads], self.a_log, self.dt_bias, row[:, cut:],
                                      ctx, *sizes, UNIT_EPS)
        o = ops.delta_scan(qkv, g, beta, row[:, :cut], ctx, *sizes)
        y = ops.head_norm_gate(o, high[:, self.a_cols:self.a_cols + self.v_cols], self.norm_w, self.eps, self.heads,
                               self.value_dim, x.dtype)
        return self.out(y, add1=residual)


register_part("mixer", "channel_delta", ChannelDeltaMixer)
