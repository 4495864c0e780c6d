"""Gated linear attention: a recurrence with a matrix state per head whose rows decay each at a rate made
from the data.

    q, k, v = W_q h * dim^(-1/2), W_k h, W_v h                  [heads, dim], [heads, dim], [heads, vdim]
    decay   = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau)              per head and key channel, in (0, 1)
    S      <- diag(decay_t) S + k_t v_t^T                       [dim, vdim], zeros before a request's first token
    o_t     = S^T q_t                                           (the read-out sees the token's own write)
    y_t     = W_o (o_t / rms(o_t) per head * norm * silu(W_g h))

The state is one float32 row per request slot (`StateSpec`).  The decay's inner projection leaves 32-bit
results, and everything behind it (the second projection, logarithm, exponential), the state, the read-out
and its norm are 32-bit in every mode.  A step's tokens of one request are walked in order by one kernel
(long portions in pieces side by side), whatever the mix of portions and single tokens.
"""
from __future__ import annotations

from typing import Dict, Optional, Sequence

import torch

from ..csrc.limits import MAX_GLA_HEAD_DIM
from ..weights.spec import INIT_NORM, INIT_NORMAL, TensorSpec
from .base import BuildContext, Mixer, StateSpec
from .linear import Linear


class GatedLinearAttention(Mixer):
    graph_safe = True

    def __init__(self, prefix: str, hidden_size: int, heads: int, dim: int, vdim: int, decay_rank: int, tau: float,
                 norm_eps: float, q_scale: Optional[float] = None, out_scale: float = 1.0,
                 names: Sequence[str] = ("q", "k", "v", "g", "a1", "a2", "a2.b", "norm", "o")):
        """`q_scale`: the factor on the queries (default dim^(-1/2)).  `out_scale`: the result is multiplied by it;
        it is folded into the 32-bit output norm's weight, so it costs no operation and no rounding of its own.
        `names`: the checkpoint's names after `prefix` of the four input projections, the decay's two projections and
        its offset, the output norm's weight [vdim] (one for all heads) and the output projection."""
        for n, what in ((dim, "key"), (vdim, "value")):
            if not 0 < n <= MAX_GLA_HEAD_DIM:
                raise ValueError(f"a head of the recurrence holds between 1 and {MAX_GLA_HEAD_DIM} {what} channels, not {n}")
        if heads <= 0 or decay_rank <= 0 or not tau > 0:
            raise ValueError("heads, the decay's inner rank and tau must be positive")
        self.prefix, self.hidden, self.H, self.dim, self.vdim, self.rank = prefix, hidden_size, heads, dim, vdim, int(decay_rank)
        self.tau, self.eps, self.out_scale = float(tau), float(norm_eps), float(out_scale)
        self.q_scale = float(dim) ** -0.5 if q_scale is None else float(q_scale)
        q, k, v, g, a1, a2, a2_b, norm, o = (prefix + n for n in names)
        self.qkvg = Linear([q, k, v, g], hidden_size, [heads * dim, heads * dim, heads * vdim, heads * vdim])
        self.a1 = Linear([a1], hidden_size, [self.rank])
        self.a2_name, self.a2_bias_name, self.norm_name = a2, a2_b, norm
        self.o = Linear([o], heads * vdim, [hidden_size])
        self.a2 = self.a2_bias = self.norm_w = None

    def state_spec(self) -> StateSpec:
        return StateSpec((self.H * self.dim * self.vdim,), torch.float32)

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        specs: Dict[str, TensorSpec] = {}
        for p in (self.qkvg, self.a1, self.o):
            specs.update(p.tensor_specs())
        specs[self.a2_name] = TensorSpec((self.H * self.dim, self.rank), INIT_NORMAL)
        specs[self.a2_bias_name] = TensorSpec((self.H * self.dim,), INIT_NORMAL)
        specs[self.norm_name] = TensorSpec((self.vdim,), INIT_NORM)
        return specs

    def bind(self, weights, ctx: BuildContext) -> None:
        self.ctx = ctx
        for p in (self.qkvg, self.a1, self.o):
            p.bind(weights, ctx)
        self.a2 = weights[self.a2_name].float().t().contiguous()  # [rank, heads * dim]: neighbouring channels side by side
        self.a2_bias = weights[self.a2_bias_name].float().reshape(-1).contiguous()
        self.norm_w = (weights[self.norm_name].float() * self.out_scale).contiguous()

    def forward(self, x, step, cache):
        ops = self.ctx.ops
        u = self.qkvg.forward(x)
        low = self.a1.forward(x, out_dtype=torch.float32)
        decay = ops.gla_decay(low, self.a2, self.a2_bias, self.tau)
        y = ops.gla_scan(u, decay, self.q_scale, self.norm_w, self.eps, cache.state, self.H, self.dim, self.vdim,
                         step.seq_slots, step.cu_tokens, step.max_q_len)
        return self.o.forward(y)
