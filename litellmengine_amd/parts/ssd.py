"""The state-space mixer of Mamba-2: a recurrence with a matrix state per head and one decay per token and head.

    [z | x | B | C | d] = W_in h                          inner = heads * vdim, inner, groups * N, groups * N, heads wide
    (x, B, C)  <- silu(conv(x, B, C) + b)                 per channel over time, J taps, zeros before a request's start
    dt     = softplus(d + dt_bias)                        one per head
    S     <- exp(-exp(A_log) dt) S + dt B x^T             [N, vdim] per head; head h reads group h // (heads // groups)
    y      = S^T C + D x                                  (the read-out sees the token's own write)
    out    = W_o [norm(y * silu(z)) * w]                  the root mean square over each of `norm_groups` equal parts

The state is one float32 row per request slot (`StateSpec`): the heads' matrices (transposed, [head][value][state], the
way the kernels read them) and, behind them, the last J - 1 rows of the convolution's inputs.  The step sizes' rows of
W_in are a product of their own (in steps of single tokens part of the convolution's launch) whose result stays in 32-bit; what enters the recurrence beyond the projections and
the convolution is 32-bit in every mode.  Requests with few tokens in a step are walked token by token, longer portions
are cut into chunks that are worked on side by side, whatever the mix.
"""
from __future__ import annotations

from typing import Dict, Sequence

import torch

from ..csrc.limits import MAX_SSD_DIM
from ..weights.spec import INIT_NORM, INIT_NORMAL, INIT_WIDE, TensorSpec
from .base import BuildContext, Mixer, StateSpec
from .linear import Linear


class StateSpaceMixer(Mixer):
    graph_safe = True

    def __init__(self, prefix: str, hidden_size: int, heads: int, vdim: int, state: int, groups: int, taps: int,
                 norm_groups: int, norm_eps: float, conv_bias: bool = True,
                 names: Sequence[str] = ("in", "conv", "conv.b", "dt_bias", "A_log", "D", "norm", "o")):
        """`state`: N.  `taps`: the convolution's length J (with one tap the state keeps no rows).  `names`: the
        checkpoint's names after `prefix` of the input projection, the taps [channels, J] (the last column the current
        token's), the convolution's bias (not with `conv_bias=False`), the step sizes' offset, the decay's logarithm and
        the skip's factor (one each per head), the output norm's weight [inner] and the output projection."""
        if heads <= 0 or groups <= 0 or heads % groups:
            raise ValueError("the heads are a multiple of the groups")
        if not 0 < vdim <= MAX_SSD_DIM or not 0 < state <= MAX_SSD_DIM:
            raise ValueError(f"a head of the recurrence holds between 1 and {MAX_SSD_DIM} channels, not {vdim} and {state}")
        if taps < 1:
            raise ValueError("a convolution has at least one tap")
        if norm_groups <= 0 or (heads * vdim) % norm_groups:
            raise ValueError("the output norm's parts are equal")
        self.prefix, self.hidden = prefix, hidden_size
        self.H, self.vdim, self.N, self.G, self.taps = heads, vdim, state, groups, int(taps)
        self.norm_groups, self.eps = int(norm_groups), float(norm_eps)
        self.inner = heads * vdim
        self.conv_cols = self.inner + 2 * groups * state
        (self.in_name, self.conv_name, conv_b, self.dt_bias_name, self.a_log_name, self.d_name, self.norm_name,
         o) = (prefix + n for n in names)
        self.conv_bias_name = conv_b if conv_bias else None
        self.o = Linear([o], self.inner, [hidden_size])
        self.zxbc = self.dt_w = self.conv_w = self.conv_b = self.dt_bias = self.a_log = self.D = self.norm_w = None

    @property
    def matrix_floats(self) -> int:
        """Of a state row; a multiple of four, so that what lies behind starts at 16 bytes."""
        return -(-self.H * self.vdim * self.N // 4) * 4

    @property
    def kept_rows(self) -> int:
        return self.taps - 1

    def state_spec(self) -> StateSpec:
        return StateSpec((-(-(self.matrix_floats + self.kept_rows * self.conv_cols) // 4) * 4,), torch.float32)

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        specs = dict(self.o.tensor_specs())
        specs[self.in_name] = TensorSpec((self.inner + self.conv_cols + self.H, self.hidden), INIT_NORMAL)
        specs[self.conv_name] = TensorSpec((self.conv_cols, self.taps), INIT_WIDE)
        if self.conv_bias_name:
            specs[self.conv_bias_name] = TensorSpec((self.conv_cols,), INIT_NORMAL)
        for name in (self.dt_bias_name, self.a_log_name, self.d_name):
            specs[name] = TensorSpec((self.H,), INIT_NORMAL)
        specs[self.norm_name] = TensorSpec((self.inner,), INIT_NORM)
        return specs

    def bind(self, weights, ctx: BuildContext) -> None:
        self.ctx = ctx
        self.o.bind(weights, ctx)
        w = weights[self.in_name].to(ctx.dtype)
        cut = self.inner + self.conv_cols
        self.zxbc, self.dt_w = w[:cut].contiguous(), w[cut:].contiguous()
        flat = lambda name: weights[name].float().reshape(-1).contiguous()
        self.conv_w = weights[self.conv_name].float().contiguous()
        self.conv_b = flat(self.conv_bias_name) if self.conv_bias_name else None
        self.dt_bias, self.a_log, self.D, self.norm_w = (flat(n) for n in (self.dt_bias_name, self.a_log_name, self.d_name,
                                                                          self.norm_name))

    def input_weight(self):
        """The rows that a mixer beside this one may stack with its own (see SideBySideMixer)."""
        return self.zxbc

    def take_input_weight(self, weight) -> None:
        self.zxbc = weight

    def forward(self, x, step, cache, projected=None):
        """`projected` = (u, col): the input projection's result is the columns from `col` on of u."""
        ops = self.ctx.ops
        state = cache.state
        kept = state[:, self.matrix_floats:] if self.kept_rows else None  # (a view: the kernels take a row stride)
        u, col = projected if projected is not None else (ops.linear(x, self.zxbc), 0)
        c, dt = ops.ssd_conv(u, col + self.inner, self.conv_w, self.conv_b, kept, step.token_seq, step.cu_tokens, step.seq_slots,
                             single=step.max_q_len == 1, x=x, dt_w=self.dt_w)
        y = ops.ssd_scan(c, dt, self.dt_bias, self.a_log, self.D, state, self.H, self.G, self.vdim, self.N, step.seq_slots,
                         step.cu_tokens, step.min_q_len, step.max_q_len)
        return self.o.forward(ops.ssd_gate_norm(y, u, col, self.norm_w, self.eps, self.norm_groups))
