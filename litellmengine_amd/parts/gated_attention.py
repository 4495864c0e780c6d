"""Grouped-query attention whose result may be gated element by element, with what a design may want of the
rest given as parameters:

    q, k, v = W_q h (+ b_q), W_k h (+ b_k), W_v h (+ b_v)
    q, k  <- rotated by their own positions (neighbouring pairs, the first elements of every head)
    v     <- rotated by its own position over all of its elements, and every head's result turned back by
             the query's position (`value_rotation`): the result depends on distances in the values too
    s_ij   = (q_i . k_j) * scale - slope_h (i - j)                               (`slopes`: a number per head)
    s_ij  <- cap tanh(s_ij / cap)                                                (`softcap`)
    keys   : `window`: i sees j <= i with i - j < window, or j < keep_first;  `chunk`: i sees j <= i of its
             own chunk of so many positions, counted from the request's first;  neither: every j <= i
    p_ij   = exp(s_ij) / (exp(sink_h) + sum_j exp(s_ij))                         (`sinks`: a learned number per head)
    p_h   <- sum_g T[h, g] p_g                                                   (`talk`: the heads' weights mixed, T [H, H])
    y      = W_o (out_scale * sigmoid(W_g h) * [heads' sum_j p_ij v_j])         (`gated=False`: W_o [heads' sum_j p_ij v_j])

Keys may be `dim` wide and values `vdim`: the cache's heads hold `cache_dim` >= both elements (a multiple of
32, which the matrix-core kernels take), the rest zeros; the gates' kernel drops the padding (without gates the
output projection has zero columns there).  The
projections are one stacked product; rotations, scores, softmax, sinks, mixing and gates are 32-bit.
"""
from __future__ import annotations

from typing import Dict, Optional, Sequence

import torch

from ..csrc.limits import check_head_dim, check_talking_sizes
from ..weights.spec import INIT_NORMAL, INIT_WIDE, TensorSpec
from .base import BuildContext, CacheSpec, KVCacheSpec, Mixer
from .linear import Linear
from .position import RotaryInterleaved


def geometric_slopes(heads: int) -> Sequence[float]:
    """2^(-8 (h + 1) / heads) for h = 0 .. heads - 1."""
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


class GatedAttention(Mixer):
    graph_safe = True

    def __init__(self, prefix: str, hidden_size: int, num_q_heads: int, num_kv_heads: int, dim: int, vdim: int, scale: float,
                 rotation: Optional[RotaryInterleaved] = None, value_rotation: Optional[RotaryInterleaved] = None,
                 window: Optional[int] = None, keep_first: int = 0, chunk: Optional[int] = None, qkv_bias: bool = False,
                 sinks: bool = False, slopes: Optional[Sequence[float]] = None, talk: bool = False, out_scale: float = 1.0,
                 names: Sequence[str] = ("q", "k", "v", "g", "o"), bias_suffix: str = ".b", sink_name: str = "sink",
                 talk_name: str = "talk", gated: bool = True, softcap: Optional[float] = None):
        """`names`: the checkpoint's names after `prefix` of the query, key, value, gate (not with `gated=False`) and
        output projections."""
        if not gated and (value_rotation is not None or out_scale != 1.0):
            raise ValueError("turned-back values and a factor on the result are the gates' kernel's work")
        if softcap is not None and not softcap > 0:
            raise ValueError("a cap on the scores must be positive")
        if num_q_heads <= 0 or num_kv_heads <= 0 or num_q_heads % num_kv_heads:
            raise ValueError("num_q_heads must be a multiple of num_kv_heads")
        self.cache_dim = -(-max(dim, vdim) // 32) * 32
        check_head_dim(self.cache_dim)
        if rotation is not None and rotation.rotary_dim > dim:
            raise ValueError("the rotation covers more elements than a key has")
        if value_rotation is not None and value_rotation.rotary_dim != vdim:
            raise ValueError("the values' rotation covers all of a value's elements")
        if window is not None and chunk is not None:
            raise ValueError("an attention has a window or chunks, not both")
        if keep_first and window is None:
            raise ValueError("first tokens are kept beside a window only")
        # chunks and distance biases are known to the kernels that mix the heads' weights (without a mix: by the identity)
        self.talking = bool(talk or slopes is not None or chunk is not None)
        if self.talking and (sinks or window is not None or softcap is not None):
            raise ValueError("the kernels that mix the heads' weights know chunks and distance biases, no windows, sinks or caps")
        if self.talking:
            check_talking_sizes(num_q_heads, self.cache_dim)
        self.prefix, self.hidden = prefix, hidden_size
        self.nq, self.nkv, self.dim, self.vdim = num_q_heads, num_kv_heads, dim, vdim
        self.scale, self.out_scale = float(scale), float(out_scale)
        self.rotation, self.value_rotation = rotation, value_rotation
        self.window, self.keep_first, self.chunk = window, int(keep_first), chunk
        self.gated, self.softcap = bool(gated), None if softcap is None else float(softcap)
        q, k, v, g, o = (prefix + n for n in (names if gated or len(names) == 5 else (*names[:3], "", names[3])))
        widths = [num_q_heads * dim, num_kv_heads * dim, num_kv_heads * vdim]
        self.gate_col = sum(widths)
        # one product for q, k, v and the gates' inputs (the gates have no bias)
        self.qkvg = Linear([q, k, v] + ([g] if gated else []), hidden_size, widths + ([num_q_heads * vdim] if gated else []))
        self.o = Linear([o], num_q_heads * vdim, [hidden_size])
        self.bias_names = [n + bias_suffix for n in (q, k, v)] if qkv_bias else []
        self.bias_widths = widths
        self.sink_name = prefix + sink_name if sinks else None
        self.slope_values = None if slopes is None else [float(s) for s in slopes]
        self.talk_name = prefix + talk_name if talk else None
        self.bias = self.sinks = self.slopes = self.talk = None

    def cache_spec(self) -> CacheSpec:
        return KVCacheSpec(self.nkv, self.cache_dim, self.window, chunk=self.chunk, keep_first=self.keep_first)

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        specs = {**self.qkvg.tensor_specs(), **self.o.tensor_specs()}
        for name, rows in zip(self.bias_names, self.bias_widths):
            specs[name] = TensorSpec((rows,), INIT_NORMAL)
        if self.sink_name:
            specs[self.sink_name] = TensorSpec((self.nq,), INIT_NORMAL)
        if self.talk_name:
            specs[self.talk_name] = TensorSpec((self.nq, self.nq), INIT_WIDE)
        return specs

    def bind(self, weights, ctx: BuildContext) -> None:
        self.ctx = ctx
        self.qkvg.bind(weights, ctx)
        if self.gated or self.cache_dim == self.vdim:
            self.o.bind(weights, ctx)
        else:  # without gates nothing drops the cache's padding: the output projection gets zero columns there
            o = weights[self.o.names[0]].to(ctx.dtype).view(self.hidden, self.nq, self.vdim)
            o = torch.nn.functional.pad(o, (0, self.cache_dim - self.vdim))
            self.o.bind_tensor(o.reshape(self.hidden, self.nq * self.cache_dim).contiguous(), ctx)
        for p in (self.rotation, self.value_rotation):
            if p is not None:
                p.bind(weights, ctx)
        if self.bias_names:
            self.bias = torch.cat([weights[n].to(ctx.dtype).reshape(-1) for n in self.bias_names]).contiguous()
        if self.sink_name:
            self.sinks = weights[self.sink_name].float().reshape(-1).contiguous()
        if self.slope_values is not None:
            self.slopes = torch.tensor(self.slope_values, dtype=torch.float32, device=ctx.device)
        if self.talk_name:
            self.talk = weights[self.talk_name].float().contiguous()
        elif self.talking:
            self.talk = torch.eye(self.nq, dtype=torch.float32, device=ctx.device)

    def input_weight(self):
        """The rows that a mixer beside this one may stack with its own (see SideBySideMixer); the kernels want them first."""
        return self.qkvg.weight

    def take_input_weight(self, weight) -> None:
        self.qkvg.weight = weight

    def forward(self, x, step, cache, projected=None):
        """`projected` = (u, 0): the input projection's result is the first columns of u."""
        ops = self.ctx.ops
        group = cache.group
        u = self.qkvg.forward(x) if projected is None else projected[0]
        turn = None if self.rotation is None else self.rotation.table(step)
        value_turn = None if self.value_rotation is None else self.value_rotation.table(step)
        q = ops.pair_rope_write(u, self.bias, group.slot_mapping, turn, value_turn, cache.kv, self.nq, self.nkv, self.dim,
                                self.vdim, cache.writes)
        where = (cache.kv, group.block_table, step.seq_slots, step.cu_tokens, step.kv_lens, step.token_seq)
        if self.talking:
            a = ops.talking_attention(q, *where, self.chunk, self.scale, self.slopes, self.talk, step.min_q_len,
                                      step.max_q_len, step.max_kv_len)
        else:
            a = ops.paged_attention(q, *where, self.window, self.scale, step.min_q_len, step.max_q_len, step.max_kv_len,
                                    sinks=self.sinks, keep_first=self.keep_first, softcap=self.softcap)
        if not self.gated:  # heads of cache_dim elements, zeros past vdim, against zero columns of the weight
            return self.o.forward(a)
        return self.o.forward(ops.turn_back_gate(a, u, self.gate_col, self.nq, self.vdim, value_turn, self.out_scale))
