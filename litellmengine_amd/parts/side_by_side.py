"""Two mixers side by side: both read the same input, and their results are added.

    y = left(h) + right(h)

Each of the two may bring its own constant factor (a mixer's `out_scale`): the sum then needs no
arithmetic of its own, the result is handed on as the pair (left, right), and the norm's kernel that
takes the mixer's result adds the two in 32-bit (`Norm.add_normed(hidden, y, extra)`).  Or the factors are
given here (`left_scale`, `right_scale`): the result is then a ScaledSum, and the factors are applied in 32-bit
by the norm's kernel that adds it into the stream (pre-norm arrangements).  At most one
of the two may keep a per-token cache; the fixed-size states of both lie one behind the other in
one state row of the request, and each mixer sees its own columns of it.

Where both mixers say which weight their input meets first (`input_weight`), the two are stacked and one product makes
both inputs; each mixer then gets the result with the column that its own begins at.

In a decode step of many requests (one that is captured into a graph) each mixer is a chain of launches that leave most of the chip
idle: the right mixer's chain then runs on a stream of its own, forked from and joined to the step's.  Whatever either
chain allocates is used by nobody else before the join, and the next fork comes after the launches that read their
results: the allocator's own order by stream is enough.
"""
from __future__ import annotations

import dataclasses
from typing import Dict, Optional

import torch

from ..weights.spec import TensorSpec
from .base import BuildContext, CacheSpec, Mixer, ScaledSum, StateSpec


_side_streams: Dict[int, "torch.cuda.Stream"] = {}


def _side_stream(device) -> "torch.cuda.Stream":
    """A stream beside the step's (one per device, default priority)."""
    index = device.index if device.index is not None else torch.cuda.current_device()
    if index not in _side_streams:
        _side_streams[index] = torch.cuda.Stream(device=device)
    return _side_streams[index]


class SideBySideMixer(Mixer):
    # decode steps of at least so many requests run the two chains on two streams (measured: 64 requests 7-10 % faster,
    # 8 requests 0-2 %, one request no faster: there the fork costs what it gains)
    ABREAST_MIN_REQUESTS = 16

    def __init__(self, left: Mixer, right: Mixer, left_scale: Optional[float] = None, right_scale: Optional[float] = None):
        if (left_scale is None) != (right_scale is None):
            raise ValueError("both mixers' factors are given, or neither")
        self.left, self.right = left, right
        self.scales = None if left_scale is None else (float(left_scale), float(right_scale))
        self.graph_safe = bool(getattr(left, "graph_safe", False) and getattr(right, "graph_safe", False))
        if left.cache_spec() is not None and right.cache_spec() is not None:
            raise ValueError("of two mixers side by side at most one keeps a per-token cache")
        self._columns = []  # per mixer: (first column, columns) of the shared state row, or None
        at = 0
        for m in (left, right):
            spec = m.state_spec()
            if spec is None:
                self._columns.append(None)
                continue
            if len(spec.shape) != 1 or spec.dtype != torch.float32:
                raise ValueError("mixers side by side keep their states as one float32 row each")
            self._columns.append((at, spec.shape[0]))
            at += spec.shape[0]
        self._state_width = at
        self.stacked: Optional[torch.Tensor] = None
        self.right_col = 0

    def cache_spec(self) -> Optional[CacheSpec]:
        return self.left.cache_spec() or self.right.cache_spec()

    def state_spec(self) -> Optional[StateSpec]:
        return StateSpec((self._state_width,), torch.float32) if self._state_width else None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {**self.left.tensor_specs(), **self.right.tensor_specs()}

    def bind(self, weights, ctx: BuildContext) -> None:
        self.ctx = ctx
        self.left.bind(weights, ctx)
        self.right.bind(weights, ctx)
        if all(hasattr(m, "input_weight") for m in (self.left, self.right)):
            a, b = self.left.input_weight(), self.right.input_weight()
            self.stacked = torch.cat([a, b], dim=0).contiguous()
            self.right_col = a.shape[0]
            self.left.take_input_weight(self.stacked[: self.right_col])  # (rows of the stack: nothing is held twice)
            self.right.take_input_weight(self.stacked[self.right_col:])

    def _share(self, cache, which: int):
        columns = self._columns[which]
        state = None if columns is None else cache.state[:, columns[0] : columns[0] + columns[1]]
        return dataclasses.replace(cache, state=state)

    def forward(self, x, step, cache):
        """-> (left's result, right's result): a pair that a norm's kernel adds up; with factors a ScaledSum."""
        shares = [{}, {}]
        if self.stacked is not None:
            u = self.ctx.ops.linear(x, self.stacked)
            shares = [{"projected": (u, 0)}, {"projected": (u, self.right_col)}]
        run = lambda which, mixer: mixer.forward(x, step, self._share(cache, which), **shares[which])
        if step.seqs is None and x.is_cuda and step.num_seqs >= self.ABREAST_MIN_REQUESTS:  # (no host-side view: a step for a graph)
            here, side = torch.cuda.current_stream(x.device), _side_stream(x.device)
            side.wait_stream(here)
            with torch.cuda.stream(side):
                right = run(1, self.right)
            left = run(0, self.left)
            here.wait_stream(side)
            y = left, right
        else:
            y = run(0, self.left), run(1, self.right)
        return y if self.scales is None else ScaledSum(*y, *self.scales)
