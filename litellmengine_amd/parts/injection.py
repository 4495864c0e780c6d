"""Vectors that enter the residual stream between two blocks.

A model that runs some of its blocks several times in a row (a loop over depth: the same weights, a cache of
its own for every pass) tells the passes apart by a vector per pass that is added to every row of the stream
right before the pass's first block.  A plan entry names the row it wants (`models.decoder.Inject`), the
model hands the sum on as a `parts.base.Injected`, and the norm that the block begins with adds it into the
32-bit stream in the same launch.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..weights.spec import INIT_NORMAL, TensorSpec
from .base import BuildContext, Part


class PassVectors(Part):
    def __init__(self, name: str, count: int, width: int):
        """`name`: the checkpoint's tensor [count, width]."""
        self.name, self.count, self.width = name, int(count), int(width)
        self.rows: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {self.name: TensorSpec((self.count, self.width), INIT_NORMAL)}

    def bind(self, weights, ctx: BuildContext) -> None:
        self.ctx = ctx
        self.rows = weights[self.name].float().contiguous()  # added in 32-bit

    def row(self, i: int) -> torch.Tensor:
        return self.rows[i]
