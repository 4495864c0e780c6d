"""Token embedding: h[t, :] = E[ids[t], :] (src/layers/embedding.cu:75-87); the
rows leave as float32, the type of the residual stream.  A design may add a learned vector of every
token's position and norm the sum before it becomes the stream's first row."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..weights.spec import INIT_NORMAL, TensorSpec
from .base import BuildContext, EmbeddedRows, Normed, Part
from .norm import RMSNorm


class Embedding(Part):
    def __init__(self, name: str, vocab_size: int, hidden_size: int, scale: float = 1.0, positions_name: Optional[str] = None,
                 max_positions: Optional[int] = None, norm: Optional[RMSNorm] = None):
        """`scale`: every row is multiplied by it on its way into the 32-bit residual stream.  `positions_name`: a
        table [max_positions, hidden_size] whose row p is added (not scaled) to a token at position p; a request may then
        be no longer than max_positions.  `norm`: the sum passes it and the result is the stream's first row."""
        if (positions_name is None) != (max_positions is None):
            raise ValueError("a position table and its length come together")
        self.positions_name, self.max_positions, self.norm = positions_name, max_positions, norm
        self.pos: Optional[torch.Tensor] = None
        self.scale = float(scale)
        self.name = name
        self.vocab_size = vocab_size
        self.hidden_size = hidden_size
        self.weight: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        specs = {self.name: TensorSpec((self.vocab_size, self.hidden_size), INIT_NORMAL)}
        if self.positions_name is not None:
            specs[self.positions_name] = TensorSpec((self.max_positions, self.hidden_size), INIT_NORMAL)
        if self.norm is not None:
            specs.update(self.norm.tensor_specs())
        return specs

    def bind(self, weights, ctx: BuildContext) -> None:
        self.ctx = ctx
        self.weight = weights[self.name].to(ctx.dtype).contiguous()
        if self.positions_name is not None:
            self.pos = weights[self.positions_name].to(ctx.dtype).contiguous()
        if self.norm is not None:
            self.norm.bind(weights, ctx)

    def again(self, step) -> EmbeddedRows:
        """The rows that forward(step.token_ids, step) gives, for whoever adds them once more later in the step."""
        if self.pos is not None or self.norm is not None:
            raise ValueError("rows that are made of more than the embedding table are not made twice")
        deferred = step.token_feedback is not None
        return EmbeddedRows(step.token_ids, self.weight, self.scale, step.token_feedback,
                            step.token_seq if deferred else None, step.seq_slots if deferred else None)

    def forward(self, ids: torch.Tensor, step=None, norm=None):
        """`step` (engine.batch.StepState): where it carries `token_feedback`, ids below zero are
        the tokens that the step before left on the device for their requests.  With `norm` (the
        parts.base.Norm that the first block begins with) the result is (rows, Normed or None):
        the norm's result comes along where one kernel makes both."""
        if self.pos is not None or self.norm is not None:
            feedback = step.token_feedback if step is not None else None
            then = norm if isinstance(norm, RMSNorm) else None  # (norms that this kernel knows)
            own = self.norm
            rows, normed = self.ctx.ops.embedding_norm(
                ids, self.weight, self.scale, step.positions if self.pos is not None else None, self.pos,
                own.weight if own is not None else None, own.eps if own is not None else 0.0,
                then.weight if then is not None else None, then.eps if then is not None else 0.0, self.ctx.dtype,
                feedback, step.token_seq if feedback is not None else None, step.seq_slots if feedback is not None else None)
            return (rows, None if normed is None else Normed(normed)) if norm is not None else rows
        if self.scale != 1.0:
            feedback = step.token_feedback if step is not None else None
            rows = self.ctx.ops.embedding(ids, self.weight, feedback, step.token_seq if feedback is not None else None,
                                          step.seq_slots if feedback is not None else None, scale=self.scale)
            return (rows, None) if norm is not None else rows
        if norm is not None:
            both = norm.of_embedding(ids, self.weight, step)
            if both is not None:
                return both[0], Normed(both[1])
            return self.forward(ids, step), None
        if step is not None and step.token_feedback is not None:
            return self.ctx.ops.embedding(ids, self.weight, step.token_feedback, step.token_seq, step.seq_slots)
        return self.ctx.ops.embedding(ids, self.weight)
