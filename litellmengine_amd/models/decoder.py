"""A decoder language model as data: an embedding, a set of blocks, the list
that says in which order they run (and with which cache), a final norm and an
output head.

The reference hard-wires embed -> layer 0..L-1 -> norm -> lm_head on all rows
(src/model/qwen3.cpp:1242-1278, :1501).  Here the order is a list of
`PlanEntry`: an entry may name a block that another entry names too (the
block's weights are then shared and it runs twice), and an entry may read the
cache that another entry writes instead of owning one.  The head runs on the
wanted rows only.
"""
from __future__ import annotations

import dataclasses
from typing import Dict, List, Optional, Sequence

import torch

from ..parts.base import Block, BuildContext, Carried, Injected, Norm, Normed, Prenormed
from ..parts.embedding import Embedding
from ..parts.injection import PassVectors
from ..parts.linear import Linear
from ..weights.spec import TensorSpec


@dataclasses.dataclass(frozen=True)
class Inject:
    """What is added to the residual stream right before a plan entry's block: row `vector` of the model's
    pass vectors (None: none), and with `embedding` the embedding's rows once more."""

    vector: Optional[int] = None
    embedding: bool = False


@dataclasses.dataclass(frozen=True)
class PlanEntry:
    """One call of a block.  `cache` names the cache layer the mixer works on
    (default: one of its own, numbered like the entry); `writes=False` makes the
    entry a reader of a cache that an earlier entry fills; `inject` adds something to
    the stream ahead of the block."""

    block: int
    cache: Optional[int] = None
    writes: bool = True
    inject: Optional[Inject] = None


def looped_plan(blocks: int, start: int, stop: int, times: int, inject: bool = True) -> List[PlanEntry]:
    """Blocks start .. stop - 1 run `times` times in a row (each time with caches and states of their own), the
    others once.  Ahead of pass t the stream gets pass vector t, and from the second pass on also the embedding's rows
    (`inject=False`: nothing enters the stream between passes)."""
    if not 0 <= start < stop <= blocks or times < 1:
        raise ValueError(f"a loop over blocks {start} .. {stop - 1}, {times} times, does not fit {blocks} blocks")
    plan = [PlanEntry(i) for i in range(start)]
    for t in range(times):
        plan += [PlanEntry(i, inject=Inject(t, t > 0) if inject and i == start else None) for i in range(start, stop)]
    return plan + [PlanEntry(i) for i in range(stop, blocks)]


class DecoderLM:
    def __init__(
        self,
        config,
        embedding: Embedding,
        blocks: Sequence[Block],
        plan: Sequence[PlanEntry],
        final_norm: Norm,
        head: Linear,
        tied_head: bool,
        logit_scale: float = 1.0,
        logit_softcap: Optional[float] = None,
        pass_vectors: Optional[PassVectors] = None,
    ):
        """`logit_scale`: the head's result is multiplied by it (in 32-bit).  `logit_softcap`: the
        logits then pass through cap * tanh(logits / cap) (in 32-bit; None: not).
        `pass_vectors`: the vectors that plan entries' `inject` names."""
        self.pass_vectors = pass_vectors
        self.logit_scale = float(logit_scale)
        self.logit_softcap = float(logit_softcap) if logit_softcap else None
        self.config = config
        self.embedding = embedding
        self.blocks = list(blocks)
        self.plan = [
            dataclasses.replace(e, cache=i if e.cache is None else e.cache) for i, e in enumerate(plan)
        ]
        self.final_norm = final_norm
        self.head = head
        self.tied_head = tied_head
        writers = {e.cache for e in self.plan if e.writes}
        for e in self.plan:
            if not 0 <= e.block < len(self.blocks):
                raise ValueError(f"plan names block {e.block}, the model has {len(self.blocks)}")
            if not e.writes and e.cache not in writers:
                raise ValueError(f"plan entry reads cache {e.cache} that no entry writes")
            if e.inject is not None and e.inject.vector is not None:
                if pass_vectors is None or not 0 <= e.inject.vector < pass_vectors.count:
                    raise ValueError(f"plan entry adds pass vector {e.inject.vector}, which the model does not have")

    # -- structure ---------------------------------------------------------
    @property
    def vocab_size(self) -> int:
        return self.embedding.vocab_size

    @property
    def max_positions(self) -> Optional[int]:
        """Most tokens of one request, where the model has a bound of its own (a table of position vectors)."""
        return getattr(self.embedding, "max_positions", None)

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        specs: Dict[str, TensorSpec] = dict(self.embedding.tensor_specs())
        for b in self.blocks:
            specs.update(b.tensor_specs())
        if self.pass_vectors is not None:
            specs.update(self.pass_vectors.tensor_specs())
        specs.update(self.final_norm.tensor_specs())
        specs.update(self.head.tensor_specs())
        return specs

    def cache_layers(self):
        """cache id -> the mixer that defines its needs (the writer)."""
        out = {}
        for e in self.plan:
            if e.writes:
                mixer = self.blocks[e.block].mixer
                if e.cache in out and out[e.cache] is not mixer:
                    raise ValueError(f"two different mixers write cache {e.cache}")
                out[e.cache] = mixer
        return out

    # -- weights -------------------------------------------------------------
    def bind(self, weights: Dict[str, torch.Tensor], ctx: BuildContext) -> None:
        self.ctx = ctx
        self.embedding.bind(weights, ctx)
        for b in self.blocks:
            b.bind(weights, ctx)
        if self.pass_vectors is not None:
            self.pass_vectors.bind(weights, ctx)
        self.final_norm.bind(weights, ctx)
        head_name = self.head.names[0]
        if head_name in weights:
            self.head.bind(weights, ctx)
        elif self.tied_head:
            self.head.bind_tensor(self.embedding.weight, ctx)
        else:
            raise KeyError(head_name)

    # -- one step --------------------------------------------------------------
    def _injected(self, inject: Inject, delta, step) -> Injected:
        """What the block before has left to be added and what enters the stream ahead of the next block."""
        if isinstance(delta, Carried):  # the block before has added everything into the stream itself
            delta = None
        return Injected(delta, None if inject.vector is None else self.pass_vectors.row(inject.vector),
                        self.embedding.again(step) if inject.embedding else None, self.ctx.ops)

    def forward(self, step, caches) -> torch.Tensor:
        """Run the tokens of `step` (engine.batch.StepState) through the plan and
        return float32 logits [len(step.logit_rows), vocab]."""
        step.scratch.clear()  # per-step tables are made anew in every run (also when a graph is captured)
        first_norm = None
        if self.plan and self.plan[0].inject is None:  # (nothing enters the stream between the embedding and the norm)
            first_norm = self.blocks[self.plan[0].block].input_norm()
        if first_norm is not None:
            hidden, delta = self.embedding.forward(step.token_ids, step, norm=first_norm)
        else:
            hidden, delta = self.embedding.forward(step.token_ids, step), None
        last = len(self.plan) - 1
        for i, e in enumerate(self.plan):
            # the norm that the next block starts with, if the products around it may do its work
            if i < last and self.plan[i + 1].inject is not None:
                next_norm = None  # something enters the stream first
            elif i < last:
                follower = self.blocks[self.plan[i + 1].block]
                next_norm = follower.entry_norm()
                if next_norm is None and self.blocks[e.block].chained_norm() is not None:
                    next_norm = follower.chained_norm()  # (between two blocks that chain their norms)
            else:  # the final norm, where the head's product can take its place (every row goes to the head)
                next_norm = self.final_norm if step.every_row_wanted and not self.head.has_bias else None
            if e.inject is not None:
                delta = self._injected(e.inject, delta, step)
            delta = self.blocks[e.block].forward(hidden, delta, step, caches.layer(i), next_norm=next_norm)
        if step.logit_rows.shape[0] == 0:
            return torch.empty((0, self.vocab_size), dtype=torch.float32, device=hidden.device)
        if isinstance(delta, Carried):  # the last block has added everything into the stream itself
            delta = None
        if isinstance(delta, Normed):  # the final norm of every row, made by the last block's last launch
            x = delta.x
        else:
            x = delta if isinstance(delta, Prenormed) else self.final_norm.forward(hidden, delta, rows=step.logit_rows)
        logits = self.head.forward(x, out_dtype=torch.float32)
        if self.logit_scale != 1.0:
            logits = self.ctx.ops.scale_(logits, self.logit_scale)
        return logits if self.logit_softcap is None else self.ctx.ops.softcap_(logits, self.logit_softcap)
