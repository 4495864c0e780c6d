"""Rorevik: how its configuration becomes parts.

The layers are listed one by one in the configuration; layer i's tensors start with `l<i>.`, its mixer's with
`l<i>.mix.` (of two mixers side by side `l<i>.mix.left.` and `l<i>.mix.right.`), its feed-forward's with `l<i>.mlp.`,
its norms are `l<i>.norm1` (before the mixer) and `l<i>.norm2` (before the feed-forward).  Every layer is a pre-norm
block; layers `loop.start` .. `loop.stop - 1` stand `loop.times` times in the plan, each time with caches and states of
their own.  The embedding's rows are scaled, get a vector of their position (`pos`) and pass `embed.norm`; the output
head is `head`.
"""
from __future__ import annotations

from ..config.registry import register_architecture
from ..config.rorevik_config import PARALLEL, RorevikConfig, RorevikLayer
from ..parts import (Embedding, GatedAttention, GatedDeltaMixer, GatedMLP, Linear, PreNormBlock, RMSNorm, RotaryInterleaved,
                     SideBySideMixer, StateSpaceMixer)
from .decoder import DecoderLM, PlanEntry, looped_plan

DELTA_NAMES = ("q", "k", "v", "b", "a1", "a2", "A_log", "dt_bias", "g1", "g2", "norm", "o")


def _mixer(c: RorevikConfig, layer: RorevikLayer, prefix: str):
    m = layer.mixer
    if layer.type == PARALLEL:
        a, r = m.left, m.right
        left = GatedAttention(prefix + "left.", c.width, a.heads, a.kv_heads, a.dim, a.vdim, a.scale,
                              rotation=RotaryInterleaved(a.rot_dims, a.rot_base), gated=False, softcap=a.softcap)
        right = StateSpaceMixer(prefix + "right.", c.width, r.heads, r.vdim, r.state, r.groups, r.conv, r.norm_groups, c.norm_eps)
        return SideBySideMixer(left, right, m.left_scale, m.right_scale)
    if m.decay_rank is None or m.gate_rank is None:
        raise ValueError("the inner ranks of the decay and the gate are not known yet: they are read from the checkpoint's shapes "
                         "(RorevikConfig.with_tensor_shapes) or given as `decay_rank` and `gate_rank`")
    return GatedDeltaMixer(prefix, c.width, m.heads, m.kv_heads, m.dim, m.vdim, m.conv, c.norm_eps, names=DELTA_NAMES,
                           decay_rank=m.decay_rank, gate_rank=m.gate_rank)


def build_rorevik(config: RorevikConfig) -> DecoderLM:
    c = config
    norm = lambda name: RMSNorm(name, c.width, c.norm_eps)
    blocks = []
    for i, layer in enumerate(c.layers):
        p = f"l{i}."
        mixer = _mixer(c, layer, p + "mix.")
        if layer.mlp is None:
            blocks.append(PreNormBlock(norm(p + "norm1"), mixer))
        else:
            ff = GatedMLP(p + "mlp.", c.width, layer.mlp.ff, names=("gate", "up", "down"), activation="clamp",
                          bias_names=("gate.b", "up.b", "down.b"), limit=layer.mlp.limit)
            blocks.append(PreNormBlock(norm(p + "norm1"), mixer, norm(p + "norm2"), ff))
    loop = c.loop
    return DecoderLM(
        config=c,
        embedding=Embedding("embed", c.vocab, c.width, scale=c.embedding_scale, positions_name="pos",
                            max_positions=c.max_positions, norm=norm("embed.norm")),
        blocks=blocks,
        plan=([PlanEntry(i) for i in range(len(blocks))] if loop is None
              else looped_plan(len(blocks), loop.start, loop.stop, loop.times, inject=False)),
        final_norm=norm("final.norm"),
        head=Linear(["head"], c.width, [c.vocab]),
        tied_head=False,
    )


register_architecture(RorevikConfig.ARCHITECTURE, RorevikConfig, build_rorevik)
