"""Telulorn: how its configuration becomes parts.

The layers are listed one by one in the configuration; layer i's tensors start with `l<i>.`, its mixer's with
`l<i>.mix.` (of two mixers side by side `l<i>.mix.left.` and `l<i>.mix.right.`), its feed-forward's with
`l<i>.mlp.`, its norms are `l<i>.norm1` (before the mixer) and `l<i>.norm2` (before the feed-forward).  Every
layer is a pre-norm block; layers `loop.start` .. `loop.stop - 1` stand `loop.times` times in the plan, each time
with caches and states of their own, and row t of `loop.step` enters the stream ahead of pass t.  The output
head is the embedding table.
"""
from __future__ import annotations

from ..config.registry import register_architecture
from ..config.telulorn_config import PARALLEL, TelulornConfig, TelulornLayer
from ..parts import (Embedding, GatedAttention, GatedLinearAttention, Linear, PassVectors, PlainMLP, PreNormBlock, RMSNorm,
                     RotaryInterleaved, SideBySideMixer, geometric_slopes)
from .decoder import DecoderLM, PlanEntry, looped_plan


def _mixer(c: TelulornConfig, layer: TelulornLayer, prefix: str):
    m = layer.mixer
    if layer.type == PARALLEL:
        a, r = m.left, m.right
        if r.decay_rank is None:
            raise ValueError("the decay's inner rank is not known yet: it is read from the checkpoint's shapes "
                             "(TelulornConfig.with_tensor_shapes) or given as `decay_rank`")
        left = GatedAttention(prefix + "left.", c.width, a.heads, a.kv_heads, a.dim, a.vdim, a.scale, chunk=a.chunk,
                              slopes=geometric_slopes(a.heads), talk=True, out_scale=m.left_scale)
        right = GatedLinearAttention(prefix + "right.", c.width, r.heads, r.dim, r.vdim, r.decay_rank, r.tau, c.norm_eps,
                                     out_scale=m.right_scale)
        return SideBySideMixer(left, right)
    return GatedAttention(prefix, c.width, m.heads, m.kv_heads, m.dim, m.vdim, m.scale,
                          rotation=RotaryInterleaved(m.rot_dims, m.rot_base),
                          value_rotation=RotaryInterleaved(m.vdim, m.rot_base), window=m.window, keep_first=m.keep_first,
                          qkv_bias=True, sinks=True)


def build_telulorn(config: TelulornConfig) -> DecoderLM:
    c = config
    norm = lambda name: RMSNorm(name, c.width, c.norm_eps)
    blocks = []
    for i, layer in enumerate(c.layers):
        p = f"l{i}."
        mixer = _mixer(c, layer, p + "mix.")
        if layer.mlp is None:
            blocks.append(PreNormBlock(norm(p + "norm1"), mixer))
        else:
            blocks.append(PreNormBlock(norm(p + "norm1"), mixer, norm(p + "norm2"),
                                       PlainMLP(p + "mlp.", c.width, layer.mlp.ff, activation="relu2", to_residual=True)))
    loop = c.loop
    return DecoderLM(
        config=c,
        embedding=Embedding("embed", c.vocab, c.width),
        blocks=blocks,
        plan=([PlanEntry(i) for i in range(len(blocks))] if loop is None
              else looped_plan(len(blocks), loop.start, loop.stop, loop.times)),
        final_norm=norm("final.norm"),
        head=Linear(["head"], c.width, [c.vocab], optional=True),
        tied_head=True,
        pass_vectors=None if loop is None else PassVectors("loop.step", loop.times, c.width),
    )


register_architecture(TelulornConfig.ARCHITECTURE, TelulornConfig, build_telulorn)
