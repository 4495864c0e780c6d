"""Tiny Rorevik configurations and helpers for the tests.  Between them every size and option differs: one key/value
head, several, or as many as query heads, values wider and narrower than keys, rotations of a pair, a part, the whole
head and none, caps from a fraction of a score to far above it, state-space heads of 8 to 100 state channels in one
group or several with output norms over a row, a part or less than a head, delta heads that share query/key heads or do
not, convolutions of one to nine taps, inner ranks of 1 to 40, loops over one layer or three, at the beginning, in the
middle and at the end of the model, once, twice or three times, and no loop, layers without a feed-forward, mixer
constants of one and others, clamps that bite seldom and often, embeddings that are scaled up, down and not."""
from __future__ import annotations

import os
from typing import Dict, List

import torch

from litellmengine_amd.config import RorevikConfig
from litellmengine_amd.weights import write_model_dir
from tests.plain import rorevik_plain as plain
from tests.visadra_util import rewrite, run_tool  # noqa: F401  (the same tool, whatever the architecture)


def parallel(heads, kv_heads, dim, vdim, scale, cap, base, dims, ssd_heads, ssd_vdim, state, groups, conv, norm_groups,
             left_scale=1.0, right_scale=1.0):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap,
            "rot": {"base": base, "dims": dims}}
    right = {"heads": ssd_heads, "vdim": ssd_vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}
    return {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}


def delta(heads, kv_heads, dim, vdim, conv, decay_rank, gate_rank):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "decay_rank": decay_rank,
            "gate_rank": gate_rank}


def layer(mixer, ff, limit=2.0):
    return {"type": "parallel" if "left" in mixer else "channel_delta", "mixer": mixer,
            "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


# odd sizes: what only the generic kernels take
R_A = {
    "architecture": "Rorevik", "vocab": 131, "width": 72, "max_positions": 512, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.0},
    "loop": {"start": 1, "stop": 4, "times": 2},
    "layers": [
        layer(delta(6, 2, 24, 20, 4, 5, 7), 52, 1.5),
        layer(parallel(6, 3, 20, 12, 0.25, 3.0, 500.0, 8, 6, 20, 24, 3, 3, 4, 0.7, 1.3), None),
        layer(delta(3, 3, 17, 33, 2, 16, 1), 36, 7.0),
        layer(parallel(2, 1, 36, 48, 0.15, 0.8, 1e4, 36, 1, 100, 12, 1, 1, 1, 1.0, 0.5), 44, 0.4),
        layer(parallel(5, 5, 17, 9, 0.2, 12.0, 1e4, 0, 5, 9, 33, 5, 9, 15), 20),
    ],
}
# sizes that the matrix-core kernels take
R_B = {
    "architecture": "Rorevik", "vocab": 256, "width": 128, "max_positions": 700, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
    "loop": {"start": 0, "stop": 2, "times": 3},
    "layers": [
        layer(parallel(8, 2, 64, 64, 0.12, 5.0, 1e5, 32, 8, 32, 64, 2, 4, 2, 0.6, 0.9), 96),
        layer(delta(4, 2, 64, 32, 4, 24, 40), 64, 3.0),
        layer(parallel(12, 3, 32, 32, 0.2, 2.0, 1e4, 2, 4, 64, 32, 1, 2, 4, 1.2, 0.8), None),
        layer(parallel(4, 1, 96, 64, 0.1, 30.0, 1e4, 96, 2, 16, 128, 2, 4, 1), 80, 1.0),
    ],
}
# one head of everything, a loop of one layer at the end
R_C = {
    "architecture": "Rorevik", "vocab": 77, "width": 50, "max_positions": 300, "norm": {"eps": 3e-5}, "embedding": {"scale": 0.5},
    "loop": {"start": 2, "stop": 3, "times": 3},
    "layers": [
        layer(parallel(1, 1, 48, 10, 0.1, 4.0, 100.0, 2, 1, 8, 8, 1, 2, 4), 20),
        layer(delta(1, 1, 100, 12, 1, 3, 2), None),
        layer(delta(5, 1, 12, 30, 3, 1, 33), 8, 0.7),
    ],
}
# no loop; one mixer after the other
R_D = {
    "architecture": "Rorevik", "vocab": 90, "width": 64, "max_positions": 400, "norm": {"eps": 1e-5}, "embedding": {"scale": 8.0},
    "layers": [layer(delta(4, 4, 32, 64, 4, 8, 16), None), layer(parallel(16, 4, 32, 64, 0.2, 6.0, 1e4, 16, 4, 48, 40, 4, 3, 2, 0.9, 1.0), 48)],
}
CONFIGS = {"A": R_A, "B": R_B, "C": R_C, "D": R_D}
PAGE_SIZES = {"A": 4, "B": 16, "C": 8, "D": 16}


def make_model_dir(tmp_path, which, seed: int = 77, dtype=torch.float32, config=None) -> str:
    cfg = RorevikConfig.from_dict(config or CONFIGS[which])
    path = os.path.join(str(tmp_path), f"rorevik_{which}_{seed}")
    write_model_dir(cfg, path, seed, dtype)
    return path


def sharpen(model_dir: str, factor: float = 1.0, memory: float = 1.0, skip=()) -> None:
    """Random weights average everything and hide faults: attention is flat and far below its cap, every decay and every
    step size is the same, gates are halves, biases and sublayers of N(0, 0.02) weights whisper beside nothing.  Here the
    attention's query and key projections grow with `factor` (single keys, near or far back, carry the softmax), norms'
    weights spread over (0.5, 1.5), the decays' rates and offsets spread so that some heads and channels forget at once
    and others, the more the larger `memory`, remember for hundreds of tokens, with inner projections that follow the
    tokens; betas, gates, biases, the embedding, the position vectors, the output head and every projection back into
    the stream grow.  `skip`: endings of tensor names that stay as they are."""

    def spread(t, lo, hi, salt):
        g = torch.Generator().manual_seed(salt + t.numel())
        return torch.rand(t.shape, generator=g) * (hi - lo) + lo

    def change(name, t):
        if any(name.endswith(x) for x in skip):
            return None
        t = t.float()
        if name.endswith("norm1") or name.endswith("norm2") or name in ("final.norm", "embed.norm") or name.endswith(".norm"):
            return spread(t, 0.5, 1.5, 1 + len(name))
        if name.endswith(".A_log"):
            return spread(t, -3.0 * memory, 1.0, 3)
        if name.endswith(".dt_bias"):
            return spread(t, -4.0 * memory, 1.0, 5)
        if name.endswith(".D"):
            return spread(t, -1.0, 1.5, 7)
        if name.endswith(".left.q") or name.endswith(".left.k"):
            return t * 4.0 * factor
        if name.endswith(".a1") or name.endswith(".g1"):
            return t * 10.0
        if name.endswith(".a2") or name.endswith(".g2"):
            return t * 25.0
        if name.endswith(".mix.b"):
            return t * 20.0
        if name.endswith(".b"):  # biases of the feed-forward and of the convolution
            return t * 15.0
        if name in ("embed", "pos", "head"):
            return t * 10.0
        if name.endswith(".o") or name.endswith(".down"):
            return t * 6.0
        if name.endswith(".in") or name.endswith(".q") or name.endswith(".k") or name.endswith(".v") or name.endswith(".gate") or name.endswith(".up"):
            return t * 4.0
        return None

    rewrite(model_dir, change)


def read(model_dir: str):
    return plain.load(model_dir)


def plain_logits(model_dir: str, requests: Dict[str, List[int]], dtype=torch.float64) -> Dict[str, torch.Tensor]:
    cfg, w = plain.load(model_dir, dtype)
    return {rid: plain.forward(cfg, w, tokens) for rid, tokens in requests.items()}


def residual_streams(model_dir: str, tokens: List[int]) -> List[torch.Tensor]:
    cfg, w = plain.load(model_dir)
    out: List[torch.Tensor] = []
    plain.forward(cfg, w, tokens, out)
    return out
