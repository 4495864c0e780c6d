"""Tiny Telulorn configurations and helpers for the tests.  Between them every size and option differs: chunks of 5
to 40 tokens and none, windows of 3 to 70 tokens with 0 to 33 kept first tokens and none, one key/value head,
several, or as many as query heads, one query head or twelve, values wider and narrower than keys, rotations of a
pair, a part or the whole head, linear attention heads of 8 to 100 key channels and other value widths, decays of
several temperatures, loops over one layer or three, at the beginning, in the middle and at the end of the model,
once, twice or three times, and no loop, layers without a feed-forward, mixer constants of one and others."""
from __future__ import annotations

import os
from typing import Dict, List

import torch

from litellmengine_amd.config import TelulornConfig
from litellmengine_amd.weights import write_model_dir
from tests.plain import telulorn_plain as plain
from tests.visadra_util import rewrite, run_tool  # noqa: F401  (the same tool, whatever the architecture)


def parallel(heads, kv_heads, dim, vdim, scale, chunk, lin_heads, lin_dim, lin_vdim, tau, rank, left_scale=1.0, right_scale=1.0):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        left["mask"] = {"size": chunk}
    right = {"heads": lin_heads, "dim": lin_dim, "vdim": lin_vdim, "tau": tau, "decay_rank": rank}
    return {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}


def attention(heads, kv_heads, dim, vdim, scale, base, dims, size=None, keep=0):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": dims}}
    if size:
        m["mask"] = {"size": size, "keep_first": keep}
    return m


def layer(mixer, ff):
    return {"type": "parallel" if "left" in mixer else "attention", "mixer": mixer,
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


# odd sizes: what only the generic kernels take
T_A = {
    "architecture": "Telulorn", "vocab": 131, "width": 72, "norm": {"eps": 1e-5}, "loop": {"start": 1, "stop": 4, "times": 2},
    "layers": [
        layer(attention(6, 2, 24, 40, 0.2, 500.0, 8, size=19, keep=4), 52),
        layer(parallel(6, 3, 20, 12, 0.25, 13, 3, 24, 20, 4.0, 5, 0.7, 1.3), None),
        layer(attention(3, 3, 40, 24, 0.15, 1e4, 40, size=5, keep=9), 36),
        layer(parallel(2, 1, 36, 48, 0.15, 40, 1, 100, 12, 16.0, 16, 1.0, 0.5), 44),
        layer(parallel(5, 5, 17, 9, 0.2, None, 2, 8, 33, 1.0, 3), 20),
    ],
}
# sizes that the matrix-core kernels take
T_B = {
    "architecture": "Telulorn", "vocab": 256, "width": 128, "norm": {"eps": 1e-6}, "loop": {"start": 0, "stop": 2, "times": 3},
    "layers": [
        layer(parallel(8, 2, 64, 64, 0.12, 24, 4, 32, 64, 8.0, 16, 0.6, 0.9), 96),
        layer(attention(8, 4, 64, 64, 0.12, 1e5, 32, size=48, keep=33), 64),
        layer(parallel(12, 3, 32, 32, 0.2, 40, 2, 64, 32, 16.0, 8, 1.2, 0.8), None),
        layer(attention(4, 1, 96, 96, 0.1, 1e4, 96, size=70, keep=1), 80),
    ],
}
# one head, a chunk of five tokens, a rotation of nothing but a pair, a window of three tokens, a loop at the end
T_C = {
    "architecture": "Telulorn", "vocab": 77, "width": 50, "norm": {"eps": 3e-5}, "loop": {"start": 2, "stop": 3, "times": 3},
    "layers": [
        layer(attention(1, 1, 48, 10, 0.1, 100.0, 2, size=3, keep=2), 20),
        layer(parallel(1, 1, 32, 32, 0.2, 5, 1, 16, 16, 2.0, 1), None),
        layer(parallel(4, 1, 12, 30, 0.3, 8, 5, 12, 100, 30.0, 7, 0.4, 2.0), 8),
    ],
}
# no loop; no window, so that nothing is kept apart
T_D = {
    "architecture": "Telulorn", "vocab": 90, "width": 64, "norm": {"eps": 1e-5},
    "layers": [layer(attention(4, 2, 32, 64, 0.2, 1e4, 16), None), layer(parallel(16, 4, 32, 32, 0.2, 17, 2, 32, 32, 16.0, 4, 0.9, 1.0), 48)],
}
CONFIGS = {"A": T_A, "B": T_B, "C": T_C, "D": T_D}
PAGE_SIZES = {"A": 4, "B": 16, "C": 8, "D": 16}


def make_model_dir(tmp_path, which, seed: int = 77, dtype=torch.float32, config=None) -> str:
    cfg = TelulornConfig.from_dict(config or CONFIGS[which])
    path = os.path.join(str(tmp_path), f"telulorn_{which}_{seed}")
    write_model_dir(cfg, path, seed, dtype)
    return path


def sharpen(model_dir: str, factor: float = 1.0, memory: float = 1.0, skip=()) -> None:
    """Random weights average everything and hide faults: attention is flat, every decay is the same, gates are
    halves, the passes' vectors and sublayers of N(0, 0.02) weights whisper beside nothing.  Here the attentions'
    query and key projections grow with `factor` (single keys, near or far back, carry the softmax, or none does and
    the sink takes the weight), biases and sinks grow, the norms' weights spread over (0.5, 1.5), the decays'
    offsets over (-4, 6 memory) (heads that forget beside heads that remember for hundreds of tokens) with decay
    projections that follow the tokens, the gates, the passes' vectors, the embedding and every projection back into
    the stream grow.  `skip`: endings of tensor names that stay as they are."""

    def spread(t, lo, hi, salt):
        g = torch.Generator().manual_seed(salt + t.numel())
        return torch.rand(t.shape, generator=g) * (hi - lo) + lo

    def change(name, t):
        if any(name.endswith(x) for x in skip):
            return None
        if ".right." not in name and (name.endswith(".q") or name.endswith(".k")):
            return t.float() * 4.0 * factor
        if name.endswith(".mix.q.b") or name.endswith(".mix.k.b") or name.endswith(".mix.v.b"):
            return t.float() * 10.0
        if name.endswith(".sink"):
            return t.float() * 50.0
        if name.endswith("norm1") or name.endswith("norm2") or name == "final.norm" or name.endswith(".right.norm"):
            return spread(t, 0.5, 1.5, 1 + len(name))
        if name.endswith(".a2.b"):
            return spread(t, -4.0, 6.0 * memory, 3)
        if name.endswith(".a1"):
            return t.float() * 10.0
        if name.endswith(".a2"):
            return t.float() * 40.0
        if name.endswith(".g"):
            return t.float() * 15.0
        if name in ("loop.step", "embed"):
            return t.float() * 10.0
        if name.endswith(".o") or name.endswith(".down"):
            return t.float() * 6.0
        if name.endswith(".v") or name.endswith(".up"):
            return t.float() * 4.0
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
