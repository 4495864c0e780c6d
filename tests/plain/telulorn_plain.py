"""Plain, slow Telulorn implementation: the oracle of the Telulorn tests.

Whole sequences, no cache, no state carried between calls, one function per
mechanism, nothing shared with the engine's code.  Everything runs on the CPU
in float64 (or the dtype of the weights handed in).  `cfg` is the dictionary of
config.json; `w` maps tensor names to tensors.

Notation: h is a sublayer's normed input [T, width]; W x means `x @ W.T` with W
stored [out, in]; positions count from 0; `p` is a tensor-name prefix.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional, Sequence

import torch


# --------------------------------------------------------------------------
# small pieces
# --------------------------------------------------------------------------
def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis (eps inside the root)."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return rms_unit(x, eps) * weight


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * sigmoid(x)


def log_sigmoid(x: torch.Tensor) -> torch.Tensor:
    """log(1 / (1 + e^-x)), written so that large |x| do not overflow."""
    return torch.clamp(x, max=0.0) - torch.log1p(torch.exp(-x.abs()))


def turn_pairs(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float, sign: float = 1.0) -> torch.Tensor:
    """x [T, heads, n >= dims]: elements 2i and 2i+1 (i < dims/2) turn by sign * pos * base^(-2i/dims);
    elements from `dims` on pass."""
    out = x.clone()
    for i in range(dims // 2):
        a = sign * positions.to(x.dtype) * (float(base) ** (-2.0 * i / dims))
        c, s = torch.cos(a).view(-1, 1), torch.sin(a).view(-1, 1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


# --------------------------------------------------------------------------
# which keys a position sees
# --------------------------------------------------------------------------
def chunk_mask(T: int, size: int) -> torch.Tensor:
    """[T, T] bool: i sees j <= i of its own chunk of `size` positions (chunks count from position 0)."""
    i, j = torch.arange(T).view(-1, 1), torch.arange(T).view(1, -1)
    return (j <= i) & (i // size == j // size)


def kept_window_mask(T: int, size: int, keep_first: int) -> torch.Tensor:
    """[T, T] bool: i sees j <= i among the last `size` positions (itself counted) or the first `keep_first`."""
    i, j = torch.arange(T).view(-1, 1), torch.arange(T).view(1, -1)
    return (j <= i) & ((i - j < size) | (j < keep_first))


# --------------------------------------------------------------------------
# attention's pieces
# --------------------------------------------------------------------------
def head_slopes(heads: int, dtype=torch.float64) -> torch.Tensor:
    """2^(-8 (h + 1) / heads) for h = 0 .. heads - 1."""
    return 2.0 ** (-8.0 * (torch.arange(heads, dtype=dtype) + 1.0) / heads)


def head_scores(q: torch.Tensor, k: torch.Tensor, scale: float) -> torch.Tensor:
    """q [T, H, d], k [T, G, d] -> [H, T, T]; query head h reads key head h // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    kk = k.repeat_interleave(H // G, dim=1)
    return torch.einsum("ihd,jhd->hij", q, kk) * scale


def distance_bias(T: int, heads: int, dtype=torch.float64) -> torch.Tensor:
    """[H, T, T]: what is taken off the score of query i and key j, slope_h * (i - j)."""
    i, j = torch.arange(T, dtype=dtype).view(-1, 1), torch.arange(T, dtype=dtype).view(1, -1)
    return head_slopes(heads, dtype).view(-1, 1, 1) * (i - j)


def softmax_weights(scores: torch.Tensor, mask: torch.Tensor, sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """scores [H, T, T]; with `sink` [H] the sum has one more place exp(sink_h) that carries no value."""
    s = scores.masked_fill(~mask, -math.inf)
    top = s.amax(dim=-1, keepdim=True)
    if sink is not None:
        top = torch.maximum(top, sink.view(-1, 1, 1))
    e = torch.exp(s - top)
    total = e.sum(dim=-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink.view(-1, 1, 1) - top)
    return e / total


def mixed_over_heads(weights: torch.Tensor, talk: torch.Tensor) -> torch.Tensor:
    """weights [H, T, T] -> sum_g talk[h, g] weights[g]."""
    return torch.einsum("hg,gij->hij", talk, weights)


def heads_values(weights: torch.Tensor, v: torch.Tensor) -> torch.Tensor:
    """weights [H, T, T] on v [T, G, d] -> [T, H, d]; head h reads value head h // (H / G)."""
    vv = v.repeat_interleave(weights.shape[0] // v.shape[1], dim=1)
    return torch.einsum("hij,jhd->ihd", weights, vv)


# --------------------------------------------------------------------------
# the mixers
# --------------------------------------------------------------------------
def talking_attention(h, w, p: str, m: dict) -> torch.Tensor:
    """Chunked attention with a distance bias, whose heads' weights are mixed; gated element by element."""
    T, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, d)
    k = (h @ w[p + "k"].T).view(T, G, d)
    v = (h @ w[p + "v"].T).view(T, G, vd)
    s = head_scores(q, k, m["scale"]) - distance_bias(T, H, h.dtype)
    a = softmax_weights(s, chunk_mask(T, (m.get("mask") or {"size": T})["size"]))  # (no mask: one chunk)
    o = heads_values(mixed_over_heads(a, w[p + "talk"]), v).reshape(T, H * vd)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def linear_recurrence(q, k, v, alpha) -> torch.Tensor:
    """q, k, alpha [T, H, d], v [T, H, vd]: S <- diag(alpha_t) S + k_t v_t^T, o_t = S^T q_t -> [T, H, vd]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    out = []
    for t in range(T):
        S = alpha[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out)


def decays(h, w, p: str, tau: float) -> torch.Tensor:
    """sigmoid(z)^(1/tau), z = W_a2 (W_a1 h) + b."""
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    return torch.exp(log_sigmoid(z) / tau)


def gated_linear_attention(h, w, p: str, m: dict, eps: float) -> torch.Tensor:
    T, H, d, vd = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, d)
    v = (h @ w[p + "v"].T).view(T, H, vd)
    o = linear_recurrence(q, k, v, decays(h, w, p, m["tau"]).view(T, H, d))
    o = rms_norm(o, w[p + "norm"], eps).reshape(T, H * vd)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel_mixer(h, w, p: str, m: dict, eps: float) -> torch.Tensor:
    return (m["left_scale"] * talking_attention(h, w, p + "left.", m["left"])
            + m["right_scale"] * gated_linear_attention(h, w, p + "right.", m["right"], eps))


def window_attention(h, w, p: str, m: dict, eps: float = 0.0) -> torch.Tensor:
    """Window with kept first tokens, sink, biases, rotated keys, queries and values; gated element by element."""
    T, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    pos = torch.arange(T)
    q = turn_pairs((h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, d), pos, dims, base)
    k = turn_pairs((h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, d), pos, dims, base)
    v = turn_pairs((h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, vd), pos, vd, base)
    mask = m.get("mask") or {"size": T}  # (no mask: every earlier token)
    a = softmax_weights(head_scores(q, k, m["scale"]), kept_window_mask(T, mask["size"], mask.get("keep_first", 0)), w[p + "sink"])
    o = turn_pairs(heads_values(a, v), pos, vd, base, sign=-1.0).reshape(T, H * vd)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


MIXERS = {"parallel": parallel_mixer, "attention": window_attention}


def squared_relu_ff(h, w, p: str) -> torch.Tensor:
    return torch.clamp(h @ w[p + "up"].T, min=0.0) ** 2 @ w[p + "down"].T


# --------------------------------------------------------------------------
# the model
# --------------------------------------------------------------------------
def layer_runs(cfg: dict) -> List[tuple]:
    """[(layer, None or the number of the loop's pass that starts with this run)] in the order of execution."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: Sequence[int],
            layers_out: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; with `layers_out`, the residual stream after every layer run is appended."""
    eps = cfg["norm"]["eps"]
    first = w["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    x = first.clone()
    for i, starts in layer_runs(cfg):
        if starts is not None:
            x = x + (first if starts > 0 else 0.0) + w["loop.step"][starts]
        spec, p = cfg["layers"][i], f"l{i}."
        x = x + MIXERS[spec["type"]](rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", spec["mixer"], eps)
        if spec.get("mlp") is not None:
            x = x + squared_relu_ff(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T


def load(model_dir: str, dtype=torch.float64):
    from safetensors.torch import load_file

    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = json.load(f)
    w = {k: v.to(dtype) for k, v in load_file(os.path.join(model_dir, "model.safetensors")).items()}
    return cfg, w


def greedy(cfg, w, prompt: Sequence[int], new_tokens: int) -> List[int]:
    ids = list(prompt)
    for _ in range(new_tokens):
        ids.append(int(torch.argmax(forward(cfg, w, ids)[-1])))
    return ids[len(prompt):]
