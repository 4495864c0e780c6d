"""Plain, slow Rorevik implementation: the oracle of the Rorevik tests.

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

UNIT_EPS = 1e-6  # inside the root that makes a vector a unit vector


# --------------------------------------------------------------------------
# small pieces
# --------------------------------------------------------------------------
def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis (eps inside the root)."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return rms_unit(x, eps) * weight


def unit_vectors(x: torch.Tensor) -> torch.Tensor:
    """x / sqrt(sum(x^2) + 1e-6) over the last axis."""
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + UNIT_EPS)


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * sigmoid(x)


def softplus(x: torch.Tensor) -> torch.Tensor:
    """log(1 + e^x), written so that large |x| do not overflow."""
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def turn_pairs(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, heads, n >= dims]: elements 2i and 2i+1 (i < dims/2) turn by pos * base^(-2i/dims);
    elements from `dims` on pass."""
    out = x.clone()
    for i in range(dims // 2):
        a = positions.to(x.dtype) * (float(base) ** (-2.0 * i / dims))
        c, s = torch.cos(a).view(-1, 1), torch.sin(a).view(-1, 1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def causal_conv(u: torch.Tensor, taps: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """u [T, C], taps [C, J]: channel c of token t is sum_j taps[c, j] u[t - J + 1 + j, c], zeros before the start."""
    T, J = u.shape[0], taps.shape[1]
    out = torch.zeros_like(u)
    for t in range(T):
        for j in range(J):
            at = t - J + 1 + j
            if at >= 0:
                out[t] = out[t] + taps[:, j] * u[at]
    return out if bias is None else out + bias


# --------------------------------------------------------------------------
# the embedding
# --------------------------------------------------------------------------
def embedded(cfg: dict, w, tokens: Sequence[int]) -> torch.Tensor:
    """norm(embed[token] * scale + pos[position])."""
    ids = torch.as_tensor(list(tokens), dtype=torch.long)
    x = w["embed"][ids] * cfg["embedding"]["scale"] + w["pos"][: len(ids)]
    return rms_norm(x, w["embed.norm"], cfg["norm"]["eps"])


# --------------------------------------------------------------------------
# the delta rule with a decay per key channel
# --------------------------------------------------------------------------
def channel_decays(h, w, p: str, heads: int, dim: int) -> torch.Tensor:
    """exp(-exp(A_log_head) * softplus(W_a2 (W_a1 h) + dt_bias)), [T, heads, dim]."""
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"].reshape(-1)
    rate = torch.exp(w[p + "A_log"].reshape(-1)).view(1, heads, 1)
    return torch.exp(-rate * softplus(z).view(-1, heads, dim))


def delta_recurrence(q, k, v, beta, g) -> torch.Tensor:
    """q, k, g [T, H, d], v [T, H, vd], beta [T, H]: S <- diag(g_t) S; u = beta_t (v_t - S^T k_t); S <- S + k_t u^T;
    o_t = S^T q_t -> [T, H, vd]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    out = []
    for t in range(T):
        S = g[t].unsqueeze(-1) * S
        u = beta[t].unsqueeze(-1) * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out)


def channel_delta(h, w, p: str, m: dict, eps: float) -> torch.Tensor:
    T, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q = unit_vectors(q.view(T, G, d)) * d ** -0.5
    k = unit_vectors(k.view(T, G, d))
    q, k = (x.repeat_interleave(H // G, dim=1) for x in (q, k))
    beta = sigmoid(h @ w[p + "b"].T)
    o = delta_recurrence(q, k, v.view(T, H, vd), beta, channel_decays(h, w, p, H, d))
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T)
    return (rms_norm(o, w[p + "norm"], eps).reshape(T, H * vd) * gate) @ w[p + "o"].T


# --------------------------------------------------------------------------
# attention with capped scores
# --------------------------------------------------------------------------
def capped(scores: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(scores / cap)


def causal_softmax(scores: torch.Tensor) -> torch.Tensor:
    """scores [H, T, T] -> weights over j <= i."""
    T = scores.shape[-1]
    later = torch.ones(T, T, dtype=torch.bool).triu(1)
    s = scores.masked_fill(later, -math.inf)
    e = torch.exp(s - s.amax(dim=-1, keepdim=True))
    return e / e.sum(dim=-1, keepdim=True)


def capped_attention(h, w, p: str, m: dict) -> torch.Tensor:
    T, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    rot = m.get("rot") or {"dims": 0, "base": 1.0}  # (no rotation)
    q = turn_pairs((h @ w[p + "q"].T).view(T, H, d), pos, rot["dims"], rot["base"])
    k = turn_pairs((h @ w[p + "k"].T).view(T, G, d), pos, rot["dims"], rot["base"])
    v = (h @ w[p + "v"].T).view(T, G, vd)
    k, v = (x.repeat_interleave(H // G, dim=1) for x in (k, v))
    a = causal_softmax(capped(torch.einsum("ihd,jhd->hij", q, k) * m["scale"], m["softcap"]))
    return torch.einsum("hij,jhd->ihd", a, v).reshape(T, H * vd) @ w[p + "o"].T


# --------------------------------------------------------------------------
# Mamba-2
# --------------------------------------------------------------------------
def ssd_recurrence(x, B, C, dt, rate, D) -> torch.Tensor:
    """x [T, H, vd], B, C [T, H, N], dt [T, H], rate, D [H]: S_t = exp(-rate dt_t) S_(t-1) + dt_t B_t x_t^T,
    y_t = S_t^T C_t + D x_t -> [T, H, vd]."""
    T, H, vd = x.shape
    S = torch.zeros(H, B.shape[2], vd, dtype=x.dtype)
    out = []
    for t in range(T):
        S = torch.exp(-rate * dt[t]).view(H, 1, 1) * S + dt[t].view(H, 1, 1) * B[t].unsqueeze(-1) * x[t].unsqueeze(1)
        out.append(torch.einsum("hnv,hn->hv", S, C[t]) + D.view(H, 1) * x[t])
    return torch.stack(out)


def gated_group_norm(y, z, weight, groups: int, eps: float) -> torch.Tensor:
    """y * silu(z), every one of `groups` equal parts of a row divided by its own root mean square, times weight."""
    a = (y * silu(z)).view(y.shape[0], groups, -1)
    return rms_unit(a, eps).reshape(y.shape) * weight


def mamba2(h, w, p: str, m: dict, eps: float) -> torch.Tensor:
    T, H, vd, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * vd
    z, xbc, dt = torch.split(h @ w[p + "in"].T, [inner, inner + 2 * G * N, H], dim=1)
    x, B, C = torch.split(silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"])), [inner, G * N, G * N], dim=1)
    dt = softplus(dt + w[p + "dt_bias"].reshape(-1))
    B, C = (t.reshape(T, G, N).repeat_interleave(H // G, dim=1) for t in (B, C))
    y = ssd_recurrence(x.reshape(T, H, vd), B, C, dt, torch.exp(w[p + "A_log"].reshape(-1)), w[p + "D"].reshape(-1))
    return gated_group_norm(y.reshape(T, inner), z, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


def parallel_mixer(h, w, p: str, m: dict, eps: float) -> torch.Tensor:
    return (m["left_scale"] * capped_attention(h, w, p + "left.", m["left"])
            + m["right_scale"] * mamba2(h, w, p + "right.", m["right"], eps))


MIXERS = {"parallel": parallel_mixer, "channel_delta": channel_delta}


# --------------------------------------------------------------------------
# the feed-forward
# --------------------------------------------------------------------------
def clamped_ff(h, w, p: str, limit: float) -> torch.Tensor:
    g = torch.clamp(h @ w[p + "gate"].T + w[p + "gate.b"], max=limit)
    u = torch.clamp(h @ w[p + "up"].T + w[p + "up.b"], min=-limit, max=limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T + w[p + "down.b"]


# --------------------------------------------------------------------------
# the model
# --------------------------------------------------------------------------
def layer_runs(cfg: dict) -> List[int]:
    """The layers in the order of execution."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    return (list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"]
            + list(range(loop["stop"], n)))


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: Sequence[int],
            layers_out: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; with `layers_out`, the residual stream after every layer run is appended."""
    eps = cfg["norm"]["eps"]
    x = embedded(cfg, w, tokens)
    for i in layer_runs(cfg):
        spec, p = cfg["layers"][i], f"l{i}."
        x = x + MIXERS[spec["type"]](rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", spec["mixer"], eps)
        if spec.get("mlp") is not None:
            x = x + clamped_ff(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", spec["mlp"]["limit"])
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


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
