"""Rorevik: a decoder whose layers are listed one by one in config.json, a run of them repeated several times with the
same weights.  The first rows of the stream are the norm of the scaled embedding plus a learned position vector.  Every
layer is pre-norm, `x <- x + mixer(norm1(x))`, then `x <- x + ff(norm2(x))` (or no second line).  The mixer is two
mixers side by side, each times a constant (attention with capped scores and rotated pairs, and Mamba-2's state-space
recurrence), or the gated delta rule with a decay per key channel.  The feed-forward is dense, gated and clamped, with
biases, or absent.  The output head is a matrix of its own.

config.json keys: `architecture` (a string), `vocab`, `width`, `max_positions`, `norm.eps`, `embedding.scale` (default
1), `loop.{start, stop, times}` (absent: every layer runs once) and `layers`: a list of
`{type, mixer: {...}, mlp: {...} | null}`:

  parallel       mixer: left  {heads, kv_heads, dim, vdim, scale, softcap, rot.{base, dims}}
                        right {heads, vdim, state, groups, conv, norm_groups}
                        left_scale, right_scale
  channel_delta  mixer: heads, kv_heads, dim, vdim, conv (the inner ranks of the decay and of the output gate are the
                 shapes of `mix.a1` and `mix.g1`; a config may also say them as `decay_rank` and `gate_rank`)
  mlp            kind "dense": ff, limit

Every size and every constant that may differ between models is read from there (or from a tensor's shape);
nothing of it stands in code.
"""
from __future__ import annotations

import dataclasses
from typing import Any, Dict, Mapping, Optional, Tuple

from .model_config import ConfigError, _optional, _required

PARALLEL, CHANNEL_DELTA = "parallel", "channel_delta"
MIXER_TYPES = (PARALLEL, CHANNEL_DELTA)
DENSE = "dense"


def _section(d: Dict[str, Any], key: str, where: str) -> Dict[str, Any]:
    v = d.get(key)
    if not isinstance(v, dict):
        raise ConfigError(f"{where} needs an object `{key}`")
    return v


def _positive(value, what: str):
    if not value > 0:
        raise ConfigError(f"Rorevik config {what} must be positive")
    return value


@dataclasses.dataclass(frozen=True)
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: Optional[float]  # None: the scores are not capped
    rot_base: float
    rot_dims: int


@dataclasses.dataclass(frozen=True)
class StateSpaceSizes:
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int  # taps
    norm_groups: int


@dataclasses.dataclass(frozen=True)
class ParallelSizes:
    left: AttentionSizes
    right: StateSpaceSizes
    left_scale: float
    right_scale: float


@dataclasses.dataclass(frozen=True)
class ChannelDeltaSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int  # taps
    decay_rank: Optional[int] = None  # None until a checkpoint's shapes have said it
    gate_rank: Optional[int] = None


@dataclasses.dataclass(frozen=True)
class DenseSizes:
    ff: int
    limit: float


@dataclasses.dataclass(frozen=True)
class RorevikLayer:
    type: str
    mixer: Any  # ParallelSizes or ChannelDeltaSizes
    mlp: Optional[DenseSizes]


@dataclasses.dataclass(frozen=True)
class LoopSizes:
    start: int
    stop: int
    times: int


def _heads(m: Dict[str, Any], key: str, where: str) -> Tuple[int, int]:
    """(`heads`, `key`): heads that come in equal shares of `key`, which is `heads` where it is not said."""
    heads = _positive(_required(m, "heads", int), f"{where}.heads")
    shares = _positive(_optional(m, key, int, heads), f"{where}.{key}")
    if heads % shares:
        raise ConfigError(f"{where}.heads must be a multiple of {key}")
    return heads, shares


def _dims(m: Dict[str, Any], where: str) -> Tuple[int, int]:
    dim = _positive(_required(m, "dim", int), f"{where}.dim")
    return dim, _positive(_optional(m, "vdim", int, dim), f"{where}.vdim")


def _attention_from(m: Dict[str, Any], where: str) -> AttentionSizes:
    heads, kv_heads = _heads(m, "kv_heads", where)
    dim, vdim = _dims(m, where)
    rot = m.get("rot") if isinstance(m.get("rot"), dict) else {"dims": 0}
    dims = _optional(rot, "dims", int, dim)
    if dims % 2 or not 0 <= dims <= dim:
        raise ConfigError(f"{where}.rot.dims must be even and at most dim")
    base = _positive(_required(rot, "base", float), f"{where}.rot.base") if dims else 1.0
    cap = _optional(m, "softcap", float, None)
    if cap is not None:
        _positive(cap, f"{where}.softcap")
    return AttentionSizes(heads, kv_heads, dim, vdim, _optional(m, "scale", float, float(dim) ** -0.5), cap, base, dims)


def _state_space_from(m: Dict[str, Any], where: str) -> StateSpaceSizes:
    heads = _positive(_required(m, "heads", int), f"{where}.heads")
    vdim = _positive(_required(m, "vdim", int), f"{where}.vdim")
    groups = _positive(_optional(m, "groups", int, 1), f"{where}.groups")
    norm_groups = _positive(_optional(m, "norm_groups", int, 1), f"{where}.norm_groups")
    if heads % groups or (heads * vdim) % norm_groups:
        raise ConfigError(f"{where}: heads must be a multiple of groups, heads * vdim one of norm_groups")
    return StateSpaceSizes(heads, vdim, _positive(_required(m, "state", int), f"{where}.state"), groups,
                           _positive(_required(m, "conv", int), f"{where}.conv"), norm_groups)


def _mixer_from(kind: str, m: Dict[str, Any], where: str):
    if kind == PARALLEL:
        return ParallelSizes(_attention_from(_section(m, "left", where), f"{where}.left"),
                             _state_space_from(_section(m, "right", where), f"{where}.right"),
                             _optional(m, "left_scale", float, 1.0), _optional(m, "right_scale", float, 1.0))
    heads, kv_heads = _heads(m, "kv_heads", where)
    dim, vdim = _dims(m, where)
    ranks = [_optional(m, key, int, None) for key in ("decay_rank", "gate_rank")]
    for key, rank in zip(("decay_rank", "gate_rank"), ranks):
        if rank is not None:
            _positive(rank, f"{where}.{key}")
    return ChannelDeltaSizes(heads, kv_heads, dim, vdim, _positive(_required(m, "conv", int), f"{where}.conv"), *ranks)


def _mlp_from(m, where: str) -> Optional[DenseSizes]:
    if m is None:
        return None
    if not isinstance(m, dict):
        raise ConfigError(f"{where}.mlp must be an object or null")
    if m.get("kind") != DENSE:
        raise ConfigError(f"{where}.mlp.kind={m.get('kind')!r} is unknown ({DENSE})")
    return DenseSizes(_positive(_required(m, "ff", int), f"{where}.mlp.ff"),
                      _positive(_required(m, "limit", float), f"{where}.mlp.limit"))


def _loop_from(d: Dict[str, Any], layers: int) -> Optional[LoopSizes]:
    if d.get("loop") is None:
        return None
    loop = _section(d, "loop", "Rorevik config")
    start, stop, times = (_required(loop, key, int) for key in ("start", "stop", "times"))
    if not 0 <= start < stop <= layers or times < 1:
        raise ConfigError(f"Rorevik config loop: layers {start} .. {stop - 1}, {times} times, do not fit {layers} layers")
    return LoopSizes(start, stop, times)


@dataclasses.dataclass(frozen=True)
class RorevikConfig:
    architecture: str
    vocab: int
    width: int
    max_positions: int
    norm_eps: float
    embedding_scale: float
    layers: Tuple[RorevikLayer, ...]
    loop: Optional[LoopSizes] = None

    ARCHITECTURE = "Rorevik"

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "RorevikConfig":
        layers = d.get("layers")
        if not isinstance(layers, list):
            raise ConfigError("Missing required config field: layers")
        out = []
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            if not isinstance(layer, dict) or layer.get("type") not in MIXER_TYPES:
                kind = layer.get("type") if isinstance(layer, dict) else layer
                raise ConfigError(f"{where}.type={kind!r} is unknown ({', '.join(MIXER_TYPES)})")
            out.append(RorevikLayer(layer["type"], _mixer_from(layer["type"], _section(layer, "mixer", where), f"{where}.mixer"),
                                    _mlp_from(layer.get("mlp"), where)))
        embedding = d.get("embedding") if isinstance(d.get("embedding"), dict) else {}
        return cls(
            architecture=str(d.get("architecture") or (d.get("architectures") or [cls.ARCHITECTURE])[0]),
            vocab=_positive(_required(d, "vocab", int), "vocab"),
            width=_positive(_required(d, "width", int), "width"),
            max_positions=_positive(_required(d, "max_positions", int), "max_positions"),
            norm_eps=_positive(_required(_section(d, "norm", "Rorevik config"), "eps", float), "norm.eps"),
            embedding_scale=_optional(embedding, "scale", float, 1.0),
            layers=tuple(out),
            loop=_loop_from(d, len(out)),
        )

    def with_tensor_shapes(self, shapes: Mapping[str, Tuple[int, ...]]) -> "RorevikConfig":
        """The sizes that config.json may leave to the checkpoint, read from its tensors' shapes: the inner ranks of
        every delta rule's decay and output gate (rows of `l<i>.mix.a1` and `l<i>.mix.g1`)."""
        layers = []
        for i, layer in enumerate(self.layers):
            if layer.type == CHANNEL_DELTA:
                found = {}
                for field, tensor in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    if getattr(layer.mixer, field) is None:
                        shape = shapes.get(f"l{i}.mix.{tensor}")
                        if shape is None or len(shape) != 2:
                            raise ConfigError(f"layers[{i}]: the checkpoint has no matrix l{i}.mix.{tensor} to read {field} from")
                        found[field] = int(shape[0])
                layer = dataclasses.replace(layer, mixer=dataclasses.replace(layer.mixer, **found))
            layers.append(layer)
        return dataclasses.replace(self, layers=tuple(layers))

    def to_dict(self) -> Dict[str, Any]:
        layers = []
        for layer in self.layers:
            m = layer.mixer
            if isinstance(m, ParallelSizes):
                a = m.left
                left: Dict[str, Any] = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale}
                if a.softcap is not None:
                    left["softcap"] = a.softcap
                if a.rot_dims:
                    left["rot"] = {"base": a.rot_base, "dims": a.rot_dims}
                mixer: Dict[str, Any] = {"left": left, "left_scale": m.left_scale, "right": dataclasses.asdict(m.right),
                                         "right_scale": m.right_scale}
            else:
                mixer = {k: v for k, v in dataclasses.asdict(m).items() if v is not None}
            layers.append({"type": layer.type, "mixer": mixer,
                           "mlp": None if layer.mlp is None else {"kind": DENSE, **dataclasses.asdict(layer.mlp)}})
        d: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                             "max_positions": self.max_positions, "norm": {"eps": self.norm_eps},
                             "embedding": {"scale": self.embedding_scale}, "layers": layers}
        if self.loop is not None:
            d["loop"] = dataclasses.asdict(self.loop)
        return d
