"""Telulorn: a decoder whose layers are listed one by one in config.json, a run of them repeated several times
with the same weights.  Every layer is pre-norm, `x <- x + mixer(norm1(x))`, then `x <- x + ff(norm2(x))` (or no
second line).  The mixer is two mixers side by side, each times a constant (chunked attention with a distance
bias whose heads' weights are mixed, and gated linear attention), or attention over a window that keeps the
first tokens in sight, with rotated values and a learned sink per head; both attentions are gated element by
element.  The feed-forward is dense without a gate (the square of relu), or absent.  Ahead of every pass of the
loop a vector of the pass is added to the stream, from the second pass on also the embedding's rows.  The
embedding table is the output head.

config.json keys: `architecture` (a string), `vocab`, `width`, `norm.eps`, `loop.{start, stop, times}` (absent:
every layer runs once) and `layers`: a list of `{type, mixer: {...}, mlp: {...} | null}`:

  parallel   mixer: left  {heads, kv_heads, dim, vdim, scale, mask.size} (no mask: one chunk of any length)
                    right {heads, dim, vdim, tau} (the decay's inner rank is the shape of `mix.right.a1`; a config
                    may also say it as `decay_rank`)
                    left_scale, right_scale
  attention  mixer: heads, kv_heads, dim, vdim, scale, rot.{base, dims}, mask.{size, keep_first} (no mask: every
                    earlier token is seen)
  mlp        kind "dense": ff

Every size and every constant that may differ between models is read from there (or from a tensor's shape);
nothing of it stands in code.
"""
from __future__ import annotations

import dataclasses
from typing import Any, Dict, Mapping, Optional, Tuple

from .model_config import ConfigError, _optional, _required

PARALLEL, ATTENTION = "parallel", "attention"
MIXER_TYPES = (PARALLEL, ATTENTION)
DENSE = "dense"


def _section(d: Dict[str, Any], key: str, where: str) -> Dict[str, Any]:
    v = d.get(key)
    if not isinstance(v, dict):
        raise ConfigError(f"{where} needs an object `{key}`")
    return v


def _positive(value, what: str):
    if not value > 0:
        raise ConfigError(f"Telulorn config {what} must be positive")
    return value


@dataclasses.dataclass(frozen=True)
class ChunkedSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: Optional[int] = None  # None: one chunk, however long


@dataclasses.dataclass(frozen=True)
class LinearSizes:
    heads: int
    dim: int
    vdim: int
    tau: float
    decay_rank: Optional[int] = None  # None until a checkpoint's shapes have said it


@dataclasses.dataclass(frozen=True)
class ParallelSizes:
    left: ChunkedSizes
    right: LinearSizes
    left_scale: float
    right_scale: float


@dataclasses.dataclass(frozen=True)
class WindowSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float
    rot_dims: int
    window: Optional[int] = None  # None: every earlier token is seen
    keep_first: int = 0


@dataclasses.dataclass(frozen=True)
class DenseSizes:
    ff: int


@dataclasses.dataclass(frozen=True)
class TelulornLayer:
    type: str
    mixer: Any  # ParallelSizes or WindowSizes
    mlp: Optional[DenseSizes]


@dataclasses.dataclass(frozen=True)
class LoopSizes:
    start: int
    stop: int
    times: int


def _heads(m: Dict[str, Any], where: str):
    heads = _positive(_required(m, "heads", int), f"{where}.heads")
    kv_heads = _positive(_optional(m, "kv_heads", int, heads), f"{where}.kv_heads")
    if heads % kv_heads:
        raise ConfigError(f"{where}.heads must be a multiple of kv_heads")
    return heads, kv_heads


def _dims(m: Dict[str, Any], where: str):
    dim = _positive(_required(m, "dim", int), f"{where}.dim")
    return dim, _positive(_optional(m, "vdim", int, dim), f"{where}.vdim")


def _mask_size(m: Dict[str, Any], where: str) -> Tuple[Dict[str, Any], Optional[int]]:
    mask = m.get("mask") if isinstance(m.get("mask"), dict) else {}
    size = _optional(mask, "size", int, None)
    if size is not None:
        _positive(size, f"{where}.mask.size")
    return mask, size


def _chunked_from(m: Dict[str, Any], where: str) -> ChunkedSizes:
    heads, kv_heads = _heads(m, where)
    dim, vdim = _dims(m, where)
    return ChunkedSizes(heads, kv_heads, dim, vdim, _optional(m, "scale", float, float(dim) ** -0.5), _mask_size(m, where)[1])


def _linear_from(m: Dict[str, Any], where: str) -> LinearSizes:
    dim, vdim = _dims(m, where)
    rank = _optional(m, "decay_rank", int, None)
    if rank is not None:
        _positive(rank, f"{where}.decay_rank")
    return LinearSizes(_positive(_required(m, "heads", int), f"{where}.heads"), dim, vdim,
                       _positive(_required(m, "tau", float), f"{where}.tau"), rank)


def _mixer_from(kind: str, m: Dict[str, Any], where: str):
    if kind == PARALLEL:
        return ParallelSizes(_chunked_from(_section(m, "left", where), f"{where}.left"),
                             _linear_from(_section(m, "right", where), f"{where}.right"),
                             _optional(m, "left_scale", float, 1.0), _optional(m, "right_scale", float, 1.0))
    heads, kv_heads = _heads(m, where)
    dim, vdim = _dims(m, where)
    rot = _section(m, "rot", where)
    dims = _optional(rot, "dims", int, dim)
    if dims % 2 or not 0 <= dims <= dim:
        raise ConfigError(f"{where}.rot.dims must be even and at most dim")
    if vdim % 2:
        raise ConfigError(f"{where}.vdim must be even: the values are rotated in pairs")
    mask, window = _mask_size(m, where)
    keep = _optional(mask, "keep_first", int, 0)
    if keep < 0:
        raise ConfigError(f"{where}.mask.keep_first must not be negative")
    return WindowSizes(heads, kv_heads, dim, vdim, _optional(m, "scale", float, float(dim) ** -0.5),
                       _positive(_required(rot, "base", float), f"{where}.rot.base"), dims, window,
                       keep if window is not None else 0)


def _mlp_from(m, where: str) -> Optional[DenseSizes]:
    if m is None:
        return None
    if not isinstance(m, dict):
        raise ConfigError(f"{where}.mlp must be an object or null")
    if m.get("kind") != DENSE:
        raise ConfigError(f"{where}.mlp.kind={m.get('kind')!r} is unknown ({DENSE})")
    return DenseSizes(_positive(_required(m, "ff", int), f"{where}.mlp.ff"))


def _loop_from(d: Dict[str, Any], layers: int) -> Optional[LoopSizes]:
    if d.get("loop") is None:
        return None
    loop = _section(d, "loop", "Telulorn config")
    start, stop, times = (_required(loop, key, int) for key in ("start", "stop", "times"))
    if not 0 <= start < stop <= layers or times < 1:
        raise ConfigError(f"Telulorn config loop: layers {start} .. {stop - 1}, {times} times, do not fit {layers} layers")
    return LoopSizes(start, stop, times)


@dataclasses.dataclass(frozen=True)
class TelulornConfig:
    architecture: str
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[TelulornLayer, ...]
    loop: Optional[LoopSizes] = None

    ARCHITECTURE = "Telulorn"

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "TelulornConfig":
        layers = d.get("layers")
        if not isinstance(layers, list):
            raise ConfigError("Missing required config field: layers")
        out = []
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            if not isinstance(layer, dict) or layer.get("type") not in MIXER_TYPES:
                kind = layer.get("type") if isinstance(layer, dict) else layer
                raise ConfigError(f"{where}.type={kind!r} is unknown ({', '.join(MIXER_TYPES)})")
            out.append(TelulornLayer(layer["type"], _mixer_from(layer["type"], _section(layer, "mixer", where), f"{where}.mixer"),
                                     _mlp_from(layer.get("mlp"), where)))
        return cls(
            architecture=str(d.get("architecture") or (d.get("architectures") or [cls.ARCHITECTURE])[0]),
            vocab=_positive(_required(d, "vocab", int), "vocab"),
            width=_positive(_required(d, "width", int), "width"),
            norm_eps=_positive(_required(_section(d, "norm", "Telulorn config"), "eps", float), "norm.eps"),
            layers=tuple(out),
            loop=_loop_from(d, len(out)),
        )

    def with_tensor_shapes(self, shapes: Mapping[str, Tuple[int, ...]]) -> "TelulornConfig":
        """The size that config.json may leave to the checkpoint, read from its tensors' shapes: the inner rank of
        every linear attention's decay (rows of `l<i>.mix.right.a1`)."""
        layers = []
        for i, layer in enumerate(self.layers):
            if layer.type == PARALLEL and layer.mixer.right.decay_rank is None:
                shape = shapes.get(f"l{i}.mix.right.a1")
                if shape is None or len(shape) != 2:
                    raise ConfigError(f"layers[{i}]: the checkpoint has no matrix l{i}.mix.right.a1 to read the decay's rank from")
                right = dataclasses.replace(layer.mixer.right, decay_rank=int(shape[0]))
                layer = dataclasses.replace(layer, mixer=dataclasses.replace(layer.mixer, right=right))
            layers.append(layer)
        return dataclasses.replace(self, layers=tuple(layers))

    def to_dict(self) -> Dict[str, Any]:
        layers = []
        for layer in self.layers:
            m = layer.mixer
            if isinstance(m, ParallelSizes):
                a, r = m.left, m.right
                left: Dict[str, Any] = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale}
                if a.chunk is not None:
                    left["mask"] = {"size": a.chunk}
                right: Dict[str, Any] = {"heads": r.heads, "dim": r.dim, "vdim": r.vdim, "tau": r.tau}
                if r.decay_rank is not None:
                    right["decay_rank"] = r.decay_rank
                mixer: Dict[str, Any] = {"left": left, "left_scale": m.left_scale, "right": right, "right_scale": m.right_scale}
            else:
                mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale,
                         "rot": {"base": m.rot_base, "dims": m.rot_dims}}
                if m.window is not None:
                    mixer["mask"] = {"size": m.window, "keep_first": m.keep_first}
            layers.append({"type": layer.type, "mixer": mixer,
                           "mlp": None if layer.mlp is None else {"kind": DENSE, "ff": layer.mlp.ff}})
        d: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                             "norm": {"eps": self.norm_eps}, "layers": layers}
        if self.loop is not None:
            d["loop"] = dataclasses.asdict(self.loop)
        return d
