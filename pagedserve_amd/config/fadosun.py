"""Typed Fadosun configuration, read from the keys of its ``config.json``.

A Fadosun model lists its layers one by one: each names its mixer (``channel_delta``, ``parallel`` or
``mlstm``) with the mixer's own sizes and constants, and its feed-forward (``dense`` or none).  Every
size and constant that may differ comes from the file; the two inner widths of a ``channel_delta``
mixer's low-rank projections, which the file may leave out, come from the stored tensors.
"""

from dataclasses import dataclass
from typing import Optional, Tuple

from .base import ConfigError, require_int, require_number

MIXERS = ("channel_delta", "parallel", "mlstm")


@dataclass(frozen=True)
class FadosunDelta:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int
    gate_rank: int

    def to_dict(self):
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
                "conv": self.conv, "decay_rank": self.decay_rank, "gate_rank": self.gate_rank}


@dataclass(frozen=True)
class FadosunAttention:
    """The attention half of a ``parallel`` mixer."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int                # 0: no rotation
    rot_base: float

    def to_dict(self):
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
               "scale": self.scale}
        if self.rot_dims:
            out["rot"] = {"dims": self.rot_dims, "base": self.rot_base}
        return out


@dataclass(frozen=True)
class FadosunStateSpace:
    """The state-space half of a ``parallel`` mixer."""

    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    def to_dict(self):
        return {"heads": self.heads, "vdim": self.vdim, "state": self.state, "groups": self.groups,
                "conv": self.conv, "norm_groups": self.norm_groups}


@dataclass(frozen=True)
class FadosunParallel:
    left: FadosunAttention
    right: FadosunStateSpace
    left_scale: float
    right_scale: float

    def to_dict(self):
        return {"left": self.left.to_dict(), "right": self.right.to_dict(),
                "left_scale": self.left_scale, "right_scale": self.right_scale}


@dataclass(frozen=True)
class FadosunMemory:
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    def to_dict(self):
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "gate_cap": self.gate_cap}


@dataclass(frozen=True)
class FadosunLayer:
    type: str
    mixer: object
    ff: Optional[int]            # inner width of the feed-forward; None: the layer has none

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(),
                "mlp": None if self.ff is None else {"kind": "dense", "ff": self.ff}}


def _part(raw, key):
    """``raw[key]`` as an object, or None where it is absent or null."""
    value = raw.get(key)
    if value is not None and not isinstance(value, dict):
        raise ConfigError(f"'{key}' must be an object")
    return value


def _shared_heads(raw, key="kv_heads"):
    heads = require_int(raw, "heads")
    shared = require_int(raw, key, default=heads)
    if heads % shared:
        raise ConfigError(f"heads ({heads}) must be a multiple of {key} ({shared})")
    return heads, shared


def _read_delta(mixer):
    heads, kv_heads = _shared_heads(mixer)
    dim = require_int(mixer, "dim")
    return FadosunDelta(heads=heads, kv_heads=kv_heads, dim=dim, vdim=require_int(mixer, "vdim", default=dim),
                        conv=require_int(mixer, "conv"), decay_rank=require_int(mixer, "decay_rank", default=dim),
                        gate_rank=require_int(mixer, "gate_rank", default=dim))


def _read_memory(mixer, where):
    dim = require_int(mixer, "dim")
    return FadosunMemory(heads=require_int(mixer, "heads"), dim=dim, vdim=require_int(mixer, "vdim", default=dim),
                         gate_cap=require_number(mixer, "gate_cap", where + ".mixer"))


def _read_parallel(mixer, where):
    left, right = _part(mixer, "left"), _part(mixer, "right")
    if left is None or right is None:
        raise ConfigError("a parallel mixer needs 'left' and 'right'")
    heads, kv_heads = _shared_heads(left)
    dim = require_int(left, "dim")
    rot = _part(left, "rot")
    rot_dims = require_int(rot, "dims", default=dim, minimum=0) if rot else 0
    if rot_dims % 2 or rot_dims > dim:
        raise ConfigError(f"'rot.dims' {rot_dims} must be even and at most dim ({dim})")
    attention = FadosunAttention(
        heads=heads, kv_heads=kv_heads, dim=dim, vdim=require_int(left, "vdim", default=dim),
        scale=require_number(left, "scale", where + ".mixer.left"), rot_dims=rot_dims,
        rot_base=require_number(rot, "base", where + ".mixer.left.rot") if rot_dims else 0.0)
    inner_heads, vdim = require_int(right, "heads"), require_int(right, "vdim")
    groups = require_int(right, "groups", default=1)
    norm_groups = require_int(right, "norm_groups", default=1)
    if inner_heads % groups:
        raise ConfigError(f"heads ({inner_heads}) must be a multiple of groups ({groups})")
    if inner_heads * vdim % norm_groups:
        raise ConfigError(f"{inner_heads * vdim} columns do not split into {norm_groups} 'norm_groups'")
    space = FadosunStateSpace(heads=inner_heads, vdim=vdim, state=require_int(right, "state"), groups=groups,
                              conv=require_int(right, "conv"), norm_groups=norm_groups)

    def factor(key):
        return require_number(mixer, key, where + ".mixer", positive=False) if key in mixer else 1.0

    return FadosunParallel(attention, space, factor("left_scale"), factor("right_scale"))


def _read_feed_forward(mlp):
    if mlp is None:
        return None
    if not isinstance(mlp, dict) or mlp.get("kind", "dense") != "dense":
        raise ConfigError(f"'mlp.kind' must be 'dense', got {mlp!r}")
    return require_int(mlp, "ff")


@dataclass(frozen=True)
class FadosunConfig:
    vocab: int
    width: int
    layers: Tuple[FadosunLayer, ...]
    norm_eps: float
    max_positions: int

    architecture = "Fadosun"
    eos_token_id = None        # the configuration names no token that ends a request
    # where the file names no bound, requests may grow to this many tokens (an engine's pool or
    # its own bound may be smaller)
    DEFAULT_MAX_POSITIONS = 32768

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @classmethod
    def from_dict(cls, raw) -> "FadosunConfig":
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json 'layers' must be a non-empty list")
        layers = []
        for index, entry in enumerate(listed):
            where = f"layers[{index}]"
            if not isinstance(entry, dict) or entry.get("type") not in MIXERS:
                raise ConfigError(f"config.json {where} 'type' must be one of {', '.join(MIXERS)}, "
                                  f"got {entry.get('type') if isinstance(entry, dict) else entry!r}")
            kind, mixer = entry["type"], entry.get("mixer")
            if not isinstance(mixer, dict):
                raise ConfigError(f"config.json {where} lacks 'mixer'")
            try:
                if kind == "channel_delta":
                    sizes = _read_delta(mixer)
                elif kind == "mlstm":
                    sizes = _read_memory(mixer, where)
                else:
                    sizes = _read_parallel(mixer, where)
                layers.append(FadosunLayer(kind, sizes, _read_feed_forward(entry.get("mlp"))))
            except ConfigError as error:
                raise ConfigError(f"{where}: {error}") from None
        return cls(
            vocab=require_int(raw, "vocab"),
            width=require_int(raw, "width"),
            layers=tuple(layers),
            norm_eps=require_number(raw.get("norm") or {}, "eps", "norm"),
            max_positions=require_int(raw, "max_positions", default=cls.DEFAULT_MAX_POSITIONS),
        )

    def to_dict(self) -> dict:
        out = {
            "architecture": self.architecture,
            "vocab": self.vocab,
            "width": self.width,
            "layers": [layer.to_dict() for layer in self.layers],
            "norm": {"eps": self.norm_eps},
        }
        if self.max_positions != self.DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        return out
