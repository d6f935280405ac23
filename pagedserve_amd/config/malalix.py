"""Typed Malalix configuration, read from the keys of its ``config.json``.

A Malalix model lists its layers one by one: each has an attention mixer (``attention``) with its
own sizes, rotation and chunk size, and a mixture of experts or no feed-forward.  ``loop`` names a
run of layers that is passed several times with the same weights.  Every size and constant that
may differ comes from the file.
"""

from dataclasses import dataclass
from typing import Optional, Tuple

from .base import ConfigError, require_int, require_number

MIXERS = ("attention",)


@dataclass(frozen=True)
class MalalixBands:
    """How the rotation's frequencies are stretched by wavelength."""

    factor: float
    low: float
    high: float
    original: float

    def to_dict(self):
        return {"factor": self.factor, "low": self.low, "high": self.high, "original": self.original}


@dataclass(frozen=True)
class MalalixAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int                   # 0: every earlier token is seen
    rot_dims: int                # 0: no rotation
    rot_base: float
    bands: Optional[MalalixBands]

    def to_dict(self):
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
               "scale": self.scale}
        if self.chunk:
            out["mask"] = {"size": self.chunk}
        if self.rot_dims:
            out["rot"] = {"dims": self.rot_dims, "base": self.rot_base}
            if self.bands is not None:
                out["rot"]["scaling"] = self.bands.to_dict()
        return out


@dataclass(frozen=True)
class MalalixExperts:
    ff: int                      # inner width of an expert
    limit: float                 # cap of the experts' gated unit
    experts: int
    top: int
    shared_ff: int = 0           # 0: no shared expert
    shared_limit: float = 0.0

    def to_dict(self):
        out = {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit},
               "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff:
            out["shared"] = {"ff": self.shared_ff, "limit": self.shared_limit}
        return out


@dataclass(frozen=True)
class MalalixLayer:
    type: str
    mixer: MalalixAttention
    mlp: Optional[MalalixExperts]

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(),
                "mlp": None if self.mlp is None else self.mlp.to_dict()}


def _part(raw, key, where):
    """``raw[key]`` as an object, or None where it is absent or null."""
    value = raw.get(key)
    if value is not None and not isinstance(value, dict):
        raise ConfigError(f"config.json {where} '{key}' must be an object")
    return value


def _read_mixer(mixer, where):
    heads = require_int(mixer, "heads")
    kv_heads = require_int(mixer, "kv_heads", default=heads)
    if heads % kv_heads:
        raise ConfigError(f"heads ({heads}) must be a multiple of kv_heads ({kv_heads})")
    dim = require_int(mixer, "dim")
    mask = _part(mixer, "mask", where)
    chunk = require_int(mask, "size") if mask and mask.get("size") is not None else 0
    rot = _part(mixer, "rot", where) or {}
    rot_dims = require_int(rot, "dims", default=dim, minimum=0) if rot else 0
    if rot_dims % 2 or rot_dims > dim:
        raise ConfigError(f"'rot.dims' {rot_dims} must be even and at most dim ({dim})")
    scaling = _part(rot, "scaling", where)
    bands = None
    if scaling and rot_dims:
        inside = where + ".mixer.rot.scaling"
        bands = MalalixBands(**{key: require_number(scaling, key, inside)
                                for key in ("factor", "low", "high", "original")})
    return MalalixAttention(
        heads=heads, kv_heads=kv_heads, dim=dim, vdim=require_int(mixer, "vdim", default=dim),
        scale=require_number(mixer, "scale", where + ".mixer"), chunk=chunk, rot_dims=rot_dims,
        rot_base=require_number(rot, "base", where + ".mixer.rot") if rot_dims else 0.0, bands=bands)


def _read_feed_forward(mlp, where):
    if mlp is None:
        return None
    if not isinstance(mlp, dict) or mlp.get("kind", "moe") != "moe":
        raise ConfigError(f"config.json {where} 'mlp.kind' must be 'moe', got {mlp!r}")
    expert, router = _part(mlp, "expert", where), _part(mlp, "router", where)
    if expert is None or router is None:
        raise ConfigError(f"config.json {where} 'mlp' needs 'expert' and 'router'")
    experts = require_int(router, "experts")
    top = require_int(router, "top")
    if top > experts:
        raise ConfigError(f"'router.top' {top} exceeds the {experts} experts")
    shared = _part(mlp, "shared", where)
    return MalalixExperts(
        ff=require_int(expert, "ff"), limit=require_number(expert, "limit", where + ".mlp.expert"),
        experts=experts, top=top, shared_ff=require_int(shared, "ff") if shared else 0,
        shared_limit=require_number(shared, "limit", where + ".mlp.shared") if shared else 0.0)


@dataclass(frozen=True)
class MalalixConfig:
    vocab: int
    width: int
    layers: Tuple[MalalixLayer, ...]
    norm_eps: float
    loop_start: int            # layers loop_start .. loop_stop - 1 run loop_times times in a row
    loop_stop: int
    loop_times: int            # 0: no loop
    max_positions: int

    architecture = "Malalix"
    eos_token_id = None        # the configuration names no token that ends a request
    # where the file names no bound, requests may grow to this many tokens (an engine's pool or
    # its own bound may be smaller)
    DEFAULT_MAX_POSITIONS = 32768

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @classmethod
    def from_dict(cls, raw) -> "MalalixConfig":
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json 'layers' must be a non-empty list")
        layers = []
        for index, entry in enumerate(listed):
            where = f"layers[{index}]"
            if not isinstance(entry, dict) or entry.get("type") not in MIXERS:
                raise ConfigError(f"config.json {where} 'type' must be one of {', '.join(MIXERS)}, "
                                  f"got {entry.get('type') if isinstance(entry, dict) else entry!r}")
            if not isinstance(entry.get("mixer"), dict):
                raise ConfigError(f"config.json {where} lacks 'mixer'")
            try:
                layers.append(MalalixLayer(entry["type"], _read_mixer(entry["mixer"], where),
                                           _read_feed_forward(entry.get("mlp"), where)))
            except ConfigError as error:
                raise ConfigError(f"{where}: {error}") from None
        loop = _part(raw, "loop", "")
        start = stop = times = 0
        if loop is not None:
            start = require_int(loop, "start", minimum=0)
            stop = require_int(loop, "stop")
            times = require_int(loop, "times")
            if not start < stop <= len(layers):
                raise ConfigError(f"config.json 'loop' {start}..{stop} does not lie within the "
                                  f"{len(layers)} layers")
        return cls(
            vocab=require_int(raw, "vocab"),
            width=require_int(raw, "width"),
            layers=tuple(layers),
            norm_eps=require_number(raw.get("norm") or {}, "eps", "norm"),
            loop_start=start, loop_stop=stop, loop_times=times,
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
        if self.loop_times:
            out["loop"] = {"start": self.loop_start, "stop": self.loop_stop, "times": self.loop_times}
        if self.max_positions != self.DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        return out

    def run_order(self):
        """(layer, number of the pass that this call opens or -1) for every call, in order."""
        order = [(index, -1) for index in range(self.loop_start)]
        for turn in range(self.loop_times):
            order += [(index, turn if index == self.loop_start else -1)
                      for index in range(self.loop_start, self.loop_stop)]
        return order + [(index, -1) for index in range(self.loop_stop, len(self.layers))]
