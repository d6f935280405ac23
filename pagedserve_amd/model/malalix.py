"""Malalix as data: a decoder whose layers are listed one by one in its configuration.

A layer norms the stream twice (RMS norms with scales of their own, of the same stream) and adds its
mixer of the one and its feed-forward of the other: attention with grouped heads, biases on its
projections, a norm per query and key head ahead of the rotation, frequencies stretched by
wavelength, and no look beyond the query's own chunk of positions; and a mixture of experts with a
capped gated unit, weights by the softmax over the chosen logits, beside a shared expert with a gate
of its own.  A run of layers may be passed several times with the same weights; every pass keeps
caches of its own, begins by adding a learned vector to the stream, and every pass but the first
adds the embedded tokens again before that.  The final norm is followed by a head matrix.
"""

import math

import torch

from ..config.malalix import MalalixConfig
from ..config.registry import Architecture, register_architecture
from ..config.spec import BlockSpec, LayerCall, ModelSpec, PartSpec
from ..weights.loader import WeightSource

# the experts' gated unit: g sigmoid(1.702 g) (u + 1) of a capped g and u
GATE_SLOPE, GATE_SHIFT = 1.702, 1.0
# heads are cached with their size rounded up to this, so that the tiled kernels take every size
HEAD_PADDING = 16


def _mixer_spec(config, mixer):
    bands = mixer.bands
    return PartSpec.make(
        "attention", heads=mixer.heads, kv_heads=mixer.kv_heads, head_dim=mixer.dim,
        value_dim=mixer.vdim, scale=mixer.scale, chunk=mixer.chunk, bias=True, out_bias=False,
        head_norm="before", norm_eps=config.norm_eps, rotary_dims=mixer.rot_dims,
        rotary_base=mixer.rot_base, rotary_layout="halves",
        rotary_bands=None if bands is None else (bands.factor, bands.low, bands.high, bands.original),
        pad_heads=HEAD_PADDING)


def _feed_forward_spec(mlp):
    return PartSpec.make(
        "moe", inner=mlp.ff, experts=mlp.experts, top=mlp.top, score="chosen_softmax",
        gate_form=(mlp.limit, GATE_SLOPE, GATE_SHIFT), shared_inner=mlp.shared_ff,
        shared_limit=mlp.shared_limit if mlp.shared_ff else None, shared_gate=mlp.shared_ff > 0)


def build_spec(config: MalalixConfig) -> ModelSpec:
    norm = PartSpec.make("rmsnorm", eps=config.norm_eps)
    blocks = []
    for layer in config.layers:
        parts = {"norm1": norm, "mixer": _mixer_spec(config, layer.mixer)}
        arrangement = "pre_norm_mixer"
        if layer.mlp is not None:
            parts.update(norm2=norm, feed_forward=_feed_forward_spec(layer.mlp))
            arrangement = "parallel_two_norms"
        blocks.append(BlockSpec.make(arrangement, **parts))
    # every call of the run order keeps a cache entry of its own: a layer that is passed again
    # shares its weights with the earlier pass, nothing else
    schedule = tuple(LayerCall(block=layer, cache=index, enter=turn, add_embedding=turn > 0)
                     for index, (layer, turn) in enumerate(config.run_order()))
    return ModelSpec(
        architecture=config.architecture,
        vocab_size=config.vocab,
        width=config.width,
        max_positions=config.max_positions,
        position=PartSpec.make("none"),
        blocks=tuple(blocks),
        schedule=schedule,
        final_norm=norm,
        tie_head=False,
        eos_token_id=None,
        embedding=PartSpec.make("lookup"),
        head=PartSpec.make("linear", bias=False),
        pass_rows=config.loop_times,
    )


def _expert_names(prefix, experts, pieces):
    return tuple(f"{prefix}e{e}.{piece}" for e in range(experts) for piece in pieces)


def weight_sources(config: MalalixConfig, spec: ModelSpec):
    """Parameter path -> checkpoint tensor(s).  Matrices are stored ``[out, in]``; projections
    that read the same input are joined into one packed product, the experts' matrices are
    stacked one behind the other."""
    sources = {
        "embedding.table": WeightSource("embed"),
        "final_norm.gamma": WeightSource("final.norm"),
        "head.weight": WeightSource("head"),
    }
    if config.loop_times:
        sources["pass_table"] = WeightSource("loop.step")
    for i, layer in enumerate(config.layers):
        b, l = f"blocks.{i}.", f"l{i}."
        m, f = l + "mix.", l + "mlp."
        sources[b + "norm1.gamma"] = WeightSource(l + "norm1")
        sources[b + "mixer.qkv.weight"] = WeightSource((m + "q", m + "k", m + "v"))
        sources[b + "mixer.qkv.bias"] = WeightSource((m + "q.b", m + "k.b", m + "v.b"))
        sources[b + "mixer.q_norm.gamma"] = WeightSource(m + "q.norm")
        sources[b + "mixer.k_norm.gamma"] = WeightSource(m + "k.norm")
        sources[b + "mixer.out.weight"] = WeightSource(m + "o")
        if layer.mlp is None:
            continue
        sources[b + "norm2.gamma"] = WeightSource(l + "norm2")
        sources[b + "feed_forward.router.weight"] = WeightSource(f + "router")
        sources[b + "feed_forward.gate_up.weight"] = WeightSource(
            _expert_names(f, layer.mlp.experts, ("gate", "up")))
        sources[b + "feed_forward.down.weight"] = WeightSource(_expert_names(f, layer.mlp.experts, ("down",)))
        if layer.mlp.shared_ff:
            s = f + "shared."
            sources[b + "feed_forward.shared.gate_up.weight"] = WeightSource((s + "gate", s + "up"))
            sources[b + "feed_forward.shared.down.weight"] = WeightSource(s + "down")
            sources[b + "feed_forward.shared_gate.weight"] = WeightSource(s + "sg")
    return sources


def complete_raw(raw: dict, shape_of) -> dict:
    """The raw configuration with the sizes that it leaves out filled in from the shapes of the
    stored tensors (``shape_of(name)``: the shape, or None where the file has no such tensor).  A
    size that the file names is never touched; one that no tensor gives stays out, and the typed
    reader then reports it."""
    import copy

    raw = copy.deepcopy(raw)

    def rows(name, axis=0):
        shape = shape_of(name)
        return None if shape is None or len(shape) <= axis else int(shape[axis])

    def fill(target, key, value):
        if isinstance(target, dict) and target.get(key) is None and value is not None and value > 0:
            target[key] = int(value)

    def ratio(a, b):
        return a // b if a is not None and b and a % b == 0 else None

    fill(raw, "vocab", rows("embed"))
    fill(raw, "width", rows("embed", 1))
    fill(raw.get("loop"), "times", rows("loop.step"))
    listed = raw.get("layers")
    for index, layer in enumerate(listed if isinstance(listed, list) else []):
        if not isinstance(layer, dict) or not isinstance(layer.get("mixer"), dict):
            continue
        m, p, f = layer["mixer"], f"l{index}.mix.", f"l{index}.mlp."
        fill(m, "dim", rows(p + "q.norm"))
        fill(m, "heads", ratio(rows(p + "q"), m.get("dim")))
        fill(m, "kv_heads", ratio(rows(p + "k"), m.get("dim")))
        fill(m, "vdim", ratio(rows(p + "v"), m.get("kv_heads")))
        mlp = layer.get("mlp")
        if isinstance(mlp, dict):
            fill(mlp.get("expert"), "ff", rows(f + "e0.gate"))
            fill(mlp.get("router"), "experts", rows(f + "router"))
            fill(mlp.get("shared"), "ff", rows(f + "shared.gate"))
    return raw


def random_tensors(config: MalalixConfig, seed: int, device="cpu"):
    """Checkpoint tensors of a random model, drawn from one seeded generator in a fixed order.
    Matrices N(0, 1/sqrt(in)); scales, biases and gates such that every part matters in the
    output."""
    generator = torch.Generator(device=device).manual_seed(int(seed))

    def normal(shape, std=1.0):
        return torch.randn(shape, generator=generator, dtype=torch.float32, device=device) * std

    def matrix(rows, columns, gain=1.0):
        return normal((rows, columns), gain / math.sqrt(columns))

    d = config.width
    tensors = {"embed": normal((config.vocab, d))}
    if config.loop_times:
        tensors["loop.step"] = normal((config.loop_times, d), 0.3)
    for i, layer in enumerate(config.layers):
        l, m, f = f"l{i}.", f"l{i}.mix.", f"l{i}.mlp."
        mixer = layer.mixer
        tensors[l + "norm1"] = 1.0 + normal((d,), 0.1)
        for name, count in (("q", mixer.heads * mixer.dim), ("k", mixer.kv_heads * mixer.dim),
                            ("v", mixer.kv_heads * mixer.vdim)):
            tensors[m + name] = matrix(count, d)
            tensors[m + name + ".b"] = normal((count,), 0.1)
        tensors[m + "q.norm"] = 1.0 + normal((mixer.dim,), 0.1)
        tensors[m + "k.norm"] = 1.0 + normal((mixer.dim,), 0.1)
        tensors[m + "o"] = matrix(d, mixer.heads * mixer.vdim)
        mlp = layer.mlp
        if mlp is None:
            continue
        tensors[l + "norm2"] = 1.0 + normal((d,), 0.1)
        names = [(f"e{e}.", mlp.ff) for e in range(mlp.experts)]
        if mlp.shared_ff:
            names.append(("shared.", mlp.shared_ff))
            tensors[f + "shared.sg"] = matrix(1, d)
        for name, ff in names:
            tensors[f + name + "gate"] = matrix(ff, d)
            tensors[f + name + "up"] = matrix(ff, d)
            tensors[f + name + "down"] = matrix(d, ff)
        tensors[f + "router"] = matrix(mlp.experts, d, 2.0)
    tensors["final.norm"] = 1.0 + normal((d,), 0.1)
    tensors["head"] = matrix(config.vocab, d)
    return tensors


MALALIX = register_architecture(Architecture(
    name="Malalix",
    config_class=MalalixConfig,
    build_spec=build_spec,
    weight_sources=weight_sources,
    random_tensors=random_tensors,
    complete_raw=complete_raw,
    model_type="malalix",
))
