"""Fadosun as data: a decoder whose layers are listed one by one in its configuration.

Every sublayer stands between two layer norms (scale and shift), and a gate made from its input
multiplies its result ahead of the second one.  The mixer is a gated delta rule with a decay per key
channel, a matrix memory with exponential gates, or attention without a softmax (rotated heads, each
visible key weighed by a sigmoid of its own) joined with a state-space mixer of one decay per head; the
feed-forward is a gated dense one with a relu, or absent.  The final norm is followed by a head matrix.
"""

import math

import torch

from ..config.fadosun import FadosunConfig
from ..config.registry import Architecture, register_architecture
from ..config.spec import BlockSpec, LayerCall, ModelSpec, PartSpec
from ..weights.loader import WeightSource

# heads are cached with their size rounded up to this, so that the tiled kernels take every size
HEAD_PADDING = 16


def _mixer_spec(config, layer):
    mixer, eps, ride = layer.mixer, config.norm_eps, config.width
    if layer.type == "channel_delta":
        return PartSpec.make("channel_delta", heads=mixer.heads, key_heads=mixer.kv_heads, key_dim=mixer.dim,
                             value_dim=mixer.vdim, taps=mixer.conv, decay_rank=mixer.decay_rank,
                             gate_rank=mixer.gate_rank, norm_eps=eps, ride=ride)
    if layer.type == "mlstm":
        return PartSpec.make("matrix_memory", heads=mixer.heads, key_dim=mixer.dim, value_dim=mixer.vdim,
                             gate_cap=mixer.gate_cap, norm_eps=eps, ride=ride)
    left, right = mixer.left, mixer.right
    attention = PartSpec.make(
        "attention", heads=left.heads, kv_heads=left.kv_heads, head_dim=left.dim, value_dim=left.vdim,
        scale=left.scale, bias=False, rotary_dims=left.rot_dims, rotary_base=left.rot_base,
        rotary_layout="halves", logistic=True, out_scale=mixer.left_scale, pad_heads=HEAD_PADDING)
    space = PartSpec.make("head_state_space", heads=right.heads, value_dim=right.vdim, states=right.state,
                          groups=right.groups, taps=right.conv, norm_groups=right.norm_groups, norm_eps=eps,
                          out_scale=mixer.right_scale)
    return PartSpec.make("joined", left=attention, right=space, ride=ride)


def build_spec(config: FadosunConfig) -> ModelSpec:
    norm = PartSpec.make("layernorm", eps=config.norm_eps)
    gate = PartSpec.make("ridden_gate")
    blocks = []
    for layer in config.layers:
        parts = {"norm1": norm, "mixer": _mixer_spec(config, layer), "gate1": gate, "post1": norm}
        arrangement = "gated_between_norms_mixer"
        if layer.ff is not None:
            parts.update(norm2=norm, gate2=gate, post2=norm, feed_forward=PartSpec.make(
                "gated", inner=layer.ff, activation="relu", ride=config.width))
            arrangement = "gated_between_norms"
        blocks.append(BlockSpec.make(arrangement, **parts))
    return ModelSpec(
        architecture=config.architecture,
        vocab_size=config.vocab,
        width=config.width,
        max_positions=config.max_positions,
        position=PartSpec.make("none"),
        blocks=tuple(blocks),
        schedule=tuple(LayerCall(block=index, cache=index) for index in range(len(blocks))),
        final_norm=norm,
        tie_head=False,
        eos_token_id=None,
        embedding=PartSpec.make("lookup"),
        head=PartSpec.make("linear", bias=False),
    )


def weight_sources(config: FadosunConfig, spec: ModelSpec):
    """Parameter path -> checkpoint tensor(s).  Matrices are stored ``[out, in]``; projections that read the
    same input are joined into one packed product, the gate on the sublayer's result among them; output
    matrices of joined mixers stand side by side."""
    sources = {
        "embedding.table": WeightSource("embed"),
        "final_norm.gamma": WeightSource("final.norm"),
        "final_norm.beta": WeightSource("final.norm.b"),
        "head.weight": WeightSource("head"),
    }

    def norms_and_gate(b, l, number):
        for path, name in ((f"norm{number}", f"norm{number}"), (f"post{number}", f"norm{number}b")):
            sources[b + path + ".gamma"] = WeightSource(l + name)
            sources[b + path + ".beta"] = WeightSource(l + name + ".b")
        sources[f"{b}gate{number}.bias"] = WeightSource(f"{l}rg{number}.b")

    for i, layer in enumerate(config.layers):
        b, l = f"blocks.{i}.", f"l{i}."
        m, p = l + "mix.", b + "mixer."
        norms_and_gate(b, l, 1)
        ride = l + "rg1"
        if layer.type == "channel_delta":
            sources[p + "in.weight"] = WeightSource(tuple(m + n for n in ("q", "k", "v", "a1", "g1", "b")) + (ride,))
            sources[p + "conv.weight"] = WeightSource((m + "q.conv", m + "k.conv", m + "v.conv"))
            sources[p + "decay.weight"] = WeightSource(m + "a2")
            sources[p + "decay.bias"] = WeightSource(m + "dt_bias")
            sources[p + "decay.log"] = WeightSource(m + "A_log")
            sources[p + "gate.weight"] = WeightSource(m + "g2")
            sources[p + "norm.gamma"] = WeightSource(m + "norm")
            sources[p + "out.weight"] = WeightSource(m + "o")
        elif layer.type == "mlstm":
            sources[p + "in.weight"] = WeightSource(tuple(m + n for n in ("q", "k", "v", "g", "i", "f")) + (ride,))
            sources[p + "input_gate.bias"] = WeightSource(m + "i.b")
            sources[p + "forget_gate.bias"] = WeightSource(m + "f.b")
            sources[p + "norm.gamma"] = WeightSource(m + "norm")
            sources[p + "out.weight"] = WeightSource(m + "o")
        else:
            a, s = m + "left.", m + "right."
            sources[p + "in.weight"] = WeightSource((a + "q", a + "k", a + "v", s + "in", ride))
            sources[p + "out.weight"] = WeightSource((a + "o", s + "o"), axis=1)
            sources[p + "left.logistic.shift"] = WeightSource(a + "pb")
            sources[p + "right.conv.weight"] = WeightSource(s + "conv")
            sources[p + "right.conv.bias"] = WeightSource(s + "conv.b")
            sources[p + "right.step.bias"] = WeightSource(s + "dt_bias")
            sources[p + "right.decay.log"] = WeightSource(s + "A_log")
            sources[p + "right.skip"] = WeightSource(s + "D")
            sources[p + "right.norm.gamma"] = WeightSource(s + "norm")
        if layer.ff is None:
            continue
        norms_and_gate(b, l, 2)
        f = l + "mlp."
        sources[b + "feed_forward.gate_up.weight"] = WeightSource((f + "gate", f + "up", l + "rg2"))
        sources[b + "feed_forward.down.weight"] = WeightSource(f + "down")
    return sources


def complete_raw(raw: dict, shape_of) -> dict:
    """The raw configuration with the sizes that it leaves out filled in from the shapes of the stored tensors
    (``shape_of(name)``: the shape, or None where the file has no such tensor).  A size that the file
    names is never touched; one that no tensor gives stays out, and the typed reader then reports it."""
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
    listed = raw.get("layers")
    for index, layer in enumerate(listed if isinstance(listed, list) else []):
        if not isinstance(layer, dict) or not isinstance(layer.get("mixer"), dict):
            continue
        m, p = layer["mixer"], f"l{index}.mix."
        if isinstance(layer.get("mlp"), dict):
            fill(layer["mlp"], "ff", rows(f"l{index}.mlp.gate"))
        if layer.get("type") == "channel_delta":
            fill(m, "decay_rank", rows(p + "a1"))
            fill(m, "gate_rank", rows(p + "g1"))
            fill(m, "heads", rows(p + "A_log"))
            fill(m, "vdim", rows(p + "norm"))
            fill(m, "dim", ratio(rows(p + "dt_bias"), m.get("heads")))
            fill(m, "kv_heads", ratio(rows(p + "q"), m.get("dim")))
            fill(m, "conv", rows(p + "q.conv", 1))
        elif layer.get("type") == "mlstm":
            fill(m, "heads", rows(p + "i.b"))
            fill(m, "dim", ratio(rows(p + "q"), m.get("heads")))
            fill(m, "vdim", ratio(rows(p + "v"), m.get("heads")))
        elif layer.get("type") == "parallel":
            left, right = m.get("left"), m.get("right")
            if isinstance(left, dict):
                fill(left, "heads", rows(p + "left.pb"))
                fill(left, "dim", ratio(rows(p + "left.q"), left.get("heads")))
                fill(left, "kv_heads", ratio(rows(p + "left.k"), left.get("dim")))
                fill(left, "vdim", ratio(rows(p + "left.v"), left.get("kv_heads")))
            if isinstance(right, dict):
                fill(right, "heads", rows(p + "right.A_log"))
                fill(right, "vdim", ratio(rows(p + "right.norm"), right.get("heads")))
                fill(right, "conv", rows(p + "right.conv", 1))
    return raw


def random_tensors(config: FadosunConfig, seed: int, device="cpu"):
    """Checkpoint tensors of a random model, drawn from one seeded generator in a fixed order.  Matrices
    N(0, 1/sqrt(in)); scales, shifts, decays and gates such that every part matters in the output and the
    recurrences neither die nor blow up."""
    generator = torch.Generator(device=device).manual_seed(int(seed))

    def normal(shape, std=1.0):
        return torch.randn(shape, generator=generator, dtype=torch.float32, device=device) * std

    def uniform(shape, low, high):
        return torch.rand(shape, generator=generator, dtype=torch.float32, device=device) * (high - low) + low

    def matrix(rows, columns, gain=1.0):
        return normal((rows, columns), gain / math.sqrt(columns))

    def steps(count):
        # softplus^-1 of step sizes between 0.001 and 0.1, log-uniform
        size = torch.exp(uniform((count,), math.log(1e-3), math.log(1e-1)))
        return size + torch.log(-torch.expm1(-size))

    d = config.width
    tensors = {"embed": normal((config.vocab, d))}

    def norm(name):
        tensors[name] = 1.0 + normal((d,), 0.1)
        tensors[name + ".b"] = normal((d,), 0.1)

    for i, layer in enumerate(config.layers):
        l, m = f"l{i}.", f"l{i}.mix."
        mixer = layer.mixer
        for number in (1, 2) if layer.ff is not None else (1,):
            norm(f"{l}norm{number}")
            norm(f"{l}norm{number}b")
            tensors[f"{l}rg{number}"] = matrix(d, d)
            tensors[f"{l}rg{number}.b"] = normal((d,), 0.5)
        if layer.type == "channel_delta":
            for name, count in (("q", mixer.kv_heads * mixer.dim), ("k", mixer.kv_heads * mixer.dim),
                                ("v", mixer.heads * mixer.vdim)):
                tensors[m + name] = matrix(count, d)
                tensors[m + name + ".conv"] = normal((count, mixer.conv), 1.0 / math.sqrt(mixer.conv))
            tensors[m + "b"] = matrix(mixer.heads, d)
            tensors[m + "A_log"] = torch.log(uniform((mixer.heads,), 1.0, 8.0))
            tensors[m + "norm"] = 1.0 + normal((mixer.vdim,), 0.1)
            tensors[m + "a1"] = matrix(mixer.decay_rank, d)
            tensors[m + "a2"] = matrix(mixer.heads * mixer.dim, mixer.decay_rank)
            tensors[m + "dt_bias"] = steps(mixer.heads * mixer.dim)
            tensors[m + "g1"] = matrix(mixer.gate_rank, d)
            tensors[m + "g2"] = matrix(mixer.heads * mixer.vdim, mixer.gate_rank)
            tensors[m + "o"] = matrix(d, mixer.heads * mixer.vdim)
        elif layer.type == "mlstm":
            for name, count in (("q", mixer.heads * mixer.dim), ("k", mixer.heads * mixer.dim),
                                ("v", mixer.heads * mixer.vdim), ("g", mixer.heads * mixer.vdim),
                                ("i", mixer.heads), ("f", mixer.heads)):
                tensors[m + name] = matrix(count, d)
            tensors[m + "i.b"] = normal((mixer.heads,), 1.0)
            tensors[m + "f.b"] = uniform((mixer.heads,), 3.0, 6.0)
            tensors[m + "norm"] = 1.0 + normal((mixer.heads * mixer.vdim,), 0.1)
            tensors[m + "o"] = matrix(d, mixer.heads * mixer.vdim)
        else:
            left, right = mixer.left, mixer.right
            a, s = m + "left.", m + "right."
            tensors[a + "q"] = matrix(left.heads * left.dim, d)
            tensors[a + "k"] = matrix(left.kv_heads * left.dim, d)
            tensors[a + "v"] = matrix(left.kv_heads * left.vdim, d)
            tensors[a + "pb"] = normal((left.heads,), 1.0) - 4.0
            tensors[a + "o"] = matrix(d, left.heads * left.vdim)
            inner = right.heads * right.vdim
            channels = inner + 2 * right.groups * right.state
            tensors[s + "in"] = matrix(inner + channels + right.heads, d)
            tensors[s + "conv"] = normal((channels, right.conv), 1.0 / math.sqrt(right.conv))
            tensors[s + "conv.b"] = normal((channels,), 0.1)
            tensors[s + "dt_bias"] = steps(right.heads)
            tensors[s + "A_log"] = torch.log(uniform((right.heads,), 1.0, 16.0))
            tensors[s + "D"] = 1.0 + normal((right.heads,), 0.1)
            tensors[s + "norm"] = 1.0 + normal((inner,), 0.1)
            tensors[s + "o"] = matrix(d, inner)
        if layer.ff is not None:
            f = l + "mlp."
            tensors[f + "gate"] = matrix(layer.ff, d)
            tensors[f + "up"] = matrix(layer.ff, d)
            tensors[f + "down"] = matrix(d, layer.ff)
    norm("final.norm")
    tensors["head"] = matrix(config.vocab, d)
    return tensors


FADOSUN = register_architecture(Architecture(
    name="Fadosun",
    config_class=FadosunConfig,
    build_spec=build_spec,
    weight_sources=weight_sources,
    random_tensors=random_tensors,
    complete_raw=complete_raw,
    model_type="fadosun",
))
