"""Small Malalix configurations for the tests: sizes, head counts, chunk sizes, layer orders, loops
and constants that differ from each other in every respect, and folders with random weights."""

import json
import os

import torch

import plain_malalix


def _rot(dims, base, scaling=None):
    out = {"dims": dims, "base": base}
    if scaling:
        out["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def _layer(heads, kv_heads, dim, vdim, scale, size=None, rot=None, mlp=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        mixer["mask"] = {"size": size}
    if rot is not None:
        mixer["rot"] = rot
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def _moe(ff, limit, experts, top, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


# grouped heads, values wider than keys, chunks of two pages, layers with other chunk sizes beside
# them, three passes over the middle layers, shared experts of other widths and limits
MODEL_A = {
    "architecture": "Malalix", "vocab": 97, "width": 64, "norm": {"eps": 1e-5},
    "loop": {"start": 1, "stop": 3, "times": 3},
    "layers": [_layer(4, 2, 16, 24, 0.3, 16, _rot(8, 100.0, (4.0, 1.0, 3.0, 40)), _moe(24, 1.2, 6, 2, (40, 2.5))),
               _layer(4, 2, 16, 24, 0.25, 9, _rot(16, 500.0), _moe(16, 0.8, 5, 3, (16, 0.7))),
               _layer(4, 2, 16, 24, 0.35, 16, _rot(8, 100.0, (4.0, 1.0, 3.0, 40)), _moe(24, 3.0, 6, 1)),
               _layer(2, 1, 8, 8, 0.5, 21, _rot(4, 30.0), None)],
}
# sizes that are multiples of nothing, a chunk of one token (a query sees itself only), no
# rotation, every expert chosen, no loop
MODEL_B = {
    "architecture": "Malalix", "vocab": 131, "width": 40, "norm": {"eps": 1e-6},
    "layers": [_layer(3, 3, 12, 20, 0.4, 7, _rot(6, 50.0), _moe(10, 1.5, 4, 4, (9, 1.0))),
               _layer(3, 1, 10, 10, 0.3, 1, None, _moe(13, 2.0, 3, 2)),
               _layer(5, 1, 6, 3, 0.6, 13, _rot(2, 10.0, (8.0, 0.5, 2.0, 12)), None)],
}
# sizes that the matrix-core kernels take as they are: eight heads on one key/value head, chunks of
# whole pages, more experts than a wave has lanes, a loop over everything
MODEL_C = {
    "architecture": "Malalix", "vocab": 256, "width": 128, "norm": {"eps": 1e-6},
    "loop": {"start": 0, "stop": 2, "times": 2},
    "layers": [_layer(8, 1, 64, 32, 0.125, 48, _rot(32, 10000.0, (8.0, 1.0, 4.0, 64)), _moe(32, 1.5, 72, 5, (64, 2.0))),
               _layer(4, 2, 64, 64, 0.11, 32, _rot(64, 150000.0), _moe(64, 1.0, 8, 2, (32, 1.2)))],
}
# heads of 128 without a mask beside a chunked layer, a single pass as a loop of the last layers
# that begins with a layer without a feed-forward
MODEL_D = {
    "architecture": "Malalix", "vocab": 77, "width": 72, "norm": {"eps": 1e-5},
    "loop": {"start": 1, "stop": 3, "times": 1},
    "layers": [_layer(2, 2, 128, 128, 0.09, None, _rot(128, 1000.0, (2.0, 1.0, 8.0, 100)), _moe(40, 2.0, 5, 2, (24, 1.5))),
               _layer(2, 1, 32, 32, 0.2, 40, _rot(10, 80.0), None),
               _layer(6, 2, 20, 40, 0.25, 100, _rot(20, 200.0), _moe(8, 0.5, 3, 1, (48, 4.0)))],
}
# a loop that begins with a layer without a feed-forward and ends the model: the launch that adds
# the embedding and the pass vector stands alone; heads cached 144 wide; rotation of two dimensions
MODEL_E = {
    "architecture": "Malalix", "vocab": 53, "width": 48, "norm": {"eps": 1e-4},
    "loop": {"start": 1, "stop": 3, "times": 4},
    "layers": [_layer(2, 1, 136, 40, 0.1, 10, _rot(2, 7.0), _moe(8, 1.0, 2, 1, (8, 1.0))),
               _layer(6, 1, 8, 40, 0.4, 4, _rot(8, 60.0, (3.0, 2.0, 2.5, 30)), None),
               _layer(1, 1, 24, 16, 0.3, 30, _rot(12, 90.0), _moe(8, 1.7, 9, 4, (32, 0.9)))],
}

# name -> (configuration, page size, seed)
MODELS = {"A": (MODEL_A, 8, 0), "B": (MODEL_B, 16, 1), "C": (MODEL_C, 16, 2), "D": (MODEL_D, 4, 3),
          "E": (MODEL_E, 8, 4)}


def write_folder(folder, raw, tensors):
    """Store a checkpoint as this design's are stored (bfloat16) and return the values as stored."""
    from safetensors.torch import save_file

    stored = {name: tensor.to(torch.bfloat16).contiguous() for name, tensor in tensors.items()}
    os.makedirs(folder, exist_ok=True)
    save_file(stored, os.path.join(folder, "model.safetensors"))
    with open(os.path.join(folder, "config.json"), "w") as handle:
        json.dump(raw, handle)
    return {name: tensor.to(torch.float64) for name, tensor in stored.items()}


def folder_of(tmp_path, which):
    """(folder, raw configuration, checkpoint tensors as stored in float64, page size)."""
    raw, page_size, seed = MODELS[which]
    folder = os.path.join(str(tmp_path), f"malalix_{which}")
    return folder, raw, write_folder(folder, raw, plain_malalix.random_checkpoint(raw, seed)), page_size


def without_close_calls(raw, weights, seed):
    """The checkpoint with routers whose choice no rounding can turn: four columns of the stream,
    which only the embedding writes, sort the tokens into four classes; a router ranks the experts
    anew for each class, a whole unit apart, with little beside that.  (A close call goes one way in
    float64 and the other in bfloat16, and the position is then off by a whole expert.)"""
    g = torch.Generator().manual_seed(seed)
    marks = torch.eye(4)[torch.randint(0, 4, (raw["vocab"],), generator=g)] * 2.0
    out = dict(weights)
    for name, tensor in weights.items():
        tensor = tensor.clone()
        if name.endswith("mlp.router"):
            tensor *= 0.02
            for column in range(4):
                tensor[:, column] = torch.randperm(tensor.shape[0], generator=g).float()
        elif name.endswith(".down") or name.endswith("mix.o"):
            tensor[:4] = 0
        elif name == "embed":
            tensor[:, :4] = marks
        elif name == "loop.step":
            tensor[:, :4] = 0
        elif name.endswith("norm2"):
            tensor[:4] = 1.0
        out[name] = tensor
    return out


def folder_for(tmp_path, which, dtype):
    """``folder_of``, for a bfloat16 engine with routers that make no close calls."""
    if dtype != "bfloat16":
        return folder_of(tmp_path, which)
    raw, page_size, seed = MODELS[which]
    weights = without_close_calls(raw, plain_malalix.random_checkpoint(raw, seed), seed)
    folder = os.path.join(str(tmp_path), f"malalix_{which}_sure")
    return folder, raw, write_folder(folder, raw, weights), page_size


LOUD, ASK = 1, 2      # tokens of the model below


def loud_key_model(tmp_path, size, heads=2, kv_heads=1, dim=16, sure=False):
    """Two layers, passed twice, in which one pair of tokens stands out: column 0 of the stream
    marks LOUD and column 1 marks ASK (nothing else writes these columns), every key has LOUD's
    mark in its last dimension and every query ASK's, so that an ASK gives nearly all its weight to a
    LOUD in its own chunk of ``size`` positions.  The second layer's chunks are 3 positions longer.
    ``sure``: with routers that make no close calls.  Returns (folder, raw, tensors)."""
    layers = [_layer(heads, kv_heads, dim, dim, 0.25, size, _rot(dim // 2, 40.0), _moe(24, 1.5, 4, 2, (16, 1.0))),
              _layer(heads, kv_heads, dim, dim, 0.25, size + 3, _rot(dim // 2, 40.0, (4.0, 1.0, 3.0, 40)), None)]
    raw = {"architecture": "Malalix", "vocab": 50, "width": 64, "norm": {"eps": 1e-5},
           "loop": {"start": 0, "stop": 2, "times": 2}, "layers": layers}
    w = plain_malalix.random_checkpoint(raw, 17)
    if sure:
        w = without_close_calls(raw, w, 17)
        for name in w:      # (their columns become 4 to 7: 0 and 1 are the marks here)
            if name.endswith("mlp.router") or name in ("embed", "loop.step"):
                w[name] = w[name].roll(4, 1)
            elif name.endswith(".down") or name.endswith("mix.o") or name.endswith("norm2"):
                w[name] = w[name].roll(4, 0)
    w["embed"][:, :2] = 0
    w["embed"][LOUD, 0] = 12.0
    w["embed"][ASK, 1] = 12.0
    w["loop.step"][:, :2] = 0
    for i in range(2):
        p = f"l{i}."
        for name in [n for n in w if n.startswith(p) and (n.endswith(".down") or n.endswith("mix.o"))]:
            w[name][:2] = 0
        w[p + "norm1"][:2] = 1.0
        for name, count, column in (("q", heads, 1), ("k", kv_heads, 0)):
            rows = w[p + "mix." + name].view(count, dim, -1)
            rows[:, :, :2] = 0
            rows[:, dim - 1] = 0
            rows[:, dim - 1, column] = 6.0
            w[p + f"mix.{name}.b"].view(count, dim)[:, dim - 1] = 0
            w[p + f"mix.{name}.norm"][dim - 1] = 3.0
        w[p + "mix.v"][:, 0] = 2.0
    folder = os.path.join(str(tmp_path), f"malalix_loud_{size}_{heads}_{int(sure)}")
    return folder, raw, write_folder(folder, raw, w)
