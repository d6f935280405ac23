"""Small Fadosun configurations for the tests: sizes, head counts, layer orders and constants that differ
from each other in every respect, and folders with random weights."""

import json
import os

import torch

import plain_fadosun


def _delta(heads, kv_heads, dim, vdim, conv, ff, **more):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, **more}
    return {"type": "channel_delta", "mixer": mixer, "mlp": _dense(ff)}


def _memory(heads, dim, vdim, cap, ff):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": _dense(ff)}


def _parallel(left, right, scales, ff):
    heads, kv_heads, dim, vdim, scale, rot = left
    a = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot is not None:
        a["rot"] = {"dims": rot[0], "base": rot[1]}
    s = dict(zip(("heads", "vdim", "state", "groups", "conv", "norm_groups"), right))
    return {"type": "parallel", "mlp": _dense(ff),
            "mixer": {"left": a, "right": s, "left_scale": scales[0], "right_scale": scales[1]}}


def _dense(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def _model(vocab, width, eps, *layers):
    return {"architecture": "Fadosun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": list(layers)}


# every mixer once; heads that share keys, values wider than keys and narrower, a layer without a
# feed-forward in the middle
MODEL_A = _model(97, 64, 1e-5,
                 _delta(4, 2, 16, 24, 4, 96),
                 _parallel((4, 2, 16, 32, 0.3, (8, 1000.0)), (6, 8, 12, 3, 3, 2), (0.7, 1.3), None),
                 _memory(2, 20, 12, 6.0, 72))
# sizes that are multiples of nothing, convolutions of one, two and five taps, one head, no rotation, a
# negative factor, a norm over everything
MODEL_B = _model(131, 42, 1e-6,
                 _memory(3, 7, 9, 2.5, 31),
                 _delta(1, 1, 10, 5, 1, None),
                 _parallel((3, 1, 9, 9, 0.4, None), (2, 15, 5, 1, 5, 1), (1.0, -0.6), 53),
                 _delta(6, 3, 6, 14, 2, 17, decay_rank=1, gate_rank=9))
# sizes that the matrix-core kernels take as they are; six heads on one key/value head; a state of 128
MODEL_C = _model(256, 128, 1e-5,
                 _parallel((6, 1, 64, 64, 0.125, (64, 10000.0)), (4, 64, 128, 1, 4, 1), (0.9, 1.1), 256),
                 _delta(2, 2, 64, 64, 4, 256, decay_rank=32, gate_rank=16),
                 _memory(2, 64, 64, 15.0, 256))
# key heads beyond 128, columns beyond one block's, more norm groups than heads, keys narrower than values
MODEL_D = _model(77, 80, 1e-5,
                 _memory(1, 136, 150, 8.0, 40),
                 _parallel((2, 2, 24, 100, 0.25, (24, 50.0)), (2, 70, 200, 2, 2, 4), (1.6, 0.4), 24),
                 _delta(2, 1, 150, 20, 3, 60))
# the smallest of everything
MODEL_E = _model(33, 24, 1e-4,
                 _delta(1, 1, 4, 3, 2, 9),
                 _memory(1, 4, 1, 1.0, None),
                 _parallel((1, 1, 4, 4, 0.7, (2, 10.0)), (1, 2, 1, 1, 1, 2), (0.5, 2.0), 7))
# name -> (configuration, page size, seed)
MODELS = {"A": (MODEL_A, 8, 0), "B": (MODEL_B, 16, 1), "C": (MODEL_C, 16, 2), "D": (MODEL_D, 4, 3),
          "E": (MODEL_E, 2, 4)}


def write_folder(folder, raw, tensors):
    """Store a checkpoint as this design's are stored (bfloat16) and return the values as stored."""
    from safetensors.torch import save_file

    stored = {name: tensor.to(torch.bfloat16).contiguous() for name, tensor in tensors.items()}
    os.makedirs(folder, exist_ok=True)
    save_file(stored, os.path.join(folder, "model.safetensors"))
    with open(os.path.join(folder, "config.json"), "w") as handle:
        json.dump(raw, handle)
    return {name: tensor.double() for name, tensor in stored.items()}


def folder_of(tmp_path, which):
    """(folder, raw configuration, checkpoint tensors as stored, page size)."""
    raw, page_size, seed = MODELS[which]
    folder = os.path.join(str(tmp_path), f"fadosun_{which}")
    return folder, raw, write_folder(folder, raw, plain_fadosun.random_checkpoint(raw, seed)), page_size


LOUD, ASK = 1, 2      # tokens of the models below


def far_model(tmp_path, kind, dim=16, heads=2):
    """A model of one layer in which an ASK reads, out of everything before it, what a LOUD has left however far
    back that was: LOUD's key and ASK's query stand in dimensions of their own, and nothing decays or
    weighs much besides.  ``kind``: the layer's type.  Returns (folder, raw, tensors)."""
    width = 64
    layer = {
        "channel_delta": _delta(heads, heads, dim, 16, 3, None),
        "mlstm": _memory(heads, dim, 16, 10.0, None),
        "parallel": _parallel((heads, 1, dim, 16, 1.0, None), (heads, 16, dim, 1, 3, 1), (1.0, 1.0), None),
        "attention": _parallel((heads, 1, dim, 16, 1.0, None), (heads, 16, dim, 1, 3, 1), (1.0, 0.0), None),
        "space": _parallel((heads, 1, dim, 16, 1.0, None), (heads, 16, dim, 1, 3, 1), (0.0, 1.0), None),
    }[kind]
    raw = _model(50, width, 1e-5, layer)
    w = plain_fadosun.random_checkpoint(raw, 17)
    # the two tokens' embeddings: long along directions 0 and 1, where no other token has anything
    w["embed"][:, :2] = 0
    for token, direction in ((LOUD, 0), (ASK, 1)):
        w["embed"][token] *= 0.05
        w["embed"][token, direction] = 8.0
    w["l0.norm1.b"][:2] = 0

    def pair(k, q, strength):
        # the first four dimensions of every head: keys of LOUD and queries of ASK only
        for matrix, direction in ((k, 0), (q, 1)):
            rows = matrix.view(-1, dim, width)
            rows[:, :, :2] = 0
            rows[:, :4] = 0
            rows[:, :4, direction] = strength

    def only_this_token(conv):
        conv[:, :-1] = 0
        conv[:, -1] = 1

    m = "l0.mix."
    if kind == "channel_delta":
        pair(w[m + "k"], w[m + "q"], 1.0)
        for name in "qkv":
            only_this_token(w[m + name + ".conv"])
        w[m + "A_log"][:] = -8.0
        w[m + "b"][:, 0] = 1.0
    elif kind == "mlstm":
        pair(w[m + "k"], w[m + "q"], 1.0)
        w[m + "i"][:, 0] = 1.0
        w[m + "f"] *= 0.1
        w[m + "f.b"][:] = 9.0
    else:
        a, s = m + "left.", m + "right."
        pair(w[a + "k"], w[a + "q"], 0.6)
        w[a + "pb"][:] = -9.0
        inner, state = heads * 16, dim
        pair(w[s + "in"][2 * inner:2 * inner + state], w[s + "in"][2 * inner + state:2 * inner + 2 * state], 1.0)
        only_this_token(w[s + "conv"])
        w[s + "conv.b"][:] = 0
        w[s + "A_log"][:] = -9.0
        w[s + "D"][:] = 0
    folder = os.path.join(str(tmp_path), f"fadosun_far_{kind}_{dim}_{heads}")
    return folder, raw, write_folder(folder, raw, w)
