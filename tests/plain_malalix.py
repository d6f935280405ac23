"""A plain, slow Malalix in float64 on the CPU, written from the design's equations: one function
per mechanism.  It shares no code with the engine; the tests hold the engine's kernels and whole
models against it.

Notation: ``x`` the stream ``[T, d]``, ``e`` the embedded tokens, ``N(x; w) = x / rms(x) * w``.
A layer is ``x <- x + A(N(x; w1)) + F(N(x; w2))``; ``F`` may be absent.  A run of layers is passed
several times: pass 0 begins with ``x <- x + s_0``, pass t > 0 with ``x <- x + e + s_t``.
"""

import math

import torch

F64 = torch.float64


def rms_norm(x, weight, eps):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


# ------------------------------------------------------------------ positions
def banded_frequencies(rot):
    """``f_i = base^(-2i / dims)``; with a scaling, a pair whose wavelength ``2 pi / f`` exceeds
    ``original / low`` turns ``factor`` times slower, one under ``original / high`` as before, and
    those between are interpolated by how many wavelengths ``original`` holds."""
    dims, base = rot["dims"], rot["base"]
    scaling = rot.get("scaling")
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling:
            wave = 2.0 * math.pi / f
            fast, slow = scaling["original"] / scaling["high"], scaling["original"] / scaling["low"]
            if wave > slow:
                f = f / scaling["factor"]
            elif wave >= fast:
                s = (scaling["original"] / wave - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def rotate_halves(x, positions, rot):
    """x ``[T, heads, dim]``: dimension i turns with dimension i + dims/2, i < dims/2."""
    if not rot or not rot["dims"]:
        return x
    out = x.clone()
    half = rot["dims"] // 2
    for i, f in enumerate(banded_frequencies(rot)):
        angle = positions.to(F64) * f
        c, s = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


# ------------------------------------------------------------------ attention inside chunks
def chunked_attention(q, k, v, scale, size=0):
    """Softmax attention of position i over the positions ``j <= i`` of its own chunk of ``size``
    positions (all earlier ones when ``size`` is 0); query head h reads key/value head ``h // (H / G)``."""
    tokens, heads, _ = q.shape
    group = heads // k.shape[1]
    out = torch.zeros((tokens, heads, v.shape[2]), dtype=F64)
    for i in range(tokens):
        first = i // size * size if size else 0
        for h in range(heads):
            scores = (k[first:i + 1, h // group] @ q[i, h]) * scale
            out[i, h] = torch.softmax(scores, 0) @ v[first:i + 1, h // group]
    return out


def attention(u, w, prefix, mixer, eps):
    tokens = u.shape[0]
    heads, groups, dim, vdim = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    q = (u @ w[prefix + "q"].T + w[prefix + "q.b"]).view(tokens, heads, dim)
    k = (u @ w[prefix + "k"].T + w[prefix + "k.b"]).view(tokens, groups, dim)
    v = (u @ w[prefix + "v"].T + w[prefix + "v.b"]).view(tokens, groups, vdim)
    positions = torch.arange(tokens)
    q = rotate_halves(rms_norm(q, w[prefix + "q.norm"], eps), positions, mixer.get("rot"))
    k = rotate_halves(rms_norm(k, w[prefix + "k.norm"], eps), positions, mixer.get("rot"))
    o = chunked_attention(q, k, v, mixer["scale"], (mixer.get("mask") or {}).get("size", 0))
    return o.reshape(tokens, heads * vdim) @ w[prefix + "o"].T


# ------------------------------------------------------------------ experts
def capped_gate(g, u, limit):
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def expert(u, w, prefix, limit):
    return capped_gate(u @ w[prefix + "gate"].T, u @ w[prefix + "up"].T, limit) @ w[prefix + "down"].T


def route(logits, top):
    """Per row: (the ``top`` experts with the largest logits, softmax over those logits)."""
    chosen, weights = [], []
    for row in logits:
        picked = sorted(range(row.numel()), key=lambda e: -float(row[e]))[:top]
        chosen.append(picked)
        weights.append(torch.softmax(row[picked], 0))
    return chosen, weights


def mixture(u, w, prefix, mlp):
    chosen, weights = route(u @ w[prefix + "router"].T, mlp["router"]["top"])
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        for e, weight in zip(chosen[t], weights[t]):
            out[t] += weight * expert(u[t:t + 1], w, f"{prefix}e{e}.", mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        s = prefix + "shared."
        out = out + torch.sigmoid(u @ w[s + "sg"].T) * expert(u, w, s, mlp["shared"]["limit"])
    return out


# ------------------------------------------------------------------ the model
def run_order(raw):
    """(layer, pass that this call opens or None) in the order in which the layers run."""
    count = len(raw["layers"])
    loop = raw.get("loop")
    if not loop:
        return [(i, None) for i in range(count)]
    order = [(i, None) for i in range(loop["start"])]
    for turn in range(loop["times"]):
        order += [(i, turn if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], count)]


def forward(raw, tensors, tokens):
    """(logits ``[T, vocab]``, the stream after every layer run) of one sequence from its start."""
    w = {name: tensor.to(F64) for name, tensor in tensors.items()}
    eps = raw["norm"]["eps"]
    embedded = w["embed"][torch.tensor(list(tokens))]
    x, after = embedded, []
    for index, turn in run_order(raw):
        if turn is not None:
            if turn > 0:
                x = x + embedded
            x = x + w["loop.step"][turn]
        layer, p = raw["layers"][index], f"l{index}."
        y = attention(rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + mixture(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"])
        x = x + y
        after.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T, after


def greedy_generate(raw, tensors, prompt, count):
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(forward(raw, tensors, tokens)[0][-1].argmax()))
    return tokens[len(prompt):]


# ------------------------------------------------------------------ random checkpoints
def random_checkpoint(raw, seed):
    """Checkpoint tensors (float32) of a random model of the raw configuration: matrices
    N(0, 1/in), scales around one, router logits a few units apart."""
    g = torch.Generator().manual_seed(seed)

    def normal(*shape, std=1.0):
        return torch.randn(shape, generator=g) * std

    def matrix(rows, columns, gain=1.0):
        return normal(rows, columns, std=gain / math.sqrt(columns))

    d = raw["width"]
    w = {"embed": normal(raw["vocab"], d), "head": matrix(raw["vocab"], d), "final.norm": 1 + normal(d, std=0.1)}
    if raw.get("loop"):
        w["loop.step"] = normal(raw["loop"]["times"], d, std=0.3)
    for i, layer in enumerate(raw["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w[p + "norm1"] = 1 + normal(d, std=0.1)
        for name, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]),
                           ("v", m["kv_heads"] * m["vdim"])):
            w[p + "mix." + name] = matrix(rows, d)
            w[p + f"mix.{name}.b"] = normal(rows, std=0.2)
        w[p + "mix.q.norm"] = 1.2 + normal(m["dim"], std=0.2)
        w[p + "mix.k.norm"] = 1.2 + normal(m["dim"], std=0.2)
        w[p + "mix.o"] = matrix(d, m["heads"] * m["vdim"])
        mlp = layer.get("mlp")
        if mlp is None:
            continue
        f = p + "mlp."
        w[p + "norm2"] = 1 + normal(d, std=0.1)
        w[f + "router"] = matrix(mlp["router"]["experts"], d, gain=3.0)
        names = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
        if mlp.get("shared"):
            names.append(("shared.", mlp["shared"]["ff"]))
            w[f + "shared.sg"] = matrix(1, d, gain=2.0)
        for name, ff in names:
            w[f + name + "gate"], w[f + name + "up"] = matrix(ff, d, gain=2.0), matrix(ff, d, gain=2.0)
            w[f + name + "down"] = matrix(d, ff)
    return w
