"""A plain, slow Fadosun in float64 on the CPU, written from the design's equations: one function
per mechanism, loops over tokens where the design has a recurrence.  It shares no code with the
engine; the tests hold the engine's kernels and whole models against it.

Notation: ``x`` the stream ``[T, d]``, ``N`` a layer norm with scale and shift.  A sublayer ``F`` reads ``u =
N1(x)`` and adds ``N1b(sigmoid(R u + r) * F(u))``; a layer is a mixer, then a feed-forward or none.
Matrices are stored ``[out, in]`` and applied as ``W u``.  Every recurrence takes the state it starts from
and returns the one it leaves, so that a sequence may be cut.

``forward(..., half=True)`` rounds to bfloat16 what a 16-bit engine may keep in 16 bits (inputs of matrix
products, queries, keys and values): how far that moves the logits says what to expect of such an engine.
"""

import math

import torch

F64 = torch.float64
_HALF = [False]


def kept(x):
    """``x``, or rounded to bfloat16 in a run that keeps 16 bits."""
    return x.to(torch.bfloat16).to(F64) if _HALF[0] else x


# ------------------------------------------------------------------ norms and small functions
def layer_norm(x, weight, bias, eps):
    mean = x.mean(-1, keepdim=True)
    var = ((x - mean) ** 2).mean(-1, keepdim=True)
    return (x - mean) / torch.sqrt(var + eps) * weight + bias


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def log_sigmoid(z):
    return torch.clamp(z, max=0.0) - torch.log1p(torch.exp(-z.abs()))


def causal_conv(raw, weight, bias=None, before=None):
    """``y_t[c] = bias[c] + sum_j weight[c, j] raw_(t - taps + 1 + j)[c]``: the last column is the current
    token's; ``before``: the ``taps - 1`` inputs ahead of the first (zeros if None)."""
    tokens, channels = raw.shape
    taps = weight.shape[1]
    if before is None:
        before = torch.zeros((taps - 1, channels), dtype=F64)
    padded = torch.cat([before, raw])
    out = torch.zeros((tokens, channels), dtype=F64)
    for t in range(tokens):
        out[t] = (padded[t:t + taps].T * weight).sum(-1) + (0.0 if bias is None else bias)
    return out


# ------------------------------------------------------------------ delta rule with a decay per channel
def delta_recurrence(q, k, v, beta, g, state=None):
    """Per head, from the state S ``[dk, dv]``: ``S <- diag(g) S``, ``e = beta (v - S^T k)``, ``S <- S + k e^T``,
    ``o = S^T q``.  q, k, g: ``[T, H, dk]``, v: ``[T, H, dv]``, beta: ``[T, H]``."""
    tokens, heads, dk = q.shape
    dv = v.shape[2]
    state = torch.zeros((heads, dk, dv), dtype=F64) if state is None else state.clone()
    out = torch.zeros((tokens, heads, dv), dtype=F64)
    for t in range(tokens):
        for h in range(heads):
            s = g[t, h][:, None] * state[h]
            e = beta[t, h] * (v[t, h] - s.T @ k[t, h])
            state[h] = s + torch.outer(k[t, h], e)
            out[t, h] = state[h].T @ q[t, h]
    return out, state


def channel_delta(u, w, p, mixer, eps):
    tokens = u.shape[0]
    heads, groups, dk, dv = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]

    def short(name, shape):
        return kept(silu(causal_conv(kept(u @ w[p + name].T), w[p + name + ".conv"]))).view(tokens, *shape)

    q = unit(short("q", (groups, dk))) * dk ** -0.5
    k = unit(short("k", (groups, dk)))
    v = short("v", (heads, dv))
    spread = torch.arange(heads) // (heads // groups)
    beta = torch.sigmoid(u @ w[p + "b"].T)
    z = kept(u @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    g = torch.exp(-torch.exp(w[p + "A_log"])[:, None] * softplus(z).view(tokens, heads, dk))
    o, _ = delta_recurrence(q[:, spread], k[:, spread], v, beta, g)
    o = rms(o, eps) * w[p + "norm"]
    gate = torch.sigmoid(kept(u @ w[p + "g1"].T) @ w[p + "g2"].T)
    return kept(o.reshape(tokens, heads * dv) * gate) @ w[p + "o"].T


# ------------------------------------------------------------------ attention without a softmax
def rotate_halves(x, positions, rot):
    """x ``[T, heads, dim]``: dimension i turns with dimension i + dims/2, i < dims/2."""
    if not rot or not rot["dims"]:
        return x
    out = x.clone()
    half = rot["dims"] // 2
    for i in range(half):
        angle = positions.to(F64) * float(rot["base"]) ** (-2.0 * i / rot["dims"])
        c, s = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        a, b = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = a * c - b * s
        out[:, :, i + half] = b * c + a * s
    return out


def logistic_attention(q, k, v, scale, shift):
    """Position i adds up the values of all ``j <= i``, each with the weight ``sigmoid(scale q_i . k_j +
    shift_h)``; query head h reads key/value head ``h // (H / G)``."""
    tokens, heads, _ = q.shape
    group = heads // k.shape[1]
    out = torch.zeros((tokens, heads, v.shape[2]), dtype=F64)
    for i in range(tokens):
        for h in range(heads):
            weights = torch.sigmoid((k[:i + 1, h // group] @ q[i, h]) * scale + shift[h])
            out[i, h] = weights @ v[:i + 1, h // group]
    return out


def attention_half(u, w, p, left):
    tokens = u.shape[0]
    heads, groups, dk, dv = left["heads"], left["kv_heads"], left["dim"], left["vdim"]
    positions = torch.arange(tokens)
    q = kept(rotate_halves((u @ w[p + "q"].T).view(tokens, heads, dk), positions, left.get("rot")))
    k = kept(rotate_halves((u @ w[p + "k"].T).view(tokens, groups, dk), positions, left.get("rot")))
    v = kept(u @ w[p + "v"].T).view(tokens, groups, dv)
    o = logistic_attention(q, k, v, left["scale"], w[p + "pb"])
    return kept(o.reshape(tokens, heads * dv)) @ w[p + "o"].T


# ------------------------------------------------------------------ state space with a decay per head
def state_space_recurrence(x, dt, a, b, c, skip, state=None):
    """``S_t = exp(a_h dt) S_(t-1) + dt b x^T`` (S: ``[N, dv]`` per head), ``y_t = S_t^T c + skip_h x``.  x: ``[T, H,
    dv]``, dt: ``[T, H]``, b, c: ``[T, H, N]``."""
    tokens, heads, dv = x.shape
    state = torch.zeros((heads, b.shape[2], dv), dtype=F64) if state is None else state.clone()
    y = torch.zeros((tokens, heads, dv), dtype=F64)
    for t in range(tokens):
        for h in range(heads):
            state[h] = torch.exp(a[h] * dt[t, h]) * state[h] + dt[t, h] * torch.outer(b[t, h], x[t, h])
            y[t, h] = state[h].T @ c[t, h] + skip[h] * x[t, h]
    return y, state


def grouped_gated_norm(y, z, weight, groups, eps):
    y = y * silu(z)
    return rms(y.view(y.shape[0], groups, -1), eps).reshape(y.shape) * weight


def state_space_half(u, w, p, right, eps):
    tokens = u.shape[0]
    heads, dv, states, groups = right["heads"], right["vdim"], right["state"], right["groups"]
    inner = heads * dv
    both = kept(u @ w[p + "in"].T)
    z, raw, dt = both[:, :inner], both[:, inner:2 * inner + 2 * groups * states], both[:, 2 * inner + 2 * groups * states:]
    act = kept(silu(causal_conv(raw, w[p + "conv"], w[p + "conv.b"])))
    x = act[:, :inner].view(tokens, heads, dv)
    b = act[:, inner:inner + groups * states].view(tokens, groups, states)
    c = act[:, inner + groups * states:].view(tokens, groups, states)
    spread = torch.arange(heads) // (heads // groups)
    dt = softplus(dt + w[p + "dt_bias"])
    y, _ = state_space_recurrence(x, dt, -torch.exp(w[p + "A_log"]), b[:, spread], c[:, spread], w[p + "D"])
    y = grouped_gated_norm(y.reshape(tokens, inner), z, w[p + "norm"], right["norm_groups"], eps)
    return kept(y) @ w[p + "o"].T


def parallel(u, w, p, mixer, eps):
    return (mixer["left_scale"] * attention_half(u, w, p + "left.", mixer["left"])
            + mixer["right_scale"] * state_space_half(u, w, p + "right.", mixer["right"], eps))


# ------------------------------------------------------------------ matrix memory with exponential gates
def matrix_memory_recurrence(q, k, v, i, f, state=None):
    """``m_t = max(f + m_(t-1), i)``; ``S_t = e^(f + m_(t-1) - m_t) S_(t-1) + e^(i - m_t) k v^T``, ``n_t`` the same with k
    alone; ``o = S_t^T q / (max(|n_t . q|, e^(-m_t)) + 1e-6)``.  State: (S, n, m), all zero at the start.  q, k:
    ``[T, H, dk]``, v: ``[T, H, dv]``, i, f: ``[T, H]`` (logarithms)."""
    tokens, heads, dk = q.shape
    dv = v.shape[2]
    if state is None:
        state = (torch.zeros((heads, dk, dv), dtype=F64), torch.zeros((heads, dk), dtype=F64),
                 torch.zeros(heads, dtype=F64))
    s, n, m = (part.clone() for part in state)
    out = torch.zeros((tokens, heads, dv), dtype=F64)
    for t in range(tokens):
        for h in range(heads):
            top = torch.maximum(f[t, h] + m[h], i[t, h])
            keep, take = torch.exp(f[t, h] + m[h] - top), torch.exp(i[t, h] - top)
            s[h] = keep * s[h] + take * torch.outer(k[t, h], v[t, h])
            n[h] = keep * n[h] + take * k[t, h]
            m[h] = top
            out[t, h] = s[h].T @ q[t, h] / (torch.maximum((n[h] @ q[t, h]).abs(), torch.exp(-top)) + 1e-6)
    return out, (s, n, m)


def memory_gates(u, w, p, cap):
    i = cap * torch.tanh((u @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f = log_sigmoid(cap * torch.tanh((u @ w[p + "f"].T + w[p + "f.b"]) / cap))
    return i, f


def matrix_memory(u, w, p, mixer, eps):
    tokens = u.shape[0]
    heads, dk, dv = mixer["heads"], mixer["dim"], mixer["vdim"]
    q = kept(u @ w[p + "q"].T).view(tokens, heads, dk) * dk ** -0.5
    k = kept(u @ w[p + "k"].T).view(tokens, heads, dk)
    v = kept(u @ w[p + "v"].T).view(tokens, heads, dv)
    i, f = memory_gates(u, w, p, mixer["gate_cap"])
    o, _ = matrix_memory_recurrence(q, k, v, i, f)
    o = rms(o, eps).reshape(tokens, heads * dv) * w[p + "norm"]
    return kept(o * torch.sigmoid(u @ w[p + "g"].T)) @ w[p + "o"].T


# ------------------------------------------------------------------ the model
def feed_forward(u, w, p):
    return kept(torch.relu(u @ w[p + "gate"].T) * (u @ w[p + "up"].T)) @ w[p + "down"].T


MIXERS = {"channel_delta": channel_delta, "parallel": parallel, "mlstm": matrix_memory}


def gated_sublayer(x, w, p, number, eps, run):
    """``x + N_b(sigmoid(R u + r) * run(u))`` with ``u = N(x)``; ``number``: 1 the mixer's, 2 the feed-forward's."""
    a, b, r = f"{p}norm{number}", f"{p}norm{number}b", f"{p}rg{number}"
    u = kept(layer_norm(x, w[a], w[a + ".b"], eps))
    y = torch.sigmoid(u @ w[r].T + w[r + ".b"]) * run(u)
    return x + layer_norm(y, w[b], w[b + ".b"], eps)


def forward(raw, tensors, tokens, half=False):
    """(logits ``[T, vocab]``, the stream after every layer) of one sequence from its start."""
    _HALF[0] = half
    try:
        return _forward(raw, tensors, tokens)
    finally:
        _HALF[0] = False


def _forward(raw, tensors, tokens):
    w = {name: tensor.to(F64) for name, tensor in tensors.items()}
    eps = raw["norm"]["eps"]
    x = w["embed"][torch.tensor(list(tokens))]
    after = []
    for index, layer in enumerate(raw["layers"]):
        p = f"l{index}."
        x = gated_sublayer(x, w, p, 1, eps, lambda u: MIXERS[layer["type"]](u, w, p + "mix.", layer["mixer"], eps))
        if layer.get("mlp") is not None:
            x = gated_sublayer(x, w, p, 2, eps, lambda u: feed_forward(u, w, p + "mlp."))
        after.append(x)
    return kept(layer_norm(x, w["final.norm"], w["final.norm.b"], eps)) @ w["head"].T, after


def greedy_generate(raw, tensors, prompt, count):
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(forward(raw, tensors, tokens)[0][-1].argmax()))
    return tokens[len(prompt):]


# ------------------------------------------------------------------ random checkpoints
def random_checkpoint(raw, seed, ranks=(6, 5)):
    """Checkpoint tensors (float32) of a random model of the raw configuration: matrices N(0, 1/in), scales
    around one, shifts and biases that matter, decays between fast and slow.  ``ranks``: inner widths of the
    low-rank decay and gate of a delta layer where the configuration names none."""
    g = torch.Generator().manual_seed(seed)

    def normal(*shape, std=1.0):
        return torch.randn(shape, generator=g) * std

    def uniform(count, low, high):
        return torch.rand(count, generator=g) * (high - low) + low

    def matrix(rows, columns, gain=1.0):
        return normal(rows, columns, std=gain / math.sqrt(columns))

    d = raw["width"]
    w = {"embed": normal(raw["vocab"], d), "head": matrix(raw["vocab"], d)}

    def norm(name):
        w[name], w[name + ".b"] = 1 + normal(d, std=0.2), normal(d, std=0.2)

    norm("final.norm")
    for i, layer in enumerate(raw["layers"]):
        p, mixer = f"l{i}.", layer["mixer"]
        m = p + "mix."
        for number in (1, 2) if layer.get("mlp") is not None else (1,):
            norm(f"{p}norm{number}")
            norm(f"{p}norm{number}b")
            w[f"{p}rg{number}"], w[f"{p}rg{number}.b"] = matrix(d, d), normal(d, std=0.5)
        if layer["type"] == "channel_delta":
            heads, groups, dk, dv = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
            for name, rows in (("q", groups * dk), ("k", groups * dk), ("v", heads * dv)):
                w[m + name] = matrix(rows, d)
                w[m + name + ".conv"] = normal(rows, mixer["conv"], std=1 / math.sqrt(mixer["conv"]))
            a, b = mixer.get("decay_rank", ranks[0]), mixer.get("gate_rank", ranks[1])
            w[m + "b"] = matrix(heads, d)
            w[m + "A_log"] = uniform(heads, -2.0, 1.0)
            w[m + "norm"] = 1 + normal(dv, std=0.2)
            w[m + "a1"], w[m + "a2"] = matrix(a, d), matrix(heads * dk, a)
            w[m + "dt_bias"] = uniform(heads * dk, -4.0, 0.0)
            w[m + "g1"], w[m + "g2"] = matrix(b, d), matrix(heads * dv, b)
            w[m + "o"] = matrix(d, heads * dv)
        elif layer["type"] == "mlstm":
            heads, dk, dv = mixer["heads"], mixer["dim"], mixer["vdim"]
            for name, rows in (("q", heads * dk), ("k", heads * dk), ("v", heads * dv), ("g", heads * dv)):
                w[m + name] = matrix(rows, d)
            w[m + "i"], w[m + "i.b"] = matrix(heads, d, 2.0), normal(heads)
            w[m + "f"], w[m + "f.b"] = matrix(heads, d), uniform(heads, 0.0, 5.0)
            w[m + "norm"] = 1 + normal(heads * dv, std=0.2)
            w[m + "o"] = matrix(d, heads * dv)
        else:
            left, right = mixer["left"], mixer["right"]
            a, s = m + "left.", m + "right."
            w[a + "q"] = matrix(left["heads"] * left["dim"], d)
            w[a + "k"] = matrix(left["kv_heads"] * left["dim"], d)
            w[a + "v"] = matrix(left["kv_heads"] * left["vdim"], d)
            w[a + "pb"] = normal(left["heads"]) - 2.0
            w[a + "o"] = matrix(d, left["heads"] * left["vdim"])
            inner = right["heads"] * right["vdim"]
            channels = inner + 2 * right["groups"] * right["state"]
            w[s + "in"] = matrix(inner + channels + right["heads"], d)
            w[s + "conv"] = normal(channels, right["conv"], std=1 / math.sqrt(right["conv"]))
            w[s + "conv.b"] = normal(channels, std=0.2)
            w[s + "dt_bias"] = uniform(right["heads"], -4.0, 0.0)
            w[s + "A_log"] = uniform(right["heads"], -2.0, 1.5)
            w[s + "D"] = normal(right["heads"])
            w[s + "norm"] = 1 + normal(inner, std=0.2)
            w[s + "o"] = matrix(d, inner)
        if layer.get("mlp") is not None:
            ff = layer["mlp"]["ff"]
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = matrix(ff, d), matrix(ff, d), matrix(d, ff)
    return w
