"""Fadosun on the GPU against the plain implementation (``plain_fadosun.py``): each new kernel or kernel option
alone (attention with logistic weights in every attention kernel, convolutions and decays that feed a
recurrence, exponential gates, the recurrences token by token and in pieces, the norm and gates of their
output, the step between two layer norms, the relu gate), then small models of several shapes stepped
whole, decoded token by token, in portions down to two tokens, and in mixed batches whose pages and slots
are used again; what stands far back in a prompt."""

import os

import pytest
import torch

import fadosun_models
import helpers
import plain_fadosun as plain

pytestmark = pytest.mark.gpu

F64 = torch.float64
# |engine - plain| <= TOLERANCE * max|plain logits|; a 16-bit engine may also differ by as much as the plain
# implementation does from itself when it keeps 16 bits, times three (norms over a head of a few numbers,
# or of a result that nearly cancels, make much of a rounding)
TOLERANCE = {"float32": 1e-4, "bfloat16": 3e-2}


def _kernels():
    from pagedserve_amd.ops import kernels

    return kernels


def _ints(values):
    return torch.tensor(values, dtype=torch.int32, device="cuda")


def _cuts(counts):
    return _ints([sum(counts[:i]) for i in range(len(counts) + 1)])


def _items(counts):
    return _ints([item for item, count in enumerate(counts) for _ in range(count)])


# ---------------------------------------------------------------- attention with logistic weights
class _Paged:
    """Keys and values of requests in a pool whose other places hold NaN, with block tables."""

    def __init__(self, dtype, kv_heads, dim, page_size, portions, seed):
        g = torch.Generator().manual_seed(seed)
        width = -(-max(start + count for start, count in portions) // page_size) + 1
        pages = len(portions) * width + 3
        self.k, self.v = [], []
        k_pool = torch.full((pages, kv_heads, page_size, dim), float("nan"))
        v_pool = torch.full_like(k_pool, float("nan"))
        tables = torch.full((len(portions), width), -1, dtype=torch.int32)
        order = torch.randperm(pages, generator=g).tolist()
        for item, (start, count) in enumerate(portions):
            total = start + count
            k = torch.randn((total, kv_heads, dim), generator=g).to(dtype)
            v = torch.randn((total, kv_heads, dim), generator=g).to(dtype)
            self.k.append(k.double())
            self.v.append(v.double())
            for logical in range(-(-total // page_size)):
                page = tables[item, logical] = order.pop()
                for place in range(min(page_size, total - logical * page_size)):
                    k_pool[page, :, place] = k[logical * page_size + place].float()
                    v_pool[page, :, place] = v[logical * page_size + place].float()
        self.k_pool, self.v_pool = k_pool.to(dtype).cuda(), v_pool.to(dtype).cuda()
        self.tables = tables.cuda()
        self.tokens = [(item, start + i) for item, (start, count) in enumerate(portions) for i in range(count)]
        self.tok_item, self.positions = _ints([t[0] for t in self.tokens]), _ints([t[1] for t in self.tokens])
        self.counts = [count for _, count in portions]
        self.cu = _cuts(self.counts)
        self.kv_lens = _ints([start + count for start, count in portions])

    def tiles(self, size, only=None):
        items = [(item, q0) for item, count in enumerate(self.counts) if only is None or item in only
                 for q0 in range(0, count, size)]
        return _ints([i for i, _ in items]), _ints([q for _, q in items])

    def expected(self, q, heads, scale, shift, norm, window=0):
        out = torch.zeros(q.shape, dtype=F64)
        for t, (item, position) in enumerate(self.tokens):
            k, v = self.k[item], self.v[item]
            first = max(0, position - window + 1) if window else 0
            for h in range(heads):
                group = h // (heads // k.shape[1])
                weights = torch.sigmoid((k[first:position + 1, group] @ q[t, h]) * scale + shift[h].double())
                out[t, h] = weights @ v[first:position + 1, group] / norm
        return out


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kv_heads,dim,page_size,norm,window", [
    (4, 2, 16, 4, 1.0, 0), (8, 1, 64, 16, 1.25, 0), (2, 2, 128, 8, 0.5, 0), (3, 1, 24, 16, 1.0, 0),
    (6, 1, 192, 16, -2.0, 0), (4, 2, 64, 8, 0.8, 40)])
def test_logistic_attention_in_every_kernel(dtype, heads, kv_heads, dim, page_size, norm, window):
    """Portions at the start of a request and behind hundreds of keys, single tokens at page borders; one key
    in a row stands out of its query's scores; ranges without keys, and a norm on the whole."""
    kernels = _kernels()
    portions = [(0, 70), (63, 5), (0, 1), (15, 1), (16, 1), (255, 2), (300, 1), (129, 33), (7, 40)]
    paged = _Paged(dtype, kv_heads, dim, page_size, portions, heads * dim)
    tokens = len(paged.tokens)
    g = torch.Generator().manual_seed(dim)
    q = torch.randn((tokens, heads, dim), generator=g).to(dtype)
    # the first key of the longest request, far away from everything, matches that request's query
    far = next(t for t, (item, _) in enumerate(paged.tokens) if item == 6)
    for h in range(heads):
        q[far, h] = (2.0 * paged.k[6][0, h // (heads // kv_heads)]).to(dtype)
    scale = dim ** -0.5
    shift = torch.randn(heads, generator=g) - 2.5
    expected = paged.expected(q.double(), heads, scale, shift, norm, window)
    logistic = (shift.cuda(), norm)
    q = q.reshape(tokens, heads * dim).cuda()
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    pools = (paged.k_pool, paged.v_pool)
    singles = [t for t in range(tokens) if paged.counts[paged.tokens[t][0]] == 1]
    several = [t for t in range(tokens) if t not in singles]
    items_of_several = [i for i, count in enumerate(paged.counts) if count > 1]
    reach = float(expected.abs().max())

    def check(out, which, what):
        got = out.double().cpu().view(tokens, heads, dim)
        worst = float((got[which] - expected[which]).abs().max())
        assert worst <= tol * reach, (what, worst / reach)

    def fresh():
        return torch.full((tokens, heads * dim), 9.0, dtype=dtype, device="cuda")

    everyone = list(range(tokens))
    index = (paged.tok_item, paged.positions, paged.tables)
    out = fresh()
    kernels.attention_rowwise(q, *pools, out, *index, heads, scale, window, logistic=logistic)
    check(out, everyone, "rowwise")
    for splits, waves in ((1, 4), (1, 16), (3, 4), (7, 4)):
        out = fresh()
        partial = torch.empty(tokens * heads * splits * (dim + 2), device="cuda")
        kernels.attention_decode(q, *pools, out, *index, heads, scale, splits, partial=partial, waves=waves,
                                 window=window, logistic=logistic)
        check(out, everyone, ("decode", splits, waves))
    if kernels.shared_decode_supported(dtype, heads, kv_heads, dim):
        for splits in (1, 3):
            out = fresh()
            partial = torch.empty(tokens * heads * splits * (dim + 2), device="cuda")
            kernels.attention_decode_shared(q, *pools, out, *index, heads, scale, splits, partial, window=window,
                                            logistic=logistic)
            check(out, everyone, ("shared decode", splits))
    if kernels.tiled_f32_supported(dtype, dim):
        out = fresh()
        kernels.attention_tiled_f32(q, *pools, out, *paged.tiles(64), paged.cu, paged.kv_lens, paged.tables, heads,
                                    scale, window, logistic=logistic)
        check(out, everyone, "tiled f32")
    if kernels.prefill_supported(dtype, dim, paged.tables.shape[1]):
        for size in [64] + ([32] if dim <= 128 else []) + ([128] if dim <= 64 else []):
            for longest in (0, 100):
                out = fresh()
                kernels.attention_prefill(q, *pools, out, *paged.tiles(size), paged.cu, paged.kv_lens, paged.tables,
                                          heads, scale, window, max_kv_len=longest, query_tile=size, logistic=logistic)
                check(out, everyone, ("prefill", size, longest))
    if kernels.mixed_supported(dtype, dim, paged.tables.shape[1]):
        out = fresh()
        kernels.attention_mixed(q, *pools, out, _ints(singles), paged.tok_item, paged.positions,
                                *paged.tiles(64, items_of_several), paged.cu, paged.kv_lens, paged.tables, heads,
                                scale, window, logistic=logistic)
        check(out, singles, "mixed, singles")
        check(out, several, "mixed, portions")
    if dtype == torch.bfloat16 and dim % 64 == 0:
        # the ranges merged inside the output projection
        first = everyone[:9]
        w = torch.randn((48, heads * dim), generator=g).to(dtype).cuda() * 0.1
        for splits in (1, 4):
            partial = torch.empty(9 * heads * splits * (dim + 2), device="cuda")
            rows = q[:9].contiguous()
            kernels.attention_decode_partial(rows, *pools, partial, paged.tok_item[:9].contiguous(),
                                             paged.positions[:9].contiguous(), paged.tables, heads, scale, splits,
                                             window=window, logistic=logistic)
            residual = torch.zeros((9, 48), device="cuda")
            kernels.attention_merge_linear(partial, 9, heads, dim, splits, w, kernels.pack_decode_weight(w), None, residual)
            want = expected[first].reshape(9, -1) @ w.double().cpu().T
            assert torch.allclose(residual.double().cpu(), want, atol=3e-2 * float(want.abs().max())), splits
    # what the far key is worth, had it been cut off
    if not window:
        cut = paged.expected(q.double().cpu().view(tokens, heads, dim), heads, scale, shift, norm, window=300)
        assert float((cut[far] - expected[far]).abs().max()) > 2 * tol * reach


def test_logistic_weights_are_checked():
    kernels = _kernels()
    paged = _Paged(torch.float32, 1, 16, 4, [(0, 3)], 1)
    q = torch.zeros((3, 32), device="cuda")
    args = (q, paged.k_pool, paged.v_pool, q.clone(), paged.tok_item, paged.positions, paged.tables, 2, 0.25)
    for bad in ((torch.zeros(3, device="cuda"), 1.0), (torch.zeros(2, device="cuda"), 0.0)):
        with pytest.raises(kernels.KernelError):
            kernels.attention_rowwise(*args, logistic=bad)


# ---------------------------------------------------------------- what a recurrence is fed with
PORTIONS = [(1,) * 5, (9, 1, 2, 30, 3), (70,), (1, 2, 3, 1), (64, 65, 8), (17, 150)]


@pytest.mark.parametrize("counts", PORTIONS)
@pytest.mark.parametrize("taps", [1, 2, 4, 6])
@pytest.mark.parametrize("key_heads,heads,dk,dv,bias", [(2, 4, 16, 24, False), (1, 1, 70, 9, False), (3, 3, 130, 64, True)])
def test_delta_inputs(counts, taps, key_heads, heads, dk, dv, bias):
    """Convolution, silu, unit norms, decays and weights of items of all lengths, with kept inputs in some
    slots; the columns lie between others in wider rows."""
    kernels = _kernels()
    g = torch.Generator().manual_seed(taps + dk)
    tokens, channels = sum(counts), 2 * key_heads * dk + heads * dv
    proj = torch.randn((tokens, channels + heads + 11), generator=g)
    col, take_col = 5, channels + 8
    weight = torch.randn((channels, taps), generator=g)
    shift = torch.randn(channels, generator=g) if bias else None
    history, slots_total = 12, len(counts) + 2
    state = torch.randn((slots_total, history + (taps - 1) * channels + 3), generator=g)
    slots = torch.randperm(slots_total, generator=g)[:len(counts)].tolist()
    z = torch.randn((tokens, heads * dk), generator=g)
    z_bias, a_log = torch.randn(heads * dk, generator=g), torch.randn(heads, generator=g)
    out, decay, take = (torch.full((tokens, n), float("nan"), device="cuda") for n in (channels, heads * dk, heads))
    kernels.state_prepare(proj.cuda(), col, weight.T.contiguous().cuda(), None if shift is None else shift.cuda(),
                          state.cuda(), history, out, "delta", decay, take, a_log.cuda(), z_bias.cuda(), take_col,
                          _items(counts), _cuts(counts), _ints(slots), z=z.cuda(), per_head=dk,
                          unit_heads=2 * key_heads, head=dk, scale_heads=key_heads, q_scale=0.3)
    want, begin = [], 0
    for slot, count in zip(slots, counts):
        before = state[slot, history:history + (taps - 1) * channels].view(taps - 1, channels).double()
        act = plain.silu(plain.causal_conv(proj[begin:begin + count, col:col + channels].double(), weight.double(),
                                           None if shift is None else shift.double(), before))
        q = plain.unit(act[:, :key_heads * dk].view(count, key_heads, dk)) * 0.3
        k = plain.unit(act[:, key_heads * dk:2 * key_heads * dk].view(count, key_heads, dk))
        want.append(torch.cat([q.reshape(count, -1), k.reshape(count, -1), act[:, 2 * key_heads * dk:]], 1))
        begin += count
    assert torch.allclose(out.double().cpu(), torch.cat(want), atol=1e-5, rtol=1e-5)
    steps = plain.softplus((z + z_bias).double()).view(tokens, heads, dk)
    want_decay = torch.exp(-torch.exp(a_log.double())[:, None] * steps).view(tokens, -1)
    assert torch.allclose(decay.double().cpu(), want_decay, atol=1e-6, rtol=1e-5)
    assert torch.allclose(take.double().cpu(), torch.sigmoid(proj[:, take_col:take_col + heads].double()), atol=1e-6)


@pytest.mark.parametrize("counts", PORTIONS)
@pytest.mark.parametrize("taps,channels,heads", [(4, 200, 3), (2, 64, 1), (5, 31, 8)])
def test_state_space_inputs(counts, taps, channels, heads):
    kernels = _kernels()
    g = torch.Generator().manual_seed(channels)
    tokens = sum(counts)
    proj = torch.randn((tokens, channels + heads + 2), generator=g)
    weight, shift = torch.randn((channels, taps), generator=g), torch.randn(channels, generator=g)
    state = torch.randn((len(counts), (taps - 1) * channels + 1), generator=g)
    step_bias, a_log = torch.randn(heads, generator=g), torch.randn(heads, generator=g)
    out, decay, take = (torch.full((tokens, n), float("nan"), device="cuda") for n in (channels, heads, heads))
    kernels.state_prepare(proj.cuda(), 1, weight.T.contiguous().cuda(), shift.cuda(), state.cuda(), 0, out, "decayed",
                          decay, take, a_log.cuda(), step_bias.cuda(), channels + 2, _items(counts), _cuts(counts),
                          _ints(list(range(len(counts)))))
    want, begin = [], 0
    for slot, count in enumerate(counts):
        before = state[slot, :(taps - 1) * channels].view(taps - 1, channels).double()
        want.append(plain.silu(plain.causal_conv(proj[begin:begin + count, 1:1 + channels].double(), weight.double(),
                                                 shift.double(), before)))
        begin += count
    assert torch.allclose(out.double().cpu(), torch.cat(want), atol=1e-5, rtol=1e-5)
    dt = plain.softplus((proj[:, channels + 2:] + step_bias).double())
    assert torch.allclose(take.double().cpu(), dt, atol=1e-6, rtol=1e-5)
    assert torch.allclose(decay.double().cpu(), -torch.exp(a_log.double()) * dt, atol=1e-6, rtol=1e-5)


@pytest.mark.parametrize("counts", PORTIONS + [(400, 1, 64, 128)])
@pytest.mark.parametrize("heads,cap", [(1, 15.0), (5, 2.5)])
def test_exponential_gates(counts, heads, cap):
    kernels = _kernels()
    g = torch.Generator().manual_seed(heads)
    tokens = sum(counts)
    proj = torch.randn((tokens, 2 * heads + 3), generator=g) * 5
    i_bias, f_bias = torch.randn(heads, generator=g), torch.randn(heads, generator=g) + 2
    state = torch.randn((len(counts) + 1, 7 + heads), generator=g) * 2
    slots = torch.randperm(len(counts) + 1, generator=g)[:len(counts)].tolist()
    device = state.cuda()
    decay, take, floor = (torch.full((tokens, heads), float("nan"), device="cuda") for _ in range(3))
    kernels.memory_gates(proj.cuda(), 1, 2 + heads, i_bias.cuda(), f_bias.cuda(), cap, device, 7, decay, take, floor,
                         _cuts(counts), _ints(slots))
    i = cap * torch.tanh((proj[:, 1:1 + heads] + i_bias).double() / cap)
    f = plain.log_sigmoid(cap * torch.tanh((proj[:, 2 + heads:2 + 2 * heads] + f_bias).double() / cap))
    begin = 0
    for slot, count in zip(slots, counts):
        m = state[slot, 7:].double()
        for t in range(begin, begin + count):
            top = torch.maximum(f[t] + m, i[t])
            for got, want in ((decay, f[t] + m - top), (take, torch.exp(i[t] - top)), (floor, torch.exp(-top))):
                assert torch.allclose(got[t].double().cpu(), want, atol=2e-5, rtol=2e-5), (slot, t)
            m = top
        assert torch.allclose(device[slot, 7:].double().cpu(), m, atol=1e-5)
        begin += count
    others = [slot for slot in range(len(counts) + 1) if slot not in slots]
    assert torch.equal(device[others].cpu(), state[others]) and torch.equal(device[:, :7].cpu(), state[:, :7])


# ---------------------------------------------------------------- the recurrences
SIZES = [(4, 2, 16, 24), (1, 1, 4, 3), (2, 1, 30, 40), (3, 3, 64, 64), (2, 2, 100, 17), (2, 1, 128, 70), (1, 1, 250, 33)]


def _recurrence_case(counts, heads, key_heads, dk, dv, rule, ones, seed, rounded=False):
    g = torch.Generator().manual_seed(seed)
    tokens = sum(counts)

    def rand(*shape):
        x = torch.randn(*shape, generator=g)
        return x.to(torch.bfloat16).float() if rounded else x

    columns = dv + (1 if ones else 0)
    case = {
        "q": rand(tokens, key_heads * dk + 4), "k": rand(tokens, key_heads * dk + 8) * dk ** -0.5, "v": rand(tokens, heads * dv),
        "take": torch.rand(tokens, heads, generator=g),
        "decay": (torch.rand(tokens, heads * dk, generator=g) if rule == "delta"
                  else -torch.rand(tokens, heads, generator=g) * 0.2),
        "state": torch.randn(len(counts) + 2, heads * columns * dk + 5, generator=g),
        "slots": torch.randperm(len(counts) + 2, generator=g)[:len(counts)].tolist(),
    }
    if rule == "delta":
        k = case["k"][:, 4:4 + key_heads * dk].reshape(tokens, key_heads, dk)
        case["k"][:, 4:4 + key_heads * dk] = plain.unit(k).reshape(tokens, -1)
    spread = torch.arange(heads) // (heads // key_heads)
    q = case["q"][:, 4:].double().view(tokens, key_heads, dk)[:, spread] * 0.7
    k = case["k"][:, 4:4 + key_heads * dk].double().reshape(tokens, key_heads, dk)[:, spread]
    v = case["v"].double().view(tokens, heads, dv)
    if ones:
        v = torch.cat([v, torch.ones((tokens, heads, 1), dtype=F64)], 2)
    outs, states, begin = [], [], 0
    for slot, count in zip(case["slots"], counts):
        part = slice(begin, begin + count)
        start = case["state"][slot, :heads * columns * dk].view(heads, columns, dk).transpose(1, 2).double()
        if rule == "delta":
            o, s = plain.delta_recurrence(q[part], k[part], v[part], case["take"][part].double(),
                                          case["decay"][part].double().view(count, heads, dk), start)
        else:
            o, s = torch.zeros((count, heads, columns), dtype=F64), start.clone()
            for t in range(count):
                for h in range(heads):
                    s[h] = (torch.exp(case["decay"][begin + t, h].double()) * s[h]
                            + case["take"][begin + t, h].double() * torch.outer(k[begin + t, h], v[begin + t, h]))
                    o[t, h] = s[h].T @ q[begin + t, h]
        outs.append(o)
        states.append(s.transpose(1, 2).reshape(-1))
        begin += count
    return case, torch.cat(outs), states


def _run_recurrence(case, counts, heads, key_heads, dk, dv, rule, ones, longest=0, chunks=None, raw=None, taps=1):
    kernels = _kernels()
    tokens, columns = sum(counts), dv + (1 if ones else 0)
    needed = heads * columns * dk
    state = case["state"].cuda()
    if raw is not None:
        state = torch.cat([case["state"][:, :needed], raw["kept"]], 1).contiguous().cuda()
    q, k = case["q"].cuda(), case["k"].cuda()
    out = torch.full((tokens, heads * columns), float("nan"), device="cuda")
    options = {} if raw is None else dict(raw=raw["rows"].cuda()[:, 1:1 + raw["channels"]], taps=taps, history=needed)
    kernels.state_scan(q[:, 4:], k[:, 4:4 + key_heads * dk], case["v"].cuda(), case["decay"].cuda(), case["take"].cuda(),
                       state, out, _cuts(counts), _ints(case["slots"]), rule, heads, key_heads, dk, dv, ones=ones,
                       q_scale=0.7, longest=longest, chunks=chunks, **options)
    return out.double().cpu().view(tokens, heads, columns), state.double().cpu()


def _check_states(state, before, case, states, atol):
    for slot, want in zip(case["slots"], states):
        got = state[slot, :want.numel()]
        assert torch.allclose(got, want, atol=atol, rtol=atol), float((got - want).abs().max())
    others = [slot for slot in range(state.shape[0]) if slot not in case["slots"]]
    assert torch.equal(state[others], before[others].double())


@pytest.mark.parametrize("counts", [(1,) * 6, (9, 1, 2, 30), (70, 17)])
@pytest.mark.parametrize("heads,key_heads,dk,dv", SIZES)
@pytest.mark.parametrize("rule,ones", [("delta", False), ("decayed", False), ("decayed", True)])
def test_recurrences_token_by_token(counts, heads, key_heads, dk, dv, rule, ones):
    case, want, states = _recurrence_case(counts, heads, key_heads, dk, dv, rule, ones, dk + dv)
    for longest in ((0, 1) if max(counts) == 1 else (0,)):
        out, state = _run_recurrence(case, counts, heads, key_heads, dk, dv, rule, ones, longest=longest)
        scale = float(want.abs().max())
        assert float((out - want).abs().max()) <= 2e-5 * scale, (longest, float((out - want).abs().max()) / scale)
        _check_states(state, case["state"], case, states, 3e-5)


@pytest.mark.parametrize("counts", [(150,), (1, 64, 65, 3, 128), (63, 200, 1, 2), (64,)])
@pytest.mark.parametrize("heads,key_heads,dk,dv", SIZES + [(2, 1, 40, 150), (1, 1, 32, 80)])
@pytest.mark.parametrize("ones", [False, True])
def test_decayed_recurrence_in_pieces(counts, heads, key_heads, dk, dv, ones):
    """Items shorter than a piece, of a piece's length, one token more, and of several; queries, keys and values
    that bfloat16 holds: what is left is the error of two-part products."""
    kernels = _kernels()
    case, want, states = _recurrence_case(counts, heads, key_heads, dk, dv, "decayed", ones, dk * dv, rounded=True)
    # (keys are scaled: round them again)
    tokens, items, size = sum(counts), len(counts), kernels.STATE_CHUNK
    case["k"] = case["k"].to(torch.bfloat16).float()
    again, want, states = _rebuild(case, counts, heads, key_heads, dk, dv, ones)
    pieces = tokens // size + items
    piece_cu, item_first = _ints([0] * (pieces + 1)), _ints([0] * (items + 1))
    kernels.scan_pieces(_cuts(counts), items, size, pieces, piece_cu, item_first)
    floats = kernels.state_chunk_floats(pieces, heads, dk, dv, ones)
    chunks = (piece_cu, item_first, pieces, torch.full((floats[0],), float("nan"), device="cuda"),
              torch.full((floats[1],), float("nan"), device="cuda"))
    out, state = _run_recurrence(again, counts, heads, key_heads, dk, dv, "decayed", ones, chunks=chunks)
    scale = float(want.abs().max())
    assert float((out - want).abs().max()) <= 1e-4 * scale, float((out - want).abs().max()) / scale
    _check_states(state, again["state"], again, states, 2e-4)


def _rebuild(case, counts, heads, key_heads, dk, dv, ones):
    """The decayed rule's results for a case whose inputs were changed."""
    tokens, columns = sum(counts), dv + (1 if ones else 0)
    spread = torch.arange(heads) // (heads // key_heads)
    q = case["q"][:, 4:].double().view(tokens, key_heads, dk)[:, spread] * 0.7
    k = case["k"][:, 4:4 + key_heads * dk].double().reshape(tokens, key_heads, dk)[:, spread]
    v = case["v"].double().view(tokens, heads, dv)
    if ones:
        v = torch.cat([v, torch.ones((tokens, heads, 1), dtype=F64)], 2)
    out, states, begin = torch.zeros((tokens, heads, columns), dtype=F64), [], 0
    for slot, count in zip(case["slots"], counts):
        s = case["state"][slot, :heads * columns * dk].view(heads, columns, dk).transpose(1, 2).double()
        for t in range(begin, begin + count):
            s = (torch.exp(case["decay"][t].double())[:, None, None] * s
                 + case["take"][t].double()[:, None, None] * k[t][:, :, None] * v[t][:, None, :])
            out[t] = (s * q[t][:, :, None]).sum(1)
        states.append(s.transpose(1, 2).reshape(-1))
        begin += count
    return case, out, states


@pytest.mark.parametrize("in_pieces", [False, True])
@pytest.mark.parametrize("taps", [1, 2, 4, 7])
@pytest.mark.parametrize("counts", [(1, 2, 3, 5), (70, 1, 4)])
def test_the_convolutions_inputs_are_kept_for_the_next_step(counts, taps, in_pieces):
    kernels = _kernels()
    heads, dk, dv, channels = 2, 8, 12, 77
    case, want, states = _recurrence_case(counts, heads, heads, dk, dv, "decayed", False, taps)
    g = torch.Generator().manual_seed(taps)
    tokens, items, total = sum(counts), len(counts), len(counts) + 2
    raw = {"rows": torch.randn((tokens, channels + 3), generator=g), "channels": channels,
           "kept": torch.randn((total, (taps - 1) * channels), generator=g)}
    chunks = None
    if in_pieces:
        pieces = tokens // kernels.STATE_CHUNK + items
        piece_cu, item_first = _ints([0] * (pieces + 1)), _ints([0] * (items + 1))
        kernels.scan_pieces(_cuts(counts), items, kernels.STATE_CHUNK, pieces, piece_cu, item_first)
        floats = kernels.state_chunk_floats(pieces, heads, dk, dv)
        chunks = (piece_cu, item_first, pieces, torch.empty(floats[0], device="cuda"), torch.empty(floats[1], device="cuda"))
    _, state = _run_recurrence(case, counts, heads, heads, dk, dv, "decayed", False, chunks=chunks, raw=raw, taps=taps)
    needed, begin = heads * dv * dk, 0
    for slot, count in zip(case["slots"], counts):
        seen = torch.cat([raw["kept"][slot].view(taps - 1, channels), raw["rows"][begin:begin + count, 1:1 + channels]])
        last = seen[seen.shape[0] - (taps - 1):].reshape(-1).double()
        assert torch.equal(state[slot, needed:], last), (slot, count)
        begin += count


# ---------------------------------------------------------------- outputs, the step between norms, the relu gate
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("tokens,heads,dv,groups,shared", [
    (3, 4, 24, 4, True), (5, 1, 7, 1, False), (130, 6, 64, 6, True), (9, 24, 64, 1, False), (4, 8, 48, 2, False),
    (2, 3, 300, 3, False), (2, 40, 64, 1, False), (3, 2, 1, 2, False)])
@pytest.mark.parametrize("form", ["delta", "memory", "space"])
def test_output_norm_and_gates(dtype, tokens, heads, dv, groups, shared, form):
    kernels = _kernels()
    g = torch.Generator().manual_seed(heads * dv)
    columns, eps = heads * dv, 1e-5
    ones = form == "memory"
    o = torch.randn((tokens, heads, dv + (1 if ones else 0)), generator=g)
    weight = torch.randn(dv if shared else columns, generator=g)
    wide = torch.randn((tokens, 2 * columns + 3), generator=g)
    floor, skip = torch.rand((tokens, heads), generator=g), torch.randn(heads, generator=g)
    x = o[:, :, :dv].double()
    options = {}
    if form == "memory":
        x = x / (torch.maximum(o[:, :, dv:].double().abs(), floor.double()[:, :, None]) + 1e-6)
        options = dict(floor=floor.cuda())
    x = x.reshape(tokens, columns)
    if form == "space":
        x = (x + wide[:, :columns].double() * skip.double().repeat_interleave(dv)) * plain.silu(wide[:, columns:2 * columns].double())
        options = dict(skip=skip.cuda(), u=wide.cuda()[:, :columns], before=wide.cuda()[:, columns:2 * columns])
    want = plain.rms(x.view(tokens, groups, -1), eps).view(tokens, columns) * (
        weight.double().repeat(heads) if shared else weight.double())
    if form != "space":
        want = want * torch.sigmoid(wide[:, 2:2 + columns].double())
        options["behind"] = wide.cuda()[:, 2:2 + columns]
    out = torch.full((tokens, columns + 5), float("nan"), dtype=dtype, device="cuda")
    kernels.state_output(o.reshape(tokens, -1).cuda(), heads, dv, weight.cuda(), eps, groups, out[:, 1:1 + columns], **options)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    assert torch.allclose(out[:, 1:1 + columns].double().cpu(), want, atol=tol * float(want.abs().max()), rtol=tol)
    assert bool(out[:, 0].isnan().all()) and bool(out[:, 1 + columns:].isnan().all())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("tokens,width", [(1, 24), (5, 256), (3, 1000), (300, 1024), (2, 2500), (300, 4096), (2, 9000)])
def test_step_between_two_layer_norms(dtype, tokens, width):
    kernels = _kernels()
    g = torch.Generator().manual_seed(width)
    eps = 1e-5
    h0, y0 = torch.randn((tokens, width), generator=g) + 3, torch.randn((tokens, width), generator=g) * 5
    gate = torch.randn((tokens, width + 6), generator=g)
    bias, w1, b1, w2, b2 = (torch.randn(width, generator=g) for _ in range(5))
    h, y = h0.cuda(), y0.cuda()
    normed = torch.full((tokens, width), float("nan"), dtype=dtype, device="cuda")
    add = (y, gate.cuda()[:, 3:3 + width], bias.cuda(), w1.cuda(), b1.cuda())
    kernels.gated_norm_step(h, tokens, width, eps, add=add, norm=(w2.cuda(), b2.cuda(), normed))
    gated = torch.sigmoid((gate[:, 3:3 + width] + bias).double()) * y0.double()
    want = h0.double() + plain.layer_norm(gated, w1.double(), b1.double(), eps)
    assert torch.allclose(h.double().cpu(), want, atol=2e-5, rtol=1e-5) and not y.any()
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    assert torch.allclose(normed.double().cpu(), plain.layer_norm(want, w2.double(), b2.double(), eps), atol=tol, rtol=tol)
    # each half alone
    h, y = h0.cuda(), y0.cuda()
    kernels.gated_norm_step(h, tokens, width, eps, add=(y,) + add[1:])
    assert torch.allclose(h.double().cpu(), want, atol=2e-5, rtol=1e-5) and not y.any()
    before = h.clone()
    kernels.gated_norm_step(h, tokens, width, eps, norm=(w2.cuda(), b2.cuda(), normed))
    assert torch.equal(h, before)
    assert torch.allclose(normed.double().cpu(), plain.layer_norm(want, w2.double(), b2.double(), eps), atol=tol, rtol=tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_relu_gate(dtype):
    kernels = _kernels()
    both = torch.randn((37, 2 * 45 + 7), generator=torch.Generator().manual_seed(1))
    out = torch.empty((37, 45), dtype=dtype, device="cuda")
    kernels.silu_gate(both.cuda()[:, :90], out, "relu")
    want = torch.relu(both[:, :45].double()) * both[:, 45:90].double()
    assert torch.allclose(out.double().cpu(), want, rtol=1e-6 if dtype == torch.float32 else 1e-2, atol=1e-6)


# ---------------------------------------------------------------- whole models
class _Reference(dict):
    """Logits per request, and how far they move where 16 bits are kept (of the largest)."""

    rounding = 0.0


def _close(rows, reference, dtype):
    worst, scale, where = helpers.max_error(rows, reference)
    allowed = TOLERANCE[dtype]
    if dtype == "bfloat16":
        allowed = max(allowed, 3 * getattr(reference, "rounding", 0.0))
    return worst <= allowed * scale, (worst / scale, allowed, where)


def _requests(raw, lengths, seed):
    return {f"r{index}": helpers.random_tokens(length, raw["vocab"], seed + index)
            for index, length in enumerate(lengths)}


def _reference(raw, tensors, requests, dtype="bfloat16"):
    out = _Reference((rid, plain.forward(raw, tensors, tokens)[0]) for rid, tokens in requests.items())
    if dtype == "bfloat16":
        scale = max(float(logits.abs().max()) for logits in out.values())
        out.rounding = max(float((plain.forward(raw, tensors, tokens, half=True)[0] - out[rid]).abs().max())
                           for rid, tokens in requests.items()) / scale
    return out


def _engine(folder, dtype, page_size, steps, max_requests=4, graphs=True):
    from pagedserve_amd.engine import Engine
    from pagedserve_amd.model import load_model

    model, _ = load_model(folder, dtype=dtype, device="cuda")
    budget = helpers.live_token_budget(steps, round_to=page_size)
    longest = max(sum(len(e["tokens"]) for e in step["entries"]) for step in steps)
    return Engine(model, num_pages=-(-budget // page_size), page_size=page_size, max_requests=max_requests,
                  max_step_tokens=max(longest, page_size), use_graphs=graphs)


LENGTHS = (58, 1, 19, 33, 7, 2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", sorted(fadosun_models.MODELS))
def test_model_whole_decoded_in_portions_and_mixed(tmp_path, which, dtype):
    folder, raw, tensors, page_size = fadosun_models.folder_of(tmp_path, which)
    requests = _requests(raw, LENGTHS, 11)
    reference = _reference(raw, tensors, requests, dtype)
    for name, steps in (("whole", helpers.trace_whole(requests)),
                        ("decoded", helpers.trace_tail_decoded(requests, tail=40)),
                        ("portions", helpers.trace_portions(requests)),
                        ("mixed", helpers.trace_mixed(requests, max_live=3))):
        engine = _engine(folder, dtype, page_size, steps, max_requests=3)
        holders = {}
        rows = helpers.replay_in_process(engine, steps, page_holders=holders)
        assert len(rows) == sum(LENGTHS)
        good, what = _close(rows, reference, dtype)
        assert good, (which, name, what)
        engine.cache.check_invariants()
        assert not engine.cache.requests and len(engine.cache.free_slots) == 3
        if name == "mixed":
            # six requests went through three slots and a pool made for the live ones only
            assert any(len(who) > 1 for who in holders.values())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_token_gives_the_same_logits_however_its_request_is_stepped(tmp_path, dtype):
    """Without an oracle between: whole, decoded and mixed runs of one engine type against each
    other, at every position."""
    folder, raw, tensors, page_size = fadosun_models.folder_of(tmp_path, "A")
    requests = _requests(raw, LENGTHS + (180,), 31)
    runs = {}
    for name, steps in (("whole", helpers.trace_whole(requests)),
                        ("decoded", helpers.trace_tail_decoded(requests, tail=60)),
                        ("mixed", helpers.trace_mixed(requests, max_live=3, seed=4))):
        engine = _engine(folder, dtype, page_size, steps, max_requests=3)
        runs[name] = helpers.replay_in_process(engine, steps)
    alone = _Reference((rid, torch.stack([runs["whole"][(rid, p)] for p in range(len(tokens))]))
                       for rid, tokens in requests.items())
    alone.rounding = _reference(raw, tensors, requests, dtype).rounding
    for name in ("decoded", "mixed"):
        good, what = _close(runs[name], alone, dtype)
        assert good, (name, what)


@pytest.mark.parametrize("which", sorted(fadosun_models.MODELS))
def test_the_stream_after_every_layer(tmp_path, which):
    from pagedserve_amd.engine import Engine, StepEntry
    from pagedserve_amd.model import load_model

    folder, raw, tensors, page_size = fadosun_models.folder_of(tmp_path, which)
    tokens = helpers.random_tokens(29, raw["vocab"], 4)
    _, after = plain.forward(raw, tensors, tokens)
    model, _ = load_model(folder, dtype="float32", device="cuda")
    caught = []
    for block in model.blocks:
        def forward(h, ctx, cache, block=block, inner=block.forward):
            out = inner(h, ctx, cache)
            block.finish(h, ctx)      # (what the block would leave to the next one's first launch)
            caught.append(h[:ctx.tokens].double().cpu())
            return out
        block.forward = forward
    engine = Engine(model, num_pages=16, page_size=page_size, max_requests=2, max_step_tokens=32, use_graphs=False)
    engine.step([StepEntry("a", tokens, [])])
    assert len(caught) == len(after) == len(raw["layers"])
    for index, (got, want) in enumerate(zip(caught, after)):
        assert torch.allclose(got, want, atol=3e-4, rtol=1e-5), (index, float((got - want).abs().max()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind,dim,heads", [("channel_delta", 16, 2), ("channel_delta", 64, 1), ("mlstm", 16, 2),
                                            ("mlstm", 64, 3), ("parallel", 16, 2), ("attention", 48, 6),
                                            ("attention", 16, 1), ("space", 16, 2), ("space", 128, 1)])
def test_what_stands_far_back_is_heard(tmp_path, kind, dim, heads, dtype):
    """One token whose key matches a query hundreds of tokens later, and nothing between them weighs much: lost
    state, a page that is not read, a maximum or a convolution that starts anew would show.  The loud token
    is the first of the request, the last of a page and the first of the next; the queries come in a prompt,
    at the start of a portion, across pieces, and decoded."""
    folder, raw, tensors = fadosun_models.far_model(tmp_path, kind, dim, heads)
    loud, ask = fadosun_models.LOUD, fadosun_models.ASK
    g = torch.Generator().manual_seed(5)
    requests = {}
    for place in (0, 7, 8, 63, 64):
        tokens = torch.randint(3, raw["vocab"], (205,), generator=g).tolist()
        tokens[place] = loud
        for at in (place + 1, 100, 128, 129, 190, 203, 204):
            tokens[at] = ask
        requests[f"p{place}"] = tokens
    reference = _reference(raw, tensors, requests, dtype)
    quiet = list(requests["p7"])
    quiet[7] = 9
    without = plain.forward(raw, tensors, quiet)[0]
    moved = (reference["p7"] - without).abs().amax(1) / reference["p7"].abs().max()
    assert float(moved[[100, 129, 204]].min()) > 2 * max(TOLERANCE[dtype], 3 * reference.rounding)
    traces = {"whole": helpers.trace_whole(requests),
              "decoded": helpers.trace_tail_decoded({"p7": requests["p7"], "p64": requests["p64"]}, tail=80),
              "portions": helpers.trace_portions(requests, sizes=(9, 2, 53, 2, 64, 65, 2, 7)),
              "mixed": helpers.trace_mixed(requests, max_live=3, portion=(66, 2, 130, 5), decode_tail=12)}
    for name, steps in traces.items():
        engine = _engine(folder, dtype, 8, steps, max_requests=3)
        rows = helpers.replay_in_process(engine, steps)
        good, what = _close(rows, reference, dtype)
        assert good, (name, what)
        engine.cache.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "C", "D"])
def test_long_prompts_whole_and_in_long_portions(tmp_path, which, dtype):
    """Prompts of several hundred tokens: the recurrences in pieces (bfloat16), attention on tiles."""
    folder, raw, tensors, page_size = fadosun_models.folder_of(tmp_path, which)
    requests = _requests(raw, (330, 200, 9), 23)
    reference = _reference(raw, tensors, requests, dtype)
    for name, steps in (("whole", helpers.trace_whole(requests)),
                        ("portions", helpers.trace_portions(requests, sizes=(160, 2, 131, 300))),
                        ("mixed", helpers.trace_mixed(requests, max_live=3, portion=(170, 129), decode_tail=3))):
        engine = _engine(folder, dtype, page_size, steps, max_requests=3)
        rows = helpers.replay_in_process(engine, steps)
        good, what = _close(rows, reference, dtype)
        assert good, (which, name, what)
        engine.cache.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B", "C", "D"])
def test_long_decoding_and_graph_replays(tmp_path, which, dtype):
    folder, raw, tensors, _ = fadosun_models.folder_of(tmp_path, which)
    requests = _requests(raw, (150, 131), 5)
    reference = _reference(raw, tensors, requests, dtype)
    # two requests decoded side by side from their third token on, pages of four tokens
    steps = [{"step": 0, "entries": [{"id": rid, "tokens": tokens[:3], "want": [0, 1, 2]}
                                      for rid, tokens in requests.items()], "end": []}]
    for index in range(3, 150):
        entries = [{"id": rid, "tokens": [tokens[index]], "want": [0]}
                   for rid, tokens in requests.items() if index < len(tokens)]
        steps.append({"step": len(steps), "entries": entries, "end": []})
    steps[-1]["end"] = list(requests)
    engine = _engine(folder, dtype, 4, steps)
    rows = helpers.replay_in_process(engine, steps)
    good, what = _close(rows, reference, dtype)
    assert good, what
    assert engine.graph_summary()["graph_replays"] > 50      # decode steps ran as recorded graphs


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_twenty_requests_decoding_together(tmp_path, dtype):
    """Lists of rows beyond the sixteen that the smallest products take."""
    folder, raw, tensors, page_size = fadosun_models.folder_of(tmp_path, "C")
    requests = _requests(raw, tuple(20 + 4 * index for index in range(20)), 71)
    reference = _reference(raw, tensors, requests, dtype)
    tail = 6
    steps = [{"step": index, "entries": [{"id": rid, "tokens": tokens[:-tail], "want": [len(tokens) - tail - 1]}],
              "end": []} for index, (rid, tokens) in enumerate(requests.items())]
    for back in range(tail, 0, -1):
        steps.append({"step": len(steps), "entries": [{"id": rid, "tokens": [tokens[-back]], "want": [0]}
                                                      for rid, tokens in requests.items()], "end": []})
    steps[-1]["end"] = list(requests)
    engine = _engine(folder, dtype, page_size, steps, max_requests=20)
    rows = helpers.replay_in_process(engine, steps)
    assert len(rows) == 20 * (tail + 1)
    good, what = _close(rows, reference, dtype)
    assert good, what
    engine.cache.check_invariants()


@pytest.mark.parametrize("which", ["A", "B", "D", "E"])
def test_greedy_generation_through_the_scheduler(tmp_path, which):
    from pagedserve_amd.engine.llm import LLM
    from pagedserve_amd.sampling import SamplingParams

    folder, raw, tensors, page_size = fadosun_models.folder_of(tmp_path, which)
    prompts = [helpers.random_tokens(length, raw["vocab"], 40 + length) for length in (9, 1, 21, 5, 14)]
    count = 10
    expected = [plain.greedy_generate(raw, tensors, prompt, count) for prompt in prompts]
    llm = LLM(folder, dtype="float32", num_kv_pages=48, block_size=page_size, max_batch_size=3,
              eos_token_id=None, prefill_chunk_size=6, scheduling_strategy="sarathi")
    outputs = llm.generate(prompts, SamplingParams(max_new_tokens=count))
    assert [output.token_ids for output in outputs] == expected
    llm.engine.cache.check_invariants()
    assert not llm.engine.cache.requests


def _drawn_configuration(seed):
    """A configuration whose every size and constant comes from a seeded generator."""
    import random

    rng = random.Random(seed)

    def ff():
        return rng.choice([None, 7, 24, 64, 100])

    layers = []
    for _ in range(rng.randint(1, 5)):
        kind = rng.choice(["delta", "memory", "parallel"])
        groups = rng.choice([1, 1, 2, 3])
        if kind == "delta":
            layers.append(fadosun_models._delta(groups * rng.choice([1, 2, 4]), groups, rng.choice([2, 6, 16, 33, 64, 96]),
                                                rng.choice([1, 5, 16, 40, 64]), rng.randint(1, 6), ff(),
                                                decay_rank=rng.choice([1, 7, 16]), gate_rank=rng.choice([3, 8, 20])))
        elif kind == "memory":
            layers.append(fadosun_models._memory(rng.choice([1, 2, 5]), rng.choice([3, 8, 32, 64, 100]),
                                                 rng.choice([2, 16, 31, 64, 90]), rng.choice([1.5, 8.0, 15.0]), ff()))
        else:
            dim = rng.choice([4, 10, 32, 64, 96, 130])
            rot = rng.choice([None, (2, 100.0), (dim // 2 // 2 * 2 or 2, 10000.0), (dim // 2 * 2, 5e5)])
            left = (groups * rng.choice([1, 2, 6, 8]), groups, dim, rng.choice([3, 16, 48, 64, 150]),
                    round(dim ** -0.5 * rng.uniform(0.5, 1.5), 4), rot)
            g = rng.choice([1, 2, 3])
            heads, vdim = g * rng.choice([1, 2, 4]), rng.choice([2, 8, 20, 48])
            norm_groups = rng.choice([n for n in (1, 2, heads, 2 * heads) if heads * vdim % n == 0])
            right = (heads, vdim, rng.choice([1, 8, 30, 64, 128]), g, rng.randint(1, 5), norm_groups)
            layers.append(fadosun_models._parallel(left, right, (round(rng.uniform(0.3, 2.0), 2),
                                                                 round(rng.uniform(-1.5, 1.5), 2)), ff()))
    raw = fadosun_models._model(rng.randint(30, 300), rng.choice([24, 40, 72, 136, 200]), rng.choice([1e-5, 1e-6]), *layers)
    return raw, rng.choice([4, 8, 16])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(16))
def test_drawn_configurations(tmp_path, seed, dtype):
    """Configurations drawn from seeds, stepped as a mixed trace of five requests through four
    slots, whole, and decoded over a tail, against the plain implementation at every position."""
    raw, page_size = _drawn_configuration(seed)
    folder = os.path.join(str(tmp_path), f"drawn_{seed}")
    tensors = fadosun_models.write_folder(folder, raw, plain.random_checkpoint(raw, 100 + seed))
    requests = _requests(raw, (150, 1, 17, 70, 2), 7 + seed)
    reference = _reference(raw, tensors, requests, dtype)
    for name, steps in (("mixed", helpers.trace_mixed(requests, max_live=4, portion=(70, 2, 31, 9), seed=seed)),
                        ("whole", helpers.trace_whole(requests)),
                        ("decoded", helpers.trace_tail_decoded({"r3": requests["r3"]}, tail=50))):
        engine = _engine(folder, dtype, page_size, steps, max_requests=4)
        rows = helpers.replay_in_process(engine, steps)
        good, what = _close(rows, reference, dtype)
        assert good, (seed, name, what, raw)
        engine.cache.check_invariants()


def test_the_trace_program_replays_a_mixed_trace(tmp_path):
    """``bin/trace_run`` as a user calls it, on a Fadosun folder: JSON lines in, ``<step>.f32``
    files and ``done`` lines out, a pool made for the live requests only."""
    import json
    import subprocess
    import sys

    import numpy as np

    folder, raw, tensors, _ = fadosun_models.folder_of(tmp_path, "C")
    requests = _requests(raw, (170, 1, 23, 40, 9), 31)
    reference = _reference(raw, tensors, requests, "float32")
    steps = helpers.trace_mixed(requests, max_live=4, seed=3)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out_dir = tmp_path / "out"
    process = subprocess.run(
        [sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
         "--out", str(out_dir), "--max-tokens", str(helpers.live_token_budget(steps))],
        input="\n".join(json.dumps(step) for step in steps) + "\n", capture_output=True, text=True, timeout=600)
    assert process.returncode == 0, process.stderr[-2000:]
    done = [line for line in process.stdout.splitlines() if line.startswith("done ")]
    assert done == [f"done {step['step']}" for step in steps]
    held, rows = {}, {}
    for step in steps:
        wanted = sum(len(entry["want"]) for entry in step["entries"])
        values = np.fromfile(out_dir / f"{step['step']}.f32", dtype="<f4").reshape(wanted, raw["vocab"])
        row = 0
        for entry in step["entries"]:
            start = held.get(entry["id"], 0)
            for place in entry["want"]:
                rows[(entry["id"], start + place)] = torch.from_numpy(values[row]).double()
                row += 1
            held[entry["id"]] = start + len(entry["tokens"])
    worst, scale, where = helpers.max_error(rows, reference)
    assert len(rows) == sum(len(tokens) for tokens in requests.values())
    assert worst <= TOLERANCE["float32"] * scale, (worst / scale, where)
