"""Malalix on the GPU against the plain implementation (``plain_malalix.py``): each new kernel or
kernel option alone (attention inside chunks in every attention kernel, heads normed ahead of the
rotation, the router over the chosen logits with a gate for the shared expert, the capped gated unit,
the stream step of two norms), then small models of several shapes stepped whole, decoded token by
token, in portions down to two tokens, and in mixed batches whose pages and slots are used again;
keys that stand out at a chunk's edges."""

import os

import pytest
import torch

import helpers
import malalix_models
import plain_malalix as plain

pytestmark = pytest.mark.gpu

F64 = torch.float64
# |engine - plain| <= TOLERANCE * max|plain logits|
TOLERANCE = {"float32": 5e-5, "bfloat16": 3e-2}


def _kernels():
    from pagedserve_amd.ops import kernels

    return kernels


def _ints(values):
    return torch.tensor(values, dtype=torch.int32, device="cuda")


# ---------------------------------------------------------------- attention inside chunks
class _Paged:
    """Keys and values of requests in a pool whose other places hold NaN, with block tables that
    list only the pages that the next positions may see (the others were given back)."""

    def __init__(self, dtype, kv_heads, dim, page_size, portions, chunk, seed):
        g = torch.Generator().manual_seed(seed)
        longest = max(start + count for start, count in portions)
        width = -(-longest // page_size) + 1
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
            first_page = (start // chunk * chunk) // page_size
            for logical in range(first_page, -(-total // page_size)):
                page = order.pop()
                tables[item, logical] = page
                for place in range(page_size):
                    position = logical * page_size + place
                    if position < total:
                        k_pool[page, :, place] = k[position].float()
                        v_pool[page, :, place] = v[position].float()
        self.k_pool, self.v_pool = k_pool.to(dtype).cuda(), v_pool.to(dtype).cuda()
        self.tables = tables.cuda()
        tokens = [(item, start + i) for item, (start, count) in enumerate(portions) for i in range(count)]
        self.tok_item, self.positions = _ints([t[0] for t in tokens]), _ints([t[1] for t in tokens])
        counts = [count for _, count in portions]
        self.cu = _ints([sum(counts[:i]) for i in range(len(counts) + 1)])
        self.kv_lens = _ints([start + count for start, count in portions])
        self.counts, self.tokens = counts, tokens

    def tiles(self, size, only=None):
        items = [(item, q0) for item, count in enumerate(self.counts) if only is None or item in only
                 for q0 in range(0, count, size)]
        return _ints([i for i, _ in items]), _ints([q for _, q in items])

    def expected(self, q, heads, scale, chunk):
        out = []
        for t, (item, position) in enumerate(self.tokens):
            k, v = self.k[item], self.v[item]
            first = position // chunk * chunk
            row = []
            for h in range(heads):
                group = h // (heads // k.shape[1])
                weights = torch.softmax((k[first:position + 1, group] @ q[t, h]) * scale, 0)
                row.append(weights @ v[first:position + 1, group])
            out.append(torch.stack(row))
        return torch.stack(out)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kv_heads,dim", [(4, 2, 16), (8, 1, 64), (2, 2, 128), (3, 1, 24)])
@pytest.mark.parametrize("chunk,page_size", [(1, 4), (16, 8), (37, 8), (64, 16), (100, 16), (512, 16)])
def test_chunked_attention_in_every_kernel(dtype, heads, kv_heads, dim, chunk, page_size):
    """Portions that begin and end inside, at and across chunk edges, single tokens at a chunk's
    first and last position; the query that a page border, a tile border and a chunk border meet."""
    kernels = _kernels()
    c = chunk
    portions = [(0, 70), (c, 5), (2 * c - 1, 2), (max(0, c - 3), 150), (3 * c, 1), (3 * c - 1, 1), (c + c // 2, 1),
                (5, 33), (7 * c, 40)]
    paged = _Paged(dtype, kv_heads, dim, page_size, portions, chunk, heads * dim + chunk)
    tokens = len(paged.tokens)
    g = torch.Generator().manual_seed(chunk)
    q = torch.randn((tokens, heads, dim), generator=g).to(dtype)
    scale = dim ** -0.5 * 1.5
    expected = paged.expected(q.double(), heads, scale, chunk)
    q = q.reshape(tokens, heads * dim).cuda()
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    pools = (paged.k_pool, paged.v_pool)
    singles = [t for t in range(tokens) if paged.counts[paged.tokens[t][0]] == 1]
    several = [t for t in range(tokens) if t not in singles]
    items_of_several = [i for i, count in enumerate(paged.counts) if count > 1]

    def check(out, which, what):
        got = out.double().cpu().view(tokens, heads, dim)
        assert torch.allclose(got[which], expected[which], atol=tol, rtol=tol), (
            what, float((got[which] - expected[which]).abs().max()))

    def fresh():
        return torch.full((tokens, heads * dim), 9.0, dtype=dtype, device="cuda")

    everyone = list(range(tokens))
    out = fresh()
    kernels.attention_rowwise(q, *pools, out, paged.tok_item, paged.positions, paged.tables, heads, scale, -chunk)
    check(out, everyone, "rowwise")
    for splits, waves in ((1, 4), (1, 16), (3, 4), (7, 4)):
        out = fresh()
        partial = torch.empty(tokens * heads * splits * (dim + 2), device="cuda")
        kernels.attention_decode(q, *pools, out, paged.tok_item, paged.positions, paged.tables, heads, scale, splits,
                                 partial=partial, window=-chunk, waves=waves)
        check(out, everyone, ("decode", splits, waves))
    if kernels.shared_decode_supported(dtype, heads, kv_heads, dim):
        for splits in (1, 3):
            out = fresh()
            partial = torch.empty(tokens * heads * splits * (dim + 2), device="cuda")
            kernels.attention_decode_shared(q, *pools, out, paged.tok_item, paged.positions, paged.tables, heads,
                                            scale, splits, partial, window=-chunk)
            check(out, everyone, ("shared decode", splits))
    if kernels.tiled_f32_supported(dtype, dim):
        out = fresh()
        kernels.attention_tiled_f32(q, *pools, out, *paged.tiles(64), paged.cu, paged.kv_lens, paged.tables, heads,
                                    scale, -chunk)
        check(out, everyone, "tiled f32")
    if kernels.prefill_supported(dtype, dim, paged.tables.shape[1]):
        sizes = [64] + ([32] if dim <= 128 else []) + ([128] if dim <= 64 else [])
        for size in sizes:
            for longest in (0, 100):
                out = fresh()
                kernels.attention_prefill(q, *pools, out, *paged.tiles(size), paged.cu, paged.kv_lens, paged.tables,
                                          heads, scale, -chunk, max_kv_len=longest, query_tile=size)
                check(out, everyone, ("prefill", size, longest))
    if kernels.mixed_supported(dtype, dim, paged.tables.shape[1]):
        out = fresh()
        kernels.attention_mixed(q, *pools, out, _ints(singles), paged.tok_item, paged.positions,
                                *paged.tiles(64, items_of_several), paged.cu, paged.kv_lens, paged.tables, heads,
                                scale, -chunk)
        check(out, singles, "mixed, single tokens")
        check(out, several, "mixed, portions")


# ---------------------------------------------------------------- kernels alone
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,rot", [(4, 2, 16, 24, (8, 100.0, (4.0, 1.0, 3.0, 40))), (3, 3, 12, 20, (6, 50.0)),
                                                         (2, 1, 136, 40, (2, 7.0)), (8, 1, 64, 32, (64, 1000.0)),
                                                         (2, 1, 10, 10, None), (1, 1, 256, 256, (256, 10000.0))])
def test_heads_normed_with_a_weight_ahead_of_the_rotation(dtype, heads, kv_heads, dim, vdim, rot):
    from pagedserve_amd.parts.position import banded_frequencies, rotary_frequencies

    kernels = _kernels()
    g = torch.Generator().manual_seed(dim + vdim)
    page_size, pages = 4, 700
    positions, items = [0, 1, 5, 2, 2047], [0, 0, 0, 1, 0]
    tokens = len(positions)
    cache_dim = -(-max(dim, vdim) // 16) * 16
    total = 3 + heads * dim + kv_heads * (dim + vdim)
    q_col, k_col, v_col = 1, 1 + heads * dim, 1 + heads * dim + kv_heads * dim
    proj = torch.randn((tokens, total), generator=g) * 3
    q_gamma, k_gamma = 1 + 0.3 * torch.randn(dim, generator=g), 1 + 0.3 * torch.randn(dim, generator=g)
    tables = torch.full((2, 600), -1, dtype=torch.int32)
    order = torch.randperm(pages, generator=g).tolist()
    for item, position in zip(items, positions):
        if tables[item, position // page_size] < 0:
            tables[item, position // page_size] = order.pop()
    k_pool = torch.full((pages, kv_heads, page_size, cache_dim), float("nan"), dtype=dtype, device="cuda")
    v_pool = torch.full_like(k_pool, float("nan"))
    q_out = torch.full((tokens, heads * cache_dim), 5.0, dtype=dtype, device="cuda")
    spec, dims, freqs = None, 0, None
    if rot:
        dims = rot[0]
        spec = malalix_models._rot(*rot)
        freqs = (banded_frequencies(dims, rot[1], *rot[2]) if len(rot) > 2 else rotary_frequencies(dims, rot[1])[0])
        freqs = freqs.float().cuda()
    kernels.attention_prepare_heads(proj.cuda(), (q_col, k_col, v_col), q_out, k_pool, v_pool, _ints(items),
                                    _ints(positions), tables.cuda(), heads, dim, vdim, freqs=freqs, rot_dims=dims,
                                    halves=True, head_norm=True, norm_first=True, q_gamma=q_gamma.cuda(),
                                    k_gamma=k_gamma.cuda(), eps=1e-5)
    at = torch.tensor(positions)
    queries = proj[:, q_col:k_col].double().view(tokens, heads, dim)
    keys = proj[:, k_col:v_col].double().view(tokens, kv_heads, dim)
    values = proj[:, v_col:v_col + kv_heads * vdim].double().view(tokens, kv_heads, vdim)
    queries = plain.rotate_halves(plain.rms_norm(queries, q_gamma.double(), 1e-5), at, spec)
    keys = plain.rotate_halves(plain.rms_norm(keys, k_gamma.double(), 1e-5), at, spec)
    # (the angle is a 32-bit product: at position 2,047 it is off by some 1e-4)
    tol = 1e-3 if dtype == torch.float32 else 3e-2
    got = q_out.double().cpu().view(tokens, heads, cache_dim)
    assert torch.allclose(got[..., :dim], queries, atol=tol, rtol=tol)
    assert torch.allclose(got[:4, :, :dim], queries[:4], atol=max(tol / 50, 1e-5) if dtype == torch.float32 else tol)
    assert float(got[..., dim:].abs().sum()) == 0.0
    for t in range(tokens):
        page, place = int(tables[items[t], positions[t] // page_size]), positions[t] % page_size
        assert torch.allclose(k_pool[page, :, place, :dim].double().cpu(), keys[t], atol=tol, rtol=tol)
        assert torch.allclose(v_pool[page, :, place, :vdim].double().cpu(), values[t], atol=tol, rtol=tol)
        assert float(k_pool[page, :, place, dim:].abs().sum()) == 0.0
        assert float(v_pool[page, :, place, vdim:].abs().sum()) == 0.0


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,top", [(6, 2), (12, 5), (4, 4), (1, 1), (64, 8), (65, 3), (130, 7)])
def test_router_over_the_chosen_logits_and_the_shared_experts_gate(dtype, experts, top):
    kernels = _kernels()
    g = torch.Generator().manual_seed(experts + top)
    tokens, width = 37, 300
    x = torch.randn((tokens, width), generator=g).to(dtype)
    router = torch.randn((experts, width), generator=g) * 0.3
    if experts > 2:
        router[0] *= 30.0       # logits far apart: a softmax over all experts would underflow
    gate = torch.randn(width, generator=g) * 0.1
    chosen, weights = plain.route(x.double() @ router.double().T, top)
    wanted = torch.sigmoid(x.double() @ gate.double())

    def check(ids, got):
        for t in range(tokens):
            assert sorted(ids[t, :top].tolist()) == sorted(chosen[t]), t
            by_id = dict(zip(chosen[t], weights[t].tolist()))
            for e, weight in zip(ids[t, :top].tolist(), got[t, :top].tolist()):
                assert abs(weight - by_id[e]) <= 2e-5

    ids = torch.full((tokens, top), -1, dtype=torch.int32, device="cuda")
    got = torch.zeros((tokens, top), device="cuda")
    kernels.moe_route(x.cuda(), router.cuda(), 1, 1, top, 1.0, ids, got, score="chosen_softmax")
    check(ids.cpu(), got.double().cpu())
    gates = torch.full((tokens + 2,), 7.0, device="cuda")
    kernels.moe_route(x.cuda(), router.cuda(), 1, 1, top, 1.0, ids, got, score="chosen_softmax", gate=gate.cuda(),
                      gate_out=gates[:tokens])
    check(ids.cpu(), got.double().cpu())
    assert torch.allclose(gates[:tokens].double().cpu(), wanted, atol=2e-6) and gates[tokens:].tolist() == [7.0, 7.0]
    ids = torch.full((tokens, top + 1), -1, dtype=torch.int32, device="cuda")
    got = torch.zeros((tokens, top + 1), device="cuda")
    kernels.moe_route(x.cuda(), router.cuda(), 1, 1, top, 1.0, ids, got, score="chosen_softmax", gate=gate.cuda(),
                      fixed=True)
    check(ids.cpu(), got.double().cpu())
    assert ids[:, top].tolist() == [experts] * tokens
    assert torch.allclose(got[:, top].double().cpu(), wanted, atol=2e-6)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,inner,shared,experts,top,tokens", [(48, 20, 36, 5, 2, 19), (128, 96, 32, 4, 3, 7),
                                                                   (44, 24, 24, 5, 1, 3), (64, 40, 8, 5, 2, 150),
                                                                   (72, 136, 200, 7, 1, 333), (24, 16, 15, 3, 2, 100)])
def test_capped_experts_by_rows_sorted_and_beside_a_gated_shared_one(dtype, width, inner, shared, experts, top, tokens):
    kernels = _kernels()
    g = torch.Generator().manual_seed(width + inner)
    limit, shared_limit = 0.9, 1.6
    form = (limit, 1.702, 1.0)
    x = torch.randn((tokens, width), generator=g).to(dtype)
    w1 = (torch.randn((experts, 2 * inner, width), generator=g) * 2 / width ** 0.5).to(dtype)
    w2 = (torch.randn((experts, width, inner), generator=g) / inner ** 0.5).to(dtype)
    s1 = (torch.randn((2 * shared, width), generator=g) * 2 / width ** 0.5).to(dtype)
    s2 = (torch.randn((width, shared), generator=g) / shared ** 0.5).to(dtype)
    ids = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(tokens)]).to(torch.int32)
    weights = torch.rand((tokens, top), generator=g)
    gate = torch.rand(tokens, generator=g)
    y0 = torch.randn((tokens, width), generator=g)

    def unit(rows, matrix, columns, cap):
        both = rows.double() @ matrix.double().T
        return plain.capped_gate(both[:, :columns], both[:, columns:], cap)

    routed = y0.double().clone()
    for t in range(tokens):
        for j in range(top):
            e = int(ids[t, j])
            routed[t] += float(weights[t, j]) * (unit(x[t:t + 1], w1[e], inner, limit) @ w2[e].double().T)[0]
    own = gate.double()[:, None] * (unit(x, s1, shared, shared_limit) @ s2.double().T)
    tol = 1e-4 if dtype == torch.float32 else 4e-2
    y = y0.clone().cuda()
    hidden = torch.empty((tokens, top * inner + shared), dtype=dtype, device="cuda")
    kernels.moe_experts(x.cuda(), w1.cuda(), w2.cuda(), ids.cuda(), weights.cuda(), hidden, y, form=form)
    assert torch.allclose(y.double().cpu(), routed, atol=tol, rtol=tol)
    # the shared expert as the last choice of every token
    ids_x = torch.cat([ids, torch.full((tokens, 1), experts, dtype=torch.int32)], 1).cuda()
    weights_x = torch.cat([weights, gate[:, None]], 1).cuda()
    y = y0.clone().cuda()
    kernels.moe_experts(x.cuda(), w1.cuda(), w2.cuda(), ids_x, weights_x, hidden, y, form=form,
                        extra=(s1.cuda(), s2.cuda()), extra_limit=shared_limit)
    assert torch.allclose(y.double().cpu(), routed + own, atol=tol, rtol=tol)
    if dtype == torch.bfloat16 and tokens * top >= kernels.MOE_GROUPED_FROM:
        assert kernels.moe_grouped_supported(dtype, width, inner)
        pairs = tokens * top
        tiles = kernels.moe_grouped_tiles(pairs, experts)
        y = y0.clone().cuda()
        kernels.moe_experts_grouped(
            x.cuda(), w1.cuda(), w2.cuda(), ids.cuda(), weights.cuda(), hidden,
            torch.empty((pairs, width), device="cuda"),
            torch.empty(tiles * kernels.MOE_TILE, dtype=torch.int32, device="cuda"),
            torch.empty(tiles, dtype=torch.int32, device="cuda"), y, form=form)
        assert torch.allclose(y.double().cpu(), routed, atol=tol, rtol=tol)
    # the unit alone, rows scaled (the shared expert of steps of many tokens)
    both = (x.double() @ s1.double().T).float()
    out = torch.empty((tokens, shared), dtype=dtype, device="cuda")
    kernels.silu_gate(both.cuda(), out, form=(shared_limit, 1.702, 1.0), row_scale=gate.cuda())
    want = plain.capped_gate(both[:, :shared].double(), both[:, shared:].double(), shared_limit) * gate.double()[:, None]
    assert torch.allclose(out.double().cpu(), want, atol=tol / 2, rtol=tol / 2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [40, 64, 300, 1030])
def test_stream_step_of_two_norms_that_adds_rows_and_the_embedding_kept(dtype, width):
    kernels = _kernels()
    g = torch.Generator().manual_seed(width)
    tokens, vocab, eps = 9, 31, 1e-5
    table = torch.randn((vocab, width), generator=g).to(dtype)
    ids = torch.randint(0, vocab, (tokens,), generator=g, dtype=torch.int32)
    h = torch.zeros((tokens + 1, width), device="cuda")
    copy = torch.full((tokens + 1, width), 3.0, device="cuda")
    kernels.embed(table.cuda(), None, ids.cuda(), None, h, copy=copy)
    embedded = table[ids.long()].double()
    assert torch.equal(h[:tokens].double().cpu(), embedded) and torch.equal(copy[:tokens], h[:tokens])
    assert float((copy[tokens:] - 3.0).abs().sum()) == 0.0
    extra = torch.randn((tokens, width), generator=g)
    h[:tokens] += extra.cuda()
    bias = torch.randn(width, generator=g)
    gamma1, gamma2 = torch.randn(width, generator=g), torch.randn(width, generator=g)
    n1 = torch.zeros((tokens, width), dtype=dtype, device="cuda")
    n2 = torch.zeros_like(n1)
    kernels.stream_step(h, tokens, width, rows=copy, bias=bias.cuda(), norm=(gamma1.cuda(), eps, n1),
                        norm2=(gamma2.cuda(), n2))
    x = embedded + extra.double() + embedded + bias.double()
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert torch.allclose(h[:tokens].double().cpu(), x, atol=1e-5)
    assert torch.allclose(n1.double().cpu(), plain.rms_norm(x, gamma1.double(), eps), atol=tol, rtol=tol)
    assert torch.allclose(n2.double().cpu(), plain.rms_norm(x, gamma2.double(), eps), atol=tol, rtol=tol)
    # nothing to add: the stream stays as it is
    before = h.clone()
    kernels.stream_step(h, tokens, width, norm=(gamma1.cuda(), eps, n1), norm2=(gamma2.cuda(), n2))
    assert torch.equal(h, before)
    with pytest.raises(Exception):
        kernels.stream_step(h, tokens, width, norm2=(gamma2.cuda(), n2))


# ---------------------------------------------------------------- whole models
def _close(rows, reference, dtype):
    """Every position within the tolerance (the bfloat16 runs use routers that make no close calls)."""
    worst, scale, where = helpers.max_error(rows, reference)
    return worst <= TOLERANCE[dtype] * scale, (worst / scale, where)


def _requests(raw, lengths, seed):
    return {f"r{index}": helpers.random_tokens(length, raw["vocab"], seed + index)
            for index, length in enumerate(lengths)}


def _reference(raw, tensors, requests):
    return {rid: plain.forward(raw, tensors, tokens)[0] for rid, tokens in requests.items()}


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
@pytest.mark.parametrize("which", sorted(malalix_models.MODELS))
def test_model_whole_decoded_in_portions_and_mixed(tmp_path, which, dtype):
    folder, raw, tensors, page_size = malalix_models.folder_for(tmp_path, which, dtype)
    requests = _requests(raw, LENGTHS, 11)
    reference = _reference(raw, tensors, requests)
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
    folder, raw, _, page_size = malalix_models.folder_for(tmp_path, "A", dtype)
    requests = _requests(raw, LENGTHS, 31)
    runs = {}
    for name, steps in (("whole", helpers.trace_whole(requests)),
                        ("decoded", helpers.trace_tail_decoded(requests, tail=60)),
                        ("mixed", helpers.trace_mixed(requests, max_live=3, seed=4))):
        engine = _engine(folder, dtype, page_size, steps, max_requests=3)
        runs[name] = helpers.replay_in_process(engine, steps)
    alone = {rid: torch.stack([runs["whole"][(rid, p)] for p in range(len(tokens))])
             for rid, tokens in requests.items()}
    for name in ("decoded", "mixed"):
        good, what = _close(runs[name], alone, dtype)
        assert good, (name, what)


@pytest.mark.parametrize("which", sorted(malalix_models.MODELS))
def test_the_stream_after_every_layer_run(tmp_path, which):
    from pagedserve_amd.engine import Engine, StepEntry
    from pagedserve_amd.model import load_model

    folder, raw, tensors, page_size = malalix_models.folder_of(tmp_path, which)
    tokens = helpers.random_tokens(29, raw["vocab"], 4)
    _, after = plain.forward(raw, tensors, tokens)
    model, _ = load_model(folder, dtype="float32", device="cuda")
    caught = []
    for block in model.blocks:
        def forward(h, ctx, cache, inner=block.forward):
            out = inner(h, ctx, cache)
            caught.append(h[:ctx.tokens].double().cpu())
            return out
        block.forward = forward
    engine = Engine(model, num_pages=8, page_size=page_size, max_requests=2, max_step_tokens=32, use_graphs=False)
    engine.step([StepEntry("a", tokens, [])])
    assert len(caught) == len(after) == len(plain.run_order(raw))
    for index, (got, want) in enumerate(zip(caught, after)):
        assert torch.allclose(got, want, atol=3e-4, rtol=1e-5), (index, float((got - want).abs().max()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("size,heads,kv_heads,dim", [(24, 2, 1, 16), (13, 6, 1, 32), (16, 2, 2, 64)])
def test_a_loud_key_just_inside_and_just_outside_the_chunk(tmp_path, size, heads, kv_heads, dim, dtype):
    """One key that takes nearly all the weight of the queries that match it and see it.  It stands
    at the first, a middle and the last place of the second chunk (a page holds 8 tokens), and
    queries that match it at every place around the chunk's end: heard up to the chunk's last
    place, not at the next one, in the second layer three places later; in a prompt, at the start
    of a portion, and decoded one by one."""
    folder, raw, tensors = malalix_models.loud_key_model(tmp_path, size, heads, kv_heads, dim, sure=dtype == "bfloat16")
    loud, ask = malalix_models.LOUD, malalix_models.ASK
    g = torch.Generator().manual_seed(5)

    def filler(count):
        return (torch.randint(3, raw["vocab"], (count,), generator=g)).tolist()

    requests = {}
    end = 2 * size
    for place in (size - 1, size, size + 5, end - 2):
        tokens = filler(end + 9)
        for at in (end - 1, end, end + 1, end + 4, end + 6):
            tokens[at] = ask
        tokens[place] = loud
        requests[f"p{place}"] = tokens
    reference = _reference(raw, tensors, requests)
    # what the loud key is worth: at the chunk's last place it is heard
    quiet = list(requests[f"p{size}"])
    quiet[size] = 5
    without, _ = plain.forward(raw, tensors, quiet)
    moved = (reference[f"p{size}"] - without).abs().amax(1) / reference[f"p{size}"].abs().max()
    assert float(moved[end - 1]) > 0.05
    # and a chunk one place longer, or shorter, would show at the queries around its end
    for other in (size - 1, size + 1):
        import copy
        changed = copy.deepcopy(raw)
        changed["layers"][0]["mixer"]["mask"]["size"] = other
        wrong, _ = plain.forward(changed, tensors, requests[f"p{size}"])
        assert float((wrong - reference[f"p{size}"]).abs().max()) > 0.05 * float(reference[f"p{size}"].abs().max())
    traces = {"whole": helpers.trace_whole(requests),
              "decoded": helpers.trace_tail_decoded(requests, tail=size + 14),
              "portions": helpers.trace_portions(requests, sizes=(9, 2, 3, 2, 11, 5, 2, 7)),
              "edges": helpers.trace_portions(requests, sizes=(size, size - 1, 2, 2, 5)),
              "mixed": helpers.trace_mixed(requests, max_live=3, decode_tail=20)}
    for name, steps in traces.items():
        engine = _engine(folder, dtype, 8, steps, max_requests=3)
        rows = helpers.replay_in_process(engine, steps)
        good, what = _close(rows, reference, dtype)
        assert good, (name, what)
        engine.cache.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "C", "D"])
def test_long_prompts_whole_and_in_long_portions(tmp_path, which, dtype):
    """Prompts of several hundred tokens: attention on tiles over many chunks whose pages were given
    back, the experts sorted onto the matrix cores with the shared one as dense products."""
    folder, raw, tensors, page_size = malalix_models.folder_for(tmp_path, which, dtype)
    requests = _requests(raw, (330, 200, 9), 23)
    reference = _reference(raw, tensors, requests)
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
def test_long_decoding_over_many_chunks_and_graph_replays(tmp_path, which, dtype):
    folder, raw, tensors, _ = malalix_models.folder_for(tmp_path, which, dtype)
    requests = _requests(raw, (150, 131), 5)
    reference = _reference(raw, tensors, requests)
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
    """Lists of rows beyond the sixteen that the smallest products take, contexts of different
    chunks side by side."""
    folder, raw, tensors, page_size = malalix_models.folder_for(tmp_path, "C", dtype)
    requests = _requests(raw, tuple(40 + 5 * index for index in range(20)), 71)
    reference = _reference(raw, tensors, requests)
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

    folder, raw, tensors, page_size = malalix_models.folder_of(tmp_path, which)
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
    """A configuration whose every size and constant comes from a seeded generator: widths and
    vocabularies that are multiples of nothing, one to eight heads on one to three key/value
    heads, keys of 4 to 200, values of 3 to 200, chunks of one token to none, rotations of none of
    the dimensions to all, 1 to 70 experts, loops of any layers."""
    import random

    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(1, 4)):
        kv_heads = rng.choice([1, 1, 2, 3])
        dim = rng.choice([4, 6, 8, 20, 32, 64, 100, 128, 200])
        rot = None
        if rng.random() < 0.85:
            dims = rng.choice([2, dim // 2 // 2 * 2 or 2, dim])
            scaling = None
            if rng.random() < 0.6:
                low = rng.choice([0.5, 1.0, 2.0])
                scaling = (rng.choice([2.0, 8.0]), low, low * rng.choice([1.5, 4.0]), rng.choice([24, 64, 500]))
            rot = malalix_models._rot(dims, rng.choice([10.0, 500.0, 10000.0, 1e6]), scaling)
        mlp = None
        if rng.random() < 0.8:
            experts = rng.choice([1, 2, 4, 7, 12, 64, 70])
            shared = rng.choice([None, (rng.choice([5, 16, 48]), round(rng.uniform(0.5, 3.0), 2))])
            mlp = malalix_models._moe(rng.choice([6, 16, 40]), round(rng.uniform(0.5, 3.0), 2), experts,
                                      rng.randint(1, min(8, experts)), shared)
        layers.append(malalix_models._layer(
            kv_heads * rng.choice([1, 1, 2, 4, 8]), kv_heads, dim, rng.choice([3, 10, 16, 40, 64, 128, 200]),
            round(dim ** -0.5 * rng.uniform(0.7, 2.0), 4), rng.choice([1, 2, 5, 8, 16, 17, 40, 64, None]), rot, mlp))
    raw = {"architecture": "Malalix", "vocab": rng.randint(30, 300), "width": rng.choice([24, 40, 72, 136, 200]),
           "norm": {"eps": rng.choice([1e-5, 1e-6])}, "layers": layers}
    if rng.random() < 0.8:
        start = rng.randrange(len(layers))
        raw["loop"] = {"start": start, "stop": rng.randint(start + 1, len(layers)), "times": rng.randint(1, 3)}
    return raw, rng.choice([4, 8, 16])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(16))
def test_drawn_configurations(tmp_path, seed, dtype):
    """Configurations drawn from seeds, stepped as a mixed trace of five requests through four
    slots, whole, and decoded over a tail that passes most chunks, against the plain
    implementation at every position."""
    raw, page_size = _drawn_configuration(seed)
    weights = plain.random_checkpoint(raw, 100 + seed)
    if dtype == "bfloat16":
        weights = malalix_models.without_close_calls(raw, weights, seed)
    folder = os.path.join(str(tmp_path), f"drawn_{seed}")
    tensors = malalix_models.write_folder(folder, raw, weights)
    requests = _requests(raw, (150, 1, 17, 70, 2), 7 + seed)
    reference = _reference(raw, tensors, requests)
    for name, steps in (("mixed", helpers.trace_mixed(requests, max_live=4, portion=(70, 2, 31, 9), seed=seed)),
                        ("whole", helpers.trace_whole(requests)),
                        ("decoded", helpers.trace_tail_decoded({"r3": requests["r3"]}, tail=50))):
        engine = _engine(folder, dtype, page_size, steps, max_requests=4)
        rows = helpers.replay_in_process(engine, steps)
        good, what = _close(rows, reference, dtype)
        assert good, (seed, name, what, raw)
        engine.cache.check_invariants()


def test_the_trace_program_replays_a_mixed_trace(tmp_path):
    """``bin/trace_run`` as a user calls it, on a Malalix folder: JSON lines in, ``<step>.f32``
    files and ``done`` lines out, a pool made for the live requests only."""
    import json
    import subprocess
    import sys

    import numpy as np

    folder, raw, tensors, _ = malalix_models.folder_of(tmp_path, "C")
    requests = _requests(raw, (170, 1, 23, 40, 9), 31)
    reference = _reference(raw, tensors, requests)
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
