"""Malalix without a GPU: the configuration reader, the model's description as parts (passes with
cache entries of their own, chunk sizes, what is added before a pass), the map from checkpoint
tensors to parameters, what the cache holds and gives back at a chunk's end, the stretched
frequencies, and the plain implementation's own consistency and sensitivity."""

import copy
import json
import math

import pytest
import torch

import malalix_models
import plain_malalix as plain
from pagedserve_amd.cache.manager import CacheGroupSpec, CacheManager
from pagedserve_amd.config.base import ConfigError
from pagedserve_amd.config.malalix import MalalixConfig
from pagedserve_amd.config.registry import resolve_architecture
from pagedserve_amd.model import load_model
from pagedserve_amd.parts.position import banded_frequencies

F64 = torch.float64


def test_the_architecture_is_found_by_its_name():
    entry = resolve_architecture({"architecture": "Malalix"})
    assert entry.name == "Malalix" and entry.config_class is MalalixConfig


@pytest.mark.parametrize("which", sorted(malalix_models.MODELS))
def test_configuration_round_trip_and_spec(which):
    raw = malalix_models.MODELS[which][0]
    config = MalalixConfig.from_dict(raw)
    assert MalalixConfig.from_dict(config.to_dict()) == config
    spec = resolve_architecture(raw).build_spec(config)
    assert spec.vocab_size == raw["vocab"] and not spec.tie_head and not spec.streams
    loop = raw.get("loop")
    assert spec.pass_rows == (loop["times"] if loop else 0)
    order = plain.run_order(raw)
    assert [call.block for call in spec.schedule] == [layer for layer, _ in order]
    assert [call.enter for call in spec.schedule] == [-1 if turn is None else turn for _, turn in order]
    assert [call.add_embedding for call in spec.schedule] == [bool(turn) for _, turn in order]
    # every pass keeps keys and values of its own
    assert [call.cache for call in spec.schedule] == list(range(len(order)))
    for layer, block in zip(raw["layers"], spec.blocks):
        mixer, wanted = dict(block.mixer.params), layer["mixer"]
        assert block.mixer.kind == "attention"
        assert (mixer["heads"], mixer["kv_heads"], mixer["head_dim"], mixer["value_dim"], mixer["scale"]) == (
            wanted["heads"], wanted["kv_heads"], wanted["dim"], wanted["vdim"], wanted["scale"])
        assert mixer["chunk"] == (wanted.get("mask") or {}).get("size", 0)
        rot = wanted.get("rot") or {}
        assert mixer["rotary_dims"] == rot.get("dims", 0)
        scaling = rot.get("scaling")
        assert mixer["rotary_bands"] == (None if not scaling else tuple(
            scaling[key] for key in ("factor", "low", "high", "original")))
        assert mixer["head_norm"] == "before" and mixer["bias"] and not mixer["out_bias"]
        mlp = layer["mlp"]
        names = [name for name, _ in block.parts]
        if mlp is None:
            assert block.arrangement == "pre_norm_mixer" and "feed_forward" not in names
            continue
        assert block.arrangement == "parallel_two_norms" and "norm2" in names
        ff = dict(block.feed_forward.params)
        assert (ff["inner"], ff["experts"], ff["top"], ff["score"]) == (
            mlp["expert"]["ff"], mlp["router"]["experts"], mlp["router"]["top"], "chosen_softmax")
        assert ff["gate_form"] == (mlp["expert"]["limit"], 1.702, 1.0)
        shared = mlp.get("shared")
        assert ff["shared_inner"] == (shared or {}).get("ff", 0) and ff["shared_gate"] == bool(shared)
        assert ff["shared_limit"] == (shared["limit"] if shared else None)


def test_configuration_errors_name_the_layer_and_key():
    raw = malalix_models.MODELS["A"][0]
    cases = [
        (lambda c: c["layers"][0].__setitem__("type", "mamba"), "layers[0]"),
        (lambda c: c["layers"][1]["mixer"].__setitem__("kv_heads", 3), "kv_heads"),
        (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
        (lambda c: c["layers"][1]["mixer"]["mask"].__setitem__("size", 0), "size"),
        (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 5), "rot.dims"),
        (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 18), "rot.dims"),
        (lambda c: c["layers"][1]["mixer"]["rot"].pop("base"), "base"),
        (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("original"), "original"),
        (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 7), "top"),
        (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "limit"),
        (lambda c: c["layers"][0]["mlp"]["shared"].pop("limit"), "limit"),
        (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "dense"), "mlp.kind"),
        (lambda c: c["loop"].__setitem__("stop", 5), "loop"),
        (lambda c: c["loop"].__setitem__("start", 3), "loop"),
        (lambda c: c["loop"].pop("times"), "times"),
        (lambda c: c["norm"].pop("eps"), "eps"),
    ]
    for change, word in cases:
        broken = copy.deepcopy(raw)
        change(broken)
        with pytest.raises(ConfigError) as caught:
            MalalixConfig.from_dict(broken)
        assert word in str(caught.value), (word, str(caught.value))


@pytest.mark.parametrize("which", sorted(malalix_models.MODELS))
def test_every_stored_tensor_feeds_a_parameter_and_the_cache_is_what_the_layers_need(tmp_path, which):
    folder, raw, tensors, _ = malalix_models.folder_of(tmp_path, which)
    model, _ = load_model(folder, dtype="float32", device="cpu")
    assert model.parameter_count == sum(t.numel() for t in tensors.values())
    groups, states = model.cache_requirements()
    order = plain.run_order(raw)
    assert not states and sum(len(group.entries) for group in groups) == len(order)
    for group in groups:
        for entry in group.entries:
            mixer = raw["layers"][order[entry][0]]["mixer"]
            assert group.chunk == (mixer.get("mask") or {}).get("size", 0) and group.window == 0
            assert group.kv_heads == mixer["kv_heads"] and group.head_dim % 16 == 0
            assert group.head_dim >= max(mixer["dim"], mixer["vdim"])
    for index, layer in enumerate(raw["layers"]):
        p, m = f"l{index}.", layer["mixer"]
        part = model.blocks[index].mixer
        assert torch.equal(part.qkv_bias.double(), torch.cat([tensors[p + f"mix.{n}.b"] for n in "qkv"]))
        assert torch.equal(part.q_gamma.double(), tensors[p + "mix.q.norm"])
        mlp = layer["mlp"]
        if mlp is None:
            continue
        experts = model.blocks[index].feed_forward
        ff = mlp["expert"]["ff"]
        assert torch.equal(experts.first_weight[1, ff:].double(), tensors[p + "mlp.e1.up"])
        assert torch.equal(experts.down_weight[-1].double(), tensors[p + f"mlp.e{mlp['router']['experts'] - 1}.down"])
        if mlp.get("shared"):
            assert torch.equal(experts.shared_gate.double(), tensors[p + "mlp.shared.sg"][0])


def test_a_missing_tensor_is_named(tmp_path):
    from safetensors.torch import load_file, save_file

    folder, _, _, _ = malalix_models.folder_of(tmp_path, "A")
    stored = load_file(folder + "/model.safetensors")
    del stored["l1.mlp.shared.sg"]
    save_file(stored, folder + "/model.safetensors")
    with pytest.raises(Exception) as caught:
        load_model(folder, dtype="float32", device="cpu")
    assert "l1.mlp.shared.sg" in str(caught.value)


@pytest.mark.parametrize("which", sorted(malalix_models.MODELS))
def test_sizes_that_the_file_leaves_out_come_from_the_tensors(tmp_path, which):
    folder, raw, _, _ = malalix_models.folder_of(tmp_path, which)
    stripped = copy.deepcopy(raw)
    for key in ("vocab", "width"):
        stripped.pop(key)
    if "loop" in stripped:
        stripped["loop"].pop("times")
    for layer in stripped["layers"]:
        for key in ("heads", "kv_heads", "dim", "vdim"):
            layer["mixer"].pop(key)
        if layer["mlp"] is not None:
            layer["mlp"]["expert"].pop("ff")
            layer["mlp"]["router"].pop("experts")
            layer["mlp"].get("shared", {}).pop("ff", None)
    with open(folder + "/config.json", "w") as handle:
        json.dump(stripped, handle)
    _, config = load_model(folder, dtype="float32", device="cpu")
    assert config == MalalixConfig.from_dict(raw)
    del stripped["layers"][0]["mixer"]["scale"]
    with open(folder + "/config.json", "w") as handle:
        json.dump(stripped, handle)
    with pytest.raises(ConfigError) as caught:
        load_model(folder, dtype="float32", device="cpu")
    assert "scale" in str(caught.value)


# ------------------------------------------------------------ frequencies
@pytest.mark.parametrize("dims,base,scaling", [(64, 500000.0, (8.0, 1.0, 4.0, 8192)), (16, 100.0, (4.0, 1.0, 3.0, 40)),
                                               (8, 60.0, (3.0, 2.0, 2.5, 30)), (2, 10.0, (8.0, 0.5, 2.0, 12))])
def test_frequencies_stretched_by_wavelength(dims, base, scaling):
    factor, low, high, original = scaling
    got = banded_frequencies(dims, base, *scaling)
    want = plain.banded_frequencies({"dims": dims, "base": base, "scaling": dict(
        zip(("factor", "low", "high", "original"), scaling))})
    assert torch.allclose(got, torch.tensor(want, dtype=F64), rtol=1e-12)
    bare = base ** (-2.0 * torch.arange(dims // 2, dtype=F64) / dims)
    kept, slowed = bare > 2 * math.pi * high / original, bare < 2 * math.pi * low / original
    assert torch.allclose(got[kept], bare[kept]) and torch.allclose(got[slowed], bare[slowed] / factor)
    between = ~(kept | slowed)
    assert bool((got[between] <= bare[between] * (1 + 1e-12)).all()) and bool((got[between] >= bare[between] / factor).all())
    if dims == 64:
        assert int(kept.sum()) and int(slowed.sum()) and int(between.sum())


# ------------------------------------------------------------ pages of a chunked group
@pytest.mark.parametrize("chunk,page_size", [(8, 4), (6, 4), (5, 8), (1, 4), (12, 3)])
def test_a_chunked_group_keeps_what_the_next_position_sees_and_gives_back_the_rest(chunk, page_size):
    group = CacheGroupSpec((0,), 1, 16, chunk=chunk)
    full = CacheGroupSpec((1,), 1, 16)
    manager = CacheManager([group, full], 24, page_size, 2, torch.float32, "cpu", max_positions=60)
    manager.admit("a")
    length = 0
    for step in (1, 1, 3, 2, 7, 1, 1, 1, 1, 12, 1, 2, 1, 1, 5):
        manager.grow("a", length + step)
        length += step
        manager.commit("a", length)
        first = length // chunk * chunk
        assert group.first_visible(length) == first
        table = manager.table("a", 0)
        for page, held in enumerate(table):
            # a page goes back exactly when the next position sees none of its places
            assert (held >= 0) == ((page + 1) * page_size - 1 >= first), (length, page)
        assert all(held >= 0 for held in manager.table("a", 1))
        manager.check_invariants()
    assert manager.pages_for_length(0, 50, longest_step=1) <= -(-(chunk + 1) // page_size) + 1
    manager.release("a")
    assert all(pool.num_allocated == 0 for pool in manager.pools)


def test_a_group_has_a_window_or_a_chunk():
    with pytest.raises(ValueError):
        CacheGroupSpec((0,), 1, 16, window=4, chunk=4)


# ------------------------------------------------------------ the plain implementation itself
@pytest.mark.parametrize("which", ["A", "B", "D", "E"])
def test_a_prompt_gives_its_prefixes_logits(which):
    raw, _, seed = malalix_models.MODELS[which]
    w = plain.random_checkpoint(raw, seed)
    tokens = torch.randint(0, raw["vocab"], (21,), generator=torch.Generator().manual_seed(3)).tolist()
    whole, _ = plain.forward(raw, w, tokens)
    for cut in (1, 8, 20):
        assert torch.allclose(plain.forward(raw, w, tokens[:cut])[0], whole[:cut], atol=1e-9)


def test_no_position_looks_beyond_its_chunk():
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(12, 1, 6, generator=g, dtype=F64) for _ in range(3))
    full = plain.chunked_attention(q, k, v, 0.4)
    assert torch.allclose(plain.chunked_attention(q, k, v, 0.4, 12), full)
    cut = plain.chunked_attention(q, k, v, 0.4, 5)
    for first in (0, 5, 10):      # a chunk is attention over its own tokens alone
        part = slice(first, min(first + 5, 12))
        assert torch.allclose(cut[part], plain.chunked_attention(q[part], k[part], v[part], 0.4))
    assert torch.allclose(plain.chunked_attention(q, k, v, 0.4, 1), v)


def test_what_the_models_are_made_of_shows_in_their_logits():
    """Each constant and branch of model A, changed a little in the plain implementation, moves the
    logits by far more than the engine may differ: a test that compares with them sees it."""
    raw, _, seed = malalix_models.MODELS["A"]
    w = plain.random_checkpoint(raw, seed)
    tokens = torch.randint(0, raw["vocab"], (45,), generator=torch.Generator().manual_seed(9)).tolist()
    right, _ = plain.forward(raw, w, tokens)
    scale = float(right.abs().max())

    def moved(change, tensors=None):
        other = copy.deepcopy(raw)
        change(other)
        return float((plain.forward(other, tensors or w, tokens)[0] - right).abs().max()) / scale

    mixer = lambda c, i: c["layers"][i]["mixer"]      # noqa: E731
    mlp = lambda c, i: c["layers"][i]["mlp"]          # noqa: E731
    for change in (lambda c: mixer(c, 0)["mask"].__setitem__("size", 17), lambda c: mixer(c, 0)["mask"].__setitem__("size", 15),
                   lambda c: mixer(c, 1)["mask"].__setitem__("size", 10), lambda c: mixer(c, 3).pop("mask"),
                   lambda c: mixer(c, 0)["rot"].pop("scaling"), lambda c: mixer(c, 1)["rot"].__setitem__("dims", 14),
                   lambda c: mixer(c, 0)["rot"]["scaling"].__setitem__("low", 0.5),
                   lambda c: mixer(c, 0).__setitem__("scale", 0.31),
                   lambda c: mlp(c, 0)["expert"].__setitem__("limit", 1.3),
                   lambda c: mlp(c, 1)["shared"].__setitem__("limit", 0.8),
                   lambda c: mlp(c, 0)["router"].__setitem__("top", 3), lambda c: mlp(c, 0).pop("shared"),
                   lambda c: c["loop"].__setitem__("times", 2), lambda c: c["loop"].__setitem__("stop", 2)):
        assert moved(change) > 1e-3
    for name in ("l0.mix.q.norm", "l2.mix.k.norm", "l1.mix.v.b", "l3.mix.k.b", "l0.mlp.shared.sg", "loop.step",
                 "l1.norm2", "l2.norm1"):
        other = dict(w)
        other[name] = w[name] * 1.2
        assert moved(lambda c: None, other) > 1e-3, name


def test_the_router_weighs_the_chosen_logits_only():
    chosen, weights = plain.route(torch.tensor([[1.0, 3.0, -2.0, 2.0]], dtype=F64), 2)
    assert chosen == [[1, 3]]
    assert torch.allclose(weights[0], torch.softmax(torch.tensor([3.0, 2.0], dtype=F64), 0))


def test_the_gated_unit_is_capped_on_both_sides():
    g = torch.tensor([5.0, -5.0, 0.5], dtype=F64)
    u = torch.tensor([-9.0, 9.0, 0.25], dtype=F64)
    s = torch.sigmoid(1.702 * torch.tensor([2.0, -5.0, 0.5], dtype=F64))
    want = torch.tensor([2.0 * -1.0, -5.0 * 3.0, 0.5 * 1.25], dtype=F64) * s
    assert torch.allclose(plain.capped_gate(g, u, 2.0), want)
