"""Fadosun without a GPU: the configuration reader, the model's description as parts, the map from
checkpoint tensors to parameters (packed products with the gate's rows riding along, output matrices side
by side), sizes from stored shapes, what a slot holds, and the plain implementation's own consistency
and sensitivity."""

import copy
import json
import os

import pytest
import torch

import fadosun_models
import plain_fadosun as plain
from pagedserve_amd.config.base import ConfigError
from pagedserve_amd.config.fadosun import FadosunConfig
from pagedserve_amd.config.registry import resolve_architecture
from pagedserve_amd.model import load_model, random_model, write_random_model
from pagedserve_amd.parts import build_part
from pagedserve_amd.parts.registry import MIXERS
from pagedserve_amd.config.spec import PartSpec

F64 = torch.float64
KINDS = {"channel_delta": "channel_delta", "mlstm": "matrix_memory", "parallel": "joined"}


def test_the_architecture_is_found_by_its_name():
    entry = resolve_architecture({"architecture": "Fadosun"})
    assert entry.name == "Fadosun" and entry.config_class is FadosunConfig


@pytest.mark.parametrize("which", sorted(fadosun_models.MODELS))
def test_configuration_round_trip_and_spec(which):
    raw = fadosun_models.MODELS[which][0]
    config = FadosunConfig.from_dict(raw)
    assert FadosunConfig.from_dict(config.to_dict()) == config
    spec = resolve_architecture(raw).build_spec(config)
    assert spec.vocab_size == raw["vocab"] and not spec.tie_head
    assert [call.block for call in spec.schedule] == list(range(len(raw["layers"])))
    assert dict(spec.final_norm.params)["eps"] == raw["norm"]["eps"]
    for layer, block in zip(raw["layers"], spec.blocks):
        mixer, wanted = dict(block.mixer.params), layer["mixer"]
        assert block.mixer.kind == KINDS[layer["type"]] and mixer["ride"] == raw["width"]
        names = [name for name, _ in block.parts]
        if layer["mlp"] is None:
            assert block.arrangement == "gated_between_norms_mixer" and "feed_forward" not in names
        else:
            ff = dict(block.feed_forward.params)
            assert (ff["inner"], ff["activation"], ff["ride"]) == (layer["mlp"]["ff"], "relu", raw["width"])
        if layer["type"] != "parallel":
            continue
        left, right = dict(mixer["left"].params), dict(mixer["right"].params)
        assert left["logistic"] and left["out_scale"] == wanted["left_scale"] and not left["bias"]
        assert (left["heads"], left["kv_heads"], left["head_dim"], left["value_dim"], left["scale"]) == tuple(
            wanted["left"][key] for key in ("heads", "kv_heads", "dim", "vdim", "scale"))
        assert left["rotary_dims"] == (wanted["left"].get("rot") or {}).get("dims", 0)
        assert right["out_scale"] == wanted["right_scale"]
        assert (right["heads"], right["value_dim"], right["states"], right["groups"], right["taps"],
                right["norm_groups"]) == tuple(wanted["right"][key] for key in
                                               ("heads", "vdim", "state", "groups", "conv", "norm_groups"))


def test_configuration_errors_name_the_layer_and_key():
    raw = fadosun_models.MODELS["A"][0]
    cases = [
        (lambda c: c["layers"][0].__setitem__("type", "mamba"), "layers[0]"),
        (lambda c: c["layers"][0]["mixer"].__setitem__("kv_heads", 3), "kv_heads"),
        (lambda c: c["layers"][0]["mixer"].pop("conv"), "conv"),
        (lambda c: c["layers"][1]["mixer"]["left"].pop("scale"), "scale"),
        (lambda c: c["layers"][1]["mixer"]["left"]["rot"].__setitem__("dims", 7), "rot.dims"),
        (lambda c: c["layers"][1]["mixer"]["left"]["rot"].__setitem__("dims", 18), "rot.dims"),
        (lambda c: c["layers"][1]["mixer"]["left"]["rot"].pop("base"), "base"),
        (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
        (lambda c: c["layers"][1]["mixer"]["right"].__setitem__("groups", 4), "groups"),
        (lambda c: c["layers"][1]["mixer"]["right"].__setitem__("norm_groups", 5), "norm_groups"),
        (lambda c: c["layers"][1]["mixer"]["right"].pop("state"), "state"),
        (lambda c: c["layers"][1]["mixer"].__setitem__("left_scale", "1"), "left_scale"),
        (lambda c: c["layers"][2]["mixer"].pop("gate_cap"), "gate_cap"),
        (lambda c: c["layers"][2]["mixer"].__setitem__("gate_cap", 0), "gate_cap"),
        (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "moe"), "mlp.kind"),
        (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff"),
        (lambda c: c["norm"].pop("eps"), "eps"),
        (lambda c: c.pop("layers"), "layers"),
    ]
    for change, word in cases:
        broken = copy.deepcopy(raw)
        change(broken)
        with pytest.raises(ConfigError) as caught:
            FadosunConfig.from_dict(broken)
        assert word in str(caught.value), (word, str(caught.value))


@pytest.mark.parametrize("which", sorted(fadosun_models.MODELS))
def test_every_stored_tensor_feeds_a_parameter_and_a_slot_holds_what_the_layers_keep(tmp_path, which):
    folder, raw, tensors, _ = fadosun_models.folder_of(tmp_path, which)
    model, _ = load_model(folder, dtype="float32", device="cpu")
    assert model.parameter_count == sum(t.numel() for t in tensors.values())
    groups, states = model.cache_requirements()
    assert model.graph_safe
    attention = [layer["mixer"]["left"] for layer in raw["layers"] if layer["type"] == "parallel"]
    assert sum(len(group.entries) for group in groups) == len(attention) and len(states) == len(raw["layers"])
    held = []
    for layer in raw["layers"]:
        m = layer["mixer"]
        if layer["type"] == "channel_delta":
            channels = 2 * m["kv_heads"] * m["dim"] + m["heads"] * m["vdim"]
            held.append(m["heads"] * m["dim"] * m["vdim"] + (m["conv"] - 1) * channels)
        elif layer["type"] == "mlstm":
            held.append(m["heads"] * (m["dim"] * (m["vdim"] + 1) + 1))
        else:
            right = m["right"]
            inner = right["heads"] * right["vdim"]
            held.append(inner * right["state"] + (right["conv"] - 1) * (inner + 2 * right["groups"] * right["state"]))
    assert sorted(-(-count // 4) * 4 for count in held) == sorted(state.shape[0] for state in states)
    d = raw["width"]
    for index, layer in enumerate(raw["layers"]):
        p, block = f"l{index}.", model.blocks[index]
        part = block.mixer
        # the gate's rows are the last of the packed product
        assert torch.equal(part.in_weight[-d:].double(), tensors[p + "rg1"])
        assert torch.equal(block.sublayers[0][2].bias.double(), tensors[p + "rg1.b"])
        assert torch.equal(block.sublayers[0][3].gamma.double(), tensors[p + "norm1b"])
        assert torch.equal(block.sublayers[0][3].beta.double(), tensors[p + "norm1b.b"])
        if layer["mlp"] is not None:
            ff = block.sublayers[1][1]
            assert torch.equal(ff.gate_up_weight[:layer["mlp"]["ff"]].double(), tensors[p + "mlp.gate"])
            assert torch.equal(ff.gate_up_weight[-d:].double(), tensors[p + "rg2"])
        m = layer["mixer"]
        if layer["type"] == "channel_delta":
            assert torch.equal(part.conv_weight.double(), torch.cat([tensors[p + f"mix.{n}.conv"] for n in "qkv"]).T)
            assert torch.equal(part.in_weight[-d - m["heads"]:-d].double(), tensors[p + "mix.b"])
        elif layer["type"] == "parallel":
            a, s = p + "mix.left.", p + "mix.right."
            left, right = part.left, part.right
            assert torch.equal(left.logistic[0].double(), tensors[a + "pb"])
            assert left.logistic[1] == pytest.approx(1.0 / m["left_scale"])
            assert torch.allclose(right.norm_gamma.double(), m["right_scale"] * tensors[s + "norm"], rtol=1e-6)
            # [left | right] columns, zero where a head is cached wider than its values
            wide = part.out_weight[:, :left.core_columns].view(d, left.heads, left.head_dim).double()
            assert torch.equal(wide[:, :, :left.value_dim].reshape(d, -1), tensors[a + "o"])
            assert not wide[:, :, left.value_dim:].any()
            assert torch.equal(part.out_weight[:, left.core_columns:].double(), tensors[s + "o"])


def test_a_missing_tensor_is_named(tmp_path):
    from safetensors.torch import load_file, save_file

    folder, _, _, _ = fadosun_models.folder_of(tmp_path, "A")
    stored = load_file(folder + "/model.safetensors")
    del stored["l1.mix.left.pb"]
    save_file(stored, folder + "/model.safetensors")
    with pytest.raises(Exception) as caught:
        load_model(folder, dtype="float32", device="cpu")
    assert "l1.mix.left.pb" in str(caught.value)


@pytest.mark.parametrize("which", sorted(fadosun_models.MODELS))
def test_sizes_that_the_file_leaves_out_come_from_the_tensors(tmp_path, which):
    folder, raw, tensors, _ = fadosun_models.folder_of(tmp_path, which)
    stripped, full = copy.deepcopy(raw), copy.deepcopy(raw)
    for key in ("vocab", "width"):
        stripped.pop(key)
    for index, (layer, other) in enumerate(zip(stripped["layers"], full["layers"])):
        if layer["mlp"] is not None:
            layer["mlp"].pop("ff")
        sizes = {"channel_delta": ("heads", "kv_heads", "dim", "vdim", "conv"), "mlstm": ("heads", "dim", "vdim")}
        for key in sizes.get(layer["type"], ()):
            layer["mixer"].pop(key)
        if layer["type"] == "parallel":
            for key in ("heads", "kv_heads", "dim", "vdim"):
                layer["mixer"]["left"].pop(key)
            for key in ("heads", "vdim", "conv"):
                layer["mixer"]["right"].pop(key)
        if layer["type"] == "channel_delta":
            # the low-rank projections' inner widths, which configurations do not name
            layer["mixer"].pop("decay_rank", None), layer["mixer"].pop("gate_rank", None)
            other["mixer"]["decay_rank"] = tensors[f"l{index}.mix.a1"].shape[0]
            other["mixer"]["gate_rank"] = tensors[f"l{index}.mix.g1"].shape[0]
    with open(os.path.join(folder, "config.json"), "w") as handle:
        json.dump(stripped, handle)
    _, config = load_model(folder, dtype="float32", device="cpu")
    assert config == FadosunConfig.from_dict(full)


def test_random_models_in_memory_and_in_a_folder(tmp_path):
    raw = fadosun_models.MODELS["A"][0]
    model, config = random_model(raw, seed=3, dtype="float32", device="cpu")
    write_random_model(str(tmp_path / "written"), raw, seed=3)
    loaded, again = load_model(str(tmp_path / "written"), dtype="float32", device="cpu")
    assert again == config and model.parameter_count == loaded.parameter_count
    assert all(torch.equal(model.tensors[name], loaded.tensors[name]) for name in model.tensors)


def test_parts_refuse_what_they_cannot_do():
    def mixer(kind, **params):
        return build_part(MIXERS, "mixer", PartSpec.make(kind, **params), width=32, dtype=torch.float32)

    plain_attention = PartSpec.make("attention", heads=2, kv_heads=1, head_dim=16, scale=0.25, bias=False)
    logistic = PartSpec.make("attention", heads=2, kv_heads=1, head_dim=16, scale=0.25, bias=False, logistic=True)
    scan = PartSpec.make("selective_scan", inner=8, states=4, dt_rank=2, taps=2)
    with pytest.raises(ValueError):
        mixer("joined", left=logistic, right=scan)          # a mixer with products of its own inside
    with pytest.raises(ValueError):
        mixer("joined", left=plain_attention, right=logistic).parameters()
    with pytest.raises(ValueError):
        mixer("attention", heads=2, kv_heads=1, head_dim=16, scale=0.25, out_scale=2.0)
    with pytest.raises(ValueError):
        mixer("attention", heads=2, kv_heads=1, head_dim=16, scale=0.25, logistic=True, sink=True)
    for kind, params in (("matrix_memory", dict(heads=1, key_dim=257, value_dim=4, gate_cap=1.0, norm_eps=1e-5)),
                         ("matrix_memory", dict(heads=1, key_dim=8, value_dim=4, gate_cap=0.0, norm_eps=1e-5)),
                         ("head_state_space", dict(heads=3, value_dim=4, states=8, groups=2, taps=2, norm_groups=1,
                                                   norm_eps=1e-5)),
                         ("channel_delta", dict(heads=2, key_heads=1, key_dim=8, value_dim=4, taps=65, decay_rank=2,
                                                gate_rank=2, norm_eps=1e-5))):
        with pytest.raises(ValueError):
            mixer(kind, **params)


# ------------------------------------------------------------ the plain implementation itself
@pytest.mark.parametrize("which", ["A", "B", "E"])
def test_a_prompt_gives_its_prefixes_logits(which):
    raw, _, seed = fadosun_models.MODELS[which]
    w = plain.random_checkpoint(raw, seed)
    tokens = torch.randint(0, raw["vocab"], (21,), generator=torch.Generator().manual_seed(3)).tolist()
    whole, _ = plain.forward(raw, w, tokens)
    for cut in (1, 8, 20):
        assert torch.allclose(plain.forward(raw, w, tokens[:cut])[0], whole[:cut], atol=1e-9)


def test_recurrences_may_be_cut_anywhere():
    g = torch.Generator().manual_seed(0)

    def rand(*shape):
        return torch.randn(*shape, generator=g, dtype=F64)

    q, k, v = rand(9, 2, 3), plain.unit(rand(9, 2, 3)), rand(9, 2, 4)
    beta, decays = torch.sigmoid(rand(9, 2)), torch.sigmoid(rand(9, 2, 3))
    i, f = rand(9, 2), plain.log_sigmoid(rand(9, 2))
    a, skip = -rand(2).abs(), rand(2)
    for name, run in (
            ("delta", lambda s, e, st: plain.delta_recurrence(q[s:e], k[s:e], v[s:e], beta[s:e], decays[s:e], st)),
            ("memory", lambda s, e, st: plain.matrix_memory_recurrence(q[s:e], k[s:e], v[s:e], i[s:e], f[s:e], st)),
            ("space", lambda s, e, st: plain.state_space_recurrence(v[s:e], beta[s:e], a, k[s:e], q[s:e], skip, st))):
        whole, _ = run(0, 9, None)
        first, state = run(0, 4, None)
        second, _ = run(4, 9, state)
        assert torch.allclose(torch.cat([first, second]), whole), name


def test_the_delta_rule_replaces_what_a_key_held():
    """A key written twice with full weight and no decay gives the second value; what stands at another key stays."""
    k = torch.eye(2, dtype=F64)[[0, 1, 0]].view(3, 1, 2)
    v = torch.tensor([[1.0, 2.0], [3.0, 4.0], [5.0, 6.0]], dtype=F64).view(3, 1, 2)
    ones = torch.ones((3, 1), dtype=F64)
    out, state = plain.delta_recurrence(k, k, v, ones, torch.ones((3, 1, 2), dtype=F64))
    assert torch.equal(out, v)
    assert torch.equal(state[0], torch.tensor([[5.0, 6.0], [3.0, 4.0]], dtype=F64))


def test_a_matrix_memory_does_not_depend_on_its_running_maximum():
    """Against the sums written out without a maximum (small gates, so that nothing overflows)."""
    g = torch.Generator().manual_seed(4)
    q, k, v = (torch.randn(7, 1, n, generator=g, dtype=F64) for n in (3, 3, 2))
    i, f = torch.randn(7, 1, generator=g, dtype=F64), plain.log_sigmoid(torch.randn(7, 1, generator=g, dtype=F64))
    out, (_, _, m) = plain.matrix_memory_recurrence(q, k, v, i, f)
    for t in range(7):
        weights = torch.stack([torch.exp(i[s, 0] + f[s + 1:t + 1, 0].sum()) for s in range(t + 1)])
        scores = weights * (k[:t + 1, 0] @ q[t, 0])
        bottom = torch.maximum(scores.sum().abs(), torch.tensor(1.0, dtype=F64))
        assert torch.allclose(out[t, 0], scores @ v[:t + 1, 0] / bottom, atol=1e-5)
    assert float(m) >= float(i[6])


def test_what_the_models_are_made_of_shows_in_their_logits():
    """Each constant and branch of model A, changed a little in the plain implementation, moves the
    logits by far more than the engine may differ: a test that compares with them sees it."""
    raw, _, seed = fadosun_models.MODELS["A"]
    w = plain.random_checkpoint(raw, seed)
    tokens = torch.randint(0, raw["vocab"], (45,), generator=torch.Generator().manual_seed(9)).tolist()
    right, _ = plain.forward(raw, w, tokens)
    scale = float(right.abs().max())

    def moved(change, tensors=None):
        other = copy.deepcopy(raw)
        change(other)
        return float((plain.forward(other, tensors or w, tokens)[0] - right).abs().max()) / scale

    mixer = lambda c, i: c["layers"][i]["mixer"]      # noqa: E731
    for change in (lambda c: mixer(c, 1)["left"].__setitem__("scale", 0.33), lambda c: mixer(c, 1)["left"].pop("rot"),
                   lambda c: mixer(c, 1)["left"]["rot"].__setitem__("dims", 10),
                   lambda c: mixer(c, 1)["left"]["rot"].__setitem__("base", 700.0),
                   lambda c: mixer(c, 1).__setitem__("left_scale", 0.75),
                   lambda c: mixer(c, 1).__setitem__("right_scale", 1.2),
                   lambda c: mixer(c, 1)["right"].__setitem__("norm_groups", 3),
                   lambda c: mixer(c, 2).__setitem__("gate_cap", 5.0),
                   lambda c: c["layers"][0].__setitem__("mlp", None)):
        assert moved(change) > 1e-3
    for name in ("l0.norm1", "l0.norm1.b", "l0.norm1b", "l0.norm1b.b", "l0.norm2b.b", "l0.rg1", "l0.rg1.b", "l0.rg2",
                 "l1.rg1.b", "l0.mix.q.conv", "l0.mix.v.conv", "l0.mix.A_log", "l0.mix.dt_bias", "l0.mix.a1",
                 "l0.mix.g2", "l0.mix.norm", "l0.mix.b", "l1.mix.left.pb", "l1.mix.right.conv.b",
                 "l1.mix.right.dt_bias", "l1.mix.right.A_log", "l1.mix.right.D", "l1.mix.right.norm", "l2.mix.i.b",
                 "l2.mix.f.b", "l2.mix.norm", "l2.mix.g", "final.norm.b"):
        # (not by one factor for all rows: a norm behind would take that out again)
        other = dict(w)
        rows = w[name].shape[0]
        ramp = 1.0 + 0.4 * torch.linspace(0.5 if rows == 1 else 0.0, 1.0, rows)
        other[name] = w[name] * ramp.view(-1, *([1] * (w[name].ndim - 1)))
        assert moved(lambda c: None, other) > 1e-3, name


@pytest.mark.parametrize("kind", ["channel_delta", "mlstm", "parallel", "attention", "space"])
def test_what_stands_far_back_is_heard_in_the_far_models(tmp_path, kind):
    raw, w = fadosun_models.far_model(tmp_path, kind)[1:]
    tokens = torch.randint(3, 50, (120,), generator=torch.Generator().manual_seed(2)).tolist()
    tokens[3], tokens[119] = fadosun_models.LOUD, fadosun_models.ASK
    quiet = list(tokens)
    quiet[3] = 9
    loud, without = (plain.forward(raw, w, t)[0][-1] for t in (tokens, quiet))
    assert float((loud - without).abs().max()) > 0.1 * float(loud.abs().max())
