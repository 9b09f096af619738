"""The Vezidra architecture without a GPU: its reader of config.json, its spec, tensor names, caches and state per
request, the random-weights folder, rotation tables, and the plain implementation's own pieces."""

import copy
import math

import pytest
import torch

import plain_vezidra as plain
import vezidra_util as vu

F64 = torch.float64


def _spec(cfg, device="meta"):
    from qwen25vl_lite_amd.config import load_config
    from qwen25vl_lite_amd.models import build_model
    return build_model(load_config(copy.deepcopy(cfg)), torch.float32, device)


@pytest.mark.parametrize("cfg", [vu.MIXED, vu.ONES, vu.ODD, vu.WIDE])
def test_the_spec_expects_the_files_tensors(cfg):
    model = _spec(cfg)
    shapes = vu.tensor_shapes(cfg)
    got = {model.spec.store_name(k): v for k, v in model.expected_tensors().items()}
    assert {k: tuple(v.shape) for k, v in got.items()} == shapes
    for name in shapes:
        assert model.spec.store_name(model.spec.map_name(name)) == name


def test_the_delta_rules_projection_is_no_bias():
    model = _spec(vu.MIXED)
    assert model.spec.map_name("l0.mix.right.b") == "l0.mix.right.b.weight"
    assert model.spec.map_name("l2.mix.left.q.b") == "l2.mix.left.q.bias"
    assert model.spec.map_name("l2.mix.right.conv.b") == "l2.mix.right.conv.bias"
    assert model.spec.map_name("l0.norm1.b") == "l0.norm1.bias" and model.spec.map_name("final.norm.b") == "final.norm.bias"


def test_caches_and_states():
    model = _spec(vu.MIXED)
    groups = {(g.need.num_kv_heads, g.need.head_dim, g.need.v_dim, g.need.window): g.num_layers for g in model.cache_groups()}
    # layers 1 and 3 share a cache that is kept for the longer of their windows
    assert groups == {(2, 24, 16, None): 1, (2, 16, 24, 37): 1, (4, 16, 24, None): 1, (1, 32, 32, None): 1,
                      (2, 48, 48, None): 1, (1, 32, 32, 9): 1}
    assert model.spec.run[3].cache_from == 1 and model.blocks[3].mixer.kv_shared and model.blocks[3].mixer.window == 37
    assert model.blocks[1].mixer.window == 21 and model.blocks[1].mixer.retain == 37
    shapes = [{name: None if model.entry_state[p] is None else tuple(model.entry_state[p].shape) for name, p in places.items()}
              for places in model.entry_places]
    assert shapes[0] == {"mix": None, "mix.left": None, "mix.right": (4, 12, 20), "mix.right.conv": (2, 128)}
    assert shapes[2] == {"mix": None, "mix.left": None, "mix.right": (6, 24, 8), "mix.right.conv": (3, 192)}
    assert shapes[1] == {"mix": None}
    assert all(s is None or s.dtype == torch.float32 for s in model.entry_state)
    assert "mix.right.conv" not in _spec(vu.ONES).entry_places[0]        # one tap: nothing to keep
    odd = _spec(vu.ODD)                                                  # a reader that sees everything keeps every page
    assert {g.need.window for g in odd.cache_groups()} == {None} and odd.blocks[1].mixer.window == 5


def test_what_the_parts_are_told():
    model = _spec(vu.MIXED)
    left, right = model.blocks[0].mixer.left, model.blocks[0].mixer.right
    assert (left.nq, left.nkv, left.hd, left.vd, left.scale, left.window) == (6, 2, 24, 16, 0.25, None)
    assert left.qk_norm_scope == "whole" and not left.interleaved and left.head_gate and left.has_sinks and not left.qkv_bias
    assert left.position.scaling == (8.0, 1.0, 4.0, 64) and left.position.rotary_dim == 16
    assert (right.heads, right.groups, right.dim, right.vdim, right.taps) == (4, 2, 12, 20, 3) and right.unit_floor == 1e-6
    assert model.blocks[0].mixer.factors == (0.7, 1.3) and not model.blocks[0].mixer.norm
    left, right = model.blocks[2].mixer.left, model.blocks[2].mixer.right
    assert left.qk_norm_scope == "whole" and left.interleaved and left.qkv_bias and left.plus_one and not left.gate_rows
    assert left.position.ramp == (4.0, 64, 8.0, 1.0) and left.position.amplitude == pytest.approx(0.1 * math.log(4.0) + 1.0)
    assert (right.heads, right.vdim, right.states, right.groups, right.norm_groups, right.conv.taps) == (6, 8, 24, 3, 4, 4)
    assert model.blocks[2].mixer.norm and model.blocks[2].mixer.factor == 0.5
    mix = model.blocks[1].mixer
    assert mix.qk_norm_scope == "head" and mix.interleaved and mix.head_gate and mix.has_sinks
    assert model.blocks[1].ffn is None and model.blocks[0].ffn.activation == "relu2" and model.blocks[0].alpha == 2.0
    assert model.embedding.scale == 3.0 and model.token_side.columns == 6 * 7
    assert [b.side.first for b in model.blocks] == [0, 6, 12, 18, 24, 30, 36]
    assert _spec(vu.ODD).token_side is None and _spec(vu.ODD).blocks[0].side is None
    assert model.graph_safe


@pytest.mark.parametrize("bad, text", [
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("postln_alpha"), "postln_alpha"),
    (lambda c: c.pop("embedding"), "embedding"),
    (lambda c: c["embedding"].pop("scale"), "scale"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["token_side"].__setitem__("dim", 0), "dim"),
    (lambda c: c["layers"][0].__setitem__("type", "conv"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("left_scale"), "left_scale"),
    (lambda c: c["layers"][0]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][0]["mixer"]["left"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"]["scaling"].pop("high"), "high"),
    (lambda c: c["layers"][0]["mixer"]["right"].__setitem__("kv_heads", 3), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["right"].__setitem__("conv", 0), "conv"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("kv_heads", 3), "multiple"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 18), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("scaling", {"factor": 2.0}), "no scaling"),
    (lambda c: c["layers"][1]["mixer"]["mask"].pop("size"), "size"),
    (lambda c: c["layers"][3]["mixer"].__setitem__("kv_from", 0), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].__setitem__("kv_from", 5), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].__setitem__("dim", 32), "differ"),
    (lambda c: c["layers"][2]["mixer"]["right"].pop("state"), "state"),
    (lambda c: c["layers"][2]["mixer"]["right"].__setitem__("groups", 4), "multiple"),
    (lambda c: c["layers"][2]["mixer"]["right"].__setitem__("norm_groups", 5), "norm_groups"),
    (lambda c: c["layers"][2]["mixer"]["left"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda c: c["layers"][2]["mlp"].__setitem__("kind", "moe"), "kind"),
    (lambda c: c["layers"][2]["mlp"].pop("ff"), "ff"),
])
def test_config_errors_name_the_key(bad, text):
    from qwen25vl_lite_amd.config import load_config
    from qwen25vl_lite_amd.config.model_config import ConfigError
    cfg = copy.deepcopy(vu.MIXED)
    bad(cfg)
    with pytest.raises(ConfigError, match=text):
        load_config(cfg)


def test_a_layer_without_a_feed_forward_has_no_second_norm():
    model = _spec(vu.MIXED)
    names = model.expected_tensors()
    assert "l1.norm2.weight" not in names and "l2.norm2.bias" in names
    for name in ("l1.norm2", "l1.norm2.b"):        # a file that stores them all the same is read
        assert model.spec.map_name(name) is None
    assert model.spec.map_name("l2.norm2.b") == "l2.norm2.bias"


def test_random_weights_folder_loads_back(tmp_path):
    from qwen25vl_lite_amd.config import load_config
    from qwen25vl_lite_amd.models import build_model
    from qwen25vl_lite_amd.weights import WeightsError, load_weights, write_random_model
    from qwen25vl_lite_amd.weights.safetensors_io import SafetensorsFile
    folder = write_random_model(load_config(copy.deepcopy(vu.MIXED)), str(tmp_path / "m"), seed=3, std=0.3)
    with SafetensorsFile(folder + "/model.safetensors") as f:
        assert {n: tuple(f.shape(n)) for n in f.keys()} == vu.tensor_shapes(vu.MIXED)
    cfg, tensors = plain.vezidra_read(folder)
    logits = plain.vezidra_forward(cfg, tensors, [1, 2, 3, 4, 5, 6, 7])
    assert logits.shape == (7, 203) and torch.isfinite(logits).all()
    model = build_model(load_config(folder), torch.float32, "cpu")
    load_weights(folder, model)
    _, t32 = plain.vezidra_read(folder, torch.float32)
    for i in range(len(cfg["layers"])):
        mixer = model.blocks[i].mixer
        parts = {"left.": mixer.left, "right.": mixer.right} if hasattr(mixer, "left") else {"": mixer}
        for prefix, part in parts.items():
            for local, w in part.named_weights().items():
                assert torch.equal(w, t32[model.spec.store_name(f"l{i}.mix.{prefix}{local}")]), (i, prefix, local)
    assert torch.equal(model.token_side.named_weights()["weight"], t32["side.embed"])
    tensors = vu.random_tensors(vu.MIXED, 4)
    del tensors["l0.mix.right.b"], tensors["l0.norm1.b"]
    tensors["l2.mix.right.D"] = tensors["l2.mix.right.D"][:4].contiguous()
    folder = vu.write_model(str(tmp_path / "p"), vu.MIXED, 4, tensors)
    with pytest.raises(WeightsError, match="(?s)l0.mix.right.b.*l0.norm1.bias|l0.norm1.bias.*l0.mix.right.b") as e:
        load_weights(folder, build_model(load_config(folder), torch.float32, "cpu"))
    assert "l2.mix.right.D" in str(e.value)


@pytest.mark.parametrize("dims", [2, 16, 48, 64])
@pytest.mark.parametrize("base", [60.0, 10000.0])
def test_rotation_tables(dims, base):
    """Frequencies stretched by wavelength and on a ramp, as the plain implementation forms them; some are kept, some
    divided, some between."""
    from qwen25vl_lite_amd.parts.base import PartSpec, build_part
    for s in (vu.waves(), vu.waves(3.0, 0.5, 2.0, 200)):
        part = build_part("position", PartSpec("rope", {"theta": base, "rotary_dim": dims, "scaling": s}), torch.float32, torch.device("cpu"))
        want = plain.by_wavelength(plain.frequencies(base, dims), s)
        assert torch.allclose(part.rotary_tables(dims)[0].double(), want, rtol=1e-6, atol=0)
    for s in (vu.ramp(), vu.ramp(2.0, 40, 4.0, 0.5)):
        part = build_part("position", PartSpec("rope", {"theta": base, "rotary_dim": dims, "scaling": {"kind": "ramp", **s}}),
                          torch.float32, torch.device("cpu"))
        want, amplitude = plain.by_ramp(plain.frequencies(base, dims), base, dims, s)
        assert torch.allclose(part.rotary_tables(dims)[0].double(), want, rtol=1e-6, atol=0)
        assert part.amplitude == pytest.approx(amplitude)


# ---------------------------------------------------------------------------------------------
# the plain implementation's pieces against what their definitions say
# ---------------------------------------------------------------------------------------------
def test_plain_norms():
    x = torch.tensor([[1.0, 3.0, -1.0, 5.0]], dtype=F64)
    y = plain.layer_norm(x, torch.full((4,), 2.0, dtype=F64), torch.full((4,), 10.0, dtype=F64), 0.0)
    assert torch.allclose(y, 10.0 + 2.0 * (x - 2.0) / math.sqrt(5.0))
    assert torch.allclose(plain.norm_in_parts(torch.tensor([[3.0, -3.0, 100.0, 100.0]], dtype=F64), 2, 0.0),
                          torch.tensor([[1.0, -1.0, 1.0, 1.0]], dtype=F64))
    assert plain.unit_vector(torch.tensor([3.0, 4.0], dtype=F64)).norm() == pytest.approx(1.0, abs=1e-6)
    assert plain.unit_vector(torch.zeros(3, dtype=F64)).norm() == 0.0


def test_plain_attention_window_and_sink():
    q = torch.zeros(5, 1, 2, dtype=F64)
    v = torch.arange(1.0, 6.0, dtype=F64).view(5, 1, 1)
    assert plain.attend(q, q, v, 1.0, 2, None)[:, 0, 0].tolist() == [1.0, 1.5, 2.5, 3.5, 4.5]
    # one in the denominator: n keys of weight 1 / (n + 1)
    out = plain.attend(q, q, v, 1.0, None, torch.zeros(1, dtype=F64))[:, 0, 0]
    assert torch.allclose(out, torch.tensor([1 / 2, 3 / 3, 6 / 4, 10 / 5, 15 / 6], dtype=F64))
    assert plain.attend(q, q, v, 1.0, None, torch.full((1,), 100.0, dtype=F64)).abs().max() < 1e-30


def test_plain_delta_rule_replaces_what_a_key_held():
    k = torch.tensor([[[1.0, 0.0]], [[1.0, 0.0]], [[0.0, 1.0]]], dtype=F64)
    v = torch.tensor([[[5.0]], [[7.0]], [[9.0]]], dtype=F64)
    one = torch.ones(3, 1, dtype=F64)
    o, S = plain.delta_rule(k, k, v, one, one)
    assert o[:, 0, 0].tolist() == [5.0, 7.0, 9.0] and S[0, :, 0].tolist() == [7.0, 9.0]
    o, S = plain.delta_rule(k, k, v, 0.5 * one, 0.5 * one)        # decay first, then half of what is missing
    assert o[:, 0, 0].tolist() == [2.5, 1.25 + 0.5 * (7 - 1.25), 4.5]


def test_plain_decayed_products_and_groups():
    one = torch.ones(2, 1, 1, dtype=F64)
    y, S = plain.decayed_products(one, one, 3 * one, torch.tensor([[1.0], [0.5]], dtype=F64), torch.tensor([[2.0], [1.0]], dtype=F64))
    assert y[:, 0, 0].tolist() == [6.0, 6.0] and S.item() == 6.0
    x = torch.arange(4.0, dtype=F64).view(1, 2, 2)
    assert plain.spread(x, 6)[0, :, 0].tolist() == [0.0, 0.0, 0.0, 2.0, 2.0, 2.0]


def test_plain_rotation_layouts():
    x = torch.randn(3, 2, 8, dtype=F64)
    f, pos = plain.frequencies(10.0, 4), torch.arange(3)
    near, halves = plain.rotate(x, pos, f, True), plain.rotate(x, pos, f, False)
    assert torch.equal(near[..., 4:], x[..., 4:]) and torch.equal(halves[..., 4:], x[..., 4:])
    order = [0, 2, 1, 3, 4, 5, 6, 7]
    assert torch.allclose(plain.rotate(x[..., order], pos, f, False), near[..., order])
    assert torch.allclose(plain.rotate(x, pos, f, True, 2.0)[..., :4], 2.0 * near[..., :4])
