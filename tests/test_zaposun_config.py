"""The Zaposun architecture without a GPU: its reader of config.json, its spec, tensor names, caches and state per
request, pages of chunks, the random-weights folder, and the plain implementation's own pieces."""

import copy
import math

import pytest
import torch

import plain_zaposun as plain
import zaposun_util as zu


def _spec(cfg):
    from qwen25vl_lite_amd.config import load_config
    from qwen25vl_lite_amd.models import build_model
    return build_model(load_config(copy.deepcopy(cfg)), torch.float32, "meta")


@pytest.mark.parametrize("cfg", [zu.MIXED, zu.ONES, zu.ODD, zu.NO_PAGES])
def test_the_spec_expects_the_files_tensors(cfg):
    model = _spec(cfg)
    shapes = zu.tensor_shapes(cfg, {0: 5, 3: 11})
    got = {model.spec.store_name(k): v for k, v in model.expected_tensors().items()}
    assert set(got) == set(shapes)
    for name, shape in shapes.items():
        assert got[name].takes(shape), name                      # the decay projections' inner size is the file's
        assert model.spec.store_name(model.spec.map_name(name)) == name
        if not got[name].free:
            assert not got[name].takes((shape[0] + 1, *shape[1:])) and not got[name].takes(shape + (1,))


def test_caches_and_states():
    model = _spec(zu.MIXED)
    groups = {(g.need.num_kv_heads, g.need.head_dim, g.need.v_dim, g.need.chunk): g.num_layers for g in model.cache_groups()}
    assert groups == {(2, 24, 16, 37): 1, (4, 16, 24, 9): 1, (1, 16, 24, 64): 1}
    shapes = [{name: None if model.entry_state[p] is None else tuple(model.entry_state[p].shape) for name, p in places.items()}
              for places in model.entry_places]
    assert shapes[0] == {"mix": (3, 16, 16), "mix.mu": (72,), "shift": (72,)}
    assert shapes[1] == {"mix": None, "mix.left": None, "mix.right": (8, 88), "mix.right.conv": (2, 88), "shift": (72,)}
    assert model.entry_state[model.embed_place].shape == (1,) and model.entry_state[model.embed_place].dtype == torch.int32
    assert all(s is None or s.dtype == torch.float32 for s in model.entry_state[:-1])
    ones = _spec(zu.ONES)          # one tap: the convolution keeps nothing
    assert "mix.right.conv" not in ones.entry_places[0] and ones.blocks[0].mixer.left.chunk == 1
    assert not _spec(zu.NO_PAGES).cache_groups()


def test_slots_of_nested_parts():
    from types import SimpleNamespace
    model = _spec(zu.MIXED)
    tensors = [object() if s is not None else None for s in model.entry_state]
    groups = model.cache_groups()
    storage = SimpleNamespace(k=[[f"k{g}"] for g in range(len(groups))], v=[[f"v{g}"] for g in range(len(groups))])
    slots = model.make_slots(storage, tensors)
    assert len(slots) == len(zu.MIXED["layers"]) + 1 and slots[-1].state is tensors[model.embed_place]
    mix = slots[1].of("mix")
    assert mix.of("left").k_cache == "k0" and mix.of("left").state is None
    assert mix.of("right").state is tensors[model.entry_places[1]["mix.right"]] and mix.of("right").group is None
    assert mix.of("right").of("conv").state is tensors[model.entry_places[1]["mix.right.conv"]]
    assert slots[0].of("mix").of("mu").state is tensors[model.entry_places[0]["mix.mu"]]
    assert slots[0].of("shift").state is tensors[model.entry_places[0]["shift"]]


def test_pages_of_a_chunk_go_back_when_the_next_begins():
    from qwen25vl_lite_amd.cache.manager import CacheGroupSpec, CacheManager
    from qwen25vl_lite_amd.parts.base import CacheNeed
    cache = CacheManager([CacheGroupSpec(CacheNeed(1, 8, chunk=37), 1)], num_pages=16, page_size=16, max_num_seqs=2)
    assert cache.prefix_cache is None
    cache.admit("a")
    at, held = 0, []
    for upto in (5, 36, 37, 38, 70, 74, 90, 111, 112):
        cache.reserve("a", upto)
        cache.commit("a", upto)
        held.append([i for i, p in enumerate(cache.table("a", 0)) if p >= 0])
    # token 37 begins a chunk inside page 2, token 74 inside page 4, token 111 inside page 6
    assert held == [[0], [0, 1, 2], [2], [2], [2, 3, 4], [4], [4, 5], [6], [6]]
    cache.release("a")
    cache.check()
    need = CacheNeed(1, 8, window=20, chunk=37)
    assert [need.first_visible(p) for p in (0, 19, 36, 37, 50, 60)] == [0, 0, 17, 37, 37, 41]


def test_what_the_parts_are_told():
    model = _spec(zu.MIXED)
    left, right = model.blocks[1].mixer.left, model.blocks[1].mixer.right
    assert (left.nq, left.nkv, left.hd, left.vd, left.chunk, left.scale, left.window) == (6, 2, 24, 16, 37, 0.25, None)
    assert left.qk_norm_scope == "head" and left.qk_norm_where == "before" and left.qk_norm_eps == 1e-5
    assert not left.gate_rows and not left.interleaved
    assert left.value_position.theta == left.position.theta == 80.0 and left.value_position.rotary_dim is None
    assert left.position.rotary_dim == 16
    assert (right.inner, right.states, right.rank, right.conv.taps) == (88, 8, 5, 3)
    assert model.blocks[1].mixer.factor == 0.5
    assert model.blocks[2].ffn is None and model.blocks[0].ffn.activation == "gelu_tanh"
    assert model.blocks[0].norm1.groups == 3 and model.final_norm.copies == 3
    assert model.head_part.scale == 0.7 and (model.embedding.buckets, model.embedding.mul_prev, model.embedding.mul_cur) == (61, 29, 5)
    assert model.graph_safe


@pytest.mark.parametrize("bad, text", [
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("streams"), "streams"),
    (lambda c: c.__setitem__("streams", 0), "streams"),
    (lambda c: c.pop("logit_scale"), "logit_scale"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["norm"].pop("groups"), "groups"),
    (lambda c: c["norm"].__setitem__("groups", 5), "groups"),
    (lambda c: c.pop("embedding"), "embedding"),
    (lambda c: c["embedding"].pop("bigram"), "bigram"),
    (lambda c: c["embedding"]["bigram"].pop("mul_cur"), "mul_cur"),
    (lambda c: c["embedding"]["bigram"].__setitem__("buckets", 0), "buckets"),
    (lambda c: c["layers"][0].__setitem__("type", "conv"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("dim"), "dim"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][1]["mixer"]["left"].__setitem__("vdim", 15), "vdim"),
    (lambda c: c["layers"][1]["mixer"]["left"].__setitem__("kv_heads", 4), "multiple"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].__setitem__("dims", 26), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].pop("size"), "size"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("dt_rank"), "dt_rank"),
    (lambda c: c["layers"][1]["mixer"]["right"].__setitem__("conv", 0), "conv"),
    (lambda c: c["layers"][1]["mlp"].__setitem__("kind", "moe"), "kind"),
    (lambda c: c["layers"][1]["mlp"].pop("ff"), "ff"),
])
def test_config_errors_name_the_key(bad, text):
    from qwen25vl_lite_amd.config import load_config
    from qwen25vl_lite_amd.config.model_config import ConfigError
    cfg = copy.deepcopy(zu.MIXED)
    bad(cfg)
    with pytest.raises(ConfigError, match=text):
        load_config(cfg)


def test_a_layer_without_a_feed_forward_has_no_second_norm():
    cfg = copy.deepcopy(zu.MIXED)
    cfg["layers"][0].pop("mlp")
    model = _spec(cfg)
    names = model.expected_tensors()
    assert "l0.norm2.weight" not in names and "l0.hc2.mix.weight" not in names and "l1.hc2.mix.weight" in names
    for name in ("l0.norm2", "l0.hc2.in", "l0.hc2.mix"):        # a file that stores them all the same is read
        assert model.spec.map_name(name) is None
    assert model.spec.map_name("l1.norm2") == "l1.norm2.weight"


def test_random_weights_folder_loads_back(tmp_path):
    from qwen25vl_lite_amd.config import load_config
    from qwen25vl_lite_amd.models import build_model
    from qwen25vl_lite_amd.weights import WeightsError, load_weights, write_random_model
    from qwen25vl_lite_amd.weights.safetensors_io import SafetensorsFile
    folder = write_random_model(load_config(copy.deepcopy(zu.MIXED)), str(tmp_path / "m"), seed=3, std=0.3)
    with SafetensorsFile(folder + "/model.safetensors") as f:
        assert {n: tuple(f.shape(n)) for n in f.keys()} == zu.tensor_shapes(zu.MIXED, {0: 64, 3: 64})
    cfg, tensors = plain.zaposun_read(folder)
    assert (tensors["l0.hc1.mix"].diagonal().mean() - 1.0).abs() < 0.6
    logits = plain.zaposun_forward(cfg, tensors, [1, 2, 3, 4, 5, 6, 7])
    assert logits.shape == (7, 203) and torch.isfinite(logits).all()
    # another file with inner sizes of its own; one whose two decay projections do not meet is refused
    folder = zu.write_model(str(tmp_path / "n"), zu.MIXED, 4, ranks=zu.RANKS)
    model = build_model(load_config(folder), torch.float32, "cpu")
    load_weights(folder, model)
    assert model.blocks[0].mixer.rank == 6 and model.blocks[3].mixer.rank == 24
    assert torch.equal(model.blocks[0].mixer.named_weights()["v.weight"],
                       plain.zaposun_read(folder, torch.float32)[1]["l0.mix.v"])
    tensors = zu.random_tensors(zu.MIXED, 4, zu.RANKS)
    tensors["l0.mix.w1"] = tensors["l0.mix.w1"][:4].contiguous()
    folder = zu.write_model(str(tmp_path / "o"), zu.MIXED, 4, tensors)
    with pytest.raises(ValueError, match="do not meet"):
        load_weights(folder, build_model(load_config(folder), torch.float32, "cpu"))
    tensors["l0.mix.r"] = tensors["l0.mix.r"][:4].contiguous()
    folder = zu.write_model(str(tmp_path / "p"), zu.MIXED, 4, tensors)
    with pytest.raises(WeightsError, match="l0.mix.r"):
        load_weights(folder, build_model(load_config(folder), torch.float32, "cpu"))


# ---------------------------------------------------------------------------------------------
# the plain implementation's pieces against what their definitions say
# ---------------------------------------------------------------------------------------------
def test_plain_bigram_rows():
    rows = plain.bigram_rows([3, 5, 2], {"buckets": 11, "mul_prev": 4, "mul_cur": 3})
    assert rows.tolist() == [11, (3 * 4 + 5 * 3) % 11, (5 * 4 + 2 * 3) % 11]


def test_plain_grouped_norm_differs_from_one_norm():
    x = torch.tensor([[3.0, -3.0, 100.0, 100.0]], dtype=torch.float64)
    assert torch.allclose(plain.grouped_norm(x, torch.ones(4, dtype=torch.float64), 2, 0.0),
                          torch.tensor([[1.0, -1.0, 1.0, 1.0]], dtype=torch.float64))


def test_plain_step_towards_the_previous_token():
    h = torch.tensor([[4.0, 4.0], [8.0, 0.0]], dtype=torch.float64)
    mu = torch.tensor([0.25, 1.0], dtype=torch.float64)
    assert plain.towards_previous(h, mu).tolist() == [[3.0, 0.0], [7.0, 4.0]]


def test_plain_chunks_and_turned_values():
    q = torch.zeros(5, 1, 2, dtype=torch.float64)
    v = torch.arange(1.0, 6.0, dtype=torch.float64).view(5, 1, 1)
    out = plain.attend_in_chunks(q, q, v, 1.0, 3)[:, 0, 0]
    assert out.tolist() == [1.0, 1.5, 2.0, 4.0, 4.5]          # tokens 3 and 4 are a chunk of their own
    x = torch.randn(4, 2, 6, dtype=torch.float64)
    f, pos = plain.frequencies(10.0, 6), torch.arange(4)
    turned = plain.rotate(x, pos, f)
    assert torch.allclose(plain.rotate(turned, -pos, f), x) and not torch.allclose(turned, x)


def test_plain_bonus_counts_for_the_current_token_only():
    one = torch.ones(2, 1, 1, dtype=torch.float64)
    out = plain.decayed_outer_products(one, one, 2 * one, 0.5 * one, torch.tensor([[3.0]], dtype=torch.float64))
    assert out[:, 0, 0].tolist() == [6.0, 8.0]                # 3*2, then the 2 that is left from before + 3*2


def test_plain_selective_scan_and_softplus():
    dt = torch.tensor([[1.0], [2.0]], dtype=torch.float64)
    x = torch.tensor([[3.0], [5.0]], dtype=torch.float64)
    a, d = torch.tensor([[-0.5]], dtype=torch.float64), torch.tensor([10.0], dtype=torch.float64)
    b, c = torch.tensor([[1.0], [2.0]], dtype=torch.float64), torch.tensor([[1.0], [1.0]], dtype=torch.float64)
    y = plain.selective_scan(x, dt, a, b, c, d)[:, 0].tolist()
    assert y[0] == pytest.approx(3.0 + 30.0) and y[1] == pytest.approx(math.exp(-1.0) * 3.0 + 20.0 + 50.0)
    z = torch.tensor([-40.0, 0.0, 40.0], dtype=torch.float64)
    assert torch.allclose(plain.softplus(z), torch.log1p(torch.exp(z)), atol=1e-12)


def test_plain_streams():
    t = {"a.mix": torch.tensor([[1.0, 2.0], [0.0, -1.0]]), "a.out": torch.tensor([0.5, 3.0]), "a.in": torch.tensor([1.0, 10.0])}
    streams = torch.tensor([[[1.0]], [[4.0]]])
    assert plain.join(streams, torch.tensor([[2.0]]), t, "a.").flatten().tolist() == [2.0, 4.0]     # mix[from, to]
    assert plain.read(streams, t, "a.").item() == 41.0
