"""Sonulorn without a GPU: the configuration reader and its errors, the list of tensors, the order of layers that run several
times, what every layer run keeps between steps, pages of chunked keys, and the plain implementation's own consistency."""
import copy

import pytest
import torch

from leone_amd.architectures import config_from_dict, model_spec_for
from leone_amd.cache.manager import CacheManager, GroupSpec
from leone_amd.config import ConfigError
from leone_amd.config.sonulorn import DenseConfig, LightningConfig, ParallelConfig, SinkAttentionConfig, SonulornConfig
from leone_amd.parts import DecoderModel
from leone_amd.parts.base import KvNeed, PartSpec, StateNeed
from tests import sonulorn_util as su
from tests.plain import sonulorn_plain as plain


def built(raw):
    return DecoderModel(model_spec_for(config_from_dict(raw)), torch.float32, "cpu")


@pytest.mark.parametrize("name", list(su.SMALL))
def test_configuration_reads_back_and_names_the_design_tensors(name):
    raw = su.SMALL[name]
    config = config_from_dict(raw)
    assert isinstance(config, SonulornConfig) and config.architecture == "Sonulorn"
    assert config_from_dict(config.to_dict()) == config and config.to_dict() == raw
    assert config.vocab_size == raw["vocab"] and config.max_position_embeddings == raw["max_positions"]
    model = built(raw)
    assert {s.name: tuple(s.shape) for s in model.tensor_specs()} == su.tensor_shapes(raw)
    assert model.graph_safe and model.spec.head == "head" and model.spec.embedding_scale == raw["embedding"]["scale"]


def test_layers_of_the_loop_run_their_parts_on_a_cache_of_every_pass():
    model = built(su.SMALL["B"])
    assert [(run.layer, run.cache) for run in model.schedule] == list(zip([0, 1, 2, 3, 4, 2, 3, 4, 2, 3, 4, 5], range(12)))
    assert model.joins == {2: 0, 5: 1, 8: 2} and len(model.layers) == 6
    assert built(su.SMALL["A"]).joins == {0: 0, 3: 1} and built(su.SMALL["C"]).joins == {3: 0, 4: 1, 5: 2, 6: 3}
    for name, raw in su.SMALL.items():
        runs = [(run.layer, built(raw).joins.get(at)) for at, run in enumerate(built(raw).schedule)]
        assert runs == plain.layer_order(raw), name
    needs = model.cache_needs()
    for run in (2, 5, 8):
        assert needs[(run, "right", "memory")] == StateNeed((4, 24, 10))
    once = {**su.SMALL["A"]}
    del once["loop"]
    straight = built(once)
    assert [run.layer for run in straight.schedule] == [0, 1, 2, 3] and straight.joins == {} and "loop.in" not in \
        {s.name for s in straight.tensor_specs()}


def test_what_every_layer_run_keeps_between_steps():
    needs = built(su.SMALL["A"]).cache_needs()
    # keys within chunks, of the layer's own run; the same again in the second pass
    assert needs[0] == KvNeed(2, 16, None, value_dim=24, chunk=20) == needs[3]
    # side by side: keys and values behind the filters, the last projected rows, the memory and its own last rows
    assert needs[(1, "left", "kv")] == KvNeed(1, 16, None, value_dim=24)
    assert needs[(1, "left", "conv")] == StateNeed((3, 4 * 16 + 16 + 24)) and needs[(1, "right", "conv")] == StateNeed((1, 24 + 24 + 36))
    assert needs[(1, "right", "memory")] == StateNeed((3, 8, 12))
    assert needs[2] == StateNeed((3, 8 * 20)) and needs[6] == KvNeed(2, 24, None, value_dim=8, chunk=16)
    single = built(su.SMALL["B"]).layers[2].mixer.branches["left"].conv      # one tap: a second one of zero ahead of it
    assert (single.file_taps, single.taps) == (1, 2) and single.cache_need() == StateNeed((1, 6 * 16 + 2 * 3 * 16))


def test_defaults_where_the_configuration_is_silent():
    raw = copy.deepcopy(su.SMALL["A"])
    del raw["max_positions"], raw["embedding"], raw["loop"]
    for m in (raw["layers"][3]["mixer"], raw["layers"][1]["mixer"]["left"]):
        for key in ("kv_heads", "vdim", "scale", "rot"):
            del m[key]
    del raw["layers"][3]["mixer"]["mask"], raw["layers"][1]["mixer"]["left"]["conv"], raw["layers"][1]["mixer"]["left_scale"]
    config = config_from_dict(raw)
    assert (config.max_positions, config.embedding_scale, config.loop) == (32768, 1.0, None)
    last, side = config.layers[3].mixer, config.layers[1].mixer
    assert last == SinkAttentionConfig(2, 2, 24, 24, 24 ** -0.5, None, None, None) and isinstance(side, ParallelConfig)
    assert side.left == SinkAttentionConfig(4, 4, 16, 16, 0.25, None, None, None) and side.left_scale == 1.0
    assert isinstance(config.layers[2].mixer, LightningConfig) and config.layers[0].mlp == DenseConfig(40, 1.2)
    assert config_from_dict(config.to_dict()) == config
    built(raw)


BROKEN = [
    (lambda r: r.pop("width"), "width"),
    (lambda r: r["norm"].pop("eps"), "norm.eps"),
    (lambda r: r["embedding"].update(scale="2"), "embedding.scale"),
    (lambda r: r.update(layers=[]), "layers"),
    (lambda r: r["layers"].append(3), "layers[4]"),
    (lambda r: r["layers"][0].update(type="mamba"), "layers[0].type"),
    (lambda r: r["layers"][0].pop("mixer"), "layers[0].mixer"),
    (lambda r: r["layers"][0]["mixer"].pop("dim"), "layers[0].mixer.dim"),
    (lambda r: r["layers"][0]["mixer"].update(kv_heads=3), "layers[0].mixer.kv_heads"),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=18), "layers[0].mixer.rot.dims"),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=7), "layers[0].mixer.rot.dims"),
    (lambda r: r["layers"][0]["mixer"]["mask"].update(size=0), "layers[0].mixer.mask.size"),
    (lambda r: r["layers"][0]["mixer"].update(scale=-1.0), "layers[0].mixer.scale"),
    (lambda r: r["layers"][1]["mixer"]["left"].update(conv=0), "layers[1].mixer.left.conv"),
    (lambda r: r["layers"][1]["mixer"]["right"].pop("conv"), "layers[1].mixer.right.conv"),
    (lambda r: r["layers"][1]["mixer"]["right"].update(kv_heads=2), "layers[1].mixer.right.kv_heads"),
    (lambda r: r["layers"][1]["mixer"].update(left_scale="1"), "layers[1].mixer.left_scale"),
    (lambda r: r["layers"][2]["mixer"].update(decay=[0.5, 0.5]), "layers[2].mixer.decay"),
    (lambda r: r["layers"][2]["mixer"].update(decay=[0.5, 0.5, 1.5]), "layers[2].mixer.decay"),
    (lambda r: r["layers"][0]["mlp"].update(kind="moe"), "layers[0].mlp.kind"),
    (lambda r: r["layers"][0]["mlp"].pop("limit"), "layers[0].mlp.limit"),
    (lambda r: r["loop"].update(start=3), "loop.stop"),
    (lambda r: r["loop"].update(stop=5), "loop.stop"),
    (lambda r: r["loop"].update(start=-1), "loop.start"),
    (lambda r: r["loop"].update(times=0), "loop.times"),
]


@pytest.mark.parametrize("break_it,field", BROKEN, ids=[f for _, f in BROKEN])
def test_errors_name_the_key(break_it, field):
    raw = copy.deepcopy(su.SMALL["A"])
    break_it(raw)
    with pytest.raises(ConfigError) as error:
        config_from_dict(raw)
    assert error.value.field == field and field in str(error.value)


def test_parts_refuse_what_they_cannot_serve():
    from leone_amd.parts import FEED_FORWARDS, MIXERS
    from leone_amd.parts.model import StreamJoin
    params = dict(model_spec_for(config_from_dict(su.SMALL["A"])).layers[0]["mixer"].params, position=None)
    with pytest.raises(ValueError, match="chunks"):
        MIXERS.build(PartSpec("gqa_attention", {**params, "window": 8}))
    with pytest.raises(ValueError, match="limit"):
        FEED_FORWARDS.build(PartSpec("swiglu", {"hidden": 8, "intermediate": 8, "gate": "g", "up": "u", "down": "d",
                                                "activation": "clamped_swish"}))
    spec = model_spec_for(config_from_dict(su.SMALL["A"]))
    spec.join = StreamJoin((0, 9), "loop.in", "loop.step")
    with pytest.raises(ValueError, match="joined"):
        DecoderModel(spec, torch.float32, "cpu")


@pytest.mark.parametrize("chunk,page", [(20, 16), (16, 16), (5, 4), (1, 8), (33, 8), (7, 16)])
def test_pages_of_a_chunk_go_back_when_the_request_has_passed_it(chunk, page):
    """After every commit exactly the pages that hold a position some later query can read are held; two requests side by
    side, portions cut anywhere."""
    m = CacheManager([GroupSpec(80, page, chunk=chunk), GroupSpec(80, page)], 2, 200)
    sizes = [3, 1, 17, 2, 30, 1, 1, 40, 5, 9]
    held = {"a": 0, "b": 0}
    for name in held:
        m.admit(name)
    for n in sizes:
        for name in held:
            size = n if name == "a" else max(1, n // 2)
            m.reserve(name, size)
            m.commit(name, size)
            held[name] += size
            first = held[name] // chunk * chunk
            table = m.table(name, 0)
            for block, at in enumerate(table):
                assert (at >= 0) == ((block + 1) * page > first), (held[name], block)
            assert all(at >= 0 for at in m.table(name, 1))
            m.check()
    for name in held:
        m.release(name)
    assert m.free_pages(0) == 80 and m.free_pages(1) == 80


def test_a_chunked_group_forks_and_is_cut_back_inside_its_chunk():
    from leone_amd.cache.manager import CacheError
    m = CacheManager([GroupSpec(30, 4, chunk=12)], 3, 100)
    m.admit("a"); m.reserve("a", 20); m.commit("a")                   # the first chunk's pages have gone back
    assert [p >= 0 for p in m.table("a", 0)] == [False, False, False, True, True]
    assert m.fork("a", "b", 16) == 16
    with pytest.raises(CacheError):
        m.fork("a", "c", 8)                                           # reads keys 0..7, which have gone back
    with pytest.raises(CacheError):
        m.truncate("a", 9)
    m.truncate("a", 17)
    m.check()
    with pytest.raises(ValueError):
        CacheManager([GroupSpec(10, 4, window=5, chunk=4)], 1, 64)


def test_plain_prefix_equals_plain_whole():
    """A position's logits do not depend on what comes after it."""
    raw = su.SMALL["A"]
    weights = su.make_weights(raw, 3, torch.float32)
    tokens = torch.randint(0, raw["vocab"], (44,), generator=torch.Generator().manual_seed(1)).tolist()
    whole = plain.forward(raw, weights, tokens)
    for n in (1, 20, 21, 40):
        assert torch.allclose(plain.forward(raw, weights, tokens[:n]), whole[:n], atol=1e-9)


def test_plain_mechanisms_do_what_they_say():
    see = plain.visible(7, 3)
    assert see.int().tolist()[4] == [0, 0, 0, 1, 1, 0, 0] and see.int().tolist()[6] == [0, 0, 0, 0, 0, 0, 1]
    x = torch.arange(12, dtype=torch.float64).view(6, 2)
    w = torch.tensor([[0.0, 0.0, 1.0], [1.0, 0.0, 0.0]], dtype=torch.float64)
    out = plain.short_convolution(x, w)
    assert torch.equal(out[:, 0], x[:, 0]) and torch.equal(out[:, 1], torch.cat([torch.zeros(2), x[:4, 1]]))
    weight = plain.softmax_with_sink(torch.zeros(1, 3, dtype=torch.float64), torch.ones(1, 3, dtype=torch.bool), torch.tensor(0.0))
    assert torch.allclose(weight, torch.full((1, 3), 0.25, dtype=torch.float64))
    assert plain.layer_order({"layers": [0, 1, 2, 3], "loop": {"start": 1, "stop": 3, "times": 2}}) == \
        [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    # without decay and with unit keys at right angles the delta rule reads back what was written
    h = torch.eye(4, dtype=torch.float64)
    m = {"heads": 1, "kv_heads": 1, "dim": 4, "vdim": 4}
    one = {"q": 9.0 * torch.eye(4), "k": 9.0 * torch.eye(4), "v": torch.randn(4, 4), "b": torch.full((1, 4), 50.0),
           "a": torch.full((1, 4), -60.0), "A_log": torch.zeros(1), "dt_bias": torch.zeros(1), "norm": torch.ones(4),
           "g": torch.ones(4, 4), "o": torch.eye(4)}
    one.update({n + ".conv": torch.ones(4, 1) for n in "qkv"})
    one = {k: v.double() for k, v in one.items()}
    got = plain.head_decay_delta(h, m, one, "", 1e-12)
    v = plain.silu(one["v"].T)
    want = plain.unit_rms(v * 0.5, 1e-12) * plain.silu(torch.ones(1, dtype=torch.float64))
    assert torch.allclose(got, want, atol=1e-5)
