"""Reverax without a GPU: the configuration reader and its errors, the list of tensors, layers that take another's weights,
what every layer keeps between steps, and the plain implementation's own consistency."""
import copy

import pytest
import torch

from leone_amd.architectures import config_from_dict, model_spec_for
from leone_amd.config import ConfigError
from leone_amd.config.reverax import (DenseConfig, MixtureConfig, ParallelConfig, ReveraxConfig, TalkingAttentionConfig)
from leone_amd.parts import DecoderModel
from leone_amd.parts.base import KvNeed, PartSpec, StateNeed
from tests import reverax_util as ru
from tests.plain import reverax_plain as plain


def ranked(raw):
    return config_from_dict(raw).with_shapes(ru.tensor_shapes(raw))


@pytest.mark.parametrize("name", list(ru.SMALL))
def test_configuration_reads_back_and_names_the_design_tensors(name):
    raw = ru.SMALL[name]
    config = config_from_dict(raw)
    assert isinstance(config, ReveraxConfig) and config.architecture == "Reverax"
    assert config_from_dict(config.to_dict()) == config and config.to_dict() == raw
    assert config.vocab_size == raw["vocab"] and config.max_position_embeddings == raw["max_positions"]
    known = config.with_shapes(ru.tensor_shapes(raw))
    assert config_from_dict(known.to_dict()) == known           # a written folder notes the ranks it was made with
    model = DecoderModel(model_spec_for(known), torch.float32, "cpu")
    assert {s.name: tuple(s.shape) for s in model.tensor_specs()} == ru.tensor_shapes(raw)
    assert model.graph_safe and model.spec.head is None
    assert model.final_norm.groups == raw["norm"]["groups"] and model.final_norm.gain_factor == raw["logit_scale"]


def test_ranks_come_with_the_tensors():
    raw = ru.SMALL["A"]
    with pytest.raises(ValueError, match="layer 0"):
        model_spec_for(config_from_dict(raw))
    ranks = [layer.mixer.right.decay_rank for layer in ranked(raw).layers if isinstance(layer.mixer, ParallelConfig)]
    assert ranks == [ru.rank_of(0), ru.rank_of(2), ru.rank_of(0)]       # the last one takes layer 0's weights
    assert {layer.mixer.right.decay_rank for layer in config_from_dict(raw).with_ranks(7).layers
            if isinstance(layer.mixer, ParallelConfig)} == {7}


def test_layers_with_anothers_weights_run_its_parts_on_a_cache_of_their_own():
    raw = ru.SMALL["B"]
    model = DecoderModel(model_spec_for(ranked(raw)), torch.float32, "cpu")
    assert len(model.layers) == 4 and [(run.layer, run.cache) for run in model.schedule] == \
        [(0, 0), (1, 1), (2, 2), (3, 3), (1, 4), (3, 5), (1, 6)]
    ahead = DecoderModel(model_spec_for(ranked(ru.SMALL["C"])), torch.float32, "cpu")
    assert [(run.layer, run.cache) for run in ahead.schedule] == [(0, 0), (1, 1), (2, 2), (2, 3), (3, 4)]
    needs = model.cache_needs()
    for slot in (1, 4, 6):
        assert needs[(slot, "left")] == KvNeed(3, 16, 16) and needs[(slot, "right", "memory")] == StateNeed((2, 24 * 24))
    chain = copy.deepcopy(raw)
    chain["layers"][6]["weights_of"] = 4                        # through a layer that has none of its own
    assert config_from_dict(chain) == config_from_dict(raw)
    for change, field in ((lambda r: r["layers"][4].update(weights_of=4), "layers[4].weights_of"),
                          (lambda r: r["layers"][4].update(weights_of=9), "layers[4].weights_of"),
                          (lambda r: r["layers"][1].update(weights_of=4), "weights_of"),
                          (lambda r: r["layers"][4].update(mlp=None), "layers[4].mlp"),
                          (lambda r: r["layers"][4].update(weights_of=0), "layers[4].type")):
        bad = copy.deepcopy(raw)
        change(bad)
        with pytest.raises(ConfigError) as error:
            config_from_dict(bad)
        assert error.value.field.endswith(field), (field, error.value.field)


def test_what_every_layer_keeps_between_steps():
    raw = ru.SMALL["A"]
    model = DecoderModel(model_spec_for(ranked(raw)), torch.float32, "cpu")
    needs = model.cache_needs()
    # side by side: the left branch's keys and values; the token before (the mixer's input) and the memory
    assert needs[(0, "left")] == KvNeed(2, 16, 20, value_dim=24)
    assert needs[(0, "right", "before")] == StateNeed((64,)) and needs[(0, "right", "memory")] == StateNeed((3, 8 * 8))
    assert needs[1] == KvNeed(2, 16, None, value_dim=24)
    assert needs[(2, "left")] == KvNeed(1, 24, None, value_dim=8) and needs[(2, "right", "memory")] == StateNeed((1, 1600))
    assert needs[3] == KvNeed(3, 8, None)
    left = model.layers[0].mixer.branches["left"]
    assert left.softcap == 5.0 and "sink" in left.names and left.value_position is not None and left.window == 20
    assert model.layers[2].mixer.branches["left"].softcap is None
    assert "talk" in model.layers[1].mixer.names and model.layers[2].feed_forward is None
    assert model.layers[0].feed_forward.weigh_input and not model.layers[0].feed_forward.gated
    assert model.spec.ignore_tensors == ("l2.norm2", "l2.ls2")


def test_defaults_where_the_configuration_is_silent():
    raw = copy.deepcopy(ru.SMALL["A"])
    del raw["max_positions"], raw["logit_scale"], raw["norm"]["groups"]
    for key in ("kv_heads", "vdim", "scale"):
        del raw["layers"][1]["mixer"][key], raw["layers"][0]["mixer"]["left"][key]
    raw["layers"] = raw["layers"][:4]
    config = config_from_dict(raw)
    assert (config.max_positions, config.logit_scale, config.norm_groups) == (32768, 1.0, 1)
    first, second = config.layers[0].mixer.left, config.layers[1].mixer
    assert isinstance(second, TalkingAttentionConfig)
    assert (second.kv_heads, second.vdim, second.scale) == (4, 16, 0.25) == (first.kv_heads, first.vdim, first.scale)
    assert config.layers[2].mixer.left.window is None and config.layers[2].mixer.left.softcap is None
    assert isinstance(config.layers[0].mlp, MixtureConfig) and isinstance(config.layers[1].mlp, DenseConfig)
    assert config.layers[2].mlp is None


BROKEN = [
    (lambda r: r.pop("width"), "width"),
    (lambda r: r["norm"].pop("eps"), "norm.eps"),
    (lambda r: r["norm"].update(groups=5), "norm.groups"),
    (lambda r: r.update(logit_scale="2"), "logit_scale"),
    (lambda r: r["layers"][0].update(type="mamba"), "layers[0].type"),
    (lambda r: r["layers"][1]["mixer"].pop("dim"), "layers[1].mixer.dim"),
    (lambda r: r["layers"][1]["mixer"].update(kv_heads=3), "layers[1].mixer.kv_heads"),
    (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=18), "layers[1].mixer.rot.dims"),
    (lambda r: r["layers"][1]["mixer"]["rot"].update(base=1.0), "layers[1].mixer.rot.base"),
    (lambda r: r["layers"][0]["mixer"]["left"].update(vdim=7), "layers[0].mixer.left.vdim"),
    (lambda r: r["layers"][0]["mixer"]["left"].update(softcap=-3.0), "layers[0].mixer.left.softcap"),
    (lambda r: r["layers"][0]["mixer"]["left"]["mask"].update(size=0), "layers[0].mixer.left.mask.size"),
    (lambda r: r["layers"][0]["mixer"]["right"].pop("heads"), "layers[0].mixer.right.heads"),
    (lambda r: r["layers"][0]["mixer"].update(left_scale=None), "layers[0].mixer.left_scale"),
    (lambda r: r["layers"][0]["mlp"]["router"].update(top=7), "layers[0].mlp.router.top"),
    (lambda r: r["layers"][0]["mlp"].update(kind="sparse"), "layers[0].mlp.kind"),
    (lambda r: r.update(layers=[]), "layers"),
]


@pytest.mark.parametrize("change,field", BROKEN, ids=[f for _, f in BROKEN])
def test_errors_name_the_key(change, field):
    raw = copy.deepcopy(ru.SMALL["A"])
    raw["layers"] = raw["layers"][:4]
    change(raw)
    with pytest.raises(ConfigError) as error:
        config_from_dict(raw)
    assert error.value.field == field


def test_parts_refuse_what_they_cannot_compute():
    from leone_amd.parts import FEED_FORWARDS, MIXERS, NORMS
    base = dict(hidden=32, q_heads=2, kv_heads=1, head_dim=16, q="q", k="k", v="v", o="o", talk="t")
    for extra in ({"softcap": 5.0}, {"sink": "s"}, {"gate": "g"}, {"distance_slopes": [0.5, 0.25]}):
        with pytest.raises(ValueError, match="mixed scores"):
            MIXERS.build(PartSpec("gqa_attention", {**base, **extra}))
    with pytest.raises(ValueError):
        NORMS.build(PartSpec("rmsnorm", {"size": 30, "eps": 1e-5, "weight": "w", "groups": 4}))
    moe = dict(hidden=32, experts=4, top=2, intermediate=8, router="r", expert="e{e}")
    with pytest.raises(ValueError, match="without a gate"):
        FEED_FORWARDS.build(PartSpec("routed_glu", {**moe, "weigh_input": True}))
    with pytest.raises(ValueError, match="unknown expert activation"):
        FEED_FORWARDS.build(PartSpec("routed_glu", {**moe, "activation": "relu2"}))


# ---- the plain implementation against itself ---------------------------------------------------------------------

def test_plain_mechanisms_by_hand():
    gen = torch.Generator().manual_seed(0)
    F = torch.float64
    x = torch.randn(3, 12, generator=gen, dtype=F)
    grouped = plain.grouped_norm(x, torch.ones(12, dtype=F), 0.0, 3)
    for part in range(3):
        assert torch.allclose((grouped[:, 4 * part:4 * part + 4] ** 2).mean(dim=-1), torch.ones(3, dtype=F))
    # a sink of minus infinity is no sink; one far above the scores leaves nothing
    see = plain.visible(3)
    score = torch.randn(3, 3, generator=gen, dtype=F)
    none = plain.softmax_with_sink(score, see, torch.tensor(-1e9, dtype=F))
    assert torch.allclose(none, torch.softmax(score.masked_fill(~see, float("-inf")), dim=-1))
    assert float(plain.softmax_with_sink(score, see, torch.tensor(80.0, dtype=F)).abs().max()) < 1e-30
    # one key and a sink of 0: the weight is a sigmoid of the score
    assert torch.allclose(plain.softmax_with_sink(score[:1, :1], see[:1, :1], torch.zeros((), dtype=F)), torch.sigmoid(score[:1, :1]))
    # a value turned by its position and turned back by the reader's is turned by their distance
    v = torch.randn(1, 1, 8, generator=gen, dtype=F)
    there = plain.rotate_halves(plain.rotate_halves(v, [5], 8, 50.0), [-9], 8, 50.0)
    assert torch.allclose(there, plain.rotate_halves(v, [-4], 8, 50.0))
    assert torch.allclose(plain.token_mix(x, torch.full((12,), 0.25, dtype=F))[1], 0.75 * x[1] + 0.25 * x[0])
    assert torch.allclose(plain.token_mix(x, torch.ones(12, dtype=F))[0], torch.zeros(12, dtype=F))
    assert float(plain.cap_scores(torch.tensor(1e6, dtype=F), 5.0)) == 5.0


def test_plain_memory_counts_the_current_token_by_its_bonus():
    """With decays near 1 and W_r = W_k = W_v = 1 the read-out is a sum over earlier tokens plus u times the own one."""
    F = torch.float64
    w = {"mu." + n: torch.zeros(2, dtype=F) for n in ("r", "k", "v", "g", "w")}
    eye = torch.eye(2, dtype=F)
    w.update(r=eye, k=eye, v=eye, g=torch.zeros(2, 2, dtype=F), w1=torch.zeros(1, 2, dtype=F), w2=torch.zeros(2, 1, dtype=F),
             w0=torch.full((2,), -40.0, dtype=F), u=torch.tensor([[3.0, 3.0]], dtype=F), norm=torch.ones(2, dtype=F), o=eye)
    h = torch.tensor([[1.0, 0.0], [0.0, 2.0], [1.0, 1.0]], dtype=F)
    got = {}
    original = plain.unit_rms
    plain.unit_rms = lambda x, eps: got.setdefault("o", x.clone())
    try:
        plain.time_mixing(h, {"heads": 1, "dim": 2}, w, "", 1e-6)
    finally:
        plain.unit_rms = original
    # o_t = sum_(s<t) (k_s . r_t) v_s + 3 (k_t . r_t) v_t
    assert torch.allclose(got["o"][:, 0], torch.tensor([[3.0, 0.0], [0.0, 24.0], [7.0, 10.0]], dtype=F))


@pytest.mark.parametrize("name", list(ru.SMALL))
def test_plain_is_causal_and_windows_end_where_they_should(name):
    raw = ru.SMALL[name]
    weights = ru.make_weights(raw, 3, torch.float32)
    gen = torch.Generator().manual_seed(1)
    tokens = torch.randint(0, raw["vocab"], (30,), generator=gen).tolist()
    full = plain.forward(raw, weights, tokens)
    assert torch.allclose(plain.forward(raw, weights, tokens[:17]), full[:17])
    m = {"heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 1.0, "rot": {"dims": 8, "base": 50.0}, "mask": {"size": 4}}
    shapes = {"q": (16, 12), "k": (8, 12), "v": (8, 12), "o": (12, 16), "q.b": (16,), "k.b": (8,), "v.b": (8,), "sink": (2,),
              "q.norm": (8,), "k.norm": (8,)}
    w = {n: ru.one_tensor(n, s, gen).double() for n, s in shapes.items()}
    h = torch.randn(10, 12, generator=gen, dtype=torch.float64)
    moved = h.clone()
    moved[3] += 1.0
    change = (plain.turned_value_attention(h, m, w, "", 1e-5) - plain.turned_value_attention(moved, m, w, "", 1e-5)).abs().amax(dim=-1)
    assert (change[3:7] > 1e-6).all() and change[:3].max() == 0 and change[7:].max() < 1e-12
