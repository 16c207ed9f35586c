"""Reverax on the GPU against the plain implementation: each mechanism alone, whole models of several sizes under every way
of cutting the work, pages and slots that are used again, keys planted far away and at the edges of windows and pages,
a memory that reaches hundreds of tokens back, long decoding, and generation through the scheduler."""
import json
import math
import os
import subprocess
import sys
import tempfile

import numpy as np
import pytest
import torch

from tests import reverax_util as ru
from tests import schedules
from tests.plain import reverax_plain as plain
from tests.test_gpu_fosulix import SCHEDULES, TOLERANCE, close, compare, make_engine, run_steps, widened
from tests.test_gpu_pamevik import run_mixer_in_cuts, step_of
from tests.test_gpu_zukinex import paged, planted

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F = torch.float64
LENGTHS = {"A": [1, 2, 37, 130, 64, 9], "B": [70, 3, 150, 33, 81], "C": [90, 17, 65, 2, 48]}
PAGE_TOKENS = {"A": 16, "B": 16, "C": 32}
CUTS = [(5, 1), (1, 1), (2, 0), (1, 3), (17, 1), (1, 16), (0, 2), (33, 1), (1, 1), (2, 40)]      # 63 and 66 rows


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    cache = {}

    def get(name, dtype_name):
        key = (name, dtype_name)
        if key not in cache:
            raw = ru.SMALL[name]
            weights = ru.make_weights(raw, 41 + len(cache), DTYPES[dtype_name], sharpen=2.0 if dtype_name == "float32" else 1.0)
            folder = ru.write_dir(str(tmp_path_factory.mktemp(f"reverax_{name}_{dtype_name}")), raw, weights)
            gen = np.random.default_rng(17 + len(cache))
            requests = {f"r{i}": gen.integers(0, raw["vocab"], size=n).tolist() for i, n in enumerate(LENGTHS[name])}
            expected = {rid: plain.forward(raw, widened(weights), toks).numpy() for rid, toks in requests.items()}
            cache[key] = (folder, requests, expected)
        return cache[key]
    return get


@pytest.mark.parametrize("schedule", list(SCHEDULES))
@pytest.mark.parametrize("dtype_name", list(DTYPES))
@pytest.mark.parametrize("name", list(ru.SMALL))
def test_engine_agrees_with_plain_however_the_work_is_cut(cases, name, dtype_name, schedule):
    """Whole prompts, tails decoded token by token (windows of 1 to 50 pass over decoded tokens), portions down to
    two tokens, and four requests at a time with portions beside single tokens, on an engine with four slots and
    just enough pages: pages and slots are used again, also pages a window has passed.  Logits at every position."""
    folder, requests, expected = cases(name, dtype_name)
    steps = SCHEDULES[schedule](requests)
    page = PAGE_TOKENS[name]
    engine = make_engine(folder, dtype_name, max_tokens=schedules.max_live_tokens(steps, page), page_tokens=page, poison_freed=True)
    outputs = run_steps(engine, steps)
    worst = compare(steps, outputs, expected, dtype_name, f"{name} {dtype_name} {schedule}")
    print(f"{name} {dtype_name} {schedule}: worst relative error {worst:.2e}")
    assert all(engine.cache.free_pages(g) == engine.cache.groups[g].num_pages for g in range(len(engine.cache.groups)))


@pytest.mark.parametrize("schedule", ["whole", "portions", "mixed"])
@pytest.mark.parametrize("name", ["A", "B"])
def test_long_portions_of_the_memory_walked_in_chunks(cases, monkeypatch, name, schedule):
    """With chunks of 8 rows from portions of 16 rows on, every longer portion is walked in chunks side by side and chained
    by the product of the chunk's decays; the results differ from the row-by-row walk by rounding only."""
    from leone_amd import ops
    monkeypatch.setattr(ops, "GATED_CHUNKS", (8, 16))
    folder, requests, expected = cases(name, "float32")
    steps = SCHEDULES[schedule](requests)
    engine = make_engine(folder, "float32", max_tokens=schedules.max_live_tokens(steps, 16), poison_freed=True)
    compare(steps, run_steps(engine, steps), expected, "float32", f"{name} chunked walk {schedule}")


ODD = ru.config(100, 301, [
    ru.layer(ru.parallel((3, 3, 12, 10, 6, 300.0, 13, 6.0), (5, 7), 0.9, 1.7), ru.dense(50)),
    ru.layer(ru.attention(5, 1, 20, 7, 14), ru.moe(12, 3, 18)),
    ru.layer(ru.attention(7, 7, 9, 30, 2, 50.0), None),
    ru.layer(ru.parallel((1, 1, 38, 2, 2, 50.0, None, None), (1, 70), -1.0, 1.0), ru.moe(3, 3, 7)),
], groups=20, logit_scale=0.3)


@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_sizes_that_are_multiples_of_nothing(dtype_name):
    """Width 100 normed in parts of 5, vocabulary 301, keys of 12, 20, 9 and 38 elements and values of 10, 7, 30 and 2 (heads
    filled up with zeros to what the cache packs, which must not count in the heads' norms), memories of 7 x 7 and 70 x 70,
    feed-forwards of 50, 18 and 7, a prompt of 300 tokens (the memories' long portions in chunks), pages of 64 tokens:
    every kernel's path for sizes that fill no run of 8 or 16."""
    weights = ru.make_weights(ODD, 3, DTYPES[dtype_name])
    gen = np.random.default_rng(1)
    requests = {f"r{i}": gen.integers(0, ODD["vocab"], size=n).tolist() for i, n in enumerate([300, 70, 5, 129])}
    expected = {rid: plain.forward(ODD, widened(weights), toks).numpy() for rid, toks in requests.items()}
    with tempfile.TemporaryDirectory() as folder:
        ru.write_dir(folder, ODD, weights)
        for name in ("whole", "mixed"):
            steps = SCHEDULES[name](requests)
            engine = make_engine(folder, dtype_name, max_tokens=schedules.max_live_tokens(steps, 64), page_tokens=64, poison_freed=True)
            got = schedules.collect(steps, run_steps(engine, steps))
            errors = np.concatenate([ru.relative_error(np.stack(got[rid]), expected[rid]) for rid in got])
            assert np.isfinite(errors).all()
            if dtype_name == "float32":
                assert errors.max() <= TOLERANCE["float32"], (name, float(errors.max()))
            else:       # a changed choice of experts moves single positions by far more: the median says what rounding does
                assert np.median(errors) <= TOLERANCE["bfloat16"], (name, float(np.median(errors)))


@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_pages_and_slots_that_held_another_request(cases, dtype_name):
    """One slot and pages enough for one request: every request runs where the one before it ran, and what freed
    pages and the slot hold is overwritten with NaN here, as a fault would leave it."""
    folder, requests, expected = cases("A", dtype_name)
    engine = make_engine(folder, dtype_name, max_tokens=144, max_requests=1)
    for rid, toks in requests.items():
        steps = schedules.portions({rid: toks}, sizes=(3, 1, 2, 40))
        outputs = run_steps(engine, steps)
        compare(steps, outputs, {rid: expected[rid]}, dtype_name, f"page reuse {rid}")
        for storage in engine.pools.paged.values():
            for pool in storage:
                pool.fill_(float("nan"))
        for storage in engine.pools.state.values():
            storage.fill_(float("nan"))


def test_long_decoding_through_recorded_steps():
    """A short prompt, then 300 tokens one by one (steps replayed from a recording), two requests side by side: the windows
    pass over decoded tokens many times, pages behind them are handed back and used again, the memory and the token before
    are carried 300 steps, by layers that share their weights but not their state."""
    raw = ru.SMALL["B"]
    weights = ru.make_weights(raw, 91, torch.float32, sharpen=2.0)
    gen = np.random.default_rng(2)
    requests = {"a": gen.integers(0, raw["vocab"], size=310).tolist(), "b": gen.integers(0, raw["vocab"], size=305).tolist()}
    expected = {rid: plain.forward(raw, weights, toks).numpy() for rid, toks in requests.items()}
    with tempfile.TemporaryDirectory() as folder:
        ru.write_dir(folder, raw, weights)
        for graphs in (True, False):
            engine = make_engine(folder, "float32", max_tokens=704, graphs=graphs, poison_freed=True)
            steps = [{"step": 0, "entries": [{"id": "a", "tokens": requests["a"][:10], "want": list(range(10))},
                                             {"id": "b", "tokens": requests["b"][:5], "want": list(range(5))}], "end": []}]
            for i in range(300):
                steps.append({"step": i + 1, "entries": [{"id": "a", "tokens": [requests["a"][10 + i]], "want": [0]},
                                                         {"id": "b", "tokens": [requests["b"][5 + i]], "want": [0]}],
                              "end": ["a", "b"] if i == 299 else []})
            assert engine.graphs == graphs
            outputs = run_steps(engine, steps)
            compare(steps, outputs, expected, "float32", f"long decoding, graphs {graphs}")


def test_greedy_generation_through_the_scheduler():
    """The framework's own entry point: prompts in, greedy tokens out, scheduled in portions with more requests
    than slots, against the plain implementation's argmax token by token."""
    from leone_amd.api import Runtime
    from leone_amd.engine.scheduler import SchedulerPolicy
    raw = ru.SMALL["A"]
    weights = ru.make_weights(raw, 23, torch.float32, sharpen=2.0)
    gen = np.random.default_rng(8)
    prompts = [gen.integers(0, raw["vocab"], size=n).tolist() for n in (3, 40, 21, 9, 57)]
    with tempfile.TemporaryDirectory() as folder:
        ru.write_dir(folder, raw, weights)
        runtime = Runtime.load(folder, "float32", max_tokens=512, page_tokens=16, max_requests=2,
                               policy=SchedulerPolicy(max_live_requests=2, prefill_chunk_tokens=16, max_step_tokens=24))
        results = runtime.generate_tokens(prompts, 12, eos_token_id=None)
    for prompt, result in zip(prompts, results):
        tokens = list(prompt)
        for i in range(12):
            logits = plain.forward(raw, weights, tokens)[-1]
            best = int(logits.argmax())
            if result.tokens[i] != best:       # a near tie may fall either way; anything else is a fault
                assert float(logits[best] - logits[result.tokens[i]]) < 1e-4, (i, best, result.tokens[i])
            tokens.append(result.tokens[i])
        assert len(result.tokens) == 12


def test_trace_replay_as_a_user_runs_it(cases, tmp_path):
    folder, requests, expected = cases("B", "float32")
    steps = schedules.mixed(requests)
    out_dir = str(tmp_path / "out")
    process = subprocess.Popen([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                                "--out", out_dir, "--max-tokens", str(schedules.max_live_tokens(steps, 64))],
                               stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    outputs = {}
    for s in steps:
        process.stdin.write(json.dumps(s) + "\n")
        process.stdin.flush()
        assert process.stdout.readline().strip() == f"done {s['step']}"
        wanted = sum(len(e["want"]) for e in s["entries"])
        if wanted:
            outputs[s["step"]] = np.fromfile(os.path.join(out_dir, f"{s['step']}.f32"), dtype="<f4").reshape(wanted, -1)
    process.stdin.close()
    assert process.wait(timeout=60) == 0
    compare(steps, outputs, expected, "float32", "trace replay")


def test_command_line_generates_from_token_ids(tmp_path):
    """``leone generate`` on a Reverax folder: greedy tokens as the plain implementation picks them; ``leone random-model``
    writes a folder of the design (from a configuration that names the decay's rank) that loads again."""
    from leone_amd import cli
    raw = ru.SMALL["C"]
    weights = ru.make_weights(raw, 61, torch.float32, sharpen=2.0)
    folder = ru.write_dir(str(tmp_path / "model"), raw, weights)
    prompt = [5, 17, 3, 99, 42, 7]
    out = str(tmp_path / "tokens.json")
    assert cli.main(["generate", "-m", folder, "--prompt-tokens", ",".join(map(str, prompt)), "-n", "8", "--dtype", "float32",
                     "--ignore-eos", "--debug-tokens", out]) == 0
    with open(out) as handle:
        got = json.load(handle)
    tokens = list(prompt)
    for token in got:
        logits = plain.forward(raw, weights, tokens)[-1]
        assert token == int(logits.argmax()) or float(logits.max() - logits[token]) < 1e-4
        tokens.append(token)
    assert len(got) == 8
    from leone_amd.architectures import config_from_dict
    config_path = str(tmp_path / "config.json")
    with open(config_path, "w") as handle:
        json.dump(config_from_dict(ru.SMALL["A"]).with_ranks(6).to_dict(), handle)
    made = str(tmp_path / "made")
    assert cli.main(["random-model", "--config", config_path, "--seed", "3", "--out", made]) == 0
    engine = make_engine(made, "bfloat16", max_tokens=64)
    from leone_amd.engine.engine import StepEntry
    logits = engine.step([StepEntry("a", [1, 2, 3], [2])]).logits
    assert logits.shape == (1, ru.SMALL["A"]["vocab"]) and torch.isfinite(logits).all()


# ---- each mechanism alone ---------------------------------------------------------------------------------------

def build_mixer(entry, dtype, width, seed, sharpen=2.0, weights=None):
    """(part, weights in double, the mixer's configuration) of one mixer from a layer entry of ``reverax_util``: the model's
    own builder makes the part's description, so the test covers what a model of this mixer alone would run."""
    from leone_amd.architectures import config_from_dict, model_spec_for
    from leone_amd.parts import MIXERS, POSITIONS
    raw = ru.config(width, 32, [ru.layer(entry)])
    spec = model_spec_for(config_from_dict(raw).with_shapes(ru.tensor_shapes(raw)))
    positions = {name: POSITIONS.build(s) for name, s in spec.positions.items()}
    for part in positions.values():
        part.prepare(512, DEV)
    mixer = MIXERS.build(spec.layers[0]["mixer"], positions=positions)
    gen = torch.Generator().manual_seed(seed)
    w = {k[len("l0.mix."):]: ru.one_tensor(k, v, gen, sharpen).to(dtype) for k, v in ru.tensor_shapes(raw).items()
         if k.startswith("l0.mix.")}
    w.update({k: v.to(dtype) for k, v in (weights or {}).items()})
    mixer.bind({"l0.mix." + k: v.to(DEV) for k, v in w.items()})
    return mixer, {k: v.to(F) for k, v in w.items()}, entry["mixer"]


def check_in_cuts(mixer, want_of, width, dtype_name, page_tokens, bound=None, rows=(63, 66)):
    dtype = DTYPES[dtype_name]
    gen = torch.Generator().manual_seed(3)
    hs = [torch.randn(n, width, generator=gen).to(dtype) for n in rows]
    got = run_mixer_in_cuts(mixer, hs, CUTS, dtype, page_tokens)
    for s in (0, 1):
        err = ru.relative_error(got[s].numpy(), want_of(hs[s].to(F)).numpy())
        assert err.max() <= (bound or (2e-5 if dtype_name == "float32" else 3e-2)), (s, int(err.argmax()), float(err.max()))


def m_seed(entry):
    return sum(ord(c) for c in json.dumps(entry, sort_keys=True)) % 1000


TALKS = [ru.attention(4, 2, 16, 24, 8, 100.0), ru.attention(1, 1, 40, 8, 40), ru.attention(6, 6, 8, 8, 2),
         ru.attention(8, 2, 64, 64, 64), ru.attention(16, 4, 32, 32, 16), ru.attention(12, 3, 128, 128, 32), ru.attention(5, 1, 20, 7, 6),
         ru.attention(24, 8, 16, 16, 16), ru.attention(4, 4, 48, 96, 24)]


@pytest.mark.parametrize("page_tokens", [16, 32])
@pytest.mark.parametrize("dtype_name", list(DTYPES))
@pytest.mark.parametrize("entry", TALKS, ids=lambda e: f"{e['mixer']['heads']}x{e['mixer']['dim']}x{e['mixer']['vdim']}")
def test_attention_with_mixed_scores_alone_in_cuts_of_every_size(entry, dtype_name, page_tokens):
    """Two sequences side by side, fed in steps of 0 to 40 rows each, pages interleaved and filled with NaN beforehand: one
    head (the mix is a factor), heads that share keys and heads that do not, biases, rotated parts of every share."""
    width = 48
    mixer, w, m = build_mixer(entry, DTYPES[dtype_name], width, seed=m_seed(entry), sharpen=2.0 if dtype_name == "float32" else 0.5)
    # the mix adds up H heads' scores: hundreds of units at 24 heads, which only magnifies float rounding
    check_in_cuts(mixer, lambda h: plain.talking_attention(h, m, w, ""), width, dtype_name, page_tokens,
                  bound=5e-5 if dtype_name == "float32" else 4e-2)


SIDES = [ru.parallel((4, 2, 16, 24, 8, 100.0, 20, 5.0), (3, 8), 0.8, -0.6),
         ru.parallel((2, 1, 24, 8, 24, 10000.0, None, None), (4, 20), 1.3, 0.4),
         ru.parallel((6, 3, 16, 16, 16, 77.0, 16, 30.0), (2, 40), 0.0, 1.0),
         ru.parallel((8, 1, 32, 32, 16, 1000.0, 24, 10.0), (8, 64), 1.0, 0.0),
         ru.parallel((1, 1, 48, 48, 2, 20.0, 1, 3.0), (1, 130), 0.5, 0.5),
         ru.parallel((8, 2, 128, 128, 64, 5000.0, 33, 20.0), (1, 16), 1.0, 0.0),
         ru.parallel((4, 2, 12, 6, 4, 100.0, 9, None), (2, 6), 1.0, 0.0)]


@pytest.mark.parametrize("page_tokens", [16, 32])
@pytest.mark.parametrize("dtype_name", list(DTYPES))
@pytest.mark.parametrize("entry", SIDES, ids=lambda e: f"{e['mixer']['left']['heads']}x{e['mixer']['left']['dim']}_{e['mixer']['right']['heads']}x{e['mixer']['right']['dim']}")
def test_attention_beside_a_memory_alone(entry, dtype_name, page_tokens):
    """Both branches and their weighted sum; a weight of zero leaves one branch alone (turned values, capped scores, sinks,
    head norms, a window; the memory with its token mixes), so a fault in either shows at full size."""
    width = 48
    mixer, w, m = build_mixer(entry, DTYPES[dtype_name], width, seed=m_seed(entry), sharpen=2.0 if dtype_name == "float32" else 1.0)
    check_in_cuts(mixer, lambda h: plain.side_by_side(h, m, w, "", 1e-5), width, dtype_name, page_tokens,
                  bound=2e-5 if dtype_name == "float32" else 4e-2)


def test_memory_reaches_hundreds_of_tokens_back():
    """Decays of exp(-exp(-9)): what a token writes is still 97 % there 250 tokens later.  A marked token at position 2 is
    read at positions 200 to 259, in a portion and token by token, in state slots that held NaN."""
    width = 32
    entry = ru.parallel((1, 1, 8, 8, 8, 100.0, 4, None), (2, 16), 0.0, 1.0)
    mixer, w, m = build_mixer(entry, torch.float32, width, seed=5,
                              weights={"right.w0": torch.full((32,), -9.0), "right.w2": torch.zeros(32, ru.rank_of(0))})
    gen = torch.Generator().manual_seed(9)
    hs = 0.05 * torch.randn(260, width, generator=gen)
    hs[2] = 4.0 * torch.randn(width, generator=gen)
    cuts = [(200, 1), (30, 1)] + [(1, 1)] * 30
    got = run_mixer_in_cuts(mixer, [hs, hs[:32]], cuts, torch.float32, 16)[0]
    want = plain.side_by_side(hs.to(F), m, w, "", 1e-5)
    quiet = hs.clone()
    quiet[2] = 0.05 * torch.randn(width, generator=gen)
    without = plain.side_by_side(quiet.to(F), m, w, "", 1e-5)
    assert float((want[200:] - without[200:]).abs().max()) > 0.1 * float(want[200:].abs().max())   # the mark is what is read
    err = ru.relative_error(got.numpy(), want.numpy())
    assert err.max() <= 2e-5, (int(err.argmax()), float(err.max()))


def key_query_value(heads, dim, vdim, width, sharp):
    """Projections that read a row's key from its first elements, every head's query from the next, the value from the rest."""
    wk = torch.zeros(dim, width)
    wk[:, :dim] = torch.eye(dim)
    wq = torch.zeros(heads * dim, width)
    for h in range(heads):
        wq[h * dim:(h + 1) * dim, dim:2 * dim] = torch.eye(dim) * sharp
    wv = torch.zeros(vdim, width)
    wv[:, 2 * dim:] = torch.randn(vdim, width - 2 * dim, generator=torch.Generator().manual_seed(1)) / 3
    return wq, wk, wv


@pytest.mark.parametrize("page_tokens", [16, 32])
@pytest.mark.parametrize("window", [None, 40, 64])
@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_left_attention_finds_planted_keys(dtype_name, window, page_tokens):
    """Keys that answer one query each are planted far back, on both sides of page borders, and at the last position a
    window still holds; a decoy stands one position outside the window of a query, with a value of its own, and must
    not be seen.  Queries come in a prompt's portion and as single decoded tokens.  Positions turn slowly enough (a large
    base, two rotated elements of each head that no planted key uses) for a key to answer wherever it stands, while
    the values turn with their positions over their whole size: a value turned by the wrong place shows in the result."""
    dtype = DTYPES[dtype_name]
    width, heads, dim, vdim = 64, 2, 16, 16
    entry = ru.parallel((heads, 1, dim, vdim, 2, 1e6, window, 60.0), (1, 8), 1.0, 0.0, scale=1.0)
    # the heads' norm makes every query as long as every other: its sharpness lies in the query norm's gain
    wq, wk, wv = key_query_value(heads, dim, vdim, width, 1.0)
    zero = torch.zeros
    mixer, w, m = build_mixer(entry, dtype, width, seed=7, weights={
        "left.q": wq, "left.k": wk, "left.v": wv, "left.q.b": zero(heads * dim), "left.k.b": zero(dim), "left.v.b": zero(vdim),
        "left.q.norm": torch.ones(dim) * (0.6 if dtype_name == "float32" else 0.5), "left.k.norm": torch.ones(dim),
        "left.sink": torch.tensor([-3.0, 1.0])})
    total = 300
    gen = torch.Generator().manual_seed(11)
    hs = torch.randn(total, width, generator=gen)
    pairs = {3: 280, 15: 281, 16: 282, 17: 283, 127: 284, 128: 285, 0: 290, 31: 291, 32: 292, 255: 295}
    if window:
        pairs = {q - window + 1: q for q in range(271, 300, 3)}
    for n, (key_at, query_at) in enumerate(pairs.items()):
        direction = torch.zeros(dim)
        direction[2 + n] = 8.0
        hs[key_at, :dim] = direction
        hs[query_at, dim:2 * dim] = direction
        hs[key_at, 2 * dim:] = 3.0 * torch.randn(width - 2 * dim, generator=gen)
        if window:                                       # the decoy just outside: same direction, the opposite value
            hs[key_at - 1, :dim] = direction
            hs[key_at - 1, 2 * dim:] = -hs[key_at, 2 * dim:]
    hs = hs.to(dtype)
    want = plain.side_by_side(hs.to(F), m, w, "", 1e-5)
    # the planted key is what its query reads: without it the result is another
    blind = hs.clone().to(F)
    for key_at in pairs:
        blind[key_at, :dim] = torch.randn(dim, generator=gen)
    gone = plain.side_by_side(blind, m, w, "", 1e-5)
    for query_at in pairs.values():
        assert float((want[query_at] - gone[query_at]).abs().max()) > 0.2 * float(want[query_at].abs().max())
    cuts = [(270, 1), (10, 1)] + [(1, 1)] * 20
    got = run_mixer_in_cuts(mixer, [hs, hs[:22]], cuts, dtype, page_tokens)[0]
    err = ru.relative_error(got.numpy(), want.numpy())
    bound = 2e-5 if dtype_name == "float32" else 3e-2
    assert err.max() <= bound, (int(err.argmax()), float(err.max()))


@pytest.mark.parametrize("page_tokens", [16, 32])
@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_mixed_scores_find_planted_keys_through_another_heads_query(dtype_name, page_tokens):
    """Head 1's queries are zero and its scores are all head 0's (the mix has one entry off the diagonal), so what it reads it
    finds through another head's query; keys are planted far back and on both sides of page borders and asked for in a
    portion and token by token.  Without the mix, or with its transpose, head 1 reads the average of everything."""
    dtype = DTYPES[dtype_name]
    width, heads, dim, vdim = 64, 2, 16, 16
    entry = ru.attention(heads, 1, dim, vdim, 2, 1e6, scale=1.0)
    wq, wk, wv = key_query_value(heads, dim, vdim, width, 0.6 if dtype_name == "float32" else 0.5)
    wq[dim:] = 0.0
    zero = torch.zeros
    mixer, w, m = build_mixer(entry, dtype, width, seed=7, weights={
        "q": wq, "k": wk, "v": wv, "q.b": zero(heads * dim), "k.b": zero(dim), "v.b": zero(vdim),
        "talk": torch.tensor([[0.2, 0.0], [1.0, -2.0]]), "o": torch.randn(width, heads * vdim, generator=torch.Generator().manual_seed(2)) / 5})
    total = 300
    gen = torch.Generator().manual_seed(11)
    hs = torch.randn(total, width, generator=gen)
    hs[:, :2 * dim] *= 0.05
    pairs = {3: 280, 15: 281, 16: 282, 17: 283, 127: 284, 128: 285, 0: 290, 31: 291, 32: 292, 255: 295}
    for n, (key_at, query_at) in enumerate(pairs.items()):
        direction = torch.zeros(dim)
        direction[2 + n] = 5.0
        hs[key_at, :dim] = direction
        hs[query_at, dim:2 * dim] = direction
        hs[key_at, 2 * dim:] = 3.0 * torch.randn(width - 2 * dim, generator=gen)
    hs = hs.to(dtype)
    want = plain.talking_attention(hs.to(F), m, w, "")
    crossed = dict(w, talk=w["talk"].T)
    other = plain.talking_attention(hs.to(F), m, crossed, "")
    for query_at in pairs.values():
        assert float((want[query_at] - other[query_at]).abs().max()) > 0.2 * float(want[query_at].abs().max())
    cuts = [(270, 1), (10, 1)] + [(1, 1)] * 20
    got = run_mixer_in_cuts(mixer, [hs, hs[:22]], cuts, dtype, page_tokens)[0]
    err = ru.relative_error(got.numpy(), want.numpy())
    assert err.max() <= (2e-5 if dtype_name == "float32" else 3e-2), (int(err.argmax()), float(err.max()))


@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_feed_forwards_and_norm_alone(dtype_name):
    """The dense feed-forward, ungated experts that read the row times its score (the score squared is what comes out: a
    weight on the wrong side shows), and the norm in groups with its factor, in steps of 1, 7, 60, 200 and 700 rows: the
    experts' products in tiles of every size."""
    from leone_amd.architectures import config_from_dict, model_spec_for
    from leone_amd.parts import FEED_FORWARDS, NORMS
    dtype = DTYPES[dtype_name]
    width = 72
    side = ru.attention(1, 1, 8, 8, 8)
    raw = ru.config(width, 32, [ru.layer(side, ru.dense(52)), ru.layer(side, ru.moe(9, 4, 24)), ru.layer(side, ru.moe(3, 1, 20)),
                                ru.layer(side, ru.moe(2, 2, 16))], groups=6, logit_scale=-1.3)
    spec = model_spec_for(config_from_dict(raw))
    weights = ru.make_weights(raw, 13, dtype)
    wide = {k: v.to(F) for k, v in weights.items()}
    gen = torch.Generator().manual_seed(4)
    for rows in (1, 7, 60, 200, 700):
        h = torch.randn(rows, width, generator=gen).to(dtype)
        step = step_of([(0, i) for i in range(rows)], dtype, [0])
        for i, layer in enumerate(spec.layers):
            part = FEED_FORWARDS.build(layer["feed_forward"])
            part.bind({k: v.to(DEV) for k, v in weights.items() if k.startswith(f"l{i}.mlp.")})
            got = part.forward(h.to(DEV), step)
            got = (got.sum(dim=0) if got.dim() == 3 else got).float().cpu()
            p = f"l{i}.mlp."
            want = plain.dense_feed_forward(h.to(F), wide, p) if i == 0 else plain.mixture(h.to(F), raw["layers"][i]["mlp"], wide, p)
            err = ru.relative_error(got.numpy(), want.numpy())
            if dtype_name == "float32":
                assert err.max() <= 2e-5, (rows, i, float(err.max()))
            else:       # a rounded router input may give a row another expert: most rows must keep the bound
                assert np.median(err) <= 3e-2 and (err > 0.15).sum() <= max(1, rows // 10), (rows, i, float(np.median(err)))
        for spec_of, name, factor in ((spec.layers[0]["norm1"], "l0.norm1", 1.0), (spec.final_norm, "final.norm", -1.3)):
            norm = NORMS.build(spec_of)
            norm.bind({name: weights[name].to(DEV)})
            x = torch.randn(rows, width, generator=gen)
            delta = torch.randn(rows, width, generator=gen)
            stream = x.clone().to(DEV)
            got = norm.add_norm(stream, delta.to(DEV), torch.float32).cpu()
            want = plain.grouped_norm((x + delta).to(F), wide[name], raw["norm"]["eps"], 6) * factor
            assert torch.allclose(got.double(), want, atol=1e-5, rtol=1e-5)
            assert torch.allclose(stream.cpu(), x + delta)


@pytest.mark.parametrize("rows,hidden,groups", [(1, 64, 1), (9, 100, 20), (3, 2048, 4), (600, 192, 3), (5, 66, 2), (2, 4096, 1), (17, 512, 64)])
def test_branch_norm_against_torch(rows, hidden, groups):
    """The sum of up to four results with factors and vectors (one of them in planes), two norms of it in groups, picked
    rows that leave the stream alone, more results than one launch takes; types mixed."""
    from leone_amd import ops
    gen = torch.Generator().manual_seed(rows)
    x = torch.randn(rows, hidden, generator=gen)
    terms = [(torch.randn(rows, hidden, generator=gen), 0.7, torch.randn(hidden, generator=gen).bfloat16()),
             (torch.randn(2, rows, hidden, generator=gen), -1.2, None),
             (torch.randn(rows, hidden, generator=gen), 1.0, torch.randn(hidden, generator=gen)),
             (torch.randn(rows, hidden, generator=gen), 2.0, None), (torch.randn(rows, hidden, generator=gen), 0.5, None),
             (torch.randn(rows, hidden, generator=gen), 0.25, None)]
    gains = [1 + 0.2 * torch.randn(hidden, generator=gen), (1 + 0.2 * torch.randn(hidden, generator=gen)).bfloat16()]

    def on(t):
        return None if t is None else t.to(DEV)
    for count in (0, 1, 3, 4, 6):
        some = terms[:count]
        want = x.double().clone()
        for t, f, s in some:
            want += f * (t.sum(dim=0) if t.dim() == 3 else t).double() * (1.0 if s is None else s.double())
        normed = [plain.grouped_norm(want, g.double(), 1e-5, groups) for g in gains]
        on_device = [(on(t), f, on(s)) for t, f, s in some]
        stream = x.clone().to(DEV)
        got = ops.branch_norm(stream, on_device, [on(g) for g in gains], 1e-5, groups, torch.float32)
        for a, b in zip(got, normed):
            assert torch.allclose(a.cpu().double(), b, atol=1e-4, rtol=1e-4), count
        assert torch.allclose(stream.cpu().double(), want, atol=1e-4, rtol=1e-5), count
        rounded = ops.branch_norm(x.clone().to(DEV), on_device, [on(gains[1])], 1e-5, groups, torch.bfloat16)[0]
        assert torch.allclose(rounded.cpu().double(), normed[1], atol=2e-2, rtol=1e-2), count
        pick = torch.tensor([rows - 1, 0], dtype=torch.int32, device=DEV)
        stream = x.clone().to(DEV)
        got = ops.branch_norm(stream, on_device, [on(gains[0])], 1e-5, groups, torch.float32, rows=pick)[0]
        assert torch.allclose(got.cpu().double(), normed[0][[rows - 1, 0]], atol=1e-4, rtol=1e-4), count
        assert torch.equal(stream.cpu(), x)


@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_token_mix_and_decays_against_torch(dtype_name):
    """Entries of one row and of several, at a sequence's start and behind it; the stored row of every entry afterwards; a
    step of single rows, which moves its state in the same launch; ranks and widths that fill nothing evenly."""
    from leone_amd import ops
    dtype = DTYPES[dtype_name]
    gen = torch.Generator().manual_seed(2)
    for hidden, counts in ((50, [3, 1, 5, 1]), (256, [1, 1, 1]), (260, [90, 2])):
        for decode_only in (False, True):
            if decode_only and max(counts) > 1:
                continue
            starts = [0, 7, 4, 0][:len(counts)]
            slots = [3, 0, 2, 1][:len(counts)]
            meta = [(e, starts[e] + i) for e in range(len(counts)) for i in range(counts[e])]
            step = step_of(meta, dtype, slots)
            step.decode_only = decode_only
            h = torch.randn(len(meta), hidden, generator=gen).to(dtype)
            mu = torch.rand(5, hidden, generator=gen).to(dtype)
            state = torch.randn(4, hidden, generator=gen)
            for e, start in enumerate(starts):
                if start == 0:
                    state[slots[e]] = float("nan")
            kept = state.clone().to(DEV)
            got = ops.token_mix(h.to(DEV), mu.to(DEV), kept, step).float().cpu()
            at = 0
            for e, count in enumerate(counts):
                before = torch.zeros(hidden) if starts[e] == 0 else state[slots[e]]
                rows = torch.cat([before[None], h[at:at + count].float()])
                for m in range(5):
                    want = (rows[1:] + (rows[:-1] - rows[1:]) * mu[m].float()).to(dtype).float()
                    assert torch.allclose(got[m, at:at + count], want, atol=1e-6 if dtype_name == "float32" else 2e-2), (hidden, e, m)
                assert torch.equal(kept[slots[e]].cpu(), h[at + count - 1].float())
                at += count
    for rows, channels, rank in ((1, 300, 8), (9, 70, 5), (40, 512, 64), (3, 256, 33), (70, 130, 64), (129, 300, 40), (200, 64, 7), (3, 128, 100)):
        low, w2, w0 = torch.randn(rows, rank + 3, generator=gen), torch.randn(channels, rank, generator=gen).to(dtype), torch.randn(channels, generator=gen).to(dtype)
        got = ops.low_rank_decay(low.to(DEV)[:, :rank], w2.to(DEV), w0.to(DEV)).cpu().double()
        want = torch.exp(-torch.exp(torch.tanh(low[:, :rank].double()) @ w2.double().T + w0.double()))
        assert torch.allclose(got, want, atol=2e-6, rtol=1e-4), (rows, channels, rank)


@pytest.mark.parametrize("rows", [1, 8, 16, 17, 40, 200])
def test_products_of_several_inputs_against_matrices_that_lie_together(rows):
    """One launch for few rows, a product each for more; with the second copies of the matrix the same bits."""
    from leone_amd import ops
    gen = torch.Generator().manual_seed(rows)
    for k, parts, dtype in ((192, [32, 32, 32, 8], torch.bfloat16), (128, [48, 48, 48], torch.bfloat16), (72, [20, 20, 7], torch.bfloat16),
                            (64, [16, 16], torch.float32), (128, [16, 40], torch.bfloat16)):
        x = torch.randn(len(parts), rows, k, generator=gen).to(dtype)
        w = (torch.randn(sum(parts), k, generator=gen) / math.sqrt(k)).to(dtype)
        on_x, on_w = x.to(DEV), w.to(DEV)
        got = [t.cpu() for t in ops.linear_planes(on_x, on_w, parts)]
        at = 0
        for p, n in enumerate(parts):
            want = x[p].double() @ w[at:at + n].double().T
            assert got[p].shape == (rows, n) and torch.allclose(got[p].double(), want, atol=2e-5, rtol=1e-5), (k, parts, p)
            at += n
        if dtype == torch.bfloat16 and k % 64 == 0:
            assert ops.keep_streamed_copy(on_w) > 0
            again = [t.cpu() for t in ops.linear_planes(on_x, on_w, parts)]
            assert all(torch.equal(a, b) if rows <= 16 or rows > 128 else torch.allclose(a, b, atol=1e-5) for a, b in zip(got, again)), (k, parts)


def shaped_reference(q, k, v, positions, scale, window, cap, sinks, turn, group):
    """Plain attention of single rows: q [rows, H, d] at ``positions`` against all keys k [n, G, d], values v [n, G, e] as they
    are cached; capped scores, a sink a head, results turned back by ``turn`` = (base, whether pairs are neighbours)."""
    out = torch.zeros(len(positions), q.shape[1], v.shape[2], dtype=F)
    keys = torch.arange(k.shape[0])
    for r, p in enumerate(positions):
        see = (keys <= p) & ((p - keys < window) if window else torch.ones_like(keys, dtype=torch.bool))
        for head in range(q.shape[1]):
            score = (k[:, head // group].double() @ q[r, head].double()) * scale
            if cap:
                score = plain.cap_scores(score, cap)
            sink = sinks[head].double() if sinks is not None else torch.tensor(-1e9, dtype=F)
            out[r, head] = plain.softmax_with_sink(score[None], see[None], sink)[0] @ v[:, head // group].double()
    if turn:
        rotate = plain.rotate_neighbours if turn[1] else plain.rotate_halves
        out = rotate(out, [-p for p in positions], v.shape[2], turn[0])
    return out


def turn_tables(base, dims, positions):
    a = plain.angles(list(range(positions)), dims, base)
    return torch.cos(a).float().to(DEV), torch.sin(a).float().to(DEV)


@pytest.mark.parametrize("page_tokens", [16, 64])
@pytest.mark.parametrize("window,cap,sunk,turn,dim", [(40, 9.0, True, (50.0, False), 32), (0, None, True, (300.0, True), 32),
                                                      (130, 5.0, False, (50.0, False), 48), (64, 20.0, True, None, 128),
                                                      (1, 3.0, True, (20.0, False), 16), (33, None, False, (20.0, True), 128)])
def test_all_three_attention_kernels_with_caps_sinks_and_turned_results(window, cap, sunk, turn, dim, page_tokens):
    """The row kernel (float32 and bfloat16), the split-KV kernel (rows one by one, and cut into several parts) and the
    prompt kernel (a portion of 420 rows that continues a request of 100, in one range of keys and in several) against
    plain attention.  Every row's query points along one key: its own, the one before, the first, one far back, the
    window's last and the one just outside it, keys on both sides of a page border; scores reach the cap, sinks lie below,
    among and above them."""
    from leone_amd import ops
    n, first, heads, q_heads = 520, 100, 2, 8
    k, v = planted(n, heads, dim, dim, 5 + window)
    positions = list(range(first, n))
    q = torch.zeros(len(positions), q_heads, dim)
    for r, i in enumerate(positions):
        kinds = [i, i - 1, 0, i // 2, i - window, i - window + 1, i - window - 1, 63, 64, i - 300]
        j = min(max(kinds[r % len(kinds)] if window else kinds[r % 4], 0), i)
        for head in range(q_heads):
            key = k[j, head // 4].bfloat16().float()
            other = k[max(j - 17, 0), head // 4].bfloat16().float()
            q[r, head] = (key / (key @ key) + (other / (other @ other) if r % 3 == 0 else 0.0)) * 12.0
    sinks = torch.linspace(-2.0, 14.0, q_heads) if sunk else None
    tables = turn_tables(turn[0], dim, n) if turn else None
    shape = ops.ScoreShape(cap, sinks.to(DEV) if sunk else None, (*tables, "adjacent" if turn[1] else "half_split") if turn else None)
    rows_at = torch.tensor(positions, dtype=torch.int32, device=DEV)
    entry = torch.zeros(len(positions), dtype=torch.int32, device=DEV)
    for dtype, bound in ((torch.float32, 2e-5), (torch.bfloat16, 1.5e-2)):
        kd, vd = k.to(dtype).float(), v.to(dtype).float()
        want = shaped_reference(q.to(dtype).float(), kd, vd, positions, 1.0, window, cap, sinks, turn, 4)
        k_pool, v_pool, table = paged(k, v, page_tokens, dtype, 9)
        flat_q = q.reshape(len(positions), -1).to(dtype).to(DEV)
        out = ops.attention_rows(flat_q, k_pool, v_pool, rows_at, entry, table, q_heads, 1.0, window, shape=shape)
        close(out.float().view(len(positions), q_heads, dim), want, bound, f"row kernel {dtype}")
        if dtype == torch.float32:
            continue
        for splits in (None, 1, 3):
            one = ops.attention_decode(flat_q, k_pool, v_pool, rows_at, entry, table, q_heads, 1.0, window, max_context=n,
                                       splits=splits, shape=shape)
            close(one.float().view(len(positions), q_heads, dim), want, bound, f"split-KV kernel, splits {splits}")
        tiles = ops.prefill_tiles([(0, 0, len(positions))]).to(DEV)
        for splits in (None, 1, 2):
            out = torch.full_like(flat_q, float("nan"))
            ops.attention_prefill(flat_q, out, k_pool, v_pool, rows_at, tiles, table, q_heads, 1.0, window, mean_keys=300,
                                  splits=splits, shape=shape)
            close(out.float().view(len(positions), q_heads, dim), want, bound, f"prompt kernel, splits {splits}")


def talking_reference(q, k, v, talk, positions, scale, window, group):
    """Plain attention of single rows whose heads' scores are mixed before the softmax."""
    out = torch.zeros(len(positions), q.shape[1], v.shape[2], dtype=F)
    keys = torch.arange(k.shape[0])
    for r, p in enumerate(positions):
        see = (keys <= p) & ((p - keys < window) if window else torch.ones_like(keys, dtype=torch.bool))
        score = torch.stack([(k[:, g // group].double() @ q[r, g].double()) * scale for g in range(q.shape[1])])
        mixed = (talk.double() @ score).masked_fill(~see, float("-inf"))
        weight = torch.softmax(mixed, dim=-1)
        for head in range(q.shape[1]):
            out[r, head] = weight[head] @ v[:, head // group].double()
    return out


@pytest.mark.parametrize("page_tokens", [16, 64])
@pytest.mark.parametrize("q_heads,kv_heads,dim,vdim,window", [(4, 4, 64, 64, 0), (8, 2, 32, 32, 40), (16, 4, 128, 128, 0), (12, 3, 128, 96, 0),
                                                              (5, 5, 24, 20, 0), (16, 16, 40, 64, 0), (24, 6, 128, 64, 0), (32, 8, 128, 128, 33),
                                                              (1, 1, 128, 128, 0), (6, 3, 64, 128, 0), (32, 8, 128, 128, 0),
                                                              (20, 5, 64, 48, 0), (24, 24, 32, 32, 0), (17, 1, 96, 128, 0), (30, 10, 80, 16, 0), (8, 1, 128, 128, 0), (2, 2, 16, 4, 64)])
def test_all_three_attention_kernels_with_mixed_scores(q_heads, kv_heads, dim, vdim, window, page_tokens):
    """The row kernel (float32 and bfloat16), the split-KV kernel (rows one by one, and cut into several parts) and the prompt
    kernel (portions that continue a request of 100 tokens, one of them of 5 rows, in one range of keys and in several)
    against plain attention.  Every row's queries point along one key each, another one for every head: its own, the one
    before, the first, one far back, keys on both sides of a page's and a stage's border; the mix has large entries off
    its diagonal, so a head reads what others ask for; scores differ by tens, so references are raised along the way."""
    from leone_amd import ops
    n, first = 333, 100
    k, v = planted(n, kv_heads, dim, vdim, 5 + dim)
    gen = torch.Generator().manual_seed(q_heads)
    talk = (0.5 * torch.eye(q_heads) + 0.7 * torch.randn(q_heads, q_heads, generator=gen) / math.sqrt(q_heads)).bfloat16()
    positions = list(range(first, n))
    q = torch.zeros(len(positions), q_heads, dim)
    for r, i in enumerate(positions):
        for head in range(q_heads):
            kinds = [i, i - 1, 0, i // 2, 63, 64, 15, 16, i - window + 1, i - window]
            j = min(max(kinds[(r + 3 * head) % (len(kinds) if window else 8)], 0), i)
            key = k[j, head * kv_heads // q_heads].bfloat16().float()
            q[r, head] = key / (key @ key) * (4.0 + 10.0 * (r % 3))
    rows_at = torch.tensor(positions, dtype=torch.int32, device=DEV)
    entry = torch.zeros(len(positions), dtype=torch.int32, device=DEV)
    for dtype, bound in ((torch.float32, 2e-5), (torch.bfloat16, 1.5e-2)):
        want = talking_reference(q.to(dtype).float(), k.to(dtype).float(), v.to(dtype).float(), talk.float(), positions, 1.0, window,
                                 q_heads // kv_heads)
        k_pool, v_pool, table = paged(k, v, page_tokens, dtype, 9)
        flat_q = q.reshape(len(positions), -1).to(dtype).to(DEV)
        on = talk.to(DEV)
        out = ops.attention_rows_talk(flat_q, k_pool, v_pool, on, rows_at, entry, table, q_heads, 1.0, window)
        close(out.float().view(len(positions), q_heads, vdim), want, bound, f"row kernel {dtype}")
        if dtype == torch.float32:
            continue
        kernels = ops.talk_attention_supported(dtype, q_heads, dim, vdim, page_tokens)
        assert kernels == {"decode": True, "prompt": True}
        for splits in (None, 1, 3, 20):
            one = ops.attention_talk_decode(flat_q, k_pool, v_pool, on, rows_at, entry, table, q_heads, 1.0, window, max_context=n,
                                            splits=splits)
            close(one.float().view(len(positions), q_heads, vdim), want, bound, f"split-KV kernel, splits {splits}")
        if not kernels["prompt"] or window:
            continue
        cuts = [(0, 5)] + [(at, min(16, len(positions) - at)) for at in range(5, len(positions), 16)]
        tiles = torch.tensor([(0, at, rows) for at, rows in cuts], dtype=torch.int32, device=DEV)
        for splits in (None, 1, 2, 7):
            out = torch.full((len(positions), q_heads * vdim), float("nan"), dtype=dtype, device=DEV)
            ops.attention_talk_prefill(flat_q, out, k_pool, v_pool, on, rows_at, tiles, table, q_heads, 1.0, mean_keys=200, splits=splits)
            close(out.float().view(len(positions), q_heads, vdim), want, bound, f"prompt kernel, splits {splits}")
