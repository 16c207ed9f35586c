"""Sonulorn on the GPU against the plain implementation: each mechanism alone, whole models of several sizes under every way
of cutting the work, pages and slots that are used again, keys planted far away and at the edges of chunks and pages,
memories that reach hundreds of tokens back, long decoding, and generation through the scheduler."""
import json
import os
import subprocess
import sys
import tempfile

import numpy as np
import pytest
import torch

from tests import schedules
from tests import sonulorn_util as su
from tests.plain import sonulorn_plain as plain
from tests.test_gpu_fosulix import SCHEDULES, close, compare, make_engine, run_steps, widened
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
            raw = su.SMALL[name]
            weights = su.make_weights(raw, 71 + len(cache), DTYPES[dtype_name], sharpen=2.0 if dtype_name == "float32" else 1.0)
            folder = su.write_dir(str(tmp_path_factory.mktemp(f"sonulorn_{name}_{dtype_name}")), raw, weights)
            gen = np.random.default_rng(29 + len(cache))
            requests = {f"r{i}": gen.integers(0, raw["vocab"], size=n).tolist() for i, n in enumerate(LENGTHS[name])}
            expected = {rid: plain.forward(raw, widened(weights), toks).numpy() for rid, toks in requests.items()}
            cache[key] = (folder, requests, expected)
        return cache[key]
    return get


@pytest.mark.parametrize("schedule", list(SCHEDULES))
@pytest.mark.parametrize("dtype_name", list(DTYPES))
@pytest.mark.parametrize("name", list(su.SMALL))
def test_engine_agrees_with_plain_however_the_work_is_cut(cases, name, dtype_name, schedule):
    """Whole prompts, tails decoded token by token (chunks of 1 to 50 positions end among decoded tokens), portions down to
    two tokens, and four requests at a time with portions beside single tokens, on an engine with four slots and
    just enough pages: pages and slots are used again, also pages of chunks that were passed.  Logits at every position."""
    folder, requests, expected = cases(name, dtype_name)
    steps = SCHEDULES[schedule](requests)
    page = PAGE_TOKENS[name]
    engine = make_engine(folder, dtype_name, max_tokens=schedules.max_live_tokens(steps, page), page_tokens=page, poison_freed=True)
    outputs = run_steps(engine, steps)
    worst = compare(steps, outputs, expected, dtype_name, f"{name} {dtype_name} {schedule}")
    print(f"{name} {dtype_name} {schedule}: worst relative error {worst:.2e}")
    assert all(engine.cache.free_pages(g) == engine.cache.groups[g].num_pages for g in range(len(engine.cache.groups)))


@pytest.mark.parametrize("how", ["products", "walks"])
@pytest.mark.parametrize("schedule", ["whole", "portions", "mixed"])
@pytest.mark.parametrize("name", ["A", "B"])
def test_long_portions_of_the_memories_in_chunks(cases, monkeypatch, name, schedule, how):
    """From portions of 16 rows on, the memories work in chunks: as products over chunks of 64 rows, or (what heads of more key
    channels take) in chunks of 8 rows walked side by side and chained, by a factor for the fixed decays and by a matrix for
    the delta rule.  The results differ by rounding only."""
    from leone_amd import ops
    monkeypatch.setattr(ops, "MEMORY_CHUNKS_FROM", 16)
    if how == "walks":
        monkeypatch.setattr(ops, "chunked_memory_supported", lambda dim: False)
        monkeypatch.setattr(ops, "OUTER_CHUNKS", (8, 16))
        monkeypatch.setattr(ops, "DELTA_CHUNKS", (8, 16))
    folder, requests, expected = cases(name, "float32")
    steps = SCHEDULES[schedule](requests)
    engine = make_engine(folder, "float32", max_tokens=schedules.max_live_tokens(steps, 16), poison_freed=True)
    compare(steps, run_steps(engine, steps), expected, "float32", f"{name} chunked walk {schedule}")


ODD = su.config(100, 301, [
    su.layer(su.parallel((3, 3, 12, 9, 6, 3), (5, 5, 7, 11, 4), 0.9, 1.7, base=300.0), su.dense(50, 1.3)),
    su.layer(su.attention(5, 1, 20, 7, 14, 13), su.dense(18)),
    su.layer(su.lightning(3, 70, 5), su.dense(7)),
    su.layer(su.attention(7, 7, 9, 30, 2, 100, base=50.0), None),
    su.layer(su.parallel((1, 1, 38, 3, 2, 6), (2, 1, 33, 66, 2), -1.0, 1.0, base=50.0), su.dense(9, 0.2)),
], (1, 5, 2), embed_scale=0.7)


@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_sizes_that_are_multiples_of_nothing(dtype_name):
    """Width 100, vocabulary 301, keys of 12, 20, 9 and 38 elements and values of 9, 7, 30 and 3 (heads filled up with zeros to
    what the cache packs, with a gate for every element too), memories of 7 x 11, 33 x 66 and 70 x 5, feed-forwards of 50, 18,
    7 and 9, a prompt of 600 tokens (the memories' long portions in chunks), pages of 64 tokens: every kernel's path for
    sizes that fill no run of 8 or 16."""
    weights = su.make_weights(ODD, 3, DTYPES[dtype_name])
    gen = np.random.default_rng(1)
    requests = {f"r{i}": gen.integers(0, ODD["vocab"], size=n).tolist() for i, n in enumerate([600, 70, 5, 129])}
    expected = {rid: plain.forward(ODD, widened(weights), toks).numpy() for rid, toks in requests.items()}
    with tempfile.TemporaryDirectory() as folder:
        su.write_dir(folder, ODD, weights)
        for name in ("whole", "mixed"):
            steps = SCHEDULES[name](requests)
            engine = make_engine(folder, dtype_name, max_tokens=schedules.max_live_tokens(steps, 64), page_tokens=64, poison_freed=True)
            compare(steps, run_steps(engine, steps), expected, dtype_name, f"odd sizes {name}")


WIDE = su.config(256, 199, [
    su.layer(su.lightning(4, 128, 256), su.dense(512)),
    su.layer(su.attention(8, 2, 64, 64, 32, 200), su.dense(512, 7.0)),
    su.layer(su.parallel((4, 2, 64, 64, 64, 4), (4, 2, 128, 128, 4), 0.5, 0.5), su.dense(512, 7.0)),
], (0, 3, 2))


@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_sizes_of_published_layers_in_long_portions(dtype_name):
    """Heads of 64 and 128, values of 256 (rows of 1,024 columns normed together), a prompt of 700 tokens beside shorter ones
    and a second portion of 300: the kernels that long portions of such sizes get."""
    weights = su.make_weights(WIDE, 5, DTYPES[dtype_name])
    gen = np.random.default_rng(4)
    requests = {f"r{i}": gen.integers(0, WIDE["vocab"], size=n).tolist() for i, n in enumerate([700, 40, 513])}
    expected = {rid: plain.forward(WIDE, widened(weights), toks).numpy() for rid, toks in requests.items()}
    with tempfile.TemporaryDirectory() as folder:
        su.write_dir(folder, WIDE, weights)
        cuts = [("r0", 400), ("r1", 39), ("r2", 200), None, ("r0", 299), ("r1", 1), ("r2", 1), None, ("r0", 1), ("r2", 312), None]
        steps, at, now = [], {rid: 0 for rid in requests}, []
        for cut in cuts:
            if cut is None:
                done = [e["id"] for e in now if at[e["id"]] == len(requests[e["id"]])]
                steps.append({"step": len(steps), "entries": now, "end": done})
                now = []
                continue
            rid, n = cut
            now.append({"id": rid, "tokens": requests[rid][at[rid]:at[rid] + n], "want": list(range(n))})
            at[rid] += n
        for way in (schedules.whole(requests), steps):
            engine = make_engine(folder, dtype_name, max_tokens=1408, page_tokens=64, poison_freed=True)
            compare(way, run_steps(engine, way), expected, dtype_name, "published sizes")


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


def test_fewer_pages_than_tokens_once_chunks_are_passed():
    """A request whose every attention layer sees chunks of 24 positions decodes 200 tokens on four pages of 16."""
    raw = su.config(48, 90, [su.layer(su.attention(2, 1, 16, 16, 8, 24), su.dense(40)), su.layer(su.lightning(2, 8, 8), None)], (0, 1, 2))
    weights = su.make_weights(raw, 6, torch.float32)
    tokens = np.random.default_rng(3).integers(0, 90, size=200).tolist()
    expected = {"a": plain.forward(raw, weights, tokens).numpy()}
    with tempfile.TemporaryDirectory() as folder:
        su.write_dir(folder, raw, weights)
        engine = make_engine(folder, "float32", num_pages=4, max_context=256, poison_freed=True)
        steps = schedules.portions({"a": tokens}, sizes=(20, 1, 1, 30, 1, 2))
        compare(steps, run_steps(engine, steps), expected, "float32", "few pages")


def test_long_decoding_through_recorded_steps():
    """A short prompt, then 300 tokens one by one (steps replayed from a recording), two requests side by side: chunks end
    among decoded tokens many times, their pages are handed back and used again, memories and filters are carried 300 steps
    by layers that run three times over, every pass with its own."""
    raw = su.SMALL["B"]
    weights = su.make_weights(raw, 91, torch.float32, sharpen=2.0)
    gen = np.random.default_rng(2)
    requests = {"a": gen.integers(0, raw["vocab"], size=310).tolist(), "b": gen.integers(0, raw["vocab"], size=305).tolist()}
    expected = {rid: plain.forward(raw, weights, toks).numpy() for rid, toks in requests.items()}
    with tempfile.TemporaryDirectory() as folder:
        su.write_dir(folder, raw, weights)
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


def test_steps_of_many_rows_of_single_tokens(cases):
    """24 requests decoded together (more rows than the folded products take), in bfloat16 with the matrices' second copies."""
    folder, requests, expected = cases("C", "bfloat16")
    raw = su.SMALL["C"]
    tokens = requests["r0"][:40]
    want = {f"n{i}": expected["r0"][:40 - i % 3] for i in range(24)}
    steps = []
    for at in range(40):
        entries = [{"id": rid, "tokens": [tokens[at]], "want": [0]} for rid, rows in want.items() if at < len(rows)]
        steps.append({"step": at, "entries": entries, "end": [e["id"] for e in entries if at == len(want[e["id"]]) - 1]})
    engine = make_engine(folder, "bfloat16", max_tokens=24 * 64, max_requests=24)
    compare(steps, run_steps(engine, steps), want, "bfloat16", f"24 rows a step of {raw['width']}")


def test_greedy_generation_through_the_scheduler():
    """The framework's own entry point: prompts in, greedy tokens out, scheduled in portions with more requests
    than slots, against the plain implementation's argmax token by token."""
    from leone_amd.api import Runtime
    from leone_amd.engine.scheduler import SchedulerPolicy
    raw = su.SMALL["A"]
    weights = su.make_weights(raw, 23, torch.float32, sharpen=2.0)
    gen = np.random.default_rng(8)
    prompts = [gen.integers(0, raw["vocab"], size=n).tolist() for n in (3, 40, 21, 9, 57)]
    with tempfile.TemporaryDirectory() as folder:
        su.write_dir(folder, raw, weights)
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
    """``leone generate`` on a Sonulorn folder: greedy tokens as the plain implementation picks them; ``leone random-model``
    writes a folder of the design that loads again."""
    from leone_amd import cli
    raw = su.SMALL["C"]
    weights = su.make_weights(raw, 61, torch.float32, sharpen=2.0)
    folder = su.write_dir(str(tmp_path / "model"), raw, weights)
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
    config_path = str(tmp_path / "config.json")
    with open(config_path, "w") as handle:
        json.dump(su.SMALL["A"], handle)
    made = str(tmp_path / "made")
    assert cli.main(["random-model", "--config", config_path, "--seed", "3", "--out", made]) == 0
    engine = make_engine(made, "bfloat16", max_tokens=64)
    from leone_amd.engine.engine import StepEntry
    logits = engine.step([StepEntry("a", [1, 2, 3], [2])]).logits
    assert logits.shape == (1, su.SMALL["A"]["vocab"]) and torch.isfinite(logits).all()


# ---- each mechanism alone ---------------------------------------------------------------------------------------

def build_mixer(entry, dtype, width, seed, sharpen=2.0, weights=None):
    """(part, weights in double, the mixer's configuration) of one mixer from a layer entry of ``sonulorn_util``: the model's
    own builder makes the part's description, so the test covers what a model of this mixer alone would run."""
    from leone_amd.architectures import config_from_dict, model_spec_for
    from leone_amd.parts import MIXERS, POSITIONS
    raw = su.config(width, 32, [su.layer(entry)])
    spec = model_spec_for(config_from_dict(raw))
    positions = {name: POSITIONS.build(s) for name, s in spec.positions.items()}
    for part in positions.values():
        part.prepare(512, DEV)
    mixer = MIXERS.build(spec.layers[0]["mixer"], positions=positions)
    gen = torch.Generator().manual_seed(seed)
    w = {k[len("l0.mix."):]: su.one_tensor(k, v, gen, sharpen).to(dtype) for k, v in su.tensor_shapes(raw).items()
         if k.startswith("l0.mix.")}
    w.update({k: v.to(dtype) for k, v in (weights or {}).items()})
    mixer.bind({"l0.mix." + k: v.to(DEV) for k, v in w.items()})
    return mixer, {k: v.to(F) for k, v in w.items()}, entry["mixer"]


def check_in_cuts(mixer, want_of, width, dtype_name, page_tokens=16, bound=None, rows=(63, 66)):
    dtype = DTYPES[dtype_name]
    gen = torch.Generator().manual_seed(3)
    hs = [torch.randn(n, width, generator=gen).to(dtype) for n in rows]
    got = run_mixer_in_cuts(mixer, hs, CUTS, dtype, page_tokens)
    for s in (0, 1):
        err = su.relative_error(got[s].numpy(), want_of(hs[s].to(F)).numpy())
        assert err.max() <= (bound or (2e-5 if dtype_name == "float32" else 4e-2)), (s, int(err.argmax()), float(err.max()))


def m_seed(entry):
    return sum(ord(c) for c in json.dumps(entry, sort_keys=True)) % 1000


CHUNKED = [su.attention(4, 2, 16, 24, 8, 20, 100.0), su.attention(1, 1, 40, 8, 40, 7), su.attention(6, 6, 8, 8, 2, 1),
           su.attention(8, 2, 64, 64, 64, 16), su.attention(16, 4, 32, 32, 16, 33), su.attention(12, 3, 128, 128, 32, 50),
           su.attention(5, 1, 20, 7, 6, 12), su.attention(4, 4, 48, 96, 24, 1000), su.attention(3, 1, 9, 5, 4, 64),
           su.attention(2, 2, 24, 8, 24, 16)]            # the rotated part is longer than a value


@pytest.mark.parametrize("page_tokens", [16, 32])
@pytest.mark.parametrize("dtype_name", list(DTYPES))
@pytest.mark.parametrize("entry", CHUNKED, ids=lambda e: f"{e['mixer']['heads']}x{e['mixer']['dim']}x{e['mixer']['vdim']}_{e['mixer']['mask']['size']}")
def test_attention_within_chunks_alone_in_cuts_of_every_size(entry, dtype_name, page_tokens):
    """Two sequences side by side, fed in steps of 0 to 40 rows each, pages interleaved and filled with NaN beforehand: chunks
    of one position, below, at and above a page, and longer than the sequence; sinks; a gate for every element."""
    width = 48
    mixer, w, m = build_mixer(entry, DTYPES[dtype_name], width, seed=m_seed(entry), sharpen=2.0 if dtype_name == "float32" else 1.0)
    check_in_cuts(mixer, lambda h: plain.sink_attention(h, m, w, "", chunk=m["mask"]["size"], gate_each=True), width, dtype_name, page_tokens)


SIDES = [su.parallel((4, 1, 16, 24, 8, 4), (3, 3, 8, 12, 2), 0.8, -0.6, 100.0),
         su.parallel((2, 1, 24, 8, 24, 1), (4, 2, 20, 33, 5), 1.3, 0.4, 10000.0),
         su.parallel((6, 3, 16, 16, 16, 3), (2, 1, 40, 16, 1), 0.0, 1.0, 77.0),
         su.parallel((8, 1, 32, 32, 16, 2), (8, 4, 64, 64, 3), 1.0, 0.0),
         su.parallel((1, 1, 48, 48, 2, 5), (1, 1, 130, 70, 4), 0.5, 0.5),
         su.parallel((8, 2, 128, 128, 64, 4), (2, 2, 64, 128, 4), 1.0, 0.0, 5000.0),
         su.parallel((4, 2, 12, 5, 4, 3), (6, 3, 6, 10, 7), 0.0, -1.0),
         su.parallel((2, 2, 8, 8, 2, 2), (4, 1, 256, 32, 2), 0.1, 1.0)]


@pytest.mark.parametrize("page_tokens", [16, 32])
@pytest.mark.parametrize("dtype_name", list(DTYPES))
@pytest.mark.parametrize("entry", SIDES, ids=lambda e: f"{e['mixer']['left']['heads']}x{e['mixer']['left']['dim']}_{e['mixer']['right']['heads']}x{e['mixer']['right']['dim']}x{e['mixer']['right']['vdim']}")
def test_attention_beside_a_delta_rule_alone(entry, dtype_name, page_tokens):
    """Both branches and their weighted sum; a weight of zero leaves one branch alone (filters of 1 to 7 taps, sinks, a gate a
    head; the delta rule with its own filters, unit vectors and decays), so a fault in either shows at full size."""
    width = 48
    mixer, w, m = build_mixer(entry, DTYPES[dtype_name], width, seed=m_seed(entry), sharpen=2.0 if dtype_name == "float32" else 1.0)
    check_in_cuts(mixer, lambda h: plain.side_by_side(h, m, w, "", 1e-5), width, dtype_name, page_tokens)


MEMORIES = [su.lightning(3, 8, 20, (0.0, 0.95, 1.0)), su.lightning(1, 40, 16), su.lightning(5, 24, 6), su.lightning(2, 256, 33),
            su.lightning(4, 64, 300), su.lightning(8, 128, 128), su.lightning(2, 100, 1)]


@pytest.mark.parametrize("dtype_name", list(DTYPES))
@pytest.mark.parametrize("entry", MEMORIES, ids=lambda e: f"{e['mixer']['heads']}x{e['mixer']['dim']}x{e['mixer']['vdim']}")
def test_memory_with_fixed_decays_alone(entry, dtype_name):
    """Decays of 0 (nothing is kept) to 1 (nothing is lost), heads normed together over 2 to 1,200 columns."""
    width = 48
    mixer, w, m = build_mixer(entry, DTYPES[dtype_name], width, seed=m_seed(entry))
    check_in_cuts(mixer, lambda h: plain.fixed_decay_memory(h, m, w, "", 1e-5), width, dtype_name)


@pytest.mark.parametrize("which", ["delta", "fixed"])
def test_memories_reach_hundreds_of_tokens_back(which):
    """What a token writes is still there 250 tokens later.  A marked token at position 2 is read at positions 200 to 259, in
    a portion and token by token, in state slots that held NaN."""
    width = 32
    if which == "delta":
        entry = su.parallel((1, 1, 8, 8, 8, 2), (1, 1, 64, 16, 2), 0.0, 1.0)
        mixer, w, m = build_mixer(entry, torch.float32, width, seed=5, weights={"right.A_log": torch.full((1,), -8.0),
                                                                                "right.b": torch.full((1, 32), -0.3)})
        want_of = lambda h: plain.side_by_side(h, m, w, "", 1e-5)                                    # noqa: E731
    else:
        entry = su.lightning(2, 16, 8, (0.9995, 0.999))
        mixer, w, m = build_mixer(entry, torch.float32, width, seed=6)
        want_of = lambda h: plain.fixed_decay_memory(h, m, w, "", 1e-5)                              # noqa: E731
    gen = torch.Generator().manual_seed(9)
    hs = 0.05 * torch.randn(260, width, generator=gen)
    hs[2] = 4.0 * torch.randn(width, generator=gen)
    cuts = [(200, 1), (30, 1)] + [(1, 1)] * 30
    got = run_mixer_in_cuts(mixer, [hs, hs[:32]], cuts, torch.float32, 16)[0]
    want = want_of(hs.to(F))
    quiet = hs.clone()
    quiet[2] = 0.05 * torch.randn(width, generator=gen)
    without = want_of(quiet.to(F))
    assert float((want[200:] - without[200:]).abs().max()) > 0.05 * float(want[200:].abs().max())   # the mark is what is read
    err = su.relative_error(got.numpy(), want.numpy())
    assert err.max() <= 3e-5, (int(err.argmax()), float(err.max()))


def memory_by_tokens(q, k, v, decay, beta, state):
    """o_t = S_t^T q_t of one head, in float64: S <- g S + k u^T with u = v, or u = beta (v - g S^T k)."""
    out = []
    for t in range(q.shape[0]):
        state = decay[t] * state
        u = v[t] if beta is None else beta[t] * (v[t] - state.T @ k[t])
        state = state + torch.outer(k[t], u)
        out.append(state.T @ q[t])
    return torch.stack(out), state


@pytest.mark.parametrize("entries", [[(70, 0)], [(64, 5), (3, 0), (130, 0)], [(17, 3), (1, 9)], [(640, 0), (129, 7)]], ids=str)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(2, 1, 32, 16), (3, 3, 7, 11), (4, 2, 128, 40), (1, 1, 65, 5), (2, 2, 100, 130), (1, 1, 136, 8)])
@pytest.mark.parametrize("kind", ["delta", "fixed", "extreme"])
def test_memories_with_one_decay_a_head_over_long_portions(monkeypatch, kind, heads, kv_heads, dim, vdim, entries):
    """Portions of 16 rows and more as products over chunks of 64 rows (the largest heads: by walking), beside shorter ones, from
    an empty and from a carried state; a fresh sequence does not read its slot.  Decays of nothing, nearly all and all."""
    from leone_amd import ops
    from leone_amd.parts.context import EntryInfo, StepContext
    monkeypatch.setattr(ops, "MEMORY_CHUNKS_FROM", 16)
    delta = kind != "fixed"
    if not delta:
        kv_heads = heads
    gen = torch.Generator().manual_seed(5)
    rows, kv = sum(count for count, _ in entries), kv_heads * dim
    x = torch.randn(rows, 2 * kv + heads * vdim, generator=gen)
    state = torch.randn(4, heads, dim, vdim, generator=gen)
    strengths, steps_ = torch.randn(rows, heads, generator=gen), torch.randn(rows, heads, generator=gen)
    rate_log, bias = torch.rand(heads, generator=gen) * 2 - 1, torch.rand(heads, generator=gen) * 5 - 6
    if kind == "extreme":       # a step size of hundreds forgets everything, one of nothing keeps it; writes at full strength
        steps_ = torch.where(torch.rand(rows, heads, generator=gen) < 0.1, 300.0, -40.0)
        strengths = strengths * 20
    fixed = torch.tensor([0.0, 0.97, 1.0][:heads] if heads <= 3 else [0.3, 0.9, 0.99, 1.0])
    slots = [2, 0, 3][:len(entries)]
    for slot, (count, start) in zip(slots, entries):
        if start == 0:
            state[slot] = float("nan")
    infos, positions, owners = [], [], []
    for i, (slot, (count, start)) in enumerate(zip(slots, entries)):
        infos.append(EntryInfo(f"r{i}", slot, len(positions), count, start))
        positions += range(start, start + count)
        owners += [i] * count
    step = StepContext(rows=rows, dtype=torch.float32, device=torch.device(DEV), positions=torch.tensor(positions, dtype=torch.int32, device=DEV),
                       row_entry=torch.tensor(owners, dtype=torch.int32, device=DEV), entries=infos,
                       entry_slots=torch.tensor(slots, dtype=torch.int32, device=DEV), want_rows=None)
    dev_x, dev_state = x.to(DEV), state.to(DEV)
    columns = {"q": 0, "k": kv, "v": 2 * kv}
    if delta:
        out = ops.delta_scan(dev_x, columns, strengths.to(DEV), steps_.to(DEV), rate_log.to(DEV), bias.to(DEV), dev_state, step, heads,
                             kv_heads, dim, vdim, dim ** -0.5, 1e-6)
    else:
        out, _ = ops.outer_scan(dev_x, columns, dev_state.view(4, heads, dim * vdim), step, heads, dim, vdim, decay=fixed.to(DEV),
                                activation="silu", k_scale=0.7)
    out, dev_state, x = out.view(rows, heads, vdim).cpu().to(F), dev_state.cpu().to(F), x.to(F)
    at = 0
    for slot, (count, start) in zip(slots, entries):
        span = slice(at, at + count)
        at += count
        for h in range(heads):
            first = (h // (heads // kv_heads)) * dim
            q, k, v = x[span, first:first + dim], x[span, kv + first:kv + first + dim], x[span, 2 * kv + h * vdim:2 * kv + (h + 1) * vdim]
            before = torch.zeros(dim, vdim, dtype=F) if start == 0 else state[slot, h].to(F)
            if delta:
                q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * dim ** -0.5
                k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
                g = torch.exp(-torch.exp(rate_log[h].to(F)) * torch.nn.functional.softplus((steps_[span, h] + bias[h]).to(F)))
                want, after = memory_by_tokens(q, k, v, g, torch.sigmoid(strengths[span, h].to(F)), before)
            else:
                q, k, v = (torch.nn.functional.silu(z) for z in (q, k, v))
                want, after = memory_by_tokens(q, 0.7 * k, v, [float(fixed[h])] * count, None, before)
            close(out[span, h], want, 2e-5, f"{kind} {slot} {h}")
            close(dev_state[slot, h], after, 2e-5, f"{kind} {slot} {h} state")


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


def plant(hs, pairs, dim, width, gen, decoys=None):
    """Every key of ``pairs`` (key position -> query position) answers its query alone; ``decoys`` (query position -> position)
    hold the same key with the opposite value."""
    hs[:, :2 * dim] *= 0.05
    for n, (key_at, query_at) in enumerate(pairs.items()):
        direction = torch.zeros(dim)
        direction[2 + n % (dim - 2)] = 5.0
        hs[key_at, :dim] = direction
        hs[query_at, dim:2 * dim] = direction
        hs[key_at, 2 * dim:] = 3.0 * torch.randn(width - 2 * dim, generator=gen)
        if decoys and query_at in decoys:
            hs[decoys[query_at], :dim] = direction
            hs[decoys[query_at], 2 * dim:] = -hs[key_at, 2 * dim:]


@pytest.mark.parametrize("page_tokens", [16, 32])
@pytest.mark.parametrize("chunk", [40, 64, 100])
@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_chunked_attention_finds_a_chunks_first_key_and_not_the_last_of_the_one_before(dtype_name, chunk, page_tokens):
    """A query asks for the first key of its chunk, for its own position's, and for others of its chunk; a decoy (the same key,
    the opposite value) is the last position of the chunk before.  Queries stand at the first, second and last positions of
    chunks, in a prompt's portion and as single decoded tokens; a portion ends inside a chunk."""
    dtype = DTYPES[dtype_name]
    width, heads, dim, vdim = 96, 2, 32, 32
    entry = su.attention(heads, 1, dim, vdim, 2, chunk, 1e6, scale=1.0)
    wq, wk, wv = key_query_value(heads, dim, vdim, width, 0.6 if dtype_name == "float32" else 0.5)
    mixer, w, m = build_mixer(entry, dtype, width, seed=7, weights={"q": wq, "k": wk, "v": wv, "sink": torch.tensor([-3.0, 1.0])})
    total, gen = 300, torch.Generator().manual_seed(11)
    hs = torch.randn(total, width, generator=gen)
    edges = list(range(chunk, total, chunk))
    queries = {}
    for edge in edges:
        queries[edge] = edge                                  # a chunk's first position sees itself alone
        if edge + 1 < total:
            queries[edge + 1] = edge + 1
        last = min(edge + chunk, total) - 1
        queries[last] = edge + 2 if edge + 2 <= last else last
    pairs = {key: query for query, key in queries.items()}
    decoys = {query: query // chunk * chunk - 1 for query in queries}
    # one decoy a chunk: its direction is the last query's of that chunk, so give each query of a chunk the same direction
    hs[:, :2 * dim] *= 0.05
    for n, edge in enumerate(edges):
        direction = torch.zeros(dim)
        direction[2 + n] = 5.0
        for query, key in queries.items():
            if query // chunk * chunk == edge:
                hs[query, dim:2 * dim] = direction
                if key == query:
                    hs[key, :dim] = direction
        hs[edge - 1, :dim] = direction
        hs[edge - 1, 2 * dim:] = 6.0 * torch.randn(width - 2 * dim, generator=gen)
    hs = hs.to(dtype)
    want = plain.sink_attention(hs.to(F), m, w, "", chunk=chunk, gate_each=True)
    seen = plain.sink_attention(hs.to(F), m, w, "", chunk=None, gate_each=True)          # what a mask without chunks would give
    late = plain.sink_attention(hs.to(F)[1:], m, w, "", chunk=chunk, gate_each=True)     # what chunks off by one would give
    for query in queries:
        assert float((want[query] - seen[query]).abs().max()) > 0.1 * float(want[query].abs().max()), query
    assert any(float((want[q] - late[q - 1]).abs().max()) > 0.2 * float(want[q].abs().max()) for q in edges)
    assert pairs and decoys
    cuts = [(chunk + 7, 1), (2, 1), (270 - chunk - 9, 1)] + [(1, 1)] * 30
    got = run_mixer_in_cuts(mixer, [hs, hs[:33]], cuts, dtype, page_tokens)[0]
    err = su.relative_error(got.numpy(), want.numpy())
    assert err.max() <= (2e-5 if dtype_name == "float32" else 3e-2), (int(err.argmax()), float(err.max()))


@pytest.mark.parametrize("page_tokens", [16, 32])
@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_convolved_attention_finds_far_keys_at_page_borders(dtype_name, page_tokens):
    """Keys that answer one query each are planted at the sequence's start, far back and on both sides of page borders, found
    through filters whose last tap counts most; queries come in a portion and token by token."""
    dtype = DTYPES[dtype_name]
    width, heads, dim, vdim = 64, 2, 16, 16
    entry = su.parallel((heads, 1, dim, vdim, 2, 3), (1, 1, 8, 8, 2), 1.0, 0.0, base=1e6, scale=1.0)
    wq, wk, wv = key_query_value(heads, dim, vdim, width, 0.6 if dtype_name == "float32" else 0.5)

    def taps(n):
        return torch.tensor([0.1, -0.2, 1.0]).repeat(n, 1)
    mixer, w, m = build_mixer(entry, dtype, width, seed=7, weights={
        "left.q": wq, "left.k": wk, "left.v": wv, "left.q.conv": taps(heads * dim), "left.k.conv": taps(dim),
        "left.v.conv": taps(vdim), "left.sink": torch.tensor([-3.0, 1.0])})
    gen = torch.Generator().manual_seed(11)
    hs = torch.randn(300, width, generator=gen)
    pairs = {3: 280, 15: 281, 17: 283, 127: 284, 0: 290, 31: 291, 33: 292, 255: 295}
    plant(hs, pairs, dim, width, gen)
    hs = hs.to(dtype)
    want = plain.side_by_side(hs.to(F), m, w, "", 1e-5)
    blind = hs.clone().to(F)
    for key_at in pairs:
        blind[key_at, :dim] = torch.randn(dim, generator=gen)
    gone = plain.side_by_side(blind, m, w, "", 1e-5)
    for query_at in pairs.values():
        assert float((want[query_at] - gone[query_at]).abs().max()) > 0.2 * float(want[query_at].abs().max())
    cuts = [(270, 1), (10, 1)] + [(1, 1)] * 20
    got = run_mixer_in_cuts(mixer, [hs, hs[:22]], cuts, dtype, page_tokens)[0]
    err = su.relative_error(got.numpy(), want.numpy())
    assert err.max() <= (2e-5 if dtype_name == "float32" else 3e-2), (int(err.argmax()), float(err.max()))


def chunked_reference(q, k, v, positions, scale, chunk, sinks, group):
    out = torch.zeros(len(positions), q.shape[1], v.shape[2], dtype=F)
    for r, p in enumerate(positions):
        first = p // chunk * chunk
        for head in range(q.shape[1]):
            score = (k[first:p + 1, head // group].double() @ q[r, head].double()) * scale
            sink = sinks[head].double() if sinks is not None else torch.tensor(-1e9, dtype=F)
            see = torch.ones_like(score, dtype=torch.bool)
            out[r, head] = plain.softmax_with_sink(score[None], see[None], sink)[0] @ v[first:p + 1, head // group].double()
    return out


@pytest.mark.parametrize("page_tokens", [16, 64])
@pytest.mark.parametrize("chunk,sunk,dim", [(40, True, 32), (64, True, 128), (130, False, 48), (1, True, 16), (33, False, 128), (1000, True, 64), (200, True, 128)])
def test_all_three_attention_kernels_within_chunks(chunk, sunk, dim, page_tokens):
    """The row kernel (float32 and bfloat16), the split-KV kernel (rows one by one, and cut into several parts) and the
    prompt kernel (a portion of 420 rows that continues a request of 100, in one range of keys and in several) against
    plain attention.  Every row's query points along one key: its own, the one before, its chunk's first, the last of the
    chunk before, keys on both sides of a page's border; sinks lie below, among and above the scores."""
    from leone_amd import ops
    n, first, heads, q_heads = 520, 100, 2, 8
    k, v = planted(n, heads, dim, dim, 5 + chunk)
    positions = list(range(first, n))
    q = torch.zeros(len(positions), q_heads, dim)
    for r, i in enumerate(positions):
        edge = i // chunk * chunk
        kinds = [i, i - 1, edge, edge - 1, edge + 1, (i + edge) // 2, 64 * (i // 64), 64 * (i // 64) - 1]
        j = min(max(kinds[r % len(kinds)], 0), i)
        for head in range(q_heads):
            key = k[j, head // 4].bfloat16().float()
            q[r, head] = key / (key @ key) * 12.0
    sinks = torch.linspace(-2.0, 14.0, q_heads) if sunk else None
    shape = ops.ScoreShape(None, sinks.to(DEV) if sunk else None)
    rows_at = torch.tensor(positions, dtype=torch.int32, device=DEV)
    entry = torch.zeros(len(positions), dtype=torch.int32, device=DEV)
    for dtype, bound in ((torch.float32, 2e-5), (torch.bfloat16, 1.5e-2)):
        want = chunked_reference(q.to(dtype).float(), k.to(dtype).float(), v.to(dtype).float(), positions, 1.0, chunk, sinks, 4)
        k_pool, v_pool, table = paged(k, v, page_tokens, dtype, 9)
        flat_q = q.reshape(len(positions), -1).to(dtype).to(DEV)
        out = ops.attention_rows(flat_q, k_pool, v_pool, rows_at, entry, table, q_heads, 1.0, shape=shape, chunk=chunk)
        close(out.float().view(len(positions), q_heads, dim), want, bound, f"row kernel {dtype}")
        if dtype == torch.float32:
            continue
        for splits in (None, 1, 3):
            one = ops.attention_decode(flat_q, k_pool, v_pool, rows_at, entry, table, q_heads, 1.0, max_context=n,
                                       splits=splits, shape=shape, chunk=chunk)
            close(one.float().view(len(positions), q_heads, dim), want, bound, f"split-KV kernel, splits {splits}")
            # gates on the result, as slices of wider rows: one a head, one an element
            wide = 2 * torch.randn(len(positions), q_heads * dim + 3, generator=torch.Generator().manual_seed(8))
            for each, factor in ((False, wide[:, 3:3 + q_heads, None]), (True, wide[:, 3:].reshape(len(positions), q_heads, dim))):
                gated = ops.attention_decode(flat_q, k_pool, v_pool, rows_at, entry, table, q_heads, 1.0, max_context=n, splits=splits,
                                             shape=shape, chunk=chunk, gate=wide.to(DEV)[:, 3:], gate_each=each)
                close(gated.float().view(len(positions), q_heads, dim), want * torch.sigmoid(factor.double()), bound, f"gated, splits {splits}")
        tiles = ops.prefill_tiles([(0, 0, len(positions))]).to(DEV)
        for splits in (None, 1, 2):
            out = torch.full_like(flat_q, float("nan"))
            ops.attention_prefill(flat_q, out, k_pool, v_pool, rows_at, tiles, table, q_heads, 1.0, mean_keys=300,
                                  splits=splits, shape=shape, chunk=chunk)
            close(out.float().view(len(positions), q_heads, dim), want, bound, f"prompt kernel, splits {splits}")
    with pytest.raises(ops.KernelError, match="chunk"):
        ops.attention_rows(flat_q, k_pool, v_pool, rows_at, entry, table, q_heads, 1.0, 5, chunk=chunk)


@pytest.mark.parametrize("limit", [0.3, 1.5, 7.0])
@pytest.mark.parametrize("dtype_name", list(DTYPES))
def test_feed_forward_held_to_a_limit(dtype_name, limit):
    """Gates and ups on both sides of the limit, in steps of 1, 7, 16, 60, 200 and 700 rows (every product kernel's epilogue
    and the kernel behind the library's product), sizes that fill runs of 8 and that do not; the matrices' second copies."""
    from leone_amd import ops
    from leone_amd.parts import FEED_FORWARDS
    from leone_amd.parts.base import PartSpec
    dtype = DTYPES[dtype_name]
    gen = torch.Generator().manual_seed(4)
    for width, ff in ((72, 52), (128, 96), (50, 7)):
        w = {"p.gate": torch.randn(ff, width, generator=gen), "p.up": torch.randn(ff, width, generator=gen),
             "p.down": torch.randn(width, ff, generator=gen) / ff ** 0.5}
        w = {k: (v * (2.5 / width ** 0.5) if k != "p.down" else v).to(dtype) for k, v in w.items()}
        part = FEED_FORWARDS.build(PartSpec("swiglu", {"hidden": width, "intermediate": ff, "gate": "p.gate", "up": "p.up",
                                                       "down": "p.down", "activation": "clamped_swish", "limit": limit,
                                                       "float_output": True}))
        part.bind({k: v.to(DEV) for k, v in w.items()})
        for copies in (False, True):
            if copies:
                for matrix in part.streamed_weights():
                    ops.keep_streamed_copy(matrix)
            for rows in (1, 7, 16, 60, 200, 700):
                h = torch.randn(rows, width, generator=gen).to(dtype)
                got = part.forward(h.to(DEV), step_of([(0, i) for i in range(rows)], dtype, [0]))
                got = (got.sum(dim=0) if got.dim() == 3 else got).float().cpu()
                want = plain.clamped_feed_forward(h.to(F), {k: v.to(F) for k, v in w.items()}, "p.", limit)
                err = su.relative_error(got.numpy(), want.numpy())
                assert err.max() <= (2e-5 if dtype_name == "float32" else 3e-2), (width, rows, copies, float(err.max()))


@pytest.mark.parametrize("rows,hidden", [(1, 64), (9, 100), (3, 2048), (600, 192), (5, 66), (17, 51)])
def test_stream_joined_with_the_embedding(rows, hidden):
    """The operand is the stream with everything pending added beside the embedding's output, the stream becomes the pass's
    vector; none to six pending results, with factors, vectors and planes; both types."""
    from leone_amd import ops
    gen = torch.Generator().manual_seed(rows)
    x, first, vector = (torch.randn(*s, generator=gen) for s in ((rows, hidden), (rows, hidden), (hidden,)))
    terms = [(torch.randn(rows, hidden, generator=gen), 0.7, torch.randn(hidden, generator=gen).bfloat16()),
             (torch.randn(2, rows, hidden, generator=gen), -1.2, None), (torch.randn(rows, hidden, generator=gen), 1.0, None),
             (torch.randn(rows, hidden, generator=gen), 2.0, None), (torch.randn(rows, hidden, generator=gen), 0.5, None),
             (torch.randn(rows, hidden, generator=gen), 0.25, None)]

    def on(t):
        return None if t is None else t.to(DEV)
    for count in (0, 1, 3, 4, 6):
        total = x.double().clone()
        for t, f, s in terms[:count]:
            total += f * (t.sum(dim=0) if t.dim() == 3 else t).double() * (1.0 if s is None else s.double())
        for following, dtype in ((vector, torch.float32), (vector.bfloat16(), torch.bfloat16), (None, torch.float32)):
            stream = x.clone().to(DEV)
            got = ops.stream_join(stream, [(on(t), f, on(s)) for t, f, s in terms[:count]], on(first), on(following), dtype)
            want = torch.cat([total, first.double()], dim=1)
            assert got.dtype == dtype and torch.allclose(got.cpu().double(), want, atol=1e-5 if dtype == torch.float32 else 3e-2, rtol=1e-2 if dtype != torch.float32 else 1e-5), count
            kept = torch.zeros(hidden) if following is None else following.float()
            assert torch.equal(stream.cpu(), kept.expand(rows, hidden))


def test_embedding_written_twice():
    from leone_amd import ops
    table = torch.randn(50, 70)
    tokens = torch.tensor([3, 49, 0, 3], dtype=torch.int32, device=DEV)
    for dtype in (torch.float32, torch.bfloat16):
        twin = torch.full((4, 70), float("nan"), device=DEV)
        out = ops.embed(table.to(dtype).to(DEV), tokens, scale=1.5, copy=twin)
        assert torch.equal(out, twin) and torch.allclose(out.cpu(), table.to(dtype).float()[[3, 49, 0, 3]] * 1.5)


@pytest.mark.parametrize("rows", [1, 5, 600])
def test_heads_normed_together(rows):
    """Runs of 96 to 5,000 columns under one root mean square, gate ahead of the norm and behind it, gains shared and not."""
    from leone_amd import ops
    gen = torch.Generator().manual_seed(rows)
    for heads, size in ((1, 96), (1, 1024), (1, 1025), (2, 1500), (1, 4096), (1, 5000)):
        if rows > 100 and size > 2000:
            continue
        o, g = torch.randn(rows, heads * size, generator=gen), torch.randn(rows, heads * size + 3, generator=gen)
        gain = 1 + 0.3 * torch.randn(size, generator=gen)
        on_gate = g.to(DEV)[:, :heads * size]
        for act, fn in (("sigmoid", torch.sigmoid), ("silu", plain.silu)):
            for gate_first in (False, True):
                got = ops.head_norm_gate(o.to(DEV), heads, size, 1e-5, torch.float32, gain=gain.to(DEV), gate=on_gate, activation=act,
                                         gate_first=gate_first).cpu().double()
                wide = o.double().view(rows, heads, size)
                opened = fn(g.double()[:, :heads * size]).view(rows, heads, size)
                want = plain.unit_rms(wide * opened, 1e-5) * gain.double() if gate_first else \
                    plain.unit_rms(wide, 1e-5) * gain.double() * opened
                assert torch.allclose(got.view_as(want), want, atol=2e-5, rtol=1e-5), (heads, size, act, gate_first)
