"""The Nidasun design on the GPU against the plain implementation of tests/plain/nidasun_plain.py: every mechanism alone
(the streams' passes, norms over a whole projection, scans of activated inputs, the gated recurrence in its three forms,
chunks and windows of keys, the sink, corrected routing), whole models of several shapes, prompts cut into portions,
token-by-token decoding, batches of unequal requests on a cache that is used again, keys and writes planted far away, at
page borders and at both sides of every window's and chunk's edge, long decoding through the recorded decode step, and
greedy generation through the Python entry point, the command line and the replay program."""
import json
import os
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import helpers
from helpers import run_batch, run_tail_one_by_one, run_whole
from plain import nidasun_plain as P
from test_nidasun_config import att, config, lin, par, random_weights

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
F32, BF16 = torch.float32, torch.bfloat16
DTYPES = ["float32", "bfloat16"]
TORCH_DT = {"float32": F32, "bfloat16": BF16}

# A: sizes in sixteens (matrix-core attention, both kinds, and products in bfloat16); a loop in the middle; windows and
#    chunks that are no multiples of a page; experts in groups; a layer without a feed-forward; three streams.
# B: sizes that are no multiple of 8 or 16 (plain products and attention, scans of odd sizes, recurrence blocks that the
#    matrix cores do not take, five taps), the whole model in the loop, nothing that turns on one side, two streams.
# C: no loop, one stream; a window and a chunk of exactly a page, blocks of 128 channels, heads of 144 key channels, decays
#    of 1 and of almost nothing, one group of experts.
# D: five streams; a window and a chunk of one key, one tap, one block of channels, one expert a token; a chunk longer
#    than any request.
CONFIGS = {
    "A": config(160, 96, 3, [
        att((6, 2, 32, 48), 90, (1e4, 32), ff=(48, 8, 3, 1.75, 4, 2)),
        par((4, 4, 32, 32), 40, (5e3, 32, 4.0), (96, 3, 4), ff=80),
        lin(3, 32, 16, (0.75, 0.96875, 0.998), ff=(32, 6, 2, 2.5, 2, 1)),
        par((2, 1, 16, 48), 101, (1e3, 8, 2.0), (64, 2, 2), scales=(0.5, 0.8)),
    ], loop=(1, 3, 3), eps=3e-4),
    "B": config(131, 60, 2, [
        par((3, 3, 10, 14), 67, (77.0, 6, 3.0), (42, 2, 5), ff=36),
        lin(2, 10, 6, (0.984375, 0.5), ff=(20, 6, 2, 1.0, 3, 2)),
        att((5, 1, 6, 10), 33, (300.0, 4)),
        par((2, 1, 22, 30), 20, (1e4, 0), (27, 1, 3), scales=(1.25, 0.5), ff=(12, 4, 2, 1.5, 2, 2)),
    ], loop=(0, 4, 2), eps=1e-6),
    "C": config(200, 64, 1, [
        par((8, 2, 16, 16), 64, (1e4, 16, 8.0), (256, 2, 3), ff=(64, 12, 4, 2.0, 1, 1)),
        att((4, 1, 64, 32), 64, (5e5, 32), ff=136),
        lin(2, 144, 80, (1.0, 0.0625), ff=72),
    ], eps=1e-5),
    "D": config(97, 48, 5, [
        att((2, 2, 16, 16), 1, (1e4, 16), ff=(16, 4, 1, 1.5, 2, 1)),
        par((3, 1, 16, 16), 1, (1e4, 16, 16.0), (32, 1, 1), scales=(0.3, 1.2), ff=40),
        att((3, 3, 32, 64), 1000, (1e6, 32), ff=24),
        lin(1, 16, 64, (0.9,)),
    ], loop=(1, 2, 2), eps=1e-5),
}
SEEDS = {"A": 41, "B": 42, "C": 43, "D": 44}
_FOLDERS, _PLAIN, _ENGINES, _WANT = {}, {}, {}, {}


def make_folder(tmp_path_factory, name, cfg, seed, coded=True):
    from safetensors.torch import save_file
    folder = str(tmp_path_factory.mktemp(f"nidasun_{name}"))
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    tensors = {k: torch.from_numpy(v).float().to(BF16).contiguous() for k, v in random_weights(cfg, seed, coded).items()}
    save_file(tensors, os.path.join(folder, "model.safetensors"), metadata={"format": "pt"})
    return folder, {k: v.float().numpy().astype(np.float64) for k, v in tensors.items()}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """name -> folder with config.json and bfloat16 weights."""
    for name, cfg in CONFIGS.items():
        if name not in _FOLDERS:
            _FOLDERS[name], _PLAIN[name] = make_folder(tmp_path_factory, name, cfg, SEEDS[name])
    return _FOLDERS


def engine_for(folder, dtype, max_tokens=64 * 24, **kw):
    from sonicboom_amd.engine import DecoderModel, Engine
    key = (folder, dtype, max_tokens, tuple(sorted(kw.items())))
    if key not in _ENGINES:
        _ENGINES[key] = Engine(DecoderModel.from_folder(folder, dtype), max_tokens, **kw)
    return _ENGINES[key]


def want_logits(name, tokens):
    key = (name, tuple(tokens))
    if key not in _WANT:
        _WANT[key] = P.forward(CONFIGS[name], _PLAIN[name], list(tokens))
    return _WANT[key]


def prompts(name, lengths, seed=0):
    rng = np.random.default_rng(seed)
    return [[int(t) for t in rng.integers(0, CONFIGS[name]["vocab"], size=n)] for n in lengths]


# Bounds.  float32 differs from the plain implementation (float64) by the rounding of float32 sums.
# bfloat16 is measured in spreads of the logits (their standard deviation): the largest difference
# and the root mean square of all differences of a request.
F32_BOUND = 3e-4
BF16_WORST, BF16_RMS = 0.6, 0.068      # what the whole file measured (0.4317 and 0.0487) times 1.4
helpers.BF16_MAX["streams that mix"], helpers.BF16_RMS["streams that mix"] = BF16_WORST, BF16_RMS


def close(got, want, dtype, what):
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    assert got.shape == want.shape, f"{what}: shape {got.shape} vs {want.shape}"
    assert np.isfinite(got).all(), f"{what}: not finite"
    spread = max(float(want.std()), 1e-30)
    err = np.abs(got - want) / spread
    if dtype in ("float32", F32):
        assert err.max() <= F32_BOUND, f"{what}: differs by {err.max():.3g} spreads at {np.unravel_index(err.argmax(), err.shape)}"
    else:
        rms = float(np.sqrt((err ** 2).mean()))
        seen = helpers.BF16_SEEN.setdefault("streams that mix", [0.0, 0.0])
        seen[0], seen[1] = max(seen[0], float(err.max())), max(seen[1], rms)
        assert err.max() <= BF16_WORST and rms <= BF16_RMS, \
            f"{what}: differs by {err.max():.3g} spreads at {np.unravel_index(err.argmax(), err.shape)}, rms {rms:.3g}"


def run_cuts(engine, tokens, cuts):
    """One request fed in portions of the given sizes; logits of every position."""
    from sonicboom_amd.engine import StepEntry
    assert sum(cuts) == len(tokens)
    s = engine.alloc_slot()
    try:
        rows, at = [], 0
        for n in cuts:
            rows.append(engine.step([StepEntry(s, tokens[at:at + n], range(n))]).cpu().numpy())
            at += n
        return np.concatenate(rows, axis=0)
    finally:
        engine.free_slot(s)


# ---- whole models -------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_requests_and_the_first_tokens(folders, name, dtype):
    eng = engine_for(folders[name], dtype)
    for tokens in prompts(name, [1, 2, 3, 17, 63, 64, 65, 200]):
        close(run_whole(eng, tokens), want_logits(name, tokens), dtype, f"{name} whole n={len(tokens)}")
    assert eng.cache.held_pages() == 0 and not eng.cache.live_slots


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_streams_after_every_layer_run_in_32_bit(folders, name):
    eng = engine_for(folders[name], "float32")
    tokens = prompts(name, [75], seed=11)[0]
    got = []
    eng.tracer = lambda what, x: got.append((what, x.detach().cpu().numpy().copy())) if ".after_" in what else None
    try:
        run_whole(eng, tokens)
    finally:
        eng.tracer = None
    last = {what.split(".")[0]: x for what, x in got}       # what an entry reports last is what it leaves
    want = []
    P.forward(CONFIGS[name], _PLAIN[name], tokens, want)
    assert len(last) == len(want)
    for i, (a, b) in enumerate(zip(last.values(), want)):
        b = b.transpose(1, 0, 2).reshape(a.shape)           # a row is its streams side by side
        assert np.abs(a - b).max() <= 2e-5 * np.abs(b).max(), f"{name}: the streams after layer run {i}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_against_token_by_token(folders, name, dtype):
    eng = engine_for(folders[name], dtype)
    for tokens in prompts(name, [40, 150], seed=1):
        got = run_tail_one_by_one(eng, tokens, tail=len(tokens) - 3)
        close(got, want_logits(name, tokens), dtype, f"{name} one by one n={len(tokens)}")
        if dtype == "float32":
            assert np.array_equal(got, run_whole(eng, tokens)), "in 32-bit the cut must not matter by a bit"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions_of_several_sizes(folders, name, dtype):
    eng = engine_for(folders[name], dtype)
    tokens = prompts(name, [331], seed=2)[0]
    whole = run_whole(eng, tokens)
    for cuts in ([2] * 20 + [291], [64, 64, 64, 139], [63, 2, 65, 1, 127, 3, 70], [130, 2, 2, 129, 68], [1, 330]):
        got = run_cuts(eng, tokens, cuts)
        close(got, want_logits(name, tokens), dtype, f"{name} cuts {cuts[:4]}")
        if dtype == "float32":
            assert np.array_equal(got, whole), f"cuts {cuts[:4]} change bits"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_unequal_batches_on_a_cache_that_is_used_again(folders, name, dtype):
    """Nine pages: every batch fills eight of them, the next gets used pages and slots."""
    eng = engine_for(folders[name], dtype, max_tokens=64 * 9, max_slots=5)
    lens = [(1, 9), (70, 4), (5, 30), (130, 12), (33, 1)]
    for round_ in range(3):
        reqs = prompts(name, [p + d for p, d in lens], seed=20 + round_)
        got = run_batch(eng, reqs, [p for p, _ in lens])
        for r, (p, _), g in zip(reqs, lens, got):
            close(g, want_logits(name, r), dtype, f"{name} batch, request of {len(r)}")
        if dtype == "float32":
            alone = run_tail_one_by_one(eng, reqs[3], tail=lens[3][1])
            assert np.array_equal(got[3], alone), "in 32-bit the batch must not matter by a bit"
        assert eng.cache.held_pages() == 0 and not eng.cache.live_slots


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_step_that_runs_in_portions(folders, dtype):
    """A step of more rows than the engine takes at once is cut inside sequences; the groups that read a window or a
    chunk have pools of their own size."""
    eng = engine_for(folders["A"], dtype, max_tokens=64 * 12, max_step_rows=100, max_slots=3)
    reqs = prompts("A", [130, 7, 220], seed=5)
    for _ in range(2):
        got = run_batch(eng, reqs, [130, 7, 220])
        for r, g in zip(reqs, got):
            close(g, want_logits("A", r), dtype, f"portions, request of {len(r)}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_long_decoding_through_the_decode_loop(folders, name, dtype):
    """150 single-token steps of two sequences past page, window and chunk borders, kernel by kernel and then replayed
    from the recorded step; logits of every step against the plain implementation."""
    eng = engine_for(folders[name], dtype)
    reqs = prompts(name, [60 + 150, 3 + 150], seed=7)
    heads = [60, 3]
    from sonicboom_amd.engine import StepEntry
    slots = [eng.alloc_slot() for _ in reqs]
    try:
        eng.step([StepEntry(s, r[:h], ()) for s, r, h in zip(slots, reqs, heads)])
        loop = eng.decode_loop()
        assert loop.use_graph, "every part of the model says its step can be recorded"
        loop.start(slots, [r[h] for r, h in zip(reqs, heads)])
        rows = [[], []]
        for k in range(150):
            logits = loop.step_logits([r[h + k] for r, h in zip(reqs, heads)]).cpu().numpy()
            for i in range(2):
                rows[i].append(logits[i])
        for r, h, got in zip(reqs, heads, rows):
            close(np.stack(got), want_logits(name, r)[h:], dtype, f"{name} long decoding")
    finally:
        for s in slots:
            eng.free_slot(s)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_random_routers_in_32_bit(tmp_path_factory, name):
    """The same models with routers of plain random weights (scores as close as chance makes them)."""
    folder, plain = make_folder(tmp_path_factory, name + "random", CONFIGS[name], 50 + SEEDS[name], coded=False)
    eng = engine_for(folder, "float32")
    tokens = prompts(name, [120], seed=12)[0]
    want = P.forward(CONFIGS[name], plain, tokens)
    close(run_whole(eng, tokens), want, "float32", f"{name} random routers")
    close(run_tail_one_by_one(eng, tokens, tail=30), want, "float32", f"{name} random routers, decoded")


def test_greedy_generation_through_the_entry_point(folders):
    from sonicboom_amd.api import Model
    for name in ("A", "B"):
        ps = prompts(name, [4, 70, 19], seed=9)
        session = Model.load(folders[name], dtype="float32").session(max_tokens=64 * 8)
        got = session.generate(ps, max_tokens=12, stop_tokens=())
        assert got == [P.greedy(CONFIGS[name], _PLAIN[name], p, 12) for p in ps]
        assert [session.generate([p], max_tokens=12, stop_tokens=())[0] for p in ps] == got
        assert not session.engine.cache.live_slots
        # bfloat16: every chosen token is the plain implementation's best or within rounding of it
        session = Model.load(folders[name], dtype="bfloat16").session(max_tokens=64 * 8)
        for p, out in zip(ps, session.generate(ps, max_tokens=12, stop_tokens=())):
            logits = want_logits(name, p + out)
            for i, t in enumerate(out):
                row = logits[len(p) - 1 + i]
                assert row[t] >= row.max() - 2 * BF16_WORST * row.std(), (name, i)


def test_command_line_and_trace_replay(folders, tmp_path):
    """The command line generates from a folder of this design; the replay program feeds a prompt, then
    its next tokens one by one beside a second request, frees one and goes on, and writes the logits
    the plain implementation gives."""
    import subprocess
    import sys
    from conftest import ROOT
    name = "B"
    ps = prompts(name, [4, 10], seed=9)
    tokens = tmp_path / "prompts.txt"
    tokens.write_text("\n".join(" ".join(map(str, p)) for p in ps) + "\n")
    cmd = [sys.executable, os.path.join(ROOT, "bin", "sb-gen"), "-m", folders[name], "--tokens", str(tokens), "-n", "6",
           "--dtype", "fp32", "--stop", ""]
    out = subprocess.run(cmd, capture_output=True, text=True, timeout=100)
    assert out.returncode == 0, out.stderr
    got = [[int(t) for t in line.split()] for line in out.stdout.strip().splitlines()]
    assert got == [P.greedy(CONFIGS[name], _PLAIN[name], p, 6) for p in ps]
    a, b = prompts(name, [75, 12], seed=10)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:70], "want": [0, 69]}, {"id": "b", "tokens": b[:9], "want": [8]}], "end": []}]
    for k in range(3):
        steps.append({"step": k + 1, "entries": [{"id": "a", "tokens": [a[70 + k]], "want": [0]},
                                                 {"id": "b", "tokens": [b[9 + k]], "want": [] if k == 1 else [0]}],
                      "end": ["b"] if k == 2 else []})
    steps.append({"step": 4, "entries": [{"id": "a", "tokens": a[73:75], "want": [1]}], "end": ["a"]})
    for dtype in DTYPES:
        outdir = tmp_path / f"out_{dtype}"
        run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders[name], "--dtype", dtype,
                              "--out", str(outdir), "--max-tokens", "256"], input="\n".join(json.dumps(x) for x in steps) + "\n",
                             capture_output=True, text=True, timeout=100)
        assert run.returncode == 0, run.stderr
        assert [ln for ln in run.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(5)]
        wa, wb = want_logits(name, a), want_logits(name, b)
        vocab = CONFIGS[name]["vocab"]
        read = lambda i: np.fromfile(outdir / f"{i}.f32", dtype="<f4").reshape(-1, vocab)
        close(read(0), np.stack([wa[0], wa[69], wb[8]]), dtype, "replay, prompts")
        close(read(1), np.stack([wa[70], wb[9]]), dtype, "replay, first single tokens")
        close(read(2), wa[71:72], dtype, "replay, a step where one request wants nothing")
        close(read(3), np.stack([wa[72], wb[11]]), dtype, "replay, last step of the short request")
        close(read(4), wa[74:75], dtype, "replay, two more tokens alone")


def drawn_configuration(seed):
    """A configuration from a seed: one to five layers in any order of kinds, head counts with one, several and as many kv
    heads as heads, sizes with and without factors of 8 and 16, windows and chunks below, at and above a page, any number of
    taps and blocks, a loop over any run of layers or none."""
    rng = np.random.default_rng(4000 + seed)
    pick = lambda *v: v[int(rng.integers(len(v)))]

    def heads():
        h = pick(1, 2, 3, 4, 6, 8)
        return h, pick(*[g for g in (1, 2, 3, 4, 6, 8) if h % g == 0]), pick(8, 16, 24, 32, 64), pick(8, 16, 24, 32, 48, 64)

    def feed_forward():
        if rng.random() < 0.5:
            return pick(None, 40, 64, 100)
        groups = pick(1, 2, 3, 4)
        each = pick(2, 3)
        keep = int(rng.integers(1, groups + 1))
        return pick(8, 16, 40, 64), groups * each, int(rng.integers(1, keep * each + 1)), float(rng.uniform(0.5, 2.5)), groups, keep
    layers = []
    for i in range(int(rng.integers(1, 6))):
        kind, ff, size = pick("attention", "lightning", "parallel"), feed_forward(), pick(1, 2, 7, 16, 63, 64, 65, 100, 128, 400)
        if kind == "lightning":
            n = pick(1, 2, 3, 5)
            layers.append(lin(n, pick(4, 6, 16, 33, 64, 100, 144), pick(2, 8, 16, 30, 64, 132),
                              tuple(float(d) for d in 1.0 - 2.0 ** -rng.uniform(0.5, 12, size=n)), ff=ff))
            continue
        h = heads()
        rot, scale = (pick(100.0, 1e4, 1e6), pick(h[2], h[2] // 2, 2, 0)), float(rng.uniform(0.5, 3.0)) / np.sqrt(h[2])
        if kind == "attention":
            layers.append(att(h, size, rot, ff=ff, scale=scale))
        else:
            blocks = pick(1, 2, 3, 4)
            layers.append(par(h, size, rot + ((pick(2.0, 8.0),) if rng.random() < 0.7 else ()),
                              (blocks * pick(5, 8, 16, 24, 40, 64, 136), blocks, pick(1, 2, 3, 4, 6)),
                              scales=(float(rng.uniform(0.3, 1.2)), float(rng.uniform(-1.0, 1.0))), ff=ff, scale=scale))
    n, loop = len(layers), None
    if rng.random() < 0.7:
        a = int(rng.integers(0, n))
        loop = (a, int(rng.integers(a + 1, n + 1)), pick(1, 2, 3))
    return config(pick(97, 128, 300), pick(48, 64, 72, 100, 128), pick(1, 2, 3, 4, 6), layers, loop=loop, eps=pick(1e-6, 1e-5, 1e-3))


@pytest.mark.parametrize("seed", range(20))
def test_configurations_drawn_from_seeds(tmp_path_factory, seed):
    cfg = drawn_configuration(seed)
    folder, plain = make_folder(tmp_path_factory, f"drawn{seed}", cfg, 500 + seed)
    rng = np.random.default_rng(seed)
    reqs = [[int(t) for t in rng.integers(0, cfg["vocab"], size=n)] for n in (150, 9, 71)]
    want = [P.forward(cfg, plain, r) for r in reqs]
    for dtype in DTYPES:
        eng = engine_for(folder, dtype, max_tokens=64 * 8)
        close(run_whole(eng, reqs[0]), want[0], dtype, f"seed {seed} whole")
        close(run_tail_one_by_one(eng, reqs[0], tail=40), want[0], dtype, f"seed {seed} tail one by one")
        for r, w, g in zip(reqs, want, run_batch(eng, reqs, [100, 3, 70])):
            close(g, w, dtype, f"seed {seed} batch, request of {len(r)}")
        assert eng.cache.held_pages() == 0 and not eng.cache.live_slots
        _ENGINES.clear()


# ---- mechanisms alone ---------------------------------------------------------------------------
def runtime(dtype, fast=True):
    from sonicboom_amd.parts import Runtime
    return Runtime(torch.device(DEV), TORCH_DT[dtype], fast)


def rand(*shape, scale=1.0, seed=0):
    g = torch.Generator().manual_seed(1000 * seed + sum(shape) + len(shape))
    return torch.randn(tuple(shape), generator=g) * scale


def i32(a):
    return torch.tensor(np.asarray(a), dtype=torch.int32, device=DEV)


def f64(t):
    return t.float().numpy().astype(np.float64)


def part_close(got, want, dtype, what, bf16=2.5e-2, f32=2e-5):
    got, want = got.detach().float().cpu().numpy().astype(np.float64), np.asarray(want, dtype=np.float64)
    scale = max(float(np.abs(want).max()), 1e-30)
    assert got.shape == want.shape, f"{what}: shape {got.shape} vs {want.shape}"
    err = np.abs(got - want).max() / scale
    assert err <= (f32 if dtype == "float32" else bf16), f"{what}: off by {err:.3g} of the largest value"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("streams, width", [(1, 64), (2, 96), (3, 2048), (4, 4096), (4, 1100), (4, 61), (6, 40), (5, 2050)])
@pytest.mark.parametrize("rows", [5, 130])
def test_a_sublayers_result_joins_streams_that_mix(dtype, streams, width, rows):
    """Whole results, K slices, experts' results with weights a row, several terms and a bias, from none to more parts than
    the kernel's registers hold; with and without what is read next."""
    from sonicboom_amd import ops
    S, act = streams, TORCH_DT[dtype]
    x, vec, w = rand(rows, S * width, scale=2.0), rand(width, seed=8).to(BF16), (1.0 + rand(width, scale=0.3, seed=9)).to(BF16)
    mix, out, read = rand(S, S, seed=3), rand(S, seed=4), rand(S, seed=5)
    whole, slices, pairs, pw = rand(rows, width), rand(5, rows, width, seed=1), rand(rows, 3, width, seed=2), rand(rows, 4, seed=6).abs()
    many = rand(9, rows, width, seed=7)
    dev = lambda t: t.to(DEV)
    cases = [[], [(whole, 1.0, False, None)], [(slices, 0.75, False, None), (whole, -0.5, False, None)], [(pairs, 1.0, True, pw[:, :3])],
             [(pairs, 1.0, True, pw[:, :3]), (whole, 1.0, False, pw[:, 3:])], [(many, 0.5, False, None), (slices, 2.0, False, None)],
             [(many, 0.5, False, None), (many, 0.25, False, None)]]
    X = f64(x).reshape(rows, S, width).transpose(1, 0, 2)
    for i, terms in enumerate(cases):
        y = np.zeros((rows, width))
        for part, scale, by_row, weights in terms:
            p = f64(part)
            p = p[None] if p.ndim == 2 else p.transpose(1, 0, 2) if by_row else p
            ws = np.ones((rows, p.shape[0])) if weights is None else f64(weights)
            y = y + scale * (p * ws.T[:, :, None]).sum(0)
        with_vec = i % 2 == 1
        y = y + f64(vec) if with_vec else y
        want = P.sublayer(X, np.zeros(S), f64(out), f64(mix), lambda u: y)
        nxt = P.rms_norm(np.tensordot(f64(read), want, axes=(0, 0)), f64(w), 1e-4)
        for follow in (True, False):
            cur = dev(x).clone()
            wide = dev(pw)
            on = [(dev(p), s, b, None if a is None else wide[:, :3] if a.shape[1] == 3 else wide[:, 3:]) for p, s, b, a in terms]
            h = ops.streams_join(cur, S, on, dev(mix), dev(out), vec=dev(vec) if with_vec else None, read=dev(read) if follow else None,
                                 weight=dev(w) if follow else None, eps=1e-4, act_dtype=act)
            part_close(cur.view(rows, S, width).permute(1, 0, 2), want, "float32", f"case {i}, the streams")
            assert (h is None) == (not follow)
            if follow:
                part_close(h, nxt, dtype, f"case {i}, what is read next", bf16=6e-3)
    part_close(ops.streams_read(dev(x), S, dev(read), dev(w), 1e-4, act), P.rms_norm(np.tensordot(f64(read), X, axes=(0, 0)), f64(w), 1e-4),
               dtype, "a read alone", bf16=6e-3)
    picked = [3, 0, 4]
    part_close(ops.streams_read(dev(x), S, None, dev(w), 1e-4, act, i32(picked)), P.rms_norm(X.sum(0)[picked], f64(w), 1e-4), dtype,
               "the sum of picked rows", bf16=6e-3)
    table = rand(11, width, seed=12).to(act)
    ids = [4, 10, 0, 4]
    e = ops.streams_embed(dev(table), i32(ids), S)
    assert torch.equal(e.cpu().view(4, S, width), table.float()[ids][:, None].expand(4, S, width))


def test_in_32_bit_a_rows_bits_do_not_depend_on_the_other_rows():
    from sonicboom_amd import ops
    S, width, rows = 4, 192, 100
    x, part, w = rand(rows, S * width).to(DEV), rand(2, rows, width, seed=1).to(DEV), rand(width, seed=2).to(DEV)
    mix, out, read = rand(S, S, seed=3).to(DEV), rand(S, seed=4).to(DEV), rand(S, seed=5).to(DEV)
    run = lambda a, p: (a, ops.streams_join(a, S, [(p, 1.0, False, None)], mix, out, read=read, weight=w, eps=1e-5))
    xa, ha = run(x.clone(), part)
    xb, hb = run(x[7:9].clone(), part[:, 7:9].contiguous())
    assert torch.equal(xa[7:9], xb) and torch.equal(ha[7:9], hb)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [3, 600])
@pytest.mark.parametrize("heads, kv_heads, dim, vdim, rot_dims", [(4, 2, 32, 16, 16), (3, 3, 10, 14, 6), (2, 1, 64, 32, 64), (5, 1, 24, 8, 0),
                                                                  (16, 4, 128, 128, 48), (1, 1, 256, 16, 32), (2, 2, 7, 3, 4)])
@pytest.mark.parametrize("slices", [1, 3])
def test_norms_over_a_whole_projection(dtype, rows, heads, kv_heads, dim, vdim, rot_dims, slices):
    """All of q and all of k normed (eps large enough to show, weights that differ from number to number), then turned by
    head, from rows that are wider than the mixer's own, whole or in K slices."""
    from sonicboom_amd import ops
    from sonicboom_amd.cache.layout import keys_in_order, values_in_order
    width, pages, eps, qw, kw = heads * dim + kv_heads * (dim + vdim), (rows + 63) // 64, 0.3, heads * dim, kv_heads * dim
    wide = rand(slices, rows, width + 24, scale=1.5)
    mine = f64(wide)[:, :, 8:8 + width].sum(0)
    act = TORCH_DT[dtype]
    wq, wk = (1.0 + rand(qw, scale=0.4, seed=1)).to(act), (1.0 + rand(kw, scale=0.4, seed=2)).to(act)
    kc = torch.zeros(pages, kv_heads, 64, dim, dtype=act, device=DEV)
    vc = torch.zeros(pages, kv_heads, vdim, 64, dtype=act, device=DEV)
    inv = None
    if rot_dims:
        inv = torch.tensor([50.0 ** (-2.0 * i / rot_dims) / 4.0 for i in range(rot_dims // 2)], dtype=F32, device=DEV)
    src = wide.to(DEV)[:, :, 8:8 + width]
    q = ops.rownorm_kv_store(src if slices > 1 else src[0], act, wq.to(DEV), wk.to(DEV), eps, i32(np.arange(rows)), i32(np.zeros(rows)), kc, vc,
                             i32(np.arange(pages)[None, ::-1].copy()), heads, kv_heads, dim, vdim, inv_freq=inv, rot_dims=rot_dims)
    rot = {"dims": rot_dims, "base": 50.0, "scaling": {"factor": 4.0}}
    pos = np.arange(rows)
    wantq = P.turn(P.rms_norm(mine[:, :qw], f64(wq), eps).reshape(rows, heads, dim), pos, rot)
    wantk = P.turn(P.rms_norm(mine[:, qw:qw + kw], f64(wk), eps).reshape(rows, kv_heads, dim), pos, rot)
    part_close(q.view(rows, heads, dim), wantq, dtype, "queries", bf16=6e-3, f32=1e-4)
    order = list(range(pages))[::-1]             # row r lies in page pages - 1 - r // 64
    keys = keys_in_order(kc.cpu())[order].permute(0, 2, 1, 3).reshape(pages * 64, kv_heads, dim)
    values = values_in_order(vc.cpu())[order].permute(0, 3, 1, 2).reshape(pages * 64, kv_heads, vdim)
    part_close(keys[:rows], wantk, dtype, "keys", bf16=6e-3, f32=1e-4)
    part_close(values[:rows], mine[:, qw + kw:].reshape(rows, kv_heads, vdim), dtype, "values", bf16=6e-3)
    assert not keys[rows:].any(), "nothing is written past the step's rows"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [64, 61, 1500, 4096, 6000, 8200])
@pytest.mark.parametrize("slices", [1, 4])
def test_a_row_norm_with_a_gate(dtype, width, slices):
    from sonicboom_amd import ops
    rows = 9
    o, g, w = rand(rows, width, scale=2.0), rand(slices, rows, width + 12, seed=1), (1.0 + rand(width, scale=0.3, seed=2)).to(BF16)
    gd = g.to(DEV)[:, :, 4:4 + width]
    y = ops.rownorm_gate(o.to(DEV), w.to(DEV), 0.2, gd if slices > 1 else gd[0], TORCH_DT[dtype])
    part_close(y, P.rms_norm(f64(o), f64(w), 0.2) * P.sigmoid(f64(g)[:, :, 4:4 + width].sum(0)), dtype, "gated row norm", bf16=6e-3)


def scan_context(lengths, slots, positions):
    cu = np.concatenate([[0], np.cumsum(lengths)])
    return SimpleNamespace(cu_rows=i32(cu), slots=i32(slots), n_seqs=len(lengths), n_rows=sum(lengths), max_new=max(lengths), shared={},
                           row_seq=i32(np.repeat(np.arange(len(lengths)), lengths)),
                           row_pos=i32(np.concatenate([np.arange(p, p + n) for n, p in zip(lengths, positions)])))


def runs_of(lengths, height):
    from sonicboom_amd.engine.step import row_runs
    return torch.from_numpy(row_runs(lengths, np.concatenate([[0], np.cumsum(lengths)]), height)).to(DEV)


@pytest.mark.parametrize("heads, D, E", [(2, 16, 16), (3, 10, 6), (1, 64, 64), (2, 33, 72), (2, 128, 128), (1, 144, 80), (1, 255, 256), (2, 4, 200)])
@pytest.mark.parametrize("turning", [False, True])
def test_scans_of_activated_inputs(heads, D, E, turning):
    """Unequal sequences on slots in any order whose states are not empty, as a walk and in chunks: what is read, as it is,
    and the states."""
    from sonicboom_amd import ops
    lengths, slots, positions = [150, 1, 64, 65, 7], [4, 0, 2, 5, 1], [0, 90, 13, 700, 64]
    n = sum(lengths)
    rows, state = rand(n, heads * (2 * D + E) + 4, seed=D + E), rand(6, heads, D, E, seed=7) * 0.5
    decay = torch.tensor([0.96875, 1.0, 0.0625][:heads])
    pos = np.concatenate([np.arange(p, p + m) for m, p in zip(lengths, positions)])
    rot = {"dims": D // 4 * 2 if turning else 0, "base": 100.0}
    act = P.silu(f64(rows))
    qn = P.turn(act[:, :heads * D].reshape(n, heads, D), pos, rot)
    kn = P.turn(act[:, heads * D:2 * heads * D].reshape(n, heads, D), pos, rot)
    vn = act[:, 2 * heads * D:heads * (2 * D + E)].reshape(n, heads, E)
    want, states, r0 = np.empty((n, heads, E)), f64(state).copy(), 0
    for m, s in zip(lengths, slots):
        for a in range(heads):
            for t in range(r0, r0 + m):
                states[s, a] = float(decay[a]) * states[s, a] + np.outer(kn[t, a], vn[t, a])
                want[t, a] = qn[t, a] @ states[s, a]
        r0 += m
    ctx, dev = scan_context(lengths, slots, positions), rows.to(DEV)
    inv = torch.tensor([100.0 ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)], dtype=F32, device=DEV) if rot["dims"] else None
    for chunked in (False, True):
        st = state.to(DEV).clone()
        q, k, v = dev[:, :heads * D], dev[:, heads * D:2 * heads * D], dev[:, 2 * heads * D:heads * (2 * D + E)]
        kw = dict(chunks=runs_of(lengths, ops.decay_chunk_rows(D)), angles=None if inv is None else ops.angle_table(ctx.row_pos, inv, n)) if chunked else {}
        got = ops.decay_scan(q, k, v, None, st, ctx, heads, D, E, 0.0, F32, decay=decay.to(DEV), act_in=True, inv_freq=inv, rot_dims=rot["dims"], **kw)
        for a in range(heads):          # (a head that keeps everything reads far larger numbers)
            part_close(got.view(n, heads, E)[:, a], want[:, a], "float32", f"{'chunks' if chunked else 'walk'}, head {a}", f32=1e-4)
        part_close(st, states, "float32", f"{'chunks' if chunked else 'walk'}, the states", f32=1e-4)
        assert torch.equal(st[3].cpu(), state[3]), "a slot that no sequence of the step has is left alone"


def lru_case(width, blocks, taps, seed=0):
    """(tensors by role, the recurrence written out over rows with a state and earlier inputs)."""
    m = width // blocks
    t = {"x_bias": rand(width, seed=seed + 1), "y_bias": rand(width, seed=seed + 2), "taps": rand(width, taps, scale=taps ** -0.5, seed=seed + 3),
         "taps_bias": rand(width, scale=0.3, seed=seed + 4), "ra": rand(blocks, m, m, scale=1.5 * m ** -0.5, seed=seed + 5).to(BF16),
         "ri": rand(blocks, m, m, scale=1.5 * m ** -0.5, seed=seed + 6).to(BF16), "ra_bias": rand(width, seed=seed + 7), "ri_bias": rand(width, seed=seed + 8)}
    lam = rand(width, scale=2.0, seed=seed + 9) - 3.0
    lam[0], lam[width // 2] = 30.0, -30.0           # a channel that forgets everything, one that keeps everything
    t["rate"] = (8.0 * torch.nn.functional.softplus(lam.double())).float()

    def reference(x, y, S, before):
        """x, y [n, width]; S [width]; before [taps - 1, width]: the inputs ahead of the rows.  (result, S, all inputs)"""
        inputs = np.concatenate([before, x + f64(t["x_bias"])])
        u = P.time_conv(inputs, f64(t["taps"]), f64(t["taps_bias"]))[len(before):]
        r = P.block_gates(u, f64(t["ra"]), f64(t["ra_bias"]).reshape(blocks, m))
        i = P.block_gates(u, f64(t["ri"]), f64(t["ri_bias"]).reshape(blocks, m))
        a = np.exp(-f64(t["rate"]) * r)
        out = np.empty_like(u)
        for k in range(len(u)):
            S = a[k] * S + np.sqrt(-np.expm1(-2.0 * f64(t["rate"]) * r[k])) * i[k] * u[k]
            out[k] = S
        return out * P.gelu_tanh(y + f64(t["y_bias"])), S, inputs
    return t, reference


@pytest.mark.parametrize("width, blocks, taps", [(64, 2, 4), (256, 2, 3), (48, 1, 2), (96, 12, 1), (40, 5, 6), (27, 1, 3), (512, 2, 4), (600, 2, 4), (36, 2, 5)])
@pytest.mark.parametrize("slices", [1, 3])
def test_the_gated_recurrence_in_its_forms(width, blocks, taps, slices):
    """Unequal sequences whose states and earlier inputs are not empty, some of them at their first positions: the walk, the
    chunked form, and a step of one row a sequence after it, against the recurrence written out; weights in both types."""
    from sonicboom_amd import ops
    t, reference = lru_case(width, blocks, taps)
    lengths, slots, positions = [150, 1, 64, 65, 2, 17], [4, 0, 2, 5, 1, 6], [0, 90, 13, 700, 1, 0]
    n, n2 = sum(lengths), len(lengths)
    rows, more = rand(slices, n, 2 * width + 8), rand(slices, n2, 2 * width + 8, seed=5)
    S0, ring0, befores = rand(8, width, seed=6) * 0.5, torch.zeros(8, taps, width), []
    for s, p in zip(slots, positions):
        if p == 0:
            S0[s] = 0.0
        have = min(p, taps - 1)
        b = torch.cat([torch.zeros(taps - 1 - have, width), rand(have, width, seed=7 + s)])
        befores.append(f64(b))
        for k in range(have):
            ring0[s, (p - 1 - k) % taps] = b[taps - 2 - k]
    ring0[3], S0[7] = 1.0, 2.0                 # slots that no sequence of the step has
    both = lambda a: (f64(a)[:, :, :width].sum(0), f64(a)[:, :, width + 4:2 * width + 4].sum(0))
    (y, x), (y2, x2) = both(rows), both(more)
    want, want2, states, r0 = [], [], {}, 0
    for i, (m, s) in enumerate(zip(lengths, slots)):
        out, S, inputs = reference(x[r0:r0 + m], y[r0:r0 + m], f64(S0)[s], befores[i])
        want.append(out)
        out2, S2, _ = reference(x2[i:i + 1], y2[i:i + 1], S, inputs[len(inputs) - (taps - 1):])
        want2.append(out2)
        states[s] = (S, S2)
        r0 += m
    ctx = scan_context(lengths, slots, positions)
    ctx2 = scan_context([1] * n2, slots, [p + m for p, m in zip(positions, lengths)])
    forms = [(F32, False), (BF16, False)] + ([(BF16, True)] if ops.gated_lru_chunked_ok(width // blocks, BF16) else [])
    for wt, chunked in forms:
        dev = {k: v.to(DEV).to(wt) if k in ("ra", "ri") else v.to(DEV) for k, v in t.items()}
        S, ring = S0.to(DEV).clone(), ring0.to(DEV).clone()

        def run(a, ctx, chunks):
            d = a.to(DEV)
            d = d if slices > 1 else d[0]
            return ops.gated_lru(d.narrow(-1, width + 4, width), d.narrow(-1, 0, width), dev["x_bias"], dev["y_bias"], dev["taps"], dev["taps_bias"],
                                 dev["ra"], dev["ri"], dev["ra_bias"], dev["ri_bias"], dev["rate"], S, ring, ctx, F32, chunks)
        what = f"{wt} {'chunked' if chunked else 'walk'}"
        part_close(run(rows, ctx, runs_of(lengths, ops.gated_lru_chunk_rows()) if chunked else None), np.concatenate(want), "float32", what, f32=5e-5)
        for s in slots:
            part_close(S[s], states[s][0], "float32", f"{what}, state of slot {s}", f32=5e-5)
        part_close(run(more, ctx2, None), np.concatenate(want2), "float32", f"{what}, the step after it", f32=5e-5)
        for s in slots:
            part_close(S[s], states[s][1], "float32", f"{what}, state of slot {s} after the step", f32=5e-5)
        assert torch.equal(ring[3].cpu(), ring0[3]) and torch.equal(S[7].cpu(), S0[7]) and torch.equal(S[3].cpu(), S0[3])


def test_the_gated_recurrence_gives_the_same_bits_however_the_rows_are_cut():
    from sonicboom_amd import ops
    width, blocks, taps, n = 72, 3, 4, 50
    t, _ = lru_case(width, blocks, taps)
    dev = {k: v.to(DEV) for k, v in t.items()}
    rows, outs = rand(n, 2 * width).to(DEV), {}
    for cuts in ([n], [1] * n, [7, 8, 9, 26], [2] * 25, [3, 1, 1, 45]):
        S, ring, got, at = torch.zeros(1, width, device=DEV), torch.zeros(1, taps, width, device=DEV), [], 0
        for m in cuts:
            d = rows[at:at + m]
            got.append(ops.gated_lru(d[:, width:], d[:, :width], dev["x_bias"], dev["y_bias"], dev["taps"], dev["taps_bias"], dev["ra"], dev["ri"],
                                     dev["ra_bias"], dev["ri_bias"], dev["rate"], S, ring, scan_context([m], [0], [at]), F32))
            at += m
        outs[str(cuts[:4])] = (torch.cat(got), S, ring)
    first = next(iter(outs.values()))
    for key, o in outs.items():
        assert all(torch.equal(a, b) for a, b in zip(o, first)), f"portions {key}"


@pytest.mark.parametrize("h_dtype", [F32, BF16])
@pytest.mark.parametrize("experts, top, groups, keep", [(10, 3, 2, 1), (6, 2, 3, 2), (64, 8, 8, 4), (200, 16, 1, 1), (12, 4, 12, 5), (130, 5, 65 // 13, 3), (4, 4, 2, 2)])
def test_the_router_by_corrected_scores(h_dtype, experts, top, groups, keep):
    from sonicboom_amd import ops
    width, rows = 96, 300
    h, w = rand(rows, width).to(h_dtype), rand(experts, width, scale=width ** -0.5, seed=1)
    corr = rand(experts, scale=0.3, seed=2) - 0.6          # choice scores on both sides of zero
    router = {"experts": experts, "top": top, "scale": 1.75, "groups": {"count": groups, "keep": keep}}
    ids, weights = ops.moe_router(h.to(DEV), w.to(DEV), experts, top, has_gate=False, score="sigmoid_corrected", score_scale=1.75,
                                  groups=groups, keep_groups=keep, correction=corr.to(DEV))
    scores = P.sigmoid(f64(h) @ f64(w).T)
    same = 0
    for r in range(rows):
        e, a = P.choose(scores[r], f64(corr), router)
        got = ids[r].cpu().numpy()
        if set(got.tolist()) == set(e.tolist()):
            same += 1
            order = np.argsort(got), np.argsort(e)
            assert np.allclose(weights[r, :top].cpu().numpy()[order[0]], a[order[1]], rtol=2e-5)
            assert np.all(np.diff((scores[r] + f64(corr))[got]) <= 1e-5), "in falling order of the choice scores"
    assert same >= rows - 2, "float32 scores may order a pair a hair apart otherwise, not more"
    # equal scores: the lower numbers win, of groups and of experts
    ids, weights = ops.moe_router(torch.zeros(2, width, device=DEV), w.to(DEV), experts, top, has_gate=False, score="sigmoid_corrected",
                                  groups=groups, keep_groups=keep, correction=torch.zeros(experts, device=DEV))
    assert ids[1].tolist() == list(range(top)) and np.allclose(weights[0, :top].cpu().numpy(), 1.0 / top)


def part_from(spec, weights, dtype, fast=True):
    """A part on the GPU from a dict of arrays by tensor name, and the arrays as the part sees them."""
    from sonicboom_amd.parts import build_part
    dev = {t.name: torch.from_numpy(np.asarray(weights[t.name])).float().to(TORCH_DT[dtype]).to(DEV) for t in spec.all_tensors()}
    ref = {k: v.float().cpu().numpy().astype(np.float64) for k, v in dev.items()}
    return build_part(spec, dev, runtime(dtype, fast)), ref


def layer_of(layer, width, weights, dtype, eps=1e-5, fast=True, what="mixer"):
    """The mixer (or feed-forward) of a layer of config.json as the model builds it."""
    from sonicboom_amd.config import architecture_of
    cfg = config(10, width, 2, [layer], eps=eps)
    spec = architecture_of(cfg).build_spec(architecture_of(cfg).config_class.from_dict(cfg))
    part, ref = part_from(spec.blocks[0].parts[what], weights, dtype, fast)
    if hasattr(part, "finish_build"):
        part.finish_build()
    return part, ref


def add_up(y, rows, width):
    """What a block would add up of a sublayer's result."""
    from sonicboom_amd.parts import Branch, Joined
    out = torch.zeros(rows, width, dtype=F32, device=DEV)
    for one in (y if isinstance(y, (list, tuple)) else [y]):
        if isinstance(one, Branch):
            out += (one.part * one.part_weights.unsqueeze(-1)).sum(1)
            continue
        one = one if isinstance(one, Joined) else Joined(one)
        out += one.scale * (one.part.sum(0) if one.part.dim() == 3 else one.part)
        if one.bias is not None:
            out += one.bias.float()
    return out


def mixer_harness(mixer, rt_dtype, width, n_tokens_cap=64 * 20):
    """A cache with the mixer's keys and states, and a function that feeds rows of one sequence in cuts and returns what
    the mixer hands over; the slot changes from call to call, its states are those of a fresh slot."""
    from sonicboom_amd.cache import PagedCache, group_entries
    from sonicboom_amd.engine.model import LayerBinding
    from sonicboom_amd.engine.step import StepContext, StepEntry
    cs, ss = mixer.cache_spec(), mixer.state_spec()
    named = ss if isinstance(ss, dict) else {} if ss is None else {"": ss}
    cache = PagedCache(group_entries({0: cs.key()} if cs is not None else {}), n_tokens_cap, TORCH_DT[rt_dtype], torch.device(DEV),
                       {k: (tuple(s.shape), s.dtype) for k, s in named.items()}, max_slots=4)
    t = getattr(mixer, "row_tile", None) or ()
    tiles = (t,) if isinstance(t, int) else tuple(t)

    def feed(h_rows, cuts):
        k, v, g = cache.entry_views(0) if cs is not None else (None, None, None)
        slot = cache.alloc_slot()
        outs, at = [], 0
        try:
            for n in cuts:
                cache.reserve([slot], [n])
                ctx = StepContext(cache, [StepEntry(slot, [0] * n, ())], torch.device(DEV), tiles)
                ctx.shared = {}
                binding = LayerBinding(0, g, k, v, True, cache.state.get(""), cache.state if isinstance(ss, dict) else None)
                outs.append(add_up(mixer.produce(h_rows[at:at + n].to(DEV).contiguous(), ctx, binding), n, width))
                cache.advance([slot], [n])
                at += n
        finally:
            cache.free_slot(slot)
        return torch.cat(outs)
    return feed


LAYERS = [
    att((6, 2, 32, 48), 90, (1e4, 16)), att((3, 3, 10, 14), 33, (77.0, 6)), att((10, 2, 64, 64), 64, (5e5, 64)), att((1, 1, 128, 128), 1, (1e4, 0)),
    lin(4, 48, 32, (0.75, 0.96875, 0.998, 1.0)), lin(1, 10, 14, (0.5,)), lin(2, 200, 132, (0.9375, 0.99)), lin(2, 128, 128, (0.9, 0.9995)),
    par((4, 4, 32, 32), 40, (5e3, 32, 4.0), (96, 3, 4)), par((3, 3, 10, 14), 67, (77.0, 6, 3.0), (42, 2, 5)),
    par((8, 2, 64, 64), 128, (1e4, 32, 8.0), (256, 2, 3), scales=(1.1, -0.4)), par((2, 1, 16, 48), 130, (1e4, 8), (272, 2, 2)),
    par((6, 1, 128, 128), 64, (1e6, 128, 2.0), (24, 1, 1)),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("i", range(len(LAYERS)))
def test_mixers_alone(dtype, i):
    """Every mixer whole, in portions, and token by token; what its positions and masks do to the result shows."""
    layer, width, n = LAYERS[i], 64, 200
    weights = random_weights(config(10, width, 2, [layer]), seed=40 + i)
    mixer, ref = layer_of(layer, width, weights, dtype)
    feed = mixer_harness(mixer, dtype, width)
    h = rand(n, width, seed=i).to(TORCH_DT[dtype])
    fn, m = P.MIXERS[layer["type"]], layer["mixer"]
    want = fn(m, 1e-5, ref, "l0.mix.", f64(h))
    for cuts in ([n], [70, 2, 60] + [1] * 68, [64, 65, 63, 8]):
        part_close(feed(h, cuts), want, dtype, f"cuts {cuts[:3]}")

    def moves(edited):
        return np.abs(fn(edited, 1e-5, ref, "l0.mix.", f64(h)) - want).max() > 0.02 * np.abs(want).max()
    if layer["type"] == "lightning":
        assert moves(dict(m, decay=[d * 0.9 for d in m["decay"]])), "the decays count"
        return
    a, put = (m, lambda x: x) if layer["type"] == "attention" else (m["left"], lambda x: dict(m, left=x))
    assert moves(put(dict(a, mask={"size": a["mask"]["size"] + 1}))), "the last key counts"
    if a["rot"]["dims"] and a["mask"]["size"] > 1:
        assert moves(put(dict(a, rot={"base": 1.0, "dims": 0}))), "positions count"


@pytest.mark.parametrize("heads, kv_heads, dim, vdim", [(4, 1, 32, 16), (6, 2, 64, 64), (16, 2, 128, 64), (5, 5, 16, 48)])
@pytest.mark.parametrize("chunk", [5, 64, 100, 300])
def test_matrix_core_attention_over_chunks_equals_the_plain_kernel(heads, kv_heads, dim, vdim, chunk):
    """bfloat16: a prompt, portions and single rows over several pages and chunks against the kernel of one wave per (row,
    head) (single rows share the pages a chunk touches out over blocks)."""
    n, width = 700, 64
    layer = att((heads, kv_heads, dim, vdim), chunk, (1e4, dim // 2))
    weights = random_weights(config(10, width, 2, [layer]), seed=3)
    h = rand(n, width).to(BF16)
    outs = {}
    for fast in (True, False):
        mixer, ref = layer_of(layer, width, weights, "bfloat16", fast=fast)
        feed = mixer_harness(mixer, "bfloat16", width)
        outs[fast] = [feed(h, cuts) for cuts in ([n], [560, 17, 3] + [1] * 120)]
    want = P.chunked_attention(layer["mixer"], 1e-5, ref, "l0.mix.", f64(h))
    for a, b in zip(outs[True], outs[False]):
        part_close(a, b.float().cpu().numpy(), "bfloat16", "matrix cores against the plain kernel", bf16=2e-2)
        part_close(a, want, "bfloat16", "matrix cores against the plain implementation")


def planted(layer, prefix, dim, heads, kv_heads, width, seed):
    """Weights of an attention whose key numbers 8.. read the input's numbers 8.. and whose query numbers 8.. the input's
    numbers dim + 8 .. (numbers below 8 may turn: they are zero)."""
    w = random_weights(config(10, width, 2, [layer]), seed=seed)
    for role, n in (("q", heads), ("k", kv_heads)):
        w[prefix + role][:] = 0.0
        if prefix + role + ".b" in w:
            w[prefix + role + ".b"][:] = 0.0
        for d in range(8, dim):
            for a in range(n):
                w[prefix + role][a * dim + d, d + (dim if role == "q" else 0)] = 1.0
    return w


@pytest.mark.parametrize("dtype, fast", [("float32", True), ("bfloat16", True), ("bfloat16", False)])
@pytest.mark.parametrize("kind, size", [("window", 1), ("window", 40), ("window", 64), ("window", 65), ("window", 321), ("chunk", 1), ("chunk", 48),
                                        ("chunk", 64), ("chunk", 100), ("chunk", 350)])
def test_one_key_stands_out_at_the_edges(dtype, fast, kind, size):
    """The last of 460 rows asks and one row answers: attention's weight falls on that key where it is just inside the window
    (or the chunk), at page borders and far back, and does not where it is just outside, as the last row of a prompt, as a
    single decoded row and behind a portion of two."""
    dim, width, n = 16, 48, 460
    t = n - 1
    if kind == "window":
        layer, prefix = par((2, 1, dim, dim), size, (1e4, 8), (8, 1, 2), scales=(1.0, 0.0), scale=0.5), "l0.mix.left."
        oldest = max(0, t - size + 1)
    else:
        layer, prefix = att((2, 1, dim, 32), size, (1e4, 8), scale=3.0), "l0.mix."
        oldest = t // size * size
    w = planted(layer, prefix, dim, 2, 1, width, 5)
    mixer, ref = layer_of(layer, width, w, dtype, fast=fast)
    feed = mixer_harness(mixer, dtype, width)
    fn = P.MIXERS[layer["type"]]
    shows = []
    places = sorted({p for p in (oldest, oldest + 1, oldest - 1, oldest - 2, t, t - 1, 0, 383, 384, 447, 448, (oldest + t) // 2) if 0 <= p <= t})
    for p in places:
        h = rand(n, width, seed=p) * 0.5
        h[:, :2 * dim] = 0.0
        h[:, 9], h[:, dim + 10] = 2.0, 2.0       # keys point along 9, queries ask for 10: nobody answers,
        h[p, 8], h[p, 9] = 2.0, 0.0              # but one key points along 8,
        h[t, dim + 8], h[t, dim + 10] = 2.0, 0.0     # which the last row asks for
        h = h.to(TORCH_DT[dtype])
        want = fn(layer["mixer"], 1e-5, ref, "l0.mix.", f64(h))
        for cuts in ([n], [n - 1, 1], [200, 196, 61, 2, 1]):
            part_close(feed(h, cuts)[t:], want[t:], dtype, f"key at {p}, cuts {cuts}")
        hidden = f64(h).copy()
        hidden[p, 8], hidden[p, 9] = 0.0, 2.0
        moved = np.abs(fn(layer["mixer"], 1e-5, ref, "l0.mix.", hidden)[t] - want[t]).max() > 0.1 * np.abs(want[t]).max()
        shows.append(moved)
        assert not moved or p >= oldest, "a key outside is seen"
    if oldest < t:
        assert all(s for s, p in zip(shows, places) if p >= oldest), "the planted key does not decide the result: the test shows nothing"


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_sink_takes_its_share_of_every_row(dtype):
    """Keys without scores: row t of a chunk gives its values the weight 1 / (k + exp(sink)) each, k the keys it sees,
    whatever the scale and however the rows are cut; a sink of one head does not move another's."""
    dim, width, n, chunk = 16, 32, 130, 50
    layer = att((3, 1, dim, 16), chunk, (1e4, 16), scale=7.0)
    w = random_weights(config(10, width, 2, [layer]), seed=6)
    for role in ("q", "k"):
        w["l0.mix." + role][:] = 0.0
        w["l0.mix." + role + ".b"][:] = 0.0
    w["l0.mix.v"][:] = 0.0
    w["l0.mix.v.b"][:] = 1.0
    w["l0.mix.o"] = np.eye(width, 48)
    w["l0.mix.o.b"][:] = 0.0
    w["l0.mix.sink"] = np.array([0.0, 3.0, -40.0])
    mixer, ref = layer_of(layer, width, w, dtype)
    feed = mixer_harness(mixer, dtype, width)
    seen = np.arange(n) % chunk + 1.0
    want = np.stack([seen / (seen + np.exp(s)) for s in (0.0, 3.0)], axis=1).repeat(16, axis=1)
    assert np.allclose(P.chunked_attention(layer["mixer"], 1e-5, ref, "l0.mix.", np.zeros((n, width))), want)
    h = rand(n, width).to(TORCH_DT[dtype])
    for cuts in ([n], [60, 2] + [1] * 68):
        part_close(feed(h, cuts), want, dtype, f"cuts {cuts[:2]}", bf16=6e-3)


FAR = [1, 2, 3, 31, 32, 33, 63, 64, 65, 127, 128, 129, 500, 699]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["lightning", "gated recurrence"])
def test_one_write_stands_out(dtype, kind):
    """One row of 700 writes into the state and the last row reads it, 1 to 699 rows later, at both sides of page and chunk
    borders: a state that is lost, moved on once too often or not at all shows."""
    n, width = 700, 48
    if kind == "lightning":
        layer = lin(2, 16, 16, (0.998, 0.9999))
        w = random_weights(config(10, width, 2, [layer]), seed=6)
        for role in ("k", "v"):
            w["l0.mix." + role][:, 20:] = 0.0                     # only the input's first numbers write
        w["l0.mix.q"][:, :20] = 0.0
        w["l0.mix.g"][:, :20] = 0.0
    else:
        layer = par((1, 1, 8, 8), 4, (1e4, 8), (64, 2, 4), scales=(0.0, 1.0))
        w = random_weights(config(10, width, 2, [layer]), seed=6)
        p = "l0.mix.right."
        w[p + "x"][:, 20:] = 0.0
        w[p + "y"][:, :20] = 0.0
        for role in ("x.b", "conv.b", "ra", "ra.b"):
            w[p + role][:] = 0.0
        w[p + "lam"] = np.linspace(-9.5, -8.5, 64)                # slow decays
    mixer, ref = layer_of(layer, width, w, dtype, eps=1e-9)
    feed = mixer_harness(mixer, dtype, width)
    fn = P.MIXERS[layer["type"]]
    t, shows = n - 1, 0
    for b in FAR:
        h = rand(n, width, seed=b)
        h[:, :20] = 0.0
        h[t - b, :20] = rand(20, seed=b + 1) * 3.0
        if kind == "lightning":
            h[0, :20] += rand(20, seed=b + 2) * 0.01              # (some state from the first row on: what is read is normed)
        h = h.to(TORCH_DT[dtype])
        want = fn(layer["mixer"], 1e-9, ref, "l0.mix.", f64(h))
        for cuts in ([n], [n - 1, 1], [300, 336, 61, 2, 1], [t - b, b + 1] if b < t else [1, t]):
            part_close(feed(h, cuts)[t:], want[t:], dtype, f"a write {b} back, cuts {cuts}", bf16=4e-2, f32=3e-4)
        hidden = f64(h).copy()
        hidden[t - b, :20] = 0.0
        shows += np.abs(fn(layer["mixer"], 1e-9, ref, "l0.mix.", hidden)[t] - want[t]).max() > 0.3 * np.abs(want[t]).max()
    assert shows == len(FAR), "the planted write does not decide the result: the test shows nothing"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 7, 150])
@pytest.mark.parametrize("ff", [80, 33, (32, 8, 3, 1.5, 4, 2), (24, 5, 2, 0.75, 1, 1), (20, 12, 1, 2.0, 4, 3), (64, 4, 4, 1.0, 2, 2)])
def test_feed_forwards_alone(dtype, rows, ff):
    width = 64
    layer = lin(1, 4, 4, (0.5,), ff=ff)
    w = random_weights(config(10, width, 2, [layer]), seed=9, coded=True)
    ffn, ref = layer_of(layer, width, w, dtype, what="ffn")
    h = rand(rows, width, seed=rows)
    h[:, -16:] = torch.where(h[:, -16:] < 0, -1.0, 1.0)           # what coded routers read
    h = h.to(TORCH_DT[dtype])
    got = add_up(ffn.produce(h.to(DEV), SimpleNamespace(shared={})), rows, width)
    part_close(got, P.feed_forward(layer["mlp"], ref, "l0.mlp.", f64(h)), dtype, "feed-forward", bf16=2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [3, 200])
def test_results_that_bring_a_bias(dtype, rows):
    """A feed-forward with biases and attention with an output bias in the blocks that take what sublayers hand over."""
    from sonicboom_amd.parts.block import parallel_block_spec, streams_block_spec
    from sonicboom_amd.parts.ffn import dense_ffn_spec
    from sonicboom_amd.parts.norm import rmsnorm_spec
    from sonicboom_amd.parts import Mixer, PartSpec, register_part

    @register_part("mixer", "toy hands over nothing")
    class Nothing(Mixer):
        def produce(self, h, ctx, binding):
            return torch.zeros(h.shape[0], h.shape[1], dtype=F32, device=DEV)
    width, inner = 64, 48
    ffn = dense_ffn_spec("up", "down", width, inner, "relu_sq", up_bias_name="up.b", down_bias_name="down.b")
    w = {"up": f64(rand(inner, width, scale=0.2)), "down": f64(rand(width, inner, scale=0.2, seed=1)), "up.b": f64(rand(inner, seed=2)),
         "down.b": f64(rand(width, seed=3)), "n1": f64(1 + rand(width, scale=0.2, seed=4)), "n2": f64(1 + rand(width, scale=0.2, seed=5))}
    x = rand(rows, width, scale=2.0, seed=6)
    relu_sq = lambda h, r: P.linear(np.maximum(P.linear(h, r["up"], r["up.b"]), 0.0) ** 2, r["down"], r["down.b"])
    block, ref = part_from(parallel_block_spec(rmsnorm_spec("n1", width, 1e-4), PartSpec("mixer", "toy hands over nothing"), None, ffn), w, dtype)
    got = x.to(DEV)
    block.forward(got, SimpleNamespace(trace=None), None)
    part_close(got, f64(x) + relu_sq(P.rms_norm(f64(x), ref["n1"], 1e-4), ref), dtype, "branches of one norm", bf16=1e-2)
    S = 3
    for q in (1, 2):
        w.update({f"{q}in": f64(rand(S, seed=10 + q)), f"{q}out": f64(rand(S, seed=12 + q)), f"{q}mix": f64(rand(S, S, seed=14 + q))})
    names = [{r: f"{q}{r}" for r in ("in", "out", "mix")} for q in (1, 2)]
    block, ref = part_from(streams_block_spec(S, rmsnorm_spec("n1", width, 1e-4), PartSpec("mixer", "toy hands over nothing"), names[0],
                                              rmsnorm_spec("n2", width, 1e-4), ffn, names[1]), w, dtype)
    x = rand(rows, S * width, scale=2.0, seed=7)
    got = x.to(DEV)
    assert block.forward(got, SimpleNamespace(trace=None), None) is None
    X = f64(x).reshape(rows, S, width).transpose(1, 0, 2)
    X = P.sublayer(X, ref["1in"], ref["1out"], ref["1mix"], lambda u: np.zeros((rows, width)))
    X = P.sublayer(X, ref["2in"], ref["2out"], ref["2mix"], lambda u: relu_sq(P.rms_norm(u, ref["n2"], 1e-4), ref))
    part_close(got.view(rows, S, width).permute(1, 0, 2), X, dtype, "streams that mix", bf16=1e-2)
