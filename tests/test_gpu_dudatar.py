"""The Dudatar design on the GPU against the plain implementation of tests/plain/dudatar_plain.py: every mechanism
alone (layer norm, the pass that joins branches, rotated head norms with a gate a head, the decaying scans as a walk and
in chunks, the decays' logarithms, both mixers, the junction), whole models of several shapes, prompts cut into portions,
token-by-token decoding, batches of unequal requests on a cache that is used again, one key and one write planted far
away and at both sides of page and chunk borders, long decoding through the recorded decode step, and greedy generation
through the Python entry point, the command line and the replay program."""
import json
import os
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import helpers
from helpers import run_batch, run_tail_one_by_one, run_whole
from plain import dudatar_plain as P
from test_dudatar_config import config, gla, random_weights, side

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
F32, BF16 = torch.float32, torch.bfloat16
DTYPES = ["float32", "bfloat16"]
TORCH_DT = {"float32": F32, "bfloat16": BF16}

# A: sizes in sixteens (the matrix-core attention and the products in bfloat16); a loop in the middle, two kv heads,
#    values wider than keys, partly rotated heads, a layer without a feed-forward.
# B: sizes that are no multiple of 8 or 16 (plain products, the plain attention kernel, scans of odd sizes), gla first, the
#    whole model in the loop, one head, nothing that turns on one side, no cap.
# C: no loop; one kv head, heads of more than 128 key channels, decays of 1 and of almost nothing, tau of 1.
CONFIGS = {
    "A": config(160, 96, [
        side((6, 2, 32, 48), (3, 32, 16, (0.75, 0.96875, 0.998)), ff=80, rot=(1e4, 16), rot_right=(1e5, 32)),
        gla(2, 32, 48, 8.0, ff=112),
        side((4, 4, 16, 32), (2, 16, 48, (0.9, 0.999)), rot_right=(1e4, 8)),
        gla(3, 16, 16, 2.0, ff=48),
    ], loop=(1, 3, 3), eps=3e-4, softcap=12.0),
    "B": config(131, 60, [
        gla(3, 10, 6, 16.0, ff=52),
        side((3, 3, 10, 14), (1, 6, 10, (0.984375,)), ff=36, rot=(77.0, 6), rot_right=(300.0, 0)),
        gla(1, 22, 30, 5.0),
        side((5, 1, 6, 10), (5, 14, 7, (0.5, 0.9, 0.97, 0.99, 0.9990234375)), rot=(300.0, 0), rot_right=(50.0, 14)),
    ], loop=(0, 4, 2), eps=1e-6),
    "C": config(200, 64, [
        side((4, 1, 64, 32), (2, 144, 80, (1.0, 0.0625)), ff=136, rot=(5e5, 32), rot_right=(1e6, 64)),
        gla(2, 80, 160, 1.0, ff=64),
        side((2, 1, 16, 16), (4, 16, 16, (0.25, 0.875, 0.9375, 0.99)), ff=72, rot=(1e3, 2)),
    ], eps=1e-5, softcap=30.0),
}
SEEDS = {"A": 31, "B": 32, "C": 33}
_FOLDERS, _PLAIN, _ENGINES, _WANT = {}, {}, {}, {}


def make_folder(tmp_path_factory, name, cfg, seed):
    from safetensors.torch import save_file
    folder = str(tmp_path_factory.mktemp(f"dudatar_{name}"))
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    tensors = {k: torch.from_numpy(v).float().to(BF16).contiguous() for k, v in random_weights(cfg, seed).items()}
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
BF16_WORST, BF16_RMS = 0.5, 0.046       # what the whole file measured (0.3535 and 0.0326) times 1.4
helpers.BF16_MAX["branches of one norm"], helpers.BF16_RMS["branches of one norm"] = BF16_WORST, BF16_RMS


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
        seen = helpers.BF16_SEEN.setdefault("branches of one norm", [0.0, 0.0])
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
def test_the_stream_after_every_layer_run_in_32_bit(folders, name):
    eng = engine_for(folders[name], "float32")
    tokens = prompts(name, [75], seed=11)[0]
    got = []
    eng.tracer = lambda what, x: got.append(x.detach().cpu().numpy().copy()) if ".after_" in what else None
    try:
        run_whole(eng, tokens)
    finally:
        eng.tracer = None
    want = []
    P.forward(CONFIGS[name], _PLAIN[name], tokens, want)
    assert len(got) == len(want)
    for i, (a, b) in enumerate(zip(got, want)):
        assert np.abs(a - b).max() <= 2e-5 * np.abs(b).max(), f"{name}: the stream after layer run {i}"


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
    """A step of more rows than the engine takes at once is cut inside sequences."""
    eng = engine_for(folders["A"], dtype, max_tokens=64 * 12, max_step_rows=100)
    reqs = prompts("A", [130, 7, 220], seed=5)
    got = run_batch(eng, reqs, [130, 7, 220])
    for r, g in zip(reqs, got):
        close(g, want_logits("A", r), dtype, f"portions, request of {len(r)}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C"])
def test_long_decoding_through_the_decode_loop(folders, name, dtype):
    """150 single-token steps of two sequences past page borders, kernel by kernel and then replayed
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
    out = subprocess.run(cmd, capture_output=True, text=True, timeout=300)
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
                             capture_output=True, text=True, timeout=300)
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
    heads as heads, sizes with and without factors of 8 and 16, partly rotated heads, scans of more than 128 key
    channels, a loop over any run of layers or none."""
    rng = np.random.default_rng(3000 + seed)
    pick = lambda *v: v[int(rng.integers(len(v)))]
    layers = []
    for i in range(int(rng.integers(1, 6))):
        ff = pick(None, 40, 64, 100, 136)
        if rng.random() < 0.4:
            layers.append(gla(pick(1, 2, 3, 5), pick(4, 6, 16, 24, 33, 64, 100, 144), pick(2, 8, 16, 30, 64, 72, 132),
                              pick(1.0, 2.0, 16.0), ff=ff))
            continue
        heads = pick(1, 2, 3, 4, 6, 8)
        dim, rdim, rheads = pick(8, 16, 24, 32, 40, 64, 128), pick(2, 8, 12, 32, 64, 96, 160), pick(1, 2, 3, 4)
        decay = tuple(float(d) for d in 1.0 - 2.0 ** -rng.uniform(0.5, 12, size=rheads))
        layers.append(side((heads, pick(*[g for g in (1, 2, 3, 4, 6, 8) if heads % g == 0]), dim, pick(8, 16, 24, 32, 48, 64)),
                           (rheads, rdim, pick(4, 16, 20, 64, 136), decay), ff=ff, rot=(pick(100.0, 1e4, 1e6), pick(dim, dim // 2, 2, 0)),
                           rot_right=(pick(100.0, 1e4, 1e6), pick(rdim, rdim // 4 * 2, 0)), scale=float(rng.uniform(0.5, 3.0)) / np.sqrt(dim)))
    n, loop = len(layers), None
    if rng.random() < 0.7:
        a = int(rng.integers(0, n))
        loop = (a, int(rng.integers(a + 1, n + 1)), pick(1, 2, 3))
    return config(pick(97, 128, 300, 512), pick(48, 64, 72, 100, 128, 192), layers, loop=loop, eps=pick(1e-6, 1e-5, 1e-3),
                  softcap=pick(0.0, 10.0, 25.0))


@pytest.mark.parametrize("seed", range(24))
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


def part_close(got, want, dtype, what, bf16=2.5e-2, f32=2e-5):
    got, want = got.detach().float().cpu().numpy().astype(np.float64), np.asarray(want, dtype=np.float64)
    scale = max(float(np.abs(want).max()), 1e-30)
    assert got.shape == want.shape, f"{what}: shape {got.shape} vs {want.shape}"
    err = np.abs(got - want).max() / scale
    assert err <= (f32 if dtype == "float32" else bf16), f"{what}: off by {err:.3g} of the largest value"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [96, 60, 35, 520, 4096, 4100, 8192])
@pytest.mark.parametrize("rows", [7, 300])
def test_layer_norm(dtype, width, rows):
    from sonicboom_amd import ops
    x = rand(rows, width, scale=3.0) + 7.0              # a mean of twice the deviation
    w = (1.0 + rand(width, seed=1)).to(TORCH_DT[dtype])
    y = ops.layernorm(x.to(DEV), w.to(DEV), 2e-3, TORCH_DT[dtype])
    part_close(y, P.layer_norm(x.numpy(), w.float().numpy(), 2e-3), dtype, "layer norm", bf16=5e-3)
    picked = torch.tensor([3, 0, 6], dtype=torch.int32)
    z = ops.layernorm(x.to(DEV), w.to(DEV), 2e-3, TORCH_DT[dtype], picked.to(DEV))
    part_close(z, P.layer_norm(x.numpy()[[3, 0, 6]], w.float().numpy(), 2e-3), dtype, "picked rows", bf16=5e-3)
    if dtype == "float32":
        assert torch.equal(z[0], y[3]), "in 32-bit a row's bits depend on the row alone"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [96, 61, 2048, 4096, 8192])
@pytest.mark.parametrize("rows", [5, 130])
@pytest.mark.parametrize("slices", [(1, 1, 1), (4, 3, 2), (8, 1, 5), (9, 2, 1), (8, 8, 4), (9, 9, 9), (2,), (1, 7), (12, 8), ()])
def test_branches_join_the_stream_in_one_pass(dtype, width, rows, slices):
    from sonicboom_amd import ops
    x, vec = rand(rows, width, scale=2.0), rand(width, seed=8).to(BF16)
    parts = [rand(s, rows, width, seed=10 + i) for i, s in enumerate(slices)]
    ws = [(1.0 + rand(width, scale=0.3, seed=20 + i)).to(BF16) if i < 2 else None for i in range(len(slices))]
    want = x.numpy().astype(np.float64) + vec.float().numpy()
    for i, p in enumerate(parts):
        s = p.numpy().astype(np.float64).sum(0)
        want = want + (0.5 * P.unit_rms(s, 1e-3) * ws[i].float().numpy() if ws[i] is not None else s)
    terms = [(p.to(DEV) if s > 1 else p[0].to(DEV).contiguous(), 0.5 if w is not None else 1.0, w is not None, None if w is None else w.to(DEV))
             for p, s, w in zip(parts, slices, ws)]
    hw = (1.0 + rand(width, seed=30)).to(BF16)
    for then, ref in (("layer", P.layer_norm(want, hw.float().numpy(), 1e-4)), ("rms", P.unit_rms(want, 1e-4) * hw.float().numpy()),
                      ("copy", want), (None, None)):
        base = x.to(DEV)
        out = torch.empty_like(base) if then == "copy" else base         # in place, or beside the base
        h = ops.join(out, base, terms, TORCH_DT[dtype], 1e-3, vec=vec.to(DEV), then=then, then_weight=hw.to(DEV) if then in ("layer", "rms") else None,
                     then_eps=1e-4, out_dtype=TORCH_DT[dtype])
        part_close(out, want, "float32", f"the sum, then {then}")
        if then is None:
            assert h is None
        else:
            part_close(h, ref, dtype, f"what follows: {then}", bf16=5e-3)


def scan_context(lengths, slots, positions):
    cu = np.concatenate([[0], np.cumsum(lengths)])
    t = lambda a: torch.tensor(np.asarray(a), dtype=torch.int32, device=DEV)
    return SimpleNamespace(cu_rows=t(cu), slots=t(slots), n_seqs=len(lengths), shared={},
                           row_pos=t(np.concatenate([np.arange(p, p + n) for n, p in zip(lengths, positions)])))


def runs_of(lengths, height):
    from sonicboom_amd.engine.step import row_runs
    return torch.from_numpy(row_runs(lengths, np.concatenate([[0], np.cumsum(lengths)]), height)).to(DEV)


@pytest.mark.parametrize("heads, D, E", [(2, 16, 16), (3, 10, 6), (1, 64, 64), (2, 33, 72), (2, 128, 128), (1, 100, 132), (1, 144, 80),
                                         (1, 255, 256), (2, 4, 200), (1, 256, 30), (1, 1, 1), (2, 48, 24)])
@pytest.mark.parametrize("channel", [False, True])
def test_decaying_scans_as_a_walk_and_in_chunks(heads, D, E, channel):
    """Unequal sequences on slots in any order whose states are not empty: both forms against the recurrence written
    out, results and states, with a decay a head (1, 0, and in between) and a decay a channel (from none to more than
    float32 can hold)."""
    from sonicboom_amd import ops
    lengths, slots, positions = [150, 1, 64, 65, 7], [4, 0, 2, 5, 1], [0, 90, 13, 700, 64]
    n, width = sum(lengths), 2 * heads * (D + E) + 3
    rows = rand(n, width, seed=D + E)
    decay = torch.tensor([1.0, 0.0, 0.96875][:heads] if heads > 1 else [0.99])
    ld = -torch.exp(rand(n, heads * D, scale=3.0, seed=5)) * 0.2
    ld[:, 0] = 0.0
    ld[n // 2, :] = -300.0
    w = 1.0 + rand(E, scale=0.3, seed=6)
    state = rand(6, heads, D, E, seed=7) * 0.5
    cut = lambda a, m: rows[:, a:a + heads * m]
    q, k, v, g = cut(0, D), cut(heads * D, D), cut(2 * heads * D, E), cut(2 * heads * D + heads * E, E)
    turn = D >= 4 and not channel
    rot = {"dims": D // 4 * 2, "base": 100.0}
    pos = np.concatenate([np.arange(p, p + m) for m, p in zip(lengths, positions)])
    qn, kn = q.numpy().astype(np.float64).reshape(n, heads, D), k.numpy().astype(np.float64).reshape(n, heads, D)
    if turn:
        qn, kn = P.turn(qn, pos, rot), P.turn(kn, pos, rot)
    qn, kn = qn * 0.75, kn * D ** -0.5
    vn = v.numpy().astype(np.float64).reshape(n, heads, E)
    want, states = np.empty((n, heads, E)), state.numpy().astype(np.float64).copy()
    al = np.exp(ld.numpy().astype(np.float64)).reshape(n, heads, D) if channel else np.broadcast_to(decay.numpy()[None, :, None].astype(np.float64), (n, heads, D))
    r0 = 0
    for m, s in zip(lengths, slots):
        for a in range(heads):
            S = states[s, a]
            for t in range(r0, r0 + m):
                S = al[t, a][:, None] * S + np.outer(kn[t, a], vn[t, a])
                want[t, a] = qn[t, a] @ S
            states[s, a] = S
        r0 += m
    want = (P.unit_rms(want, 1e-4) * (w.numpy() if channel else 1.0)).reshape(n, heads * E) * P.silu(g.numpy())
    ctx = scan_context(lengths, slots, positions)
    dev = rows.to(DEV)
    inv = torch.tensor([100.0 ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)], dtype=F32, device=DEV) if turn else None
    for chunked in (False, True):
        st = state.to(DEV).clone()
        parts = [dev[:, x:x + heads * m] for x, m in ((0, D), (heads * D, D), (2 * heads * D, E), (2 * heads * D + heads * E, E))]
        kw = dict(log_decay=ld.to(DEV), weight=w.to(DEV)) if channel else dict(decay=decay.to(DEV))
        if chunked:
            kw.update(chunks=runs_of(lengths, ops.decay_chunk_rows(D)), angles=ops.angle_table(ctx.row_pos, inv, n) if turn else None)
        got = ops.decay_scan(*parts, st, ctx, heads, D, E, 1e-4, F32, q_scale=0.75, k_scale=D ** -0.5, inv_freq=inv,
                             rot_dims=rot["dims"] if turn else 0, **kw)
        what = f"{'chunks' if chunked else 'walk'}"
        got = got.cpu().numpy().astype(np.float64)
        assert np.isfinite(got).all(), what
        # (a head that reads almost nothing is normed to order one: its rounding is that of what it cancels)
        err = np.abs(got - want).max() / np.abs(want).max()
        assert err <= (2e-3 if E == 1 else 2e-4), f"{what}: off by {err:.3g}"
        part_close(st, states, "float32", f"{what}, the states")
        assert torch.equal(st[3].cpu(), state[3]), "a slot that no sequence of the step has is left alone"


def test_the_walk_gives_the_same_bits_however_the_rows_are_cut():
    from sonicboom_amd import ops
    heads, D, E, n = 2, 40, 72, 50
    rows, st = rand(n, 2 * heads * (D + E)).to(DEV), {}
    ld = -torch.exp(rand(n, heads * D, seed=2)).to(DEV)
    outs = {}
    for cuts in ([n], [1] * n, [7, 8, 9, 26], [2] * 25):
        state, got, at = torch.zeros(1, heads, D, E, device=DEV), [], 0
        for m in cuts:
            part = rows[at:at + m]
            views = [part[:, x:x + heads * s] for x, s in ((0, D), (heads * D, D), (2 * heads * D, E), (2 * heads * D + heads * E, E))]
            got.append(ops.decay_scan(*views, state, scan_context([m], [0], [at]), heads, D, E, 1e-5, F32, log_decay=ld[at:at + m].contiguous()))
            at += m
        outs[len(cuts)] = (torch.cat(got), state)
    for key, (o, s) in outs.items():
        assert torch.equal(o, outs[1][0]) and torch.equal(s, outs[1][1]), f"{key} portions"


@pytest.mark.parametrize("rank, width, rows", [(16, 192, 40), (1, 30, 3), (7, 300, 9), (130, 64, 17)])
def test_logarithms_of_decays(rank, width, rows):
    from sonicboom_amd import ops
    a, w, b = rand(rows, rank + 5, scale=2.0), rand(rank, width), rand(width, scale=8.0, seed=1)
    got = ops.log_decay(a.to(DEV)[:, 2:2 + rank], w.to(DEV), b.to(DEV), 0.125)
    z = a.numpy()[:, 2:2 + rank].astype(np.float64) @ w.numpy().astype(np.float64) + b.numpy()
    want = np.where(z > 0, -np.log1p(np.exp(-np.abs(z))), z - np.log1p(np.exp(-np.abs(z)))) * 0.125
    assert np.allclose(got.cpu().numpy(), want, rtol=1e-5, atol=1e-6 * rank)
    if width % 2 == 0:          # the walk makes the same decays in its own kernel
        heads, D, E = 2, width // 2, 20
        x = rand(rows, 2 * heads * (D + E), seed=3).to(DEV)
        views = [x[:, c:c + heads * m] for c, m in ((0, D), (heads * D, D), (2 * heads * D, E), (2 * heads * D + heads * E, E))]
        outs = []
        for kw in (dict(log_decay=got), dict(decay_from=(a.to(DEV)[:, 2:2 + rank], w.to(DEV), b.to(DEV), 0.125))):
            state = torch.ones(1, heads, D, E, device=DEV)
            outs.append((ops.decay_scan(*views, state, scan_context([rows], [0], [0]), heads, D, E, 1e-5, F32, **kw), state))
        assert torch.equal(outs[0][0], outs[1][0]) and torch.equal(outs[0][1], outs[1][1])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [3, 600])
@pytest.mark.parametrize("heads, kv_heads, dim, vdim, rot_dims", [(4, 2, 32, 16, 16), (3, 3, 10, 14, 6), (2, 1, 64, 32, 64), (5, 1, 24, 8, 0),
                                                                  (2, 2, 128, 128, 48), (1, 1, 256, 16, 32)])
def test_rotated_head_norms(dtype, rows, heads, kv_heads, dim, vdim, rot_dims):
    """Queries and keys turned, then divided by their root mean square a head (eps large enough to show), from rows that
    are wider than the mixer's own."""
    from sonicboom_amd import ops
    from sonicboom_amd.cache.layout import keys_in_order, values_in_order
    width, pages, eps = heads * dim + kv_heads * (dim + vdim), (rows + 63) // 64, 0.3
    wide = rand(rows, width + 24, scale=1.5)
    mine = wide[:, 8:8 + width]
    kc = torch.zeros(pages, kv_heads, 64, dim, dtype=TORCH_DT[dtype], device=DEV)
    vc = torch.zeros(pages, kv_heads, vdim, 64, dtype=TORCH_DT[dtype], device=DEV)
    t = lambda a: torch.tensor(np.asarray(a), dtype=torch.int32, device=DEV)
    inv = None
    if rot_dims:
        inv = torch.tensor([50.0 ** (-2.0 * i / rot_dims) for i in range(rot_dims // 2)], dtype=F32, device=DEV)
    q = ops.headnorm_kv_store(wide.to(DEV)[:, 8:8 + width], TORCH_DT[dtype], None, None, eps, t(np.arange(rows)), t(np.zeros(rows)), kc, vc,
                              t(np.arange(pages)[None, ::-1].copy()), heads, kv_heads, dim, vdim, inv_freq=inv, rot_dims=rot_dims, unit=True)
    rot = {"dims": rot_dims, "base": 50.0}
    qk = mine[:, :(heads + kv_heads) * dim].numpy().reshape(rows, heads + kv_heads, dim)
    want = P.unit_rms(P.turn(qk, np.arange(rows), rot), eps)
    # (an angle is a float32 product: at position 600 it is right to 600 * 2^-24)
    part_close(q.view(rows, heads, dim), want[:, :heads], dtype, "queries", bf16=6e-3, f32=1e-4)
    order = list(range(pages))[::-1]             # row r lies in page pages - 1 - r // 64
    keys = keys_in_order(kc.cpu())[order].permute(0, 2, 1, 3).reshape(pages * 64, kv_heads, dim)
    values = values_in_order(vc.cpu())[order].permute(0, 3, 1, 2).reshape(pages * 64, kv_heads, vdim)
    part_close(keys[:rows], want[:, heads:], dtype, "keys", bf16=6e-3, f32=1e-4)
    part_close(values[:rows], mine[:, (heads + kv_heads) * dim:].numpy().reshape(rows, kv_heads, vdim), dtype, "values", bf16=6e-3)
    assert not keys[rows:].any(), "nothing is written past the step's rows"


def part_from(spec, weights, dtype, fast=True):
    """A part on the GPU from a dict of arrays by tensor name, and the arrays as the part sees them."""
    from sonicboom_amd.parts import build_part
    dev = {t.name: torch.from_numpy(np.asarray(weights[t.name])).float().to(TORCH_DT[dtype]).to(DEV) for t in spec.all_tensors()}
    ref = {k: v.float().cpu().numpy().astype(np.float64) for k, v in dev.items()}
    return build_part(spec, dev, runtime(dtype, fast)), ref


def mixer_of(layer, width, weights, dtype, eps=1e-5, fast=True):
    """The mixer of a layer of config.json as the model builds it."""
    from sonicboom_amd.config import architecture_of
    cfg = config(10, width, [layer], eps=eps)
    spec = architecture_of(cfg).build_spec(architecture_of(cfg).config_class.from_dict(cfg))
    part, ref = part_from(spec.blocks[0].parts["mixer"], weights, dtype, fast)
    if hasattr(part, "finish_build"):
        part.finish_build()
    return part, ref


def mixer_harness(mixer, rt_dtype, width, n_tokens_cap=64 * 20):
    """A cache with the mixer's keys and states, and a function that feeds rows of one sequence in cuts and returns what
    the mixer adds into an empty stream; the slot changes from call to call, its states are those of a fresh slot."""
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
                x = torch.zeros(n, width, dtype=F32, device=DEV)
                binding = LayerBinding(0, g, k, v, True, cache.state.get(""), cache.state if isinstance(ss, dict) else None)
                mixer.forward(h_rows[at:at + n].to(DEV).contiguous(), x, ctx, binding)
                outs.append(x)
                cache.advance([slot], [n])
                at += n
        finally:
            cache.free_slot(slot)
        return torch.cat(outs)
    return feed


SIDES = [
    side((4, 2, 32, 16), (3, 32, 16, (0.75, 0.96875, 0.998)), rot=(1e4, 16), rot_right=(1e5, 32)),
    side((3, 3, 10, 14), (1, 6, 10, (0.984375,)), rot=(77.0, 6), rot_right=(300.0, 0)),
    side((5, 1, 16, 64), (2, 144, 72, (0.5, 0.999)), rot=(1e4, 0), rot_right=(1e4, 64)),
    side((8, 1, 64, 48), (1, 64, 128, (0.99,)), rot=(5e5, 64), rot_right=(1e4, 16)),
    side((1, 1, 128, 128), (4, 128, 32, (1.0, 0.9, 0.25, 0.997)), rot=(1e6, 32), rot_right=(1e6, 128)),
]
GLAS = [gla(4, 48, 32, 16.0), gla(1, 10, 14, 1.0), gla(3, 24, 72, 3.0), gla(2, 128, 128, 16.0), gla(1, 200, 256, 8.0), gla(5, 16, 8, 2.0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("i", range(len(SIDES) + len(GLAS)))
def test_mixers_alone(dtype, i):
    """Both mixers whole, in portions, and token by token; what each mechanism does to the result shows."""
    layer, width, n = (SIDES + GLAS)[i], 64, 200
    weights = random_weights(config(10, width, [layer]), seed=40 + i, rank=(9, 300)[i % 2])
    mixer, ref = mixer_of(layer, width, weights, dtype)
    feed = mixer_harness(mixer, dtype, width)
    h = rand(n, width, seed=i).to(TORCH_DT[dtype])
    hn = h.float().numpy()
    fn = P.side_by_side if layer["type"] == "parallel" else P.gated_linear_attention
    want = fn(layer["mixer"], 1e-5, ref, "l0.mix.", hn)
    for cuts in ([n], [70, 2, 60] + [1] * 68, [64, 65, 63, 8]):
        part_close(feed(h, cuts), want, dtype, f"cuts {cuts[:3]}")
    m = layer["mixer"]
    if layer["type"] == "parallel":
        for name in ("left", "right"):
            if m[name]["rot"]["dims"]:
                still = dict(m, **{name: dict(m[name], rot=dict(m[name]["rot"], dims=0))})
                assert np.abs(fn(still, 1e-5, ref, "l0.mix.", hn) - want).max() > 0.02 * np.abs(want).max(), f"{name}: positions count"
    else:
        slow = dict(m, tau=m["tau"] * 2)
        assert np.abs(fn(slow, 1e-5, ref, "l0.mix.", hn) - want).max() > 0.02 * np.abs(want).max(), "the decays count"


@pytest.mark.parametrize("heads, kv_heads, dim, vdim", [(4, 1, 32, 16), (6, 2, 64, 64), (16, 2, 128, 64), (5, 5, 16, 48)])
def test_matrix_core_attention_equals_the_plain_kernel(heads, kv_heads, dim, vdim):
    """bfloat16: a prompt, portions and single rows over several pages (the pages of a step of few rows are shared out
    over blocks and merged, the gate applied once) against the kernel of one wave per (row, head)."""
    n, width = 700, 64
    layer = side((heads, kv_heads, dim, vdim), (1, 8, 8, (0.9,)), rot=(1e4, dim // 2))
    weights = random_weights(config(10, width, [layer]), seed=3)
    h = rand(n, width).to(BF16)
    outs = {}
    for fast in (True, False):
        mixer, ref = mixer_of(layer, width, weights, "bfloat16", fast=fast)
        feed = mixer_harness(mixer, "bfloat16", width)
        outs[fast] = [feed(h, cuts) for cuts in ([n], [560, 17, 3] + [1] * 120)]
    want = P.side_by_side(layer["mixer"], 1e-5, ref, "l0.mix.", h.float().numpy())
    for a, b in zip(outs[True], outs[False]):
        part_close(a, b.float().cpu().numpy(), "bfloat16", "matrix cores against the plain kernel", bf16=2e-2)
        part_close(a, want, "bfloat16", "matrix cores against the plain implementation")


FAR = [1, 2, 31, 32, 33, 63, 64, 65, 127, 128, 129, 500, 636, 699]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("fast", [True, False])
def test_one_key_stands_out(dtype, fast):
    """A prompt of 700 rows in which the last row asks and one row answers: attention's weight falls on that key however
    far back it lies, at both sides of page borders and at the very first row, as the last row of a prompt, as a single
    decoded row and behind a portion of two.  Every other key points elsewhere with the same length (keys are normed), and
    the side of the retention is switched off by its norm's weight."""
    if fast and dtype == "float32":
        pytest.skip("the 32-bit path has one attention kernel")
    dim, vdim, width, n = 16, 16, 48, 700
    layer = side((2, 1, dim, vdim), (1, 8, 8, (0.9,)), rot=(1e4, 8), scale=0.9)
    w = random_weights(config(10, width, [layer]), seed=5)
    z = {k: np.zeros_like(v) for k, v in w.items() if k.startswith("l0.mix.left.") and k.rsplit(".", 1)[1] in ("q", "k")}
    w.update(z)
    for d in range(8, dim):
        w["l0.mix.left.k"][d, d] = 1.0                           # key numbers 8.. read the input's numbers 8..
        for a in range(2):
            w["l0.mix.left.q"][a * dim + d, dim + d] = 1.0       # query numbers 8.. the input's numbers dim + 8 ..
    w["l0.mix.right.out"][:] = 0.0
    mixer, ref = mixer_of(layer, width, w, dtype, fast=fast)
    feed = mixer_harness(mixer, dtype, width)
    t, shows = n - 1, 0
    for b in FAR:
        h = rand(n, width, seed=b) * 0.5
        h[:, :2 * dim] = 0.0
        h[:, 9], h[:, dim + 10] = 2.0, 2.0       # keys point along 9, queries ask for 10: nobody answers,
        h[t - b, 8], h[t - b, 9] = 2.0, 0.0      # but one key points along 8,
        h[t, dim + 8], h[t, dim + 10] = 2.0, 0.0     # which the last row asks for
        h = h.to(TORCH_DT[dtype])
        hn = h.float().numpy()
        want = P.side_by_side(layer["mixer"], 1e-5, ref, "l0.mix.", hn)
        for cuts in ([n], [n - 1, 1], [300, 336, 61, 2, 1]):
            part_close(feed(h, cuts)[t:], want[t:], dtype, f"key {b} back, cuts {cuts}")
        hidden = hn.copy()
        hidden[t - b, 8], hidden[t - b, 9] = 0.0, 2.0
        other = P.side_by_side(layer["mixer"], 1e-5, ref, "l0.mix.", hidden)
        shows += np.abs(other[t] - want[t]).max() > 0.3 * np.abs(want[t]).max()
    assert shows == len(FAR), "the planted key does not decide the result: the test shows nothing"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["retention", "gla", "wide gla"])
def test_one_write_stands_out(dtype, kind):
    """One row of 700 writes into the state and the last row reads it, 1 to 699 rows later, at both sides of page and
    chunk borders: the norm after the read-out brings even a faded write to order one, so a state that is lost, moved on
    once too often or not at all shows.  (What is left of a write after hundreds of decays is a sum over channels that
    partly cancels, and the norm enlarges its rounding with it.)"""
    n, width = 700, 48
    if kind == "retention":
        layer = side((1, 1, 8, 8), (2, 16, 16, (0.998, 0.9999)), rot_right=(1e4, 8))
        q, out = "l0.mix.right.", "l0.mix.left.out"
    else:
        layer = gla(2, 16, 16, 16.0) if kind == "gla" else gla(1, 160, 24, 16.0)
        q, out = "l0.mix.", None
    w = random_weights(config(10, width, [layer]), seed=6, rank=5)
    if out:
        w[out][:] = 0.0
    else:
        w[q + "a2.b"] = np.abs(w[q + "a2.b"]) + 3.0              # slow decays
    for role in ("k", "v"):
        w[q + role][:, 20:] = 0.0                                 # only the input's first numbers write
    w[q + "q"][:, :20] = 0.0
    mixer, ref = mixer_of(layer, width, w, dtype, eps=1e-9)
    feed = mixer_harness(mixer, dtype, width)
    fn = P.side_by_side if out else P.gated_linear_attention
    t, shows = n - 1, 0
    for b in FAR:
        h = rand(n, width, seed=b)
        h[:, :20] = 0.0
        h[t - b, :20] = rand(20, seed=b + 1) * 3.0
        h[0, :20] += rand(20, seed=b + 2) * 0.01                  # (some state from the first row on)
        h = h.to(TORCH_DT[dtype])
        hn = h.float().numpy()
        want = fn(layer["mixer"], 1e-9, ref, "l0.mix.", hn)
        for cuts in ([n], [n - 1, 1], [300, 336, 61, 2, 1], [t - b, b + 1] if b < t else [1, t]):
            part_close(feed(h, cuts)[t:], want[t:], dtype, f"a write {b} back, cuts {cuts}", bf16=4e-2, f32=3e-4)
        hidden = hn.copy()
        hidden[t - b, :20] = 0.0
        other = fn(layer["mixer"], 1e-9, ref, "l0.mix.", hidden)
        shows += np.abs(other[t] - want[t]).max() > 0.3 * np.abs(want[t]).max()
    assert shows == len(FAR), "the planted write does not decide the result: the test shows nothing"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 5, 80, 300])
@pytest.mark.parametrize("width", [64, 60, 35])
def test_the_junction(dtype, rows, width):
    """x <- W [x; x0] + step[turn], turn by turn, with and without the norm that follows in the same pass."""
    from sonicboom_amd.parts import build_part
    from sonicboom_amd.parts.junction import mix_embedding_spec
    from sonicboom_amd.parts.norm import layernorm_spec
    w = random_weights(config(10, width, [gla(1, 4, 4, 1.0)], loop=(0, 1, 3)), seed=8)
    junction, ref = part_from(mix_embedding_spec("loop.in", "loop.step", width, 3), w, dtype)
    norm, nref = part_from(layernorm_spec("l0.norm1", width, 1e-4), w, dtype)
    x0, x = rand(rows, width, scale=2.0), rand(rows, width, scale=3.0, seed=1)
    ctx = SimpleNamespace(shared={})
    h0 = junction.begin(x0.to(DEV), ctx)
    part_close(h0, x0.numpy(), dtype, "the embedding in the activation type", bf16=5e-3)
    cur, want = x.to(DEV), x.numpy().astype(np.float64)
    for turn in (0, 2, 1):
        h = junction.forward(cur, ctx, turn, next_norm=norm if turn != 2 else None)
        want = P.begin_pass(ref, want, x0.numpy().astype(np.float64), turn)
        part_close(cur, want, dtype, f"turn {turn}", bf16=2e-2)
        assert (h is None) == (turn == 2)
        if h is not None:
            part_close(h, P.layer_norm(want, nref["l0.norm1"], 1e-4), dtype, "the norm that follows", bf16=4e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_block_whose_branches_do_not_hand_their_results_over(dtype):
    """Sublayers that add into the stream themselves, in a block of one norm: both still read the norm of the stream before
    either result has joined it."""
    from sonicboom_amd.parts import PartSpec, build_part, register_part
    from sonicboom_amd.parts.base import Mixer, Part
    from sonicboom_amd.parts.block import parallel_block_spec
    from sonicboom_amd.parts.norm import layernorm_spec

    @register_part("mixer", "toy adds three times its input")
    class ToyMixer(Mixer):
        def forward(self, h, x, ctx, binding):
            x += 3.0 * h.float()

    @register_part("ffn", "toy adds half its input")
    class ToyFFN(Part):
        def forward(self, h, x, ctx):
            x += 0.5 * h.float()
    w = {"n": 1.0 + rand(40, scale=0.2).numpy()}
    spec = parallel_block_spec(layernorm_spec("n", 40, 1e-4), PartSpec("mixer", "toy adds three times its input"), None,
                               PartSpec("ffn", "toy adds half its input"))
    block, ref = part_from(spec, w, dtype)
    x = rand(9, 40, seed=2)
    got = x.to(DEV)
    block.forward(got, SimpleNamespace(trace=None), None)
    part_close(got, x.numpy() + 3.5 * P.layer_norm(x.numpy(), ref["n"], 1e-4), dtype, "the block", bf16=1e-2)


@pytest.mark.parametrize("slices", [1, 3, 9])
def test_a_products_slices_are_added_where_they_are_read(slices):
    """The rows of the stacked product in K slices, handed to the storing kernel and to the walk, give the bits of the rows
    added up before."""
    from sonicboom_amd import ops
    heads, kv, dim, vdim, rows = 4, 2, 32, 16, 9
    width = heads * dim + kv * (dim + vdim) + heads
    parts = rand(slices, rows, width + 12).to(DEV)
    whole = parts[0].clone()
    for s in range(1, slices):
        whole += parts[s]
    t = lambda a: torch.tensor(np.asarray(a), dtype=torch.int32, device=DEV)
    outs = []
    for src in (parts[..., 4:4 + width], whole[:, 4:4 + width]):
        kc, vc = torch.zeros(1, kv, 64, dim, device=DEV), torch.zeros(1, kv, vdim, 64, device=DEV)
        inv = torch.tensor([0.5 ** i for i in range(8)], device=DEV)
        q, gate = ops.headnorm_kv_store(src, F32, None, None, 1e-3, t(np.arange(rows)), t(np.zeros(rows)), kc, vc, t([[0]]), heads, kv, dim, vdim,
                                        inv_freq=inv, rot_dims=16, unit=True, gate_n=heads)
        outs.append((q, gate, kc, vc))
    assert all(torch.equal(a, b) for a, b in zip(*outs))
    assert torch.equal(outs[0][1], whole[:, 4 + width - heads:4 + width])
    H, D, E, rank = 2, 20, 36, 5
    parts = rand(slices, rows, 2 * H * (D + E) + rank + 3, seed=2).to(DEV)
    whole = parts[0].clone()
    for s in range(1, slices):
        whole += parts[s]
    up, bias = rand(rank, H * D).to(DEV), rand(H * D, seed=1).to(DEV)
    outs = []
    for src in (parts[..., 3:], whole[:, 3:]):
        cut = [src[..., c:c + n] for c, n in ((0, H * D), (H * D, H * D), (2 * H * D, H * E), (2 * H * D + H * E, H * E), (2 * H * (D + E), rank))]
        state = torch.zeros(1, H, D, E, device=DEV)
        outs.append((ops.decay_scan(*cut[:4], state, scan_context([rows], [0], [5]), H, D, E, 1e-5, F32, decay_from=(cut[4], up, bias, 0.25)), state))
    assert torch.equal(outs[0][0], outs[1][0]) and torch.equal(outs[0][1], outs[1][1])
