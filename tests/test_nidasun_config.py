"""The Nidasun configuration, its model spec, the cache of a mixer that sees chunks of keys, and the plain implementation,
without a GPU."""
import copy

import numpy as np
import pytest

from plain import nidasun_plain as P


def mlp_of(ff):
    """None, the inner size of a dense feed-forward, or (ff, experts, top, scale, groups, keep)."""
    if ff is None:
        return None
    if isinstance(ff, int):
        return {"kind": "dense", "ff": ff}
    ff, experts, top, scale, groups, keep = ff
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "scale": scale, "groups": {"count": groups, "keep": keep}}}


def attention(heads, size, rot, scale):
    H, G, D, E = heads
    r = {"base": rot[0], "dims": rot[1]}
    if len(rot) > 2:
        r["scaling"] = {"factor": rot[2]}
    return {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": scale if scale is not None else 2.5 / D ** 0.5,
            "mask": {"size": size}, "rot": r}


def att(heads, chunk, rot, ff=None, scale=None):
    return {"type": "attention", "mixer": attention(heads, chunk, rot, scale), "mlp": mlp_of(ff)}


def lin(heads, dim, vdim, decay, ff=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}, "mlp": mlp_of(ff)}


def par(left, window, rot, right, scales=(0.75, 0.625), ff=None, scale=None):
    """``right``: (width, blocks, taps)."""
    return {"type": "parallel", "mlp": mlp_of(ff), "mixer": {
        "left": attention(left, window, rot, scale), "left_scale": scales[0], "right_scale": scales[1],
        "right": dict(zip(("width", "blocks", "conv"), right))}}


def config(vocab, width, streams, layers, loop=None, eps=1e-5):
    d = {"architecture": "Nidasun", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


CFG = config(50, 24, 3, [
    lin(2, 6, 10, (0.5, 0.96875), ff=20),
    par((4, 2, 6, 10), 5, (500.0, 4, 4.0), (12, 3, 4), ff=(14, 6, 2, 1.25, 3, 2)),
    att((3, 3, 8, 4), 7, (1e4, 8), ff=18),
    par((2, 1, 8, 4), 9, (1e4, 0), (10, 1, 2), scales=(1.0, -0.5)),
], loop=(1, 3, 3), eps=2e-5)

# numbers no two pairs of which have the same sum
APART = np.array([0, 1, 3, 7, 12, 20, 30, 44, 65, 80, 96, 122])


def random_weights(cfg, seed=0, coded=False):
    """Weights by the file's names for a config.json dict, drawn here (not by the package): projections of unit outputs
    for unit inputs, norm weights, stream numbers and biases that are not near what would hide them.

    ``coded``: routers whose choice does not hang on a close call (bfloat16 rounds what a router reads, and two scores a
    hair apart would be ordered differently).  As many channels of the embedding as there are experts hold +1 or -1, no
    sublayer writes to them, and expert e reads channel e alone: all scores of a token are one of two numbers, and the
    corrections, no two pairs of which add up to the same, order those that are equal."""
    rng = np.random.default_rng(seed)
    d, S, w = cfg["width"], cfg["streams"], {}
    codes = max([lay["mlp"]["router"]["experts"] for lay in cfg["layers"] if lay["mlp"] and lay["mlp"]["kind"] == "moe"], default=0)
    codes = codes if coded else 0

    def mat(name, n_out, n_in, times=1.0):
        w[name] = rng.normal(0, times / np.sqrt(n_in), (n_out, n_in))

    def into(name, n_in, times=1.0):          # a matrix that writes into the stream
        mat(name, d, n_in, times)
        if codes:
            w[name][-codes:] = 0.0

    def vec(name, n, mean=1.0, spread=0.25):
        w[name] = rng.normal(mean, spread, n)

    def plus_minus(*shape):
        return np.where(rng.random(shape) < 0.5, -1.0, 1.0)
    w["embed"] = rng.normal(0.1, 1.0, (cfg["vocab"], d))
    if codes:
        w["embed"][:, -codes:] = plus_minus(cfg["vocab"], codes)
    mat("head", cfg["vocab"], d, 2.0)
    vec("final.norm", d)
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        vec(p + "norm1", d)
        for q in (1, 2) if f else (1,):
            w[f"{p}hc{q}.in"] = np.abs(rng.normal(1.0, 0.3, S)) / S
            w[f"{p}hc{q}.out"] = rng.normal(0.7, 0.3, S)
            w[f"{p}hc{q}.mix"] = 0.7 * np.eye(S) + np.abs(rng.normal(0.0, 0.3, (S, S))) / S
        mp = p + "mix."
        if layer["type"] == "lightning":
            for role, n in (("q", m["heads"] * m["dim"]), ("k", m["heads"] * m["dim"]), ("v", m["heads"] * m["vdim"]),
                            ("g", m["heads"] * m["vdim"])):
                mat(mp + role, n, d)
            vec(mp + "norm", m["heads"] * m["vdim"])
            into(mp + "o", m["heads"] * m["vdim"])
        else:
            a, ap = (m, mp) if layer["type"] == "attention" else (m["left"], mp + "left.")
            sizes = {"q": a["heads"] * a["dim"], "k": a["kv_heads"] * a["dim"], "v": a["kv_heads"] * a["vdim"]}
            for role, n in sizes.items():
                mat(ap + role, n, d)
                if layer["type"] == "attention":
                    vec(ap + role + ".b", n, 0.0, 0.5)
            into(ap + "o", a["heads"] * a["vdim"])
            if layer["type"] == "attention":
                vec(ap + "o.b", d, 0.0, 0.5)
                if codes:
                    w[ap + "o.b"][-codes:] = 0.0
                vec(ap + "sink", a["heads"], 1.0, 1.5)
            else:
                vec(ap + "q.norm", sizes["q"]), vec(ap + "k.norm", sizes["k"])
                r, rp = m["right"], mp + "right."
                n, b = r["width"], r["width"] // r["blocks"]
                for role in ("y", "x"):
                    mat(rp + role, n, d)
                    vec(rp + role + ".b", n, 0.0, 0.5)
                mat(rp + "conv", n, r["conv"])
                vec(rp + "conv.b", n, 0.0, 0.3)
                for role in ("ra", "ri"):
                    w[rp + role] = rng.normal(0, 1.5 / np.sqrt(b), (r["blocks"], b, b))
                    w[rp + role + ".b"] = rng.normal(0, 0.5, (r["blocks"], b))
                vec(rp + "lam", n, -3.0, 2.0)
                into(rp + "o", n)
        if f:
            vec(p + "norm2", d)
            if f["kind"] == "dense":
                mat(p + "mlp.up", f["ff"], d), into(p + "mlp.down", f["ff"])
            else:
                n = f["router"]["experts"]
                for e in range(n):
                    q = f"{p}mlp.e{e}."
                    mat(q + "gate", f["expert"]["ff"], d, 1.5), mat(q + "up", f["expert"]["ff"], d), into(q + "down", f["expert"]["ff"])
                if codes:
                    w[p + "norm2"][-codes:] = 1.0
                    w[p + "mlp.router"] = np.zeros((n, d))
                    w[p + "mlp.router"][np.arange(n), d - codes + np.arange(n)] = 2.0
                    w[p + "mlp.correction"] = rng.permutation(APART[:n]) / 512.0
                else:
                    mat(p + "mlp.router", n, d)
                    vec(p + "mlp.correction", n, 0.0, 0.2)
    return w


def test_configuration_round_trip_and_spec():
    from sonicboom_amd.config import architecture_of
    arch = architecture_of(CFG)
    cfg = arch.config_class.from_dict(CFG)
    assert cfg.to_dict() == CFG
    spec = arch.build_spec(cfg)
    shapes = {t.name: t.shape for t in spec.all_tensors()}
    want = random_weights(CFG)
    assert set(shapes) == set(want), "the spec names the tensors of the file, no more and no fewer"
    for name, a in want.items():
        assert shapes[name] == a.shape, name
    # layers 1 and 2 run three times, each time with a cache of its own; nothing stands between the passes
    assert [e.block for e in spec.order] == [0, 1, 2, 1, 2, 1, 2, 3] and not spec.junctions
    caches = [e.cache for e in spec.order]
    assert caches[0] is None and len(set(caches[1:])) == 7 and all(e.writes_cache for e in spec.order)
    light, both, chunked = (spec.blocks[i].parts["mixer"] for i in (0, 1, 2))
    assert light.kind == "lightning" and light.params["decay"] == [0.5, 0.96875] and light.params["eps"] == 2e-5
    left, right = both.parts["left"], both.parts["right"]
    assert both.kind == "side_by_side" and both.params["weight"] == (0.75, 0.625) and not both.tensors
    assert (left.params["window"], left.params["chunk"], left.params["qk_norm"], left.params["v_dim"]) == (5, 0, "row", 10)
    assert left.tensors["q_norm"].shape == (24,) and left.tensors["k_norm"].shape == (12,)
    assert np.allclose(left.parts["position"].params["frequencies"], [0.25, 0.25 * 500.0 ** -0.5])
    assert (right.params["inner"], right.params["blocks"], right.params["taps"]) == (12, 3, 4)
    assert (chunked.params["window"], chunked.params["chunk"], chunked.params["sink_scores"], chunked.params["out_bias"]) == (0, 7, True, True)
    assert spec.blocks[3].parts["mixer"].parts["left"].parts["position"].kind == "none", "no pair turns"
    moe = spec.blocks[1].parts["ffn"].params
    assert (moe["router_score"], moe["router_scale"], moe["groups"], moe["keep_groups"], moe["activation"]) == \
        ("sigmoid_corrected", 1.25, 3, 2, "silu")
    assert spec.blocks[0].parts["ffn"].params["activation"] == "relu_sq" and "ffn" not in spec.blocks[3].parts
    assert spec.final_norm.kind == "streams_sum" and spec.embedding.params["streams"] == 3
    assert "l3.norm2" in spec.ignorable_tensors and "l3.hc2.mix" in spec.ignorable_tensors


def test_absent_keys_mean_absent_mechanisms():
    from sonicboom_amd.config import architecture_of
    bare = copy.deepcopy(CFG)
    bare.pop("loop")
    bare["layers"][1]["mlp"]["router"].pop("groups")
    bare["layers"][1]["mixer"]["left"]["rot"].pop("scaling")
    spec = architecture_of(bare).build_spec(architecture_of(bare).config_class.from_dict(bare))
    assert [e.block for e in spec.order] == [0, 1, 2, 3]
    assert spec.blocks[1].parts["ffn"].params["groups"] == 1
    left = spec.blocks[1].parts["mixer"].parts["left"]
    assert np.allclose(left.parts["position"].params["frequencies"], [1.0, 500.0 ** -0.5])


@pytest.mark.parametrize("edit, message", [
    (lambda c: c["layers"][1]["mixer"]["left"].pop("heads"), "layers[1].mixer.left.heads"),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("mask"), "layers[1].mixer.left.mask"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("conv"), "layers[1].mixer.right.conv"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(blocks=5), "do not divide"),
    (lambda c: c["layers"][1]["mixer"].pop("left_scale"), "layers[1].mixer.left_scale"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].pop("factor"), "rot.scaling.factor"),
    (lambda c: c["layers"][2]["mixer"]["mask"].update(size=0), "mask.size must be positive"),
    (lambda c: c["layers"][2]["mixer"].update(kv_heads=2), "not a multiple"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=10), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["decay"].pop(), "layers[0].mixer.decay"),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5, 1.5]), "between 0 and 1"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=7), "router"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4), "groups"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), "hold fewer"),
    (lambda c: c["layers"][1]["mlp"]["router"].pop("scale"), "layers[1].mlp.router.scale"),
    (lambda c: c["layers"][0]["mlp"].update(kind="gated"), "unknown feed-forward"),
    (lambda c: c["layers"][0].update(type="lstm"), "unknown layer type"),
    (lambda c: c["loop"].update(stop=5), "loop"),
    (lambda c: c["loop"].pop("times"), "loop.times"),
    (lambda c: c.update(streams=0), "streams"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_configuration_errors_name_the_key(edit, message):
    from sonicboom_amd.config import ConfigError, architecture_of
    bad = copy.deepcopy(CFG)
    edit(bad)
    with pytest.raises(ConfigError, match=message.replace("[", r"\[").replace("]", r"\]")):
        architecture_of(bad).config_class.from_dict(bad)


def test_a_chunk_of_keys_gives_its_pages_back_when_the_next_begins():
    from sonicboom_amd.cache.paged import PAGE, PagedCache, group_entries, pages_for
    groups = group_entries({0: (1, 32, 0, 32, 100), 1: (1, 32, 0, 32), 2: (1, 32, 0, 32, 100), 3: (1, 32, 100, 32)})
    assert [(g.entries, g.chunk, g.window, g.span) for g in groups] == [((0, 2), 100, 0, 100), ((1,), 0, 0, 0), ((3,), 0, 100, 100)]
    c = PagedCache(groups, PAGE * 40, max_slots=3, allocate=False, step_rows=70)
    assert c.windowed(True) == [0, 2] and c.pools[0].n_pages == 3 * (pages_for(100) + 2) + pages_for(70) < c.pools[1].n_pages
    s, length = c.alloc_slot(), 0
    for n in (70, 29, 1, 1, 60, 39, 1, 64, 70):
        c.reserve([s], [n])
        c.advance([s], [n])
        length += n
        first = length // 100 * 100 // PAGE          # the page of the first key that position `length` reads
        held = [i for i, p in enumerate(c.page_table(0, [s])[0]) if p >= 0]
        assert held == list(range(first, pages_for(length))), length
        assert c.held_pages(1) == pages_for(length)
    assert c.can_truncate(s, length - 1) and not c.can_truncate(s, 100)
    c.free_slot(s)
    assert c.held_pages(0) == c.held_pages(1) == c.held_pages(2) == 0
    # many sequences at their bounds, steps of every size up to the promised: never out of pages
    rng = np.random.default_rng(0)
    slots = [c.alloc_slot() for _ in range(3)]
    for _ in range(60):
        cut = np.diff([0, *sorted(rng.integers(1, 70, size=2)), 70])
        live = [(s, int(n)) for s, n in zip(slots, cut) if n > 0]
        for s, n in live:
            if c.length(s) + n > PAGE * 12:
                c.free_slot(s)
                assert c.alloc_slot() == s
        c.reserve([s for s, _ in live], [n for _, n in live])
        c.advance([s for s, _ in live], [n for _, n in live])


def test_the_plain_implementation_is_causal_and_every_mechanism_counts():
    w = random_weights(CFG, seed=3)
    tokens = [int(t) for t in np.random.default_rng(1).integers(0, 50, size=23)]
    whole = P.forward(CFG, w, tokens)
    assert np.allclose(whole[:9], P.forward(CFG, w, tokens[:9]), atol=1e-9), "a prefix's logits do not change"
    assert P.run_order(CFG) == [0, 1, 2, 1, 2, 1, 2, 3]

    def moves(cfg=CFG, **edits):
        return np.abs(P.forward(cfg, dict(w, **edits), tokens) - whole).max() > 1e-3 * whole.std()
    for name in w:
        if name in ("l0.hc1.in", "l3.hc1.out"):
            continue          # (the sum alone counts: the streams are equal before the first, and added after the last)
        assert moves(**{name: np.roll(w[name].reshape(-1), 1).reshape(w[name].shape)}), name
    assert moves(**{"l1.hc1.mix": w["l1.hc1.mix"].T}), "the mixing matrix is indexed from, to"
    for path, key, value in ((("layers", 1, "mixer", "left", "mask"), "size", 6), (("layers", 2, "mixer", "mask"), "size", 8),
                             (("layers", 1, "mixer", "left", "rot", "scaling"), "factor", 2.0), (("layers", 1, "mixer"), "left_scale", 0.5),
                             (("layers", 3, "mixer"), "right_scale", 0.5), (("layers", 1, "mlp", "router"), "scale", 1.0),
                             (("layers", 1, "mlp", "router", "groups"), "keep", 1), (("loop",), "times", 2)):
        other = copy.deepcopy(CFG)
        at = other
        for k in path:
            at = at[k]
        at[key] = value
        assert moves(other), (path, key)


def test_the_plain_pieces():
    assert P.chunk_mask(5, 2).astype(int).tolist() == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [0, 0, 1, 0, 0], [0, 0, 1, 1, 0], [0, 0, 0, 0, 1]]
    assert P.window_mask(4, 2).astype(int).tolist() == [[1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]]
    q, k, v = np.ones((1, 1, 1)), np.zeros((1, 1, 1)), np.full((1, 1, 1), 6.0)
    assert np.allclose(P.attend(q, k, v, 1.0, P.window_mask(1, 1), [np.log(2.0)]), 2.0), "weight 1 / (1 + 2)"
    assert np.allclose(P.time_conv([[1.0], [2.0], [4.0]], [[10.0, 100.0]], [0.5]), [[100.5], [210.5], [420.5]])
    assert np.allclose(P.lightning_reads(np.ones((2, 1)), np.array([[1.0], [2.0]]), np.array([[3.0], [5.0]]), 0.5), [[3.0], [11.5]])
    a = np.exp(-8.0 * 0.5 * np.log(2.0))
    got = P.gated_recurrence(np.array([[1.0], [1.0]]), np.full((2, 1), 0.5), np.ones((2, 1)), [0.0])
    assert np.allclose(got, [[np.sqrt(1 - a * a)], [(1 + a) * np.sqrt(1 - a * a)]])
    router = {"experts": 6, "top": 2, "scale": 2.0, "groups": {"count": 3, "keep": 1}}
    # choice scores .9 .1 | .6 .6 | .0 -.5: the second group's two best add up to the most
    ids, weights = P.choose(np.array([0.9, 0.1, 0.5, 0.5, 0.2, 0.2]), [0, 0, 0.1, 0.1, -0.2, -0.7], router)
    assert sorted(ids) == [2, 3] and np.allclose(weights, [1.0, 1.0]), "weights leave the correction out"
    # a choice score below zero still beats a closed group's
    ids, _ = P.choose(np.array([0.1, 0.1, 0.9, 0.0, 0.0, 0.0]), [-0.2, -0.3, -2.0, -2.0, -2.0, -2.0], router)
    assert sorted(ids) == [0, 1]
    X = np.array([[[1.0]], [[10.0]]])
    out = P.sublayer(X, [1.0, 2.0], [0.5, 3.0], [[1.0, 0.1], [0.0, 2.0]], lambda u: u)
    assert np.allclose(out[:, 0, 0], [1.0 + 0.5 * 21.0, 0.1 + 20.0 + 3.0 * 21.0])


def test_coded_routers_make_no_close_calls():
    cfg = config(40, 40, 2, [lin(2, 4, 4, (0.5, 0.9), ff=(8, 12, 4, 1.0, 4, 2)), att((2, 1, 4, 4), 6, (100.0, 4), ff=(8, 10, 3, 2.0, 2, 1))],
                 loop=(0, 2, 3))
    w = random_weights(cfg, seed=4, coded=True)
    gaps, chosen = [], set()
    real = P.choose

    def watched(scores, correction, router):
        ids, weights = real(scores, correction, router)
        choice = scores + correction
        m = router["experts"] // router["groups"]["count"]
        sums = np.sort([np.sort(choice[g:g + m])[-2:].sum() for g in range(0, router["experts"], m)])[::-1]
        kept = set(int(e) // m for e in ids)
        rest = [choice[e] for e in range(router["experts"]) if e // m in kept and e not in ids]
        gaps.append(min(sums[router["groups"]["keep"] - 1] - sums[router["groups"]["keep"]], choice[ids].min() - max(rest, default=-9.0)))
        chosen.add((router["experts"], tuple(sorted(int(e) for e in ids))))
        return ids, weights
    P.choose = watched
    try:
        P.forward(cfg, w, [int(t) for t in np.random.default_rng(0).integers(0, 40, size=60)])
    finally:
        P.choose = real
    assert min(gaps) > 1e-3 and len(chosen) > 20, (min(gaps), len(chosen))
