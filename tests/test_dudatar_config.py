"""The Dudatar configuration, its model spec and the plain implementation, without a GPU."""
import copy

import numpy as np
import pytest

from plain import dudatar_plain as P


def side(left, right, ff=None, rot=(1e4, None), rot_right=(1e3, None), scale=None):
    """A ``parallel`` layer: left = (heads, kv_heads, dim, vdim), right = (heads, dim, vdim, decay)."""
    H, G, D, E = left
    R, K, V, decay = right
    return {"type": "parallel", "mlp": None if ff is None else {"kind": "dense", "ff": ff}, "mixer": {
        "left": {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": scale if scale is not None else 3.0 / D ** 0.5,
                 "rot": {"base": rot[0], "dims": D if rot[1] is None else rot[1]}},
        "right": {"heads": R, "dim": K, "vdim": V, "decay": list(decay),
                  "rot": {"base": rot_right[0], "dims": K if rot_right[1] is None else rot_right[1]}}}}


def gla(heads, dim, vdim, tau, ff=None, rank=None):
    mixer = {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}
    if rank is not None:
        mixer["rank"] = rank
    return {"type": "gla", "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(vocab, width, layers, loop=None, eps=1e-5, softcap=0.0):
    d = {"architecture": "Dudatar", "vocab": vocab, "width": width, "logit_softcap": softcap, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


CFG = config(50, 24, [
    gla(2, 6, 10, 4.0, ff=20, rank=3),
    side((4, 2, 6, 10), (3, 8, 4, (0.5, 0.875, 0.99)), ff=28, rot=(500.0, 4), rot_right=(100.0, 6)),
    gla(1, 8, 4, 1.0, rank=5),
    side((3, 3, 8, 4), (1, 4, 12, (0.9,)), rot=(1e4, 0)),
], loop=(1, 3, 3), eps=2e-5, softcap=9.0)


def random_weights(cfg, seed=0, rank=7, gain=1.0):
    """Weights by the file's names for a config.json dict, drawn here (not by the package): projections of unit
    outputs for unit inputs, times ``gain``; norm weights that are not near 1.  The recurrences' keys lean towards their
    queries, so that a token's read of its own write is no small difference of large numbers: what is read is normed to
    order one, and where it nearly cancelled (a first token with q.k near 0) rounding would decide its sign."""
    rng = np.random.default_rng(seed)
    d, w = cfg["width"], {}

    def lin(name, n_out, n_in, times=1.0):
        w[name] = rng.normal(0, gain * times / np.sqrt(n_in), (n_out, n_in))

    def vec(name, n, mean=1.0, spread=0.25):
        w[name] = rng.normal(mean, spread, n)
    w["embed"] = rng.normal(0.1, 1.0, (cfg["vocab"], d))
    lin("head", cfg["vocab"], d, 2.0)
    vec("final.norm", d)
    if cfg.get("loop"):
        lin("loop.in", d, 2 * d)
        w["loop.step"] = rng.normal(0, 0.5, (cfg["loop"]["times"], d))
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        vec(p + "norm1", d)
        if layer["type"] == "parallel":
            a, b = m["left"], m["right"]
            q = p + "mix.left."
            lin(q + "q", a["heads"] * a["dim"], d), lin(q + "k", a["kv_heads"] * a["dim"], d)
            lin(q + "v", a["kv_heads"] * a["vdim"], d), lin(q + "g", a["heads"], d, 2.0), lin(q + "o", d, a["heads"] * a["vdim"])
            q = p + "mix.right."
            for role, n in (("q", b["heads"] * b["dim"]), ("k", b["heads"] * b["dim"]), ("v", b["heads"] * b["vdim"]),
                            ("g", b["heads"] * b["vdim"])):
                lin(q + role, n, d)
            w[q + "k"] = 0.8 * w[q + "q"] + 0.6 * w[q + "k"]
            lin(q + "o", d, b["heads"] * b["vdim"])
            vec(p + "mix.left.out", d), vec(p + "mix.right.out", d)
        else:
            q, H = p + "mix.", m["heads"]
            for role, n in (("q", H * m["dim"]), ("k", H * m["dim"]), ("v", H * m["vdim"]), ("g", H * m["vdim"])):
                lin(q + role, n, d)
            w[q + "k"] = 0.8 * w[q + "q"] + 0.6 * w[q + "k"]
            r = m.get("rank") or rank
            lin(q + "a1", r, d), lin(q + "a2", H * m["dim"], r, 1.5)
            w[q + "a2.b"] = rng.normal(1.0, 2.0, H * m["dim"])
            vec(q + "norm", m["vdim"])
            lin(q + "o", d, H * m["vdim"])
        if layer["mlp"] is not None:
            f = layer["mlp"]["ff"]
            lin(p + "mlp.gate", f, d, 1.5), lin(p + "mlp.up", f, d), lin(p + "mlp.down", d, f)
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
    # layers 1 and 2 run three times; every pass begins with the junction and has a cache of its own
    assert [e.block for e in spec.order] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert [(e.junction, e.turn) for e in spec.order] == [(None, 0), (0, 0), (None, 0), (0, 1), (None, 0), (0, 2), (None, 0), (None, 0)]
    caches = [e.cache for e in spec.order]
    assert [c is None for c in caches] == [True, False, True, False, True, False, True, False]
    assert len({c for c in caches if c is not None}) == 4 and all(e.writes_cache for e in spec.order)
    m = spec.blocks[1].parts["mixer"]
    left, right = m.parts["left"], m.parts["right"]
    assert m.kind == "side_by_side" and m.params["weight"] == 0.5 and m.params["eps"] == 2e-5
    assert (left.params["heads_kv"], left.params["v_dim"], left.params["out_gate"], left.params["qk_norm"]) == (2, 10, "head", True)
    assert left.params["scale"] == CFG["layers"][1]["mixer"]["left"]["scale"] and "q_norm" not in left.tensors
    assert np.allclose(left.parts["position"].params["frequencies"], [1.0, 500.0 ** -0.5]) and left.parts["position"].params["rot_dims"] == 4
    assert spec.blocks[3].parts["mixer"].parts["left"].parts["position"].kind == "none", "no pair turns"
    assert right.params["decay"] == [0.5, 0.875, 0.99]
    assert spec.blocks[0].parts["mixer"].params["tau"] == 4.0 and spec.blocks[0].parts["ffn"].params["activation"] == "gelu_tanh"
    assert "ffn" not in spec.blocks[2].parts and "ffn_norm" not in spec.blocks[0].parts
    assert spec.head.params["softcap"] == 9.0 and spec.final_norm.kind == "layernorm"


def test_absent_keys_mean_absent_mechanisms():
    from sonicboom_amd.config import architecture_of
    bare = copy.deepcopy(CFG)
    bare.pop("logit_softcap"), bare.pop("loop")
    bare["layers"][0]["mixer"].pop("rank")
    cfg = architecture_of(bare).config_class.from_dict(bare)
    spec = architecture_of(bare).build_spec(cfg)
    assert spec.head.params["softcap"] == 0.0 and not spec.junctions and [e.block for e in spec.order] == [0, 1, 2, 3]
    assert {t.name: t.shape for t in spec.all_tensors()}["l0.mix.a1"] == (-1, 24), "left to the file"
    once = dict(copy.deepcopy(CFG), loop={"start": 0, "stop": 4, "times": 1})
    spec = architecture_of(once).build_spec(architecture_of(once).config_class.from_dict(once))
    assert [(e.junction, e.turn) for e in spec.order] == [(0, 0)] + [(None, 0)] * 3, "one pass still begins with its junction"


@pytest.mark.parametrize("edit, message", [
    (lambda c: c["layers"][1]["mixer"]["left"].pop("heads"), "layers[1].mixer.left.heads"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("rot"), "layers[1].mixer.right.rot"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("decay"), "layers[1].mixer.right.decay"),
    (lambda c: c["layers"][1]["mixer"]["right"]["decay"].pop(), "layers[1].mixer.right.decay"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.5, 1.5, 0.9]), "between 0 and 1"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), "not a multiple"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["right"]["rot"].update(dims=10), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"].pop("tau"), "layers[0].mixer.tau"),
    (lambda c: c["layers"][0]["mixer"].update(tau=0), "tau must be positive"),
    (lambda c: c["layers"][2].update(type="lstm"), "unknown layer type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "unknown feed-forward"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "layers[0].mlp.ff"),
    (lambda c: c["loop"].update(stop=5), "loop"),
    (lambda c: c["loop"].update(start=3), "loop"),
    (lambda c: c["loop"].pop("times"), "loop.times"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_configuration_errors_name_the_key(edit, message):
    from sonicboom_amd.config import ConfigError, architecture_of
    bad = copy.deepcopy(CFG)
    edit(bad)
    with pytest.raises(ConfigError, match=message.replace("[", r"\[").replace("]", r"\]")):
        architecture_of(bad).config_class.from_dict(bad)


def test_an_order_entry_names_a_junction_that_exists():
    from sonicboom_amd.config import architecture_of
    spec = architecture_of(CFG).build_spec(architecture_of(CFG).config_class.from_dict(CFG))
    spec.junctions = []
    with pytest.raises(ValueError, match="junction"):
        spec.validate()


def test_the_plain_implementation_is_causal_and_its_passes_differ():
    w = random_weights(CFG, seed=3)
    tokens = [int(t) for t in np.random.default_rng(1).integers(0, 50, size=17)]
    whole = P.forward(CFG, w, tokens)
    assert np.allclose(whole[:9], P.forward(CFG, w, tokens[:9]), atol=1e-12), "a prefix's logits do not change"
    assert np.all(np.abs(whole) <= 9.0), "the cap bounds the logits"
    assert [s for _, s in P.run_order(CFG)] == [None, 0, None, 1, None, 2, None, None]
    swapped = dict(w, **{"loop.step": w["loop.step"][[1, 0, 2]]})
    assert np.abs(P.forward(CFG, swapped, tokens) - whole).max() > 1e-3, "every pass has its own vector"
    turned = dict(w, **{"loop.in": np.concatenate([w["loop.in"][:, 24:], w["loop.in"][:, :24]], axis=1)})
    assert np.abs(P.forward(CFG, turned, tokens) - whole).max() > 1e-3, "x comes first, the embedding second"


def test_the_plain_recurrence():
    q, k, v = np.array([[1.0, 2.0], [3.0, 0.0]]), np.array([[1.0, 0.0], [0.0, 1.0]]), np.array([[5.0], [7.0]])
    got = P.decayed_reads(q, k, v, np.array([[0.5, 0.25], [0.5, 0.25]]))
    # S after the first token is [[5], [0]], after the second [[2.5], [7]]
    assert np.allclose(got, [[5.0], [7.5]])
    assert np.allclose(P.layer_norm(np.array([1.0, 3.0]), np.array([2.0, 1.0]), 0.0), [-2.0, 1.0])
    assert np.allclose(P.gelu_tanh(np.array([0.0, 1.0])), [0.0, 0.8411919906])
    c, s = np.cos(0.5), np.sin(0.5)
    out = P.turn(np.array([[[1.0, 2.0, 3.0, 4.0, 9.0]]]), [5], {"dims": 4, "base": 100.0})[0, 0]
    assert np.allclose(out[[1, 3]], [2 * c - 4 * s, 4 * c + 2 * s]) and out[4] == 9.0, "pair 1 turns by 5 / 10"
