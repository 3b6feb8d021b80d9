"""Lolulorn's configuration, plan and random-weights mode, and the twin's own small checks (no GPU)."""

import json

import numpy as np
import pytest

import plain_lolulorn as plain
from liyab_amd.config import config_from_dict
from liyab_amd.config.lolulorn import LolulornConfig
from liyab_amd.errors import InvalidArgument, InvalidModel, Unsupported

RAW = {
    "architecture": "Lolulorn", "vocab": 97, "width": 40, "embedding": {"scale": 3.0}, "norm": {"eps": 1e-5},
    "layers": [
        {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 10, "scale": 0.3, "mask": {"size": 5, "keep_first": 2},
                                        "rot": {"dims": 4, "base": 100.0, "scaling": {"factor": 3.0}}},
         "mlp": {"kind": "moe", "expert": {"ff": 12}, "router": {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 2}}}},
        {"type": "delta", "mixer": {"heads": 6, "kv_heads": 3, "dim": 8, "vdim": 5, "conv": 3}, "mlp": {"kind": "dense", "ff": 30}},
        {"type": "gla", "mixer": {"heads": 2, "dim": 8, "vdim": 12, "tau": 6.0}, "mlp": None},
        {"type": "attention", "mixer": {"heads": 2, "kv_heads": 2, "dim": 6, "vdim": 10, "scale": 0.2, "kv_from": 0, "mask": {"size": 9, "keep_first": 0},
                                        "rot": {"dims": 4, "base": 100.0, "scaling": {"factor": 3.0}}},
         "mlp": {"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 3, "top": 1}}},
    ],
}


def fresh():
    return json.loads(json.dumps(RAW))


def test_the_registry_finds_it_and_the_keys_come_back():
    cfg = config_from_dict(fresh())
    assert isinstance(cfg, LolulornConfig)
    assert config_from_dict(cfg.to_json()) == cfg
    a, d, g, s = (layer.mixer for layer in cfg.layers)
    assert (a.n_head, a.n_kv_head, a.head_dim, a.value_dim, a.window, a.keep_first, a.rot_dims, a.rot_factor, a.kv_from) == (4, 2, 6, 10, 5, 2, 4, 3.0, None)
    assert (d.n_head, d.n_kv_head, d.head_dim, d.value_dim, d.taps) == (6, 3, 8, 5, 3)
    assert (g.n_head, g.head_dim, g.value_dim, g.tau, g.decay_rank) == (2, 8, 12, 6.0, 16)
    assert (s.kv_from, s.window, s.keep_first) == (0, 9, 0)
    m = cfg.layers[0].mlp
    assert (m.kind, m.ff, m.experts, m.top, m.groups, m.keep) == ("moe", 12, 6, 2, 3, 2)
    assert (cfg.layers[3].mlp.groups, cfg.layers[3].mlp.keep) == (1, 1)  # (nothing says otherwise)
    assert cfg.embedding_scale == 3.0 and cfg.layers[2].mlp is None


def test_the_decays_rank_is_the_narrow_matrix_shape():
    cfg = LolulornConfig.from_json(fresh(), shapes={"l2.mix.a1": (7, 40)})
    assert cfg.layers[2].mixer.decay_rank == 7
    assert config_from_dict(cfg.to_json()).layers[2].mixer.decay_rank == 7


def test_the_plan_names_the_tensors_and_whose_cache_is_read():
    plan = config_from_dict(fresh()).plan()
    assert [spec.arrangement for spec in plan.layers] == ["post_norm_gated"] * 4
    assert [(e.layer, e.cache_layer, e.writes_cache) for e in plan.order] == [(0, 0, True), (1, 1, True), (2, 2, True), (3, 0, False)]
    a, d, g, s = (spec.mixer for spec in plan.layers)
    assert a.qk_norm_rows and not a.qk_norm and a.keep_first == 2 and a.rotary.linear == 3.0 and not a.rotary.halves and not a.kv_shared
    assert s.kv_shared and not {"k", "v", "k_norm"} & set(s.tensors) and s.tensors["q_norm"].name == "l3.mix.q.norm"
    assert (d.key_eps, d.q_scale, d.tensors["dt_bias"].name, d.tensors["k_conv"].name) == (1e-6, 8 ** -0.5, "l1.mix.dt_bias", "l1.mix.k.conv")
    assert (g.tau, g.q_scale, g.tensors["w2_bias"].name) == (6.0, 8 ** -0.5, "l2.mix.a2.b")
    norm = plan.layers[0].norm_ffn
    assert (norm.kind, norm.tensors["weight"].name, norm.tensors["bias"].name) == ("layernorm", "l0.norm2", "l0.norm2.b") and plan.layers[2].norm_ffn is None
    ffn = plan.layers[0].ffn
    assert (ffn.scores, ffn.groups, ffn.gated, ffn.activation, ffn.tensors["correction"].name, ffn.tensors[("gate", 5)].name) == (
        "logistic", (3, 2), True, "silu", "l0.mlp.correction", "l0.mlp.e5.gate")
    assert plan.layers[1].ffn.activation == "gelu_tanh" and plan.embedding.scale == 3.0


@pytest.mark.parametrize("change,error", [
    (lambda r: r.pop("vocab"), InvalidModel),
    (lambda r: r["norm"].pop("eps"), InvalidModel),
    (lambda r: r["layers"][0].update(type="convolution"), Unsupported),
    (lambda r: r["layers"][0]["mixer"].update(kv_heads=3), InvalidModel),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=5), InvalidModel),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=8), InvalidModel),
    (lambda r: r["layers"][0]["mixer"]["rot"]["scaling"].pop("factor"), InvalidModel),
    (lambda r: r["layers"][0]["mixer"]["mask"].update(size=0), InvalidModel),
    (lambda r: r["layers"][0]["mixer"]["mask"].update(keep_first=-1), InvalidModel),
    (lambda r: r["layers"][1]["mixer"].pop("conv"), InvalidModel),
    (lambda r: r["layers"][1]["mixer"].update(kv_heads=4), InvalidModel),
    (lambda r: r["layers"][2]["mixer"].update(tau=0.0), InvalidModel),
    (lambda r: r["layers"][3]["mixer"].update(kv_from=1), InvalidModel),
    (lambda r: r["layers"][3]["mixer"].update(kv_from=3), InvalidModel),
    (lambda r: r["layers"][3]["mixer"].update(dim=8), InvalidModel),
    (lambda r: r["layers"][0]["mlp"]["router"].update(top=5), InvalidModel),
    (lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(count=4), InvalidModel),
    (lambda r: r["layers"][1]["mlp"].update(kind="gated"), Unsupported),
])
def test_what_is_wrong_is_refused(change, error):
    raw = fresh()
    change(raw)
    with pytest.raises(error):
        config_from_dict(raw)


def test_a_cache_read_by_another_layer_keeps_what_either_reads():
    from liyab_amd.cache import KVSpec

    rows = (("k", 2, 16), ("v", 2, 16))
    spec = KVSpec(2, 16, 20, rows=rows, keep_first=3)
    assert spec.covering(KVSpec(2, 16, 50, rows=rows, keep_first=1)) == KVSpec(2, 16, 50, rows=rows, keep_first=3)
    assert spec.covering(KVSpec(2, 16, 0, rows=rows)).window == 0
    with pytest.raises(InvalidArgument):
        spec.covering(KVSpec(2, 8, 50, rows=(("k", 2, 8), ("v", 2, 16))))
    assert spec.key != KVSpec(2, 16, 20, rows=rows, keep_first=4).key and KVSpec(2, 16, 0, keep_first=4).key == KVSpec(2, 16, 0).key


def test_random_weights_fit_the_twin(tmp_path):
    """The random-weights mode draws every tensor the twin reads; the twin runs on them, and a change of any constant of the
    configuration changes its logits."""
    from liyab_amd.weights import write_random_model
    from plain_gpt2 import read_model

    d = write_random_model(str(tmp_path / "m"), fresh(), 3)
    raw, t = read_model(d)
    assert {"embed", "head", "final.norm", "final.norm.b", "l0.mix.q.norm", "l0.mix.k.norm", "l0.mlp.correction", "l0.mlp.e5.gate", "l1.mix.q.conv", "l1.mix.A_log",
            "l1.mix.dt_bias", "l1.mix.b", "l1.norm2.b", "l2.mix.a1", "l2.mix.a2.b", "l3.mix.q.norm"} <= set(t)
    assert "l2.norm2" not in t and "l3.mix.k" not in t and "l3.mix.k.norm" not in t
    assert t["l1.mix.v.conv"].shape == (30, 3) and t["l1.mix.norm"].shape == (5,) and t["l2.mix.a2"].shape == (16, 16) and t["l0.mix.q.norm"].shape == (24,)
    toks = [5, 17, 3, 9, 11, 60, 2, 4, 8, 1, 96, 33, 7, 21]
    streams = []
    base = plain.forward(raw, t, toks, streams)
    assert base.shape == (len(toks), 97) and np.isfinite(base).all() and len(streams) == 4
    for change in (lambda r: r["layers"][0]["mixer"]["rot"]["scaling"].update(factor=2.0), lambda r: r["layers"][0]["mixer"]["mask"].update(size=6),
                   lambda r: r["layers"][0]["mixer"]["mask"].update(keep_first=1), lambda r: r["layers"][3]["mixer"]["mask"].update(size=10),
                   lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(keep=1), lambda r: r["layers"][2]["mixer"].update(tau=5.0),
                   lambda r: r["embedding"].update(scale=1.0), lambda r: r["norm"].update(eps=1e-2), lambda r: r["layers"][3]["mixer"].update(scale=0.5)):
        other = json.loads(json.dumps(raw))
        change(other)
        assert np.abs(plain.forward(other, t, toks) - base).max() > 1e-6


def test_the_twins_parts_on_cases_worked_by_hand():
    # who sees whom: the window's last position, the first one behind it, the kept first ones
    seen = plain.visible(6, {"size": 2, "keep_first": 1})
    assert seen[5].tolist() == [True, False, False, False, True, True] and seen[0].tolist() == [True] + [False] * 5
    assert plain.visible(3, None).tolist() == np.tril(np.ones((3, 3), dtype=bool)).tolist()
    # a turn keeps a pair's length and leaves what lies behind the turned entries alone; a factor divides the angle
    v = np.arange(1.0, 13.0).reshape(1, 1, 12)
    out = plain.turn_pairs(v, np.array([3.0]), {"dims": 8, "base": 10.0})
    assert np.allclose(out[..., 8:], v[..., 8:]) and np.allclose(out[0, 0, 0] ** 2 + out[0, 0, 1] ** 2, 1.0 + 4.0)
    assert np.allclose(plain.turn_pairs(v, np.array([6.0]), {"dims": 8, "base": 10.0, "scaling": {"factor": 2.0}}), out)
    # the delta rule: a second token with the same key and rate one leaves only its own value, whatever the first one's was
    H = {"p.q": np.eye(2), "p.k": np.eye(2), "p.v": np.eye(2), "p.b": np.full((1, 2), 50.0), "p.a": np.zeros((1, 2)), "p.A_log": np.array([-60.0]),
         "p.dt_bias": np.zeros(1), "p.norm": np.ones(2), "p.g": np.ones((2, 2)), "p.o": np.eye(2)}
    for c in "qkv":
        H[f"p.{c}.conv"] = np.ones((2, 1))
    m = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "conv": 1}
    x = np.array([[2.0, 2.0], [2.0, 2.0]])
    out = plain.delta(x, H, "p.", m, 0.0)
    assert np.allclose(out[0], out[1], atol=1e-5)
    # gated linear attention forgets a channel whose decay's logit is far below zero, and keeps all of one far above
    G = {"p.q": np.ones((1, 1)), "p.k": np.ones((1, 1)), "p.v": np.array([[1.0], [-1.0]]), "p.a1": np.zeros((1, 1)), "p.a2": np.zeros((1, 1)), "p.norm": np.ones(2),
         "p.g": np.ones((2, 1)), "p.o": np.eye(2)}
    m = {"heads": 1, "dim": 1, "vdim": 2, "tau": 2.0}
    x = np.array([[1.0], [2.0]])
    for bias, kept in ((800.0, 1.0), (-800.0, 0.0)):
        out = plain.gla(x, dict(G, **{"p.a2.b": np.array([bias])}), "p.", m, 1.0)
        o = 2.0 * (kept * np.array([1.0, -1.0]) + 2.0 * np.array([2.0, -2.0]))
        assert np.allclose(out[1], o / np.sqrt((o * o).mean() + 1.0) * plain.silu(2.0))
    # a group with two good scores beats one with the best; the weights are the scores themselves
    s = np.array([[0.9, 0.1, 0.6, 0.55]])
    chosen, weights = plain.route(np.log(s / (1 - s)), np.zeros(4), 2, 2, 1)
    assert chosen.tolist() == [[2, 3]] and np.allclose(weights, [[0.6, 0.55]])
    chosen, weights = plain.route(np.log(s / (1 - s)), np.array([-9.0, -9.0, -10.0, -10.0]), 2, 2, 1)
    assert chosen.tolist() == [[0, 1]] and np.allclose(weights, [[0.9, 0.1]])
