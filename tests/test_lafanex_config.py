"""Lafanex's configuration, plan and random-weights mode, and the twin's own small checks (no GPU)."""

import json

import numpy as np
import pytest
import torch

import plain_lafanex as plain
from liyab_amd.config import config_from_dict
from liyab_amd.config.lafanex import LafanexConfig
from liyab_amd.errors import InvalidModel, Unsupported

RAW = {
    "architecture": "Lafanex", "vocab": 97, "width": 40, "norm": {"eps": 1e-5}, "streams": 3, "loop": {"start": 1, "stop": 3, "times": 2},
    "layers": [
        {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 10, "scale": 0.3, "rot": {"dims": 4, "base": 100.0}},
         "mlp": {"kind": "moe", "expert": {"ff": 12, "limit": 0.9}, "router": {"experts": 6, "top": 3, "identity": 2, "scale": 1.4}, "shared": {"ff": 14, "limit": 0.5}}},
        {"type": "mamba1", "mixer": {"inner": 30, "state": 5, "dt_rank": 3, "conv": 4}, "mlp": {"kind": "dense", "ff": 28}},
        {"type": "mamba1", "mixer": {"inner": 20, "state": 7, "dt_rank": 2, "conv": 2}, "mlp": None},
        {"type": "attention", "mixer": {"heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 0.2},
         "mlp": {"kind": "moe", "expert": {"ff": 8, "limit": 2.0}, "router": {"experts": 3, "top": 1}}},
    ],
}


def fresh():
    return json.loads(json.dumps(RAW))


def test_the_registry_finds_it_and_the_keys_come_back():
    cfg = config_from_dict(fresh())
    assert isinstance(cfg, LafanexConfig)
    assert config_from_dict(cfg.to_json()) == cfg
    a, m, n, b = (layer.mixer for layer in cfg.layers)
    assert (a.n_head, a.n_kv_head, a.head_dim, a.value_dim, a.scale, a.rot_dims, a.rot_base) == (4, 2, 6, 10, 0.3, 4, 100.0)
    assert (m.inner, m.n_state, m.dt_rank, m.taps) == (30, 5, 3, 4) and (n.inner, n.n_state, n.dt_rank, n.taps) == (20, 7, 2, 2)
    assert b.rot_dims == 0
    f = cfg.layers[0].mlp
    assert (f.kind, f.ff, f.limit, f.experts, f.top, f.identity, f.scale, f.shared_ff, f.shared_limit) == ("moe", 12, 0.9, 6, 3, 2, 1.4, 14, 0.5)
    g = cfg.layers[3].mlp
    assert (g.identity, g.scale, g.shared_ff) == (0, 1.0, 0)  # (nothing says otherwise)
    assert cfg.streams == 3 and cfg.runs() == [0, 1, 2, 1, 2, 3] and cfg.layers[2].mlp is None
    for change, runs in ((None, [0, 1, 2, 3]), ({"start": 0, "stop": 4, "times": 1}, [0, 1, 2, 3]), ({"start": 3, "stop": 4, "times": 3}, [0, 1, 2, 3, 3, 3])):
        raw = fresh()
        raw["loop"] = change
        assert config_from_dict(raw).runs() == runs == plain.runs(raw)


def test_sizes_of_a_scan_that_the_file_leaves_to_its_tensors():
    raw = fresh()
    raw["layers"][1]["mixer"] = {}
    shapes = {"l1.mix.A_log": (30, 5), "l1.mix.dt": (30, 3), "l1.mix.conv": (30, 4)}
    assert LafanexConfig.from_json(raw, shapes=shapes).layers[1].mixer == config_from_dict(fresh()).layers[1].mixer
    with pytest.raises(InvalidModel):
        config_from_dict(raw)


def test_the_plan_lists_a_looped_layer_once_a_run():
    plan = config_from_dict(fresh()).plan()
    assert plan.streams == 3 and [spec.arrangement for spec in plan.layers] == ["streams"] * 6
    assert [(e.layer, e.cache_layer) for e in plan.order] == [(i, i) for i in range(6)]
    assert plan.layers[1].mixer.tensors["in"].name == plan.layers[3].mixer.tensors["in"].name == "l1.mix.in"
    a, m = plan.layers[0].mixer, plan.layers[1].mixer
    assert a.qk_norm and not a.qk_norm_weights and a.sink_value == 0.0 and not a.sink and a.rotary.dims == 4 and not a.rotary.halves and plan.layers[5].mixer.rotary is None
    assert (m.kind, m.inner, m.n_state, m.dt_rank, m.taps, m.tensors["dt_bias"].name, m.tensors["A_log"].name) == ("selective_scan", 30, 5, 3, 4, "l1.mix.dt.b", "l1.mix.A_log")
    f = plan.layers[0].ffn
    assert (f.scores, f.identity, f.scale, f.clamp, f.shared_clamp, f.shared_inner, f.shared_weighed) == ("softmax_all", 2, 1.4, (0.9, 1.702, 1.0), (0.5, 1.702, 1.0), 14, True)
    assert f.tensors["shared_weight"].name == "l0.mlp.shared.sg" and f.tensors[("down", 5)].name == "l0.mlp.e5.down" and ("down", 6) not in f.tensors
    c = plan.layers[0].connect_ffn
    assert (c.streams, c.tensors["take"].name, c.tensors["give"].name, c.tensors["mix"].name) == (3, "l0.hc2.in", "l0.hc2.out", "l0.hc2.mix")
    assert plan.layers[2].connect_ffn is None and plan.layers[2].connect_mixer is not None and plan.layers[2].norm_ffn is None
    assert plan.final_norm.weight_offset == 1.0 and plan.layers[0].norm_mixer.weight_offset == 1.0
    assert plan.head.tensors["weight"].name == plan.embedding.tensors["table"].name == "embed"
    raw = fresh()
    raw.pop("streams")
    plan = config_from_dict(raw).plan()
    assert plan.streams == 1 and plan.layers[0].connect_mixer is None and plan.layers[0].connect_ffn is None


@pytest.mark.parametrize("change,error", [
    (lambda r: r.pop("vocab"), InvalidModel),
    (lambda r: r["norm"].pop("eps"), InvalidModel),
    (lambda r: r.update(streams=0), InvalidModel),
    (lambda r: r["loop"].update(stop=5), InvalidModel),
    (lambda r: r["loop"].update(start=3, stop=2), InvalidModel),
    (lambda r: r["loop"].update(times=0), InvalidModel),
    (lambda r: r["layers"][0].update(type="convolution"), Unsupported),
    (lambda r: r["layers"][0].update(mixer=None), InvalidModel),
    (lambda r: r["layers"][0]["mixer"].update(kv_heads=3), InvalidModel),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=5), InvalidModel),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=8), InvalidModel),
    (lambda r: r["layers"][0]["mixer"].pop("scale"), InvalidModel),
    (lambda r: r["layers"][1]["mixer"].pop("state"), InvalidModel),
    (lambda r: r["layers"][1]["mixer"].update(conv=0), InvalidModel),
    (lambda r: r["layers"][0]["mlp"]["router"].update(top=9), InvalidModel),
    (lambda r: r["layers"][0]["mlp"]["router"].update(identity=-1), InvalidModel),
    (lambda r: r["layers"][0]["mlp"]["expert"].update(limit=0.0), InvalidModel),
    (lambda r: r["layers"][0]["mlp"]["shared"].pop("limit"), InvalidModel),
    (lambda r: r["layers"][1]["mlp"].update(kind="gated"), Unsupported),
])
def test_what_is_wrong_is_refused(change, error):
    raw = fresh()
    change(raw)
    with pytest.raises(error):
        config_from_dict(raw)


def test_parts_that_do_not_go_together_are_refused():
    """Identity experts behind a block that norms its sublayers' results; streams among blocks that know one."""
    import dataclasses

    from liyab_amd.models.decoder import DecoderModel
    from liyab_amd.weights.random_init import DrawingStore

    plan = config_from_dict(fresh()).plan()
    other = [dataclasses.replace(spec, arrangement="pre_norm", connect_mixer=None, connect_ffn=None) for spec in plan.layers]
    with pytest.raises(ValueError):
        DecoderModel(dataclasses.replace(plan, layers=other), DrawingStore(1), torch.float32)
    layer = dataclasses.replace(plan.layers[0], arrangement="post_norm_gated", connect_mixer=None, connect_ffn=None)
    with pytest.raises(Unsupported):
        DecoderModel(dataclasses.replace(plan, streams=0, layers=[layer], order=plan.order[:1]), DrawingStore(1), torch.float32)


def test_random_weights_fit_the_twin(tmp_path):
    """The random-weights mode draws every tensor the twin reads; the twin runs on them, and a change of any constant of the
    configuration changes its logits."""
    from liyab_amd.weights import write_random_model
    from plain_gpt2 import read_model

    d = write_random_model(str(tmp_path / "m"), fresh(), 3)
    raw, t = read_model(d)
    assert {"embed", "final.norm", "l0.hc1.in", "l0.hc2.mix", "l0.mlp.correction", "l0.mlp.e5.gate", "l0.mlp.shared.sg", "l1.mix.A_log", "l1.mix.conv.b", "l1.mix.dt.b",
            "l1.mix.D", "l2.hc1.out", "l3.mix.o"} <= set(t)
    assert not {"head", "l2.norm2", "l2.hc2.in", "l0.mlp.e6.gate", "l3.mlp.shared.gate"} & set(t)
    assert t["l0.mlp.router"].shape == (8, 40) and t["l0.mlp.correction"].shape == (8,) and t["l0.hc1.mix"].shape == (3, 3)
    assert t["l1.mix.x"].shape == (13, 30) and t["l1.mix.dt"].shape == (30, 3) and t["l1.mix.in"].shape == (60, 40)
    toks = [5, 17, 3, 9, 11, 60, 2, 4, 8, 1, 96, 33, 7, 21]
    streams = []
    base = plain.forward(raw, t, toks, streams)
    assert base.shape == (len(toks), 97) and np.isfinite(base).all() and len(streams) == 6
    for change in (lambda r: r["layers"][0]["mixer"]["rot"].update(base=99.0), lambda r: r["layers"][0]["mixer"]["rot"].update(dims=2), lambda r: r["loop"].update(times=3),
                   lambda r: r["layers"][0]["mlp"]["router"].update(scale=1.3), lambda r: r["layers"][0]["mlp"]["expert"].update(limit=0.8),
                   lambda r: r["layers"][0]["mlp"]["shared"].update(limit=0.6), lambda r: r["layers"][0]["mlp"]["router"].update(top=2),
                   lambda r: r["norm"].update(eps=1e-2), lambda r: r["layers"][3]["mixer"].update(scale=0.5)):
        other = json.loads(json.dumps(raw))
        change(other)
        assert np.abs(plain.forward(other, t, toks) - base).max() > 1e-6


def test_a_layer_without_a_feed_forward_may_carry_what_nobody_reads():
    from liyab_amd.models.decoder import DecoderModel
    from liyab_amd.weights.loader import WeightStore
    from liyab_amd.weights.random_init import random_tensors

    cfg = config_from_dict(fresh())
    plan, tensors = cfg.plan(), random_tensors(cfg, 2)
    tensors.update({"l2.norm2": torch.zeros(40), "l2.hc2.in": torch.zeros(3), "l2.hc2.out": torch.zeros(3), "l2.hc2.mix": torch.zeros(3, 3)})
    for extra, fits in ((None, True), ("l1.mix.bonus", False)):
        have = dict(tensors, **({extra: torch.zeros(1)} if extra else {}))
        store = WeightStore(have, device="cpu", compute_dtype=torch.float32, name_prefixes=plan.name_prefixes, ignorable=plan.ignorable)
        DecoderModel(plan, store, torch.float32)
        if fits:
            store.finish()
        else:
            with pytest.raises(InvalidModel):
                store.finish()


def test_the_twins_parts_on_cases_worked_by_hand():
    # a turn keeps a pair's length and leaves what lies behind the turned entries alone
    v = np.arange(1.0, 13.0).reshape(1, 1, 12)
    out = plain.turn_pairs(v, np.array([3.0]), {"dims": 8, "base": 10.0})
    assert np.allclose(out[..., 8:], v[..., 8:]) and np.allclose(out[0, 0, 0] ** 2 + out[0, 0, 1] ** 2, 1.0 + 4.0)
    # one in the denominator: two scores of zero take a third each, scores far below zero nothing, and large ones everything
    seen = np.array([True, True])
    assert np.allclose(plain.weights_with_one(np.array([[0.0, 0.0]]), seen), 1.0 / 3.0)
    assert np.allclose(plain.weights_with_one(np.array([[-800.0, -800.0]]), seen), 0.0)
    assert np.allclose(plain.weights_with_one(np.array([[900.0, 900.0]]), seen), 0.5)
    # the walk: a state without decay adds up, one with a strong decay forgets
    x, ones = np.array([[2.0], [3.0]]), np.ones((2, 1))
    assert np.allclose(plain.selective_walk(x, ones, ones, ones, np.array([[0.0]]), np.array([0.5])), [[3.0], [6.5]])
    assert np.allclose(plain.selective_walk(x, ones, ones, ones, np.array([[-900.0]]), np.array([0.0])), [[2.0], [3.0]])
    assert np.allclose(plain.selective_walk(x, 2.0 * ones, ones, 3.0 * ones, np.array([[-0.5]]), np.array([0.0])), [[12.0], [3.0 * (4.0 * np.exp(-1.0) + 6.0)]])
    # the convolution's last column is the current row's
    assert np.allclose(plain.short_convolution(np.array([[1.0], [10.0], [100.0]]), np.array([[2.0, 3.0]]), np.array([0.5])), [[3.5], [32.5], [320.5]])
    # streams: the mix is indexed [from, to], every stream from the old ones
    X = np.stack([np.full((1, 1), 1.0), np.full((1, 1), 10.0)])
    t = {"p.in": np.array([1.0, 0.5]), "p.out": np.array([1.0, -1.0]), "p.mix": np.array([[0.0, 1.0], [2.0, 0.0]])}
    assert np.allclose(plain.connected(X, t, "p.", lambda u: 100.0 * u)[:, 0, 0], [20.0 + 600.0, 1.0 - 600.0])
    # the choice goes by the corrected score, the weight is the score itself
    z = np.log(np.array([[0.5, 0.2, 0.3]]))
    chosen, weights = plain.route(z, np.array([-1.0, 0.0, 0.0]), 2, 2.0)
    assert chosen.tolist() == [[2, 1]] and np.allclose(weights, [[0.6, 0.4]])
    # an identity expert gives the input itself
    m = {"expert": {"limit": 1.0}, "router": {"experts": 1, "top": 1, "identity": 1, "scale": 3.0}}
    h = np.array([[1.0, -2.0]])
    T = {"router": np.zeros((2, 2)), "correction": np.array([0.0, 1.0]), "e0.gate": np.ones((1, 2)), "e0.up": np.ones((1, 2)), "e0.down": np.ones((2, 1))}
    assert np.allclose(plain.routed_feed_forward(h, T, "", m), 1.5 * h)
    # clamps: the gate from above only, the other half from both sides
    G = {"gate": np.array([[5.0], [-5.0]]), "up": np.array([[-9.0], [9.0]]), "down": np.eye(2)}
    assert np.allclose(plain.clamped_unit(np.array([[1.0]]), G, "", 2.0), [[2.0 * plain.logistic(3.404) * -1.0, -5.0 * plain.logistic(-8.51) * 3.0]])
