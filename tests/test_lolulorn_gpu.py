"""Lolulorn through the engine against its plain twin (`plain_lolulorn.py`): each mechanism alone, then whole models of
several geometries under every way of cutting and batching the work, in 32-bit and in bfloat16 (needs the GPU). The
geometries differ from each other in every size and in the order of their layers; one has sizes no kernel tiles evenly,
one nothing but recurrences (no cache at all), one nothing but attention, one the values that other geometries happen to share
or make one (one head, one tap, one expert, one group, a window of one position, no kept position, a factor of one)."""

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_lolulorn as plain
import trace_tools as tt
from conftest import ROOT, TOL
from plain_gpt2 import read_model

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
# float32: the largest difference of a row relative to its largest |logit|, as for the other models.
# bfloat16, against the twin in float64 with the same rounded matrices: the root mean square of a row's difference over
# that of the row's logits, both with their means taken off; a fault in a mechanism makes it about 1. Every sublayer's result
# passes a norm before it joins the stream, which brings each rounding back to the stream's own size, layer after layer.
TOL_B = {"float32": TOL["float32"], "bfloat16": 6e-2}
TOL_DRAWN = 2e-1
KEPT_32BIT = (".conv", ".a2")  # 2-D tensors that the engine keeps in 32 bits


def check_logits(got, reqs, ref, dtype, what, family=None, tol=None):
    if dtype == "float32":
        return tt.check_against_plain(got, reqs, ref, TOL_B[dtype], what, family=family)
    tol = tol or TOL_B[dtype]
    key = ((family or what.split(" ")[0]) + " (rms)", tol)
    for rid, toks in reqs.items():
        assert rid in got, f"{what}: no logits for request {rid}"
        for p in sorted(got[rid]):
            row, want = np.asarray(got[rid][p], dtype=np.float64), ref[rid][p]
            assert np.isfinite(row).all(), f"{what}: request {rid} position {p}: non-finite logits"
            diff = row - want
            e = float(np.sqrt(np.mean((diff - diff.mean()) ** 2)) / np.sqrt(np.mean((want - want.mean()) ** 2)))
            tt.WORST[key] = max(tt.WORST.get(key, 0.0), e)
            assert e <= tol, f"{what}: request {rid} (length {len(toks)}) first differs at position {p}: {e:.3e} > {tol:.1e}"


# ---------------------------------------------------------------------------
# configurations
# ---------------------------------------------------------------------------
def att(heads, kv_heads, dim, vdim, mask=None, rot=None, kv_from=None, scale=None):
    """mask = (size, keep_first); rot = (dims, base) or (dims, base, factor)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5}
    if mask:
        m["mask"] = {"size": mask[0], "keep_first": mask[1]}
    if rot:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
        if len(rot) > 2:
            m["rot"]["scaling"] = {"factor": rot[2]}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def delta(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def gla(heads, dim, vdim, tau, rank):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, groups=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if groups:
        m["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    return m


def layer(kind, m, mlp=None):
    return {"type": kind, "mixer": m, "mlp": mlp}


def config(vocab, width, eps, layers, scale=1.0):
    return {"architecture": "Lolulorn", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # every kind of layer and feed-forward; two layers read another's keys and values, under windows of their own
    "mix": (config(300, 96, 1e-5, [
        layer("delta", delta(6, 3, 16, 24, 3), moe(24, 8, 3, groups=(4, 2))),
        layer("attention", att(4, 2, 24, 16, mask=(30, 5), rot=(12, 10000.0, 3.0)), dense(80)),
        layer("gla", gla(3, 32, 20, 8.0, 12), moe(16, 6, 2, groups=(2, 1))),
        layer("attention", att(6, 2, 24, 16, mask=(70, 9), rot=(12, 10000.0, 3.0), kv_from=1), moe(20, 9, 2, groups=(3, 2))),
        layer("attention", att(2, 2, 24, 16, rot=(12, 10000.0, 3.0), kv_from=1, scale=0.3), None),
        layer("delta", delta(2, 1, 40, 16, 5), dense(64)),
    ], scale=4.0), 61),
    # sizes that no kernel tiles evenly; two taps; a window smaller than what it keeps
    "odd": (config(211, 100, 1e-6, [
        layer("gla", gla(3, 10, 6, 3.0, 5), moe(13, 6, 3, groups=(3, 2))),
        layer("attention", att(3, 3, 10, 6, mask=(17, 33), rot=(6, 777.0)), dense(30)),
        layer("delta", delta(3, 1, 7, 11, 2), moe(9, 5, 2)),
        layer("attention", att(5, 1, 6, 10, mask=(23, 2), rot=(2, 30.0, 7.0)), None),
        layer("gla", gla(2, 5, 13, 20.0, 3), dense(50)),
    ], scale=9.0), 72),
    # recurrences only: no cache at all; one tap (no history), wide heads
    "recurrent": (config(128, 64, 1e-5, [
        layer("delta", delta(2, 2, 32, 72, 1), moe(32, 4, 1)),
        layer("gla", gla(1, 72, 40, 1.5, 24), None),
        layer("delta", delta(4, 1, 72, 8, 6), dense(40)),
    ]), 63),
    # attention only (no state at all): heads of 64 and 128, a window of many pages, one that keeps more than a page, and no window
    "keys": (config(150, 64, 1e-5, [
        layer("attention", att(1, 1, 64, 64, mask=(64, 40), rot=(64, 10000.0)), dense(48)),
        layer("attention", att(2, 1, 128, 8, mask=(100, 3)), None),
        layer("attention", att(8, 4, 8, 8, rot=(8, 20.0, 2.0)), moe(8, 4, 4, groups=(2, 2))),
        layer("attention", att(2, 1, 128, 8, mask=(20, 60), kv_from=1), moe(12, 4, 1, groups=(4, 3))),
    ], scale=0.5), 64),
    # what other geometries share or make one
    "ones": (config(128, 72, 1e-5, [
        layer("attention", att(1, 1, 16, 16, mask=(1, 0), rot=(16, 100.0, 1.0)), moe(20, 1, 1, groups=(1, 1))),
        layer("delta", delta(1, 1, 8, 8, 1), moe(12, 5, 1)),
        layer("gla", gla(1, 8, 8, 1.0, 1), dense(24)),
        layer("attention", att(2, 1, 8, 8, mask=(12, 0)), moe(8, 4, 2, groups=(4, 2))),
    ], scale=20.0), 115),
}
# (the seeds are such that rounding the sublayers' inputs to bfloat16 in the twin itself moves no row by more than about 0.01: a head
# whose result all but vanishes before its norm, as a head of one or two entries' worth of weight may, makes a row of any size)
LENGTHS = {"mix": [1, 2, 23, 70, 131, 260], "odd": [3, 40, 97, 200], "recurrent": [1, 50, 140, 230], "keys": [2, 65, 150, 300], "ones": [4, 5, 66, 150]}


def weigh_all(cfg):
    """The same model with routers that weigh every expert: in bfloat16 a rounding ahead of a router whose candidates lie a
    rounding apart takes another expert than the twin, and the row then differs by far more than any rounding. The choice
    itself is compared in 32-bit throughout, and in bfloat16 where the router is run alone."""
    cfg = json.loads(json.dumps(cfg))
    for entry in cfg["layers"]:
        mlp = entry["mlp"]
        if mlp is not None and mlp["kind"] == "moe":
            mlp["router"]["top"] = mlp["router"]["experts"]
            if "groups" in mlp["router"]:
                mlp["router"]["groups"]["keep"] = mlp["router"]["groups"]["count"]
    return cfg


def twin_tensors(tensors, dtype):
    if dtype == "float32":
        return tensors
    return {k: (plain.round_to_bf16(v) if (v.ndim == 2 and not k.endswith(KEPT_32BIT)) else v) for k, v in tensors.items()}


def write_model(folder, cfg, seed, dtype):
    """A folder with random weights for `cfg` (in bfloat16 runs: its routers weigh every expert; the tensors are the same)."""
    from liyab_amd.weights import write_random_model

    write_random_model(folder, json.loads(json.dumps(cfg if dtype == "float32" else weigh_all(cfg))), seed)
    raw, tensors = read_model(folder)
    return raw, twin_tensors(tensors, dtype)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, (cfg, seed) in CONFIGS.items():
        for dtype in DTYPES:
            d = str(tmp_path_factory.mktemp(f"lolulorn_{name}_{dtype}"))
            out[(name, dtype)] = (d,) + write_model(d, cfg, seed, dtype)
    return out


def make_requests(name):
    cfg, seed = CONFIGS[name]
    return {f"{name}{i}": tt.random_tokens(seed * 50 + i, n, cfg["vocab"]) for i, n in enumerate(LENGTHS[name])}


@pytest.fixture(scope="module")
def reference(models):
    return {(name, dtype): {rid: plain.forward(raw, t, toks) for rid, toks in make_requests(name).items()}
            for (name, dtype), (_, raw, t) in models.items()}


def make_core(model_dir, dtype, max_tokens, page_size=16, max_requests=4, **kw):
    from liyab_amd.engine import EngineCore

    core = EngineCore(model_dir, dtype=dtype, page_size=page_size, max_tokens=max_tokens, max_requests=max_requests, **kw)
    # free pages and unused state hold NaN: a kernel that reads past a request's length, or a slot's old state, shows it
    for c in core.storage.layers.values():
        for t in c.rows.values():
            t.fill_(float("nan"))
    for t in core.storage.states.values():
        t.fill_(float("nan"))
    torch.cuda.synchronize()
    return core


def rand(rng, *shape, scale=1.0, mean=0.0):
    return torch.from_numpy((rng.standard_normal(shape) * scale + mean).astype(np.float32))


def f64(t):
    return t.detach().float().cpu().numpy().astype(np.float64)


# ---------------------------------------------------------------------------
# each mechanism alone
# ---------------------------------------------------------------------------
class _Layer:
    """A model of one layer, for driving its parts by hand through steps of one request."""

    def __init__(self, dtype, entry, width=64, tensors=None, page_size=8, eps=1e-5):
        from liyab_amd.config import config_from_dict
        from liyab_amd.engine import EngineCore
        from liyab_amd.weights.random_init import random_tensors

        self.raw = config(50, width, eps, [entry])
        cfg = config_from_dict(self.raw)
        t = random_tensors(cfg, 5)
        for k, v in (tensors or {}).items():
            assert k in t and tuple(t[k].shape) == tuple(v.shape), (k, tuple(v.shape))
            t[k] = v
        if dtype == "bfloat16":
            t = {k: (v.to(torch.bfloat16).float() if (v.dim() == 2 and not k.endswith(KEPT_32BIT)) else v) for k, v in t.items()}
        self.t = {k: f64(v) for k, v in t.items()}
        self.core = EngineCore.from_plan(cfg.plan(), t, dtype=dtype, page_size=page_size, num_pages=300, max_requests=3, use_graphs=False)
        for s in self.core.storage.states.values():
            s.fill_(float("nan"))
        for c in self.core.storage.layers.values():
            for rows in c.rows.values():
                rows.fill_(float("nan"))
        self.block = self.core.model.blocks[0]
        self.width, self.dtype, self.eps, self.entry = width, dtype, eps, entry

    def run(self, rid, rows, portions, fn):
        from liyab_amd.engine import StepItem

        out, done = [], 0
        for take in portions:
            item = StepItem(rid, [1] * take, [])
            ctx, lengths = self.core.step_fn.prepare([item])
            out.append(fn(ctx, rows[done:done + take].to(DEV)))
            self.core.step_fn.commit([item], lengths)
            done += take
        assert done == rows.shape[0]
        return np.concatenate(out)


def _mixer_alone(p, x, portions, rid="m"):
    """The layer's mixer over the rows x of one request, in portions."""
    core, mix = p.core, p.block.mixer
    core.open(rid)

    def step(ctx, xs):
        y = torch.empty(xs.shape[0], p.width, dtype=torch.float32, device=DEV)
        mix.forward(xs.to(core.dtype), ctx, core.storage.layer(0), core.storage.state(0), None, out=y)
        return f64(y)

    got = p.run(rid, x, portions, step)
    core.close(rid)
    core.manager.check()
    return got


def _inputs(p, rng, n, scale=1.0):
    x = rand(rng, n, p.width, scale=scale)
    return x, f64(x.to(torch.bfloat16).float() if p.dtype == "bfloat16" else x)


MIXER_TOL = {"float32": 2e-5, "bfloat16": 3e-2}
PORTIONS = ((75,), (25, 1, 9, 1, 1, 2, 36), (2,) * 10 + (1,) * 5 + (50,), (1,) * 75)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", [att(4, 2, 24, 16, mask=(20, 3), rot=(12, 10000.0, 4.0)), att(3, 3, 10, 6, mask=(9, 14), rot=(6, 777.0)), att(2, 1, 128, 48, mask=(33, 1), rot=(32, 2e4, 2.0)),
                               att(8, 4, 8, 8, rot=(8, 20.0)), att(1, 1, 64, 64, mask=(16, 16)), att(5, 1, 6, 10, mask=(38, 0), rot=(2, 3.0, 5.0)), att(6, 3, 80, 80, mask=(24, 8), rot=(40, 1e4))])
def test_attention_alone_in_portions(dtype, m):
    """Norms over the whole queries and keys, pairs turned under a divided frequency, grouped keys, keys and values of their own
    widths, a window with kept first positions, from portion to portion down to single tokens; a second request finds pages that
    were used before."""
    p = _Layer(dtype, layer("attention", m), width=72)
    rng = np.random.default_rng(3)
    for k, portions in enumerate(PORTIONS + ((130,), (100, 2, 90))):
        x, xs = _inputs(p, rng, sum(portions))
        pos = np.arange(len(xs), dtype=np.float64)
        want = plain.attention(xs, p.t, "l0.mix.", m, pos, p.eps, plain.keys_and_values(xs, p.t, "l0.mix.", m, pos, p.eps))
        got = _mixer_alone(p, x, portions, rid=f"a{k}")
        assert tt.rel_err(got, want) < MIXER_TOL[dtype], (m, portions[:4])


def _marked_layer(dtype, H, G, D, V, mask, width, page_size):
    """An attention layer whose queries and keys see two channels only: a row large in channel 0 has queries and keys along one
    entry of a head (behind the turned ones), a row large in channel 1 along another. Rows of the first kind attend to each other
    with nearly all their weight (the norms fix every query's and key's length, so only the direction can mark one)."""
    q, kk = torch.zeros(H * D, width), torch.zeros(G * D, width)
    for h in range(H):
        q[h * D + 12, 0] = q[h * D + 13, 1] = 1.0
    for g in range(G):
        kk[g * D + 12, 0] = kk[g * D + 13, 1] = 1.0
    m = att(H, G, D, V, mask=mask, rot=(8, 10000.0), scale=1.0)
    ones = {"l0.mix.q.norm": torch.ones(H * D), "l0.mix.k.norm": torch.ones(G * D)}
    return m, _Layer(dtype, layer("attention", m), width=width, tensors={"l0.mix.q": q, "l0.mix.k": kk, **ones}, page_size=page_size)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep,page_size", [(41, 5, 8), (41, 5, 16), (33, 70, 16), (100, 3, 16), (129, 0, 8), (150, 20, 64), (17, 130, 8)])
def test_a_marked_key_at_the_edges_of_the_window_and_of_the_kept_positions(dtype, window, keep, page_size):
    """One earlier row matches the last query and holds values of its own: just inside and just outside the window, the last of
    the kept first positions and the next one, at the very start, beside the query, on either side of pages' borders. Seen, it
    holds about half the query's weight; unseen, it changes nothing. In one prompt, in portions, and decoded token by token."""
    H, G, D, V, width, n = 4, 2, 16, 8, 48, 420
    m, p = _marked_layer(dtype, H, G, D, V, (window, keep), width, page_size)
    pos = np.arange(n, dtype=np.float64)
    last = n - 1
    places = {last - window + 1, last - window, keep, max(keep - 1, 0), 0, last - 1, last - window + 1 - page_size, 2 * page_size - 1, 2 * page_size, last - 2 * page_size}
    for case, j in enumerate(sorted(j for j in places if 0 <= j < last)):
        rng = np.random.default_rng(10 + case)
        x = rand(rng, n, width, scale=0.3)
        x[:, 0] *= 0.05
        x[:, 1] = 4.0
        blind = x.clone()
        for row in (j, last):
            x[row, 0], x[row, 1] = 4.0, 0.02
        blind[last, 0], blind[last, 1] = 4.0, 0.02
        x[j, 2:] *= 6.0
        rounded = (lambda a: f64(a.to(torch.bfloat16).float())) if dtype == "bfloat16" else f64
        xs, bs = rounded(x), rounded(blind)
        want = plain.attention(xs, p.t, "l0.mix.", m, pos, p.eps, plain.keys_and_values(xs, p.t, "l0.mix.", m, pos, p.eps))
        without = plain.attention(bs, p.t, "l0.mix.", m, pos, p.eps, plain.keys_and_values(bs, p.t, "l0.mix.", m, pos, p.eps))
        moved = np.abs(want[last] - without[last]).max() / np.abs(want).max()
        seen = last - j < window or j < keep
        assert (moved > 0.2) if seen else (moved < 1e-9), (j, seen, moved)
        for k, portions in enumerate(((n,), (n - 40,) + (1,) * 40, (100, 2, 150, 37, 2, n - 291))):
            got = _mixer_alone(p, x, portions, rid=f"k{case}_{k}")
            assert tt.rel_err(got, want) < (2e-5 if dtype == "float32" else 3e-2), (j, seen, portions[:3])


@pytest.mark.parametrize("dtype", DTYPES)
def test_keys_and_values_of_another_layer_are_found_behind_its_own_window(dtype, tmp_path):
    """Three layers read the first one's keys and values, under a window of their own, a longer one and none: the pages that the
    first layer's window has passed must still be there for them. The longer one's result differs from what the first layer's
    window would give; whole, in portions, token by token and mixed, in pools just large enough."""
    rot = (8, 100.0, 2.0)
    cfg = config(90, 48, 1e-5, [layer("attention", att(2, 1, 16, 8, mask=(9, 2), rot=rot)), layer("attention", att(4, 1, 16, 8, mask=(50, 5), rot=rot, kv_from=0), dense(32)),
                                layer("attention", att(2, 2, 8, 8, mask=(12, 1))), layer("attention", att(1, 1, 16, 8, rot=rot, kv_from=0)),
                                layer("attention", att(2, 2, 8, 8, mask=(30, 0), kv_from=2))])
    d = str(tmp_path / "m")
    raw, t = write_model(d, cfg, 3, dtype)
    reqs = {f"v{i}": tt.random_tokens(30 + i, n, 90) for i, n in enumerate([1, 40, 150])}
    ref = {rid: plain.forward(raw, t, toks) for rid, toks in reqs.items()}
    for changed in ((1, (9, 2)), (4, (12, 1))):
        other = json.loads(json.dumps(raw))
        other["layers"][changed[0]]["mixer"]["mask"] = {"size": changed[1][0], "keep_first": changed[1][1]}
        assert np.abs(plain.forward(other, t, reqs["v2"]) - ref["v2"]).max() > 0.05 * np.abs(ref["v2"]).max()
    for steps in (tt.schedule_whole(reqs), tt.schedule_bulk_tail(reqs, tail=60), tt.schedule_portions(reqs, (2, 5, 1, 9)), tt.schedule_mixed(reqs, seed=2, max_live=3)):
        core = make_core(d, dtype, None, page_size=8, max_requests=3, num_pages=tt.max_live_pages(steps, 8))
        check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lolulorn-shared {dtype}", family="lolulorn-shared")
        core.manager.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", [delta(4, 2, 16, 16, 4), delta(3, 3, 10, 6, 2), delta(2, 1, 33, 70, 1), delta(6, 2, 64, 128, 5), delta(1, 1, 128, 64, 3), delta(8, 1, 8, 12, 7),
                               delta(2, 2, 200, 20, 4), delta(1, 1, 96, 256, 2)])
def test_the_gated_delta_rule_alone_in_portions(dtype, m):
    """The state and the convolution's last inputs travel from portion to portion, down to single tokens, and through steps long
    enough for segments; a second request in a slot that was used before starts from zeros whatever the slot holds; one tap
    keeps no inputs."""
    p = _Layer(dtype, layer("delta", m), width=72)
    rng = np.random.default_rng(5)
    for k, portions in enumerate(PORTIONS + ((260,), (3, 255, 2))):
        x, xs = _inputs(p, rng, sum(portions))
        got = _mixer_alone(p, x, portions, rid=f"r{k}")
        assert tt.rel_err(got, plain.delta(xs, p.t, "l0.mix.", m, p.eps)) < MIXER_TOL[dtype], (m, portions[:4])


def test_the_delta_rule_replaces_what_its_key_holds_and_carries_a_token_far():
    """States that hardly decay carry one early token to the end of a long sequence, and a later token with the same key takes
    it out again: both change the last output by much. The engine follows the twin whole, in portions and token by token."""
    m, width, n = delta(2, 1, 24, 16, 1), 64, 400
    t = {"l0.mix.A_log": torch.full((2,), -9.0), "l0.mix.b": torch.zeros(2, width), "l0.mix.q.conv": torch.ones(24, 1), "l0.mix.k.conv": torch.ones(24, 1), "l0.mix.v.conv": torch.ones(32, 1)}
    t["l0.mix.b"][:, 0] = 8.0  # the rate is one where channel 0 is large, nearly nothing elsewhere
    p = _Layer("float32", layer("delta", m), width=width, tensors=t)
    rng = np.random.default_rng(6)
    x = rand(rng, n, width)
    x[:, 0] = -1.5
    x[5] = 3.0 * rand(rng, width)
    x[5, 0] = 2.0
    x[n - 1, 1:] = x[5, 1:]
    again = x.clone()
    again[200] = x[5] * 1.0
    again[200, 40:] = -2.0 * x[5, 40:]
    runs = []
    for rows in (x, again):
        xs = f64(rows)
        want = plain.delta(xs, p.t, "l0.mix.", m, p.eps)
        runs.append(want)
        for k, portions in enumerate(((n,), (n - 40,) + (1,) * 40, (100, 2, 150, 37, 2, 107, 2))):
            assert tt.rel_err(_mixer_alone(p, rows, portions, rid=f"f{k}"), want) < 2e-5
    blind = f64(x)
    blind[5] = f64(x)[6]
    scale_of = np.abs(runs[0]).max()
    assert np.abs(plain.delta(blind, p.t, "l0.mix.", m, p.eps)[-1] - runs[0][-1]).max() > 0.05 * scale_of
    assert np.abs(runs[1][-1] - runs[0][-1]).max() > 0.05 * scale_of


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", [gla(4, 24, 16, 8.0, 12), gla(3, 10, 6, 3.0, 5), gla(2, 64, 128, 16.0, 16), gla(1, 128, 64, 1.0, 1), gla(8, 8, 12, 5.0, 40), gla(1, 40, 256, 12.0, 8)])
def test_gated_linear_attention_alone_in_portions(dtype, m):
    """As for the delta rule: portions down to single tokens, steps long enough for segments, slots used again."""
    p = _Layer(dtype, layer("gla", m), width=72)
    rng = np.random.default_rng(7)
    for k, portions in enumerate(PORTIONS + ((260,), (3, 255, 2))):
        x, xs = _inputs(p, rng, sum(portions))
        got = _mixer_alone(p, x, portions, rid=f"g{k}")
        assert tt.rel_err(got, plain.gla(xs, p.t, "l0.mix.", m, p.eps)) < MIXER_TOL[dtype], (m, portions[:4])


def test_gated_linear_attention_carries_a_token_far():
    """Channels that hardly decay carry one early token to the end; channels whose decay's logit is very low forget at once."""
    m, width, n = gla(2, 16, 8, 16.0, 4), 64, 400
    bias = torch.full((32,), 9.0)
    bias[::2] = -700.0
    p = _Layer("float32", layer("gla", m), width=width, tensors={"l0.mix.a2.b": bias})
    rng = np.random.default_rng(8)
    x = rand(rng, n, width)
    x[3] *= 30.0
    xs = f64(x)
    want = plain.gla(xs, p.t, "l0.mix.", m, p.eps)
    blind = xs.copy()
    blind[3] = 0.0
    assert np.abs(plain.gla(blind, p.t, "l0.mix.", m, p.eps)[-1] - want[-1]).max() > 0.05 * np.abs(want[-1]).max()
    for k, portions in enumerate(((n,), (n - 40,) + (1,) * 40, (100, 2, 150, 37, 2, 107, 2))):
        assert tt.rel_err(_mixer_alone(p, x, portions, rid=f"f{k}"), want) < 2e-5


def _ffn_alone(p, x):
    from liyab_amd.engine import StepItem

    n = x.shape[0]
    ffn = p.block.ffn
    k = int(getattr(ffn, "rows_a_token", 1))
    y = torch.zeros(n * k, p.width, dtype=torch.float32, device=DEV)
    p.core.open("f")
    ctx, _ = p.core.step_fn.prepare([StepItem("f", [1] * n, [])])
    ffn.forward(x.to(DEV).to(p.core.dtype), ctx, None, out=y)
    p.core.close("f")
    return f64(y).reshape(n, k, p.width)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [96, 50, 200])
def test_the_gated_feed_forward_alone(dtype, ff):
    p = _Layer(dtype, layer("attention", att(1, 1, 8, 8), dense(ff)), width=72)
    for n, scale in ((1, 1.0), (37, 3.0), (150, 0.3)):
        x, xs = _inputs(p, np.random.default_rng(8 + n), n, scale=scale)
        want = plain.feed_forward(xs, p.t, "l0.mlp.", dense(ff))
        assert tt.rel_err(_ffn_alone(p, x)[:, 0], want) < MIXER_TOL[dtype]


def _choice(z, correction, top, groups):
    from liyab_amd.kernels import ops

    n, E = z.shape
    tiles = ops.moe_tiles(n * top, E, ops.GROUPED_ROWS)
    ids = torch.empty(n * top, dtype=torch.int32, device=DEV)
    w = torch.empty(n * top, dtype=torch.float32, device=DEV)
    rows = torch.empty(tiles * ops.GROUPED_ROWS, dtype=torch.int32, device=DEV)
    tile_group = torch.empty(tiles, dtype=torch.int32, device=DEV)
    ops.moe_route(z.to(DEV).contiguous(), top, ids, w, rows, tile_group, groups=groups, scores="logistic",
                  correction=correction.to(DEV) if correction is not None else None)
    listed = rows[rows >= 0].cpu().numpy()
    assert sorted(listed.tolist()) == list(range(n * top))  # every entry is listed once, in a tile of its expert
    for place in np.flatnonzero(rows.cpu().numpy() >= 0):
        assert int(tile_group[place // ops.GROUPED_ROWS]) == int(ids[int(rows[place])])
    return ids.cpu().numpy().reshape(n, top), f64(w).reshape(n, top)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", [moe(24, 8, 2, groups=(4, 2)), moe(13, 6, 3, groups=(3, 2)), moe(16, 6, 3), moe(20, 1, 1, groups=(1, 1)), moe(8, 4, 4, groups=(2, 2)),
                               moe(12, 12, 5, groups=(6, 3)), moe(48, 16, 5, groups=(4, 2)), moe(8, 8, 3, groups=(8, 5)), moe(8, 80, 6, groups=(5, 2))])
def test_experts_chosen_by_corrected_logistic_scores_alone(dtype, m):
    """Who is chosen, with which weight, and the experts' sum, for few rows (one workgroup, the small tiles) and many; the twin's
    router reads the same rounded rows, so the choice is compared in bfloat16 too."""
    p = _Layer(dtype, layer("attention", att(1, 1, 8, 8), m), width=72)
    r = m["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    for n in (1, 9, 64, 65, 300):
        x, xs = _inputs(p, np.random.default_rng(9 + n), n, scale=1.5)
        want = plain.routed_feed_forward(xs, p.t, "l0.mlp.", m)
        got = _ffn_alone(p, x)
        assert got.shape[1] == r["top"]
        assert tt.rel_err(got.sum(axis=1), want) < MIXER_TOL[dtype], (m, n)
        z = torch.from_numpy(xs @ p.t["l0.mlp.router"].T).float()
        ids, w = _choice(z, torch.from_numpy(p.t["l0.mlp.correction"]).float(), r["top"], (g["count"], g["keep"]))
        chosen, weights = plain.route(f64(z), p.t["l0.mlp.correction"], r["top"], g["count"], g["keep"])
        assert (ids == chosen).all()
        assert np.abs(w - weights).max() < 1e-6


def test_choices_worked_by_hand():
    """Choice scores below zero still beat what is not allowed; a group's score is the sum of its two largest, so a group with one
    large score loses to one with two good ones; the weights are the scores without the correction, not divided by anything."""
    logit = lambda s: np.log(s / (1.0 - s))  # noqa: E731
    s = np.array([[0.9, 0.1, 0.1, 0.1, 0.6, 0.55, 0.1, 0.1]])
    z = torch.from_numpy(logit(s)).float()
    ids, w = _choice(z, None, 2, (2, 1))
    assert ids.tolist() == [[4, 5]] and np.abs(w - [[0.6, 0.55]]).max() < 1e-6
    # every allowed choice score is negative, and the kept group's third is chosen before any of the other group
    correction = torch.tensor([-1.2, -1.5, -3.0, -3.5, -4.0, -4.0, -4.0, -4.0])
    ids, w = _choice(z, correction, 3, (2, 1))
    assert ids.tolist() == [[0, 1, 2]] and np.abs(w - [[0.9, 0.1, 0.1]]).max() < 1e-6
    # the correction decides the choice alone
    ids, w = _choice(z, torch.tensor([0.0, 0.0, 0.0, 5.0, 0.0, 0.0, 0.0, 5.0]), 2, (1, 1))
    assert sorted(ids[0].tolist()) == [3, 7] and np.abs(w - 0.1).max() < 1e-6
    # equal scores: the lower number first
    ids, _ = _choice(torch.zeros(70, 6), None, 3, (3, 2))
    assert (ids == [0, 1, 2]).all()


@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("d,n_sum", [(72, 1), (96, 3), (1000, 2), (2048, 1), (2300, 2)])
def test_a_layer_norm_behind_a_sublayer(out_dtype, d, n_sum):
    """The rows' update with the mean taken off: rows whose mean is far larger than their spread, several rows a token, widths
    that a thread's registers hold and not."""
    from liyab_amd.kernels import ops

    rng = np.random.default_rng(d)
    n = 5
    x, y = rand(rng, n, d), rand(rng, n * n_sum, d, mean=3.0)
    y[0] += 40.0
    w, b = rand(rng, d, scale=0.2, mean=1.0), rand(rng, d, scale=0.5)
    s = f64(y).reshape(n, n_sum, d).sum(axis=1)
    want = f64(x) + plain.centred_norm(s, f64(w), f64(b), 1e-5)
    xd, cast = x.to(DEV), torch.empty(n, d, dtype=out_dtype, device=DEV)
    ops.gated_norm_add(xd, y.to(DEV), w.to(DEV), 1e-5, n_sum=n_sum, bias=b.to(DEV), centred=True, cast_out=cast)
    assert tt.rel_err(f64(xd), want) < 1e-5
    assert torch.equal(cast, xd.to(out_dtype))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_rows_of_no_request_write_no_keys(dtype):
    """Slot -1 (padding rows) leaves the pages alone; turned halves, the other layout of the pairs; rows wider than the heads."""
    from liyab_amd.kernels import ops

    rng = np.random.default_rng(1)
    H, G, D, V, P, n, page = 4, 2, 10, 6, 16, 3, 4
    src = rand(rng, n, H * D + G * D + G * V)
    qn, kn = rand(rng, H * D, mean=1.0), rand(rng, G * D, mean=1.0)
    freqs = torch.tensor([1.0, 0.25, 0.0625], dtype=torch.float64)
    q = torch.empty(n, H * P, dtype=dtype, device=DEV)
    kc, vc = (torch.full((2, G, page, P), 7.0, dtype=dtype, device=DEV) for _ in range(2))
    slots = torch.tensor([5, -1, 2], dtype=torch.int32, device=DEV)
    positions = torch.tensor([9, 0, 3], dtype=torch.int32, device=DEV)
    for halves in (False, True):
        kc.fill_(7.0)
        vc.fill_(7.0)
        ops.qk_prepare_rows(src.to(DEV), q, kc, vc, slots, positions, q_off=0, k_off=H * D, v_off=H * D + G * D, n_head=H, n_kv_head=G, head_dim=D, value_dim=V,
                            q_norm=qn.to(DEV), k_norm=kn.to(DEV), eps=1e-5, freqs=freqs.to(DEV), rot_dims=6, rot_halves=halves)
        s = f64(src)
        for at, heads, norm in ((0, H, qn), (H * D, G, kn)):
            want = (plain.unit(s[:, at:at + heads * D], 1e-5) * f64(norm)).reshape(n, heads, D)
            a = f64(positions)[:, None] * f64(freqs)[None, :]
            c, sn = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
            one, two = (slice(0, 3), slice(3, 6)) if halves else (slice(0, 6, 2), slice(1, 6, 2))
            u, v = want[..., one].copy(), want[..., two].copy()
            want[..., one], want[..., two] = u * c - v * sn, v * c + u * sn
            if at == 0:
                got = f64(q).reshape(n, H, P)
                assert np.abs(got[..., :D] - want).max() < (1e-5 if dtype == torch.float32 else 2e-2) and np.abs(got[..., D:]).max() == 0.0
            else:
                for t, slot in ((0, 5), (2, 2)):
                    got = f64(kc)[slot // page, :, slot % page]
                    assert np.abs(got[:, :D] - want[t]).max() < (1e-5 if dtype == torch.float32 else 2e-2) and np.abs(got[:, D:]).max() == 0.0
        kept = f64(kc).copy()
        for slot in (5, 2):
            kept[slot // page, :, slot % page] = 7.0
        assert (kept == 7.0).all()
        assert (f64(vc)[1, :, 1, V:] == 0.0).all() and (f64(vc)[0, :, 0] == 7.0).all()
    before = q.clone()
    ops.qk_prepare_rows(src[:, :H * D].contiguous().to(DEV), q, None, None, slots, positions, q_off=0, k_off=0, v_off=0, n_head=H, n_kv_head=G, head_dim=D, value_dim=V,
                        q_norm=qn.to(DEV), k_norm=None, eps=1e-5, freqs=freqs.to(DEV), rot_dims=6, rot_halves=True)
    assert torch.equal(before, q)


# ---------------------------------------------------------------------------
# whole models
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_each_request_alone_and_whole_and_every_layer(name, dtype, models, reference):
    reqs = make_requests(name)
    steps = tt.schedule_whole(reqs)
    core = make_core(models[(name, dtype)][0], dtype, tt.max_live_tokens(steps))
    got = tt.run_schedule(core, steps)
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lolulorn-whole {name} {dtype}")
    core.manager.check()
    assert not core.manager.groups or core.manager.pages_in_use() == 0
    if dtype == "float32":
        from liyab_amd.engine import StepItem

        rid, toks = list(reqs.items())[2]
        streams, caught = [], []
        plain.forward(models[(name, dtype)][1], models[(name, dtype)][2], toks, streams)
        plain_core = make_core(models[(name, dtype)][0], dtype, 512, use_graphs=False)
        plain_core.model.replay_layers = False
        for block in plain_core.model.blocks:
            def wrapped(x, ctx, cache, state, writes_cache=True, _f=block.forward):
                out = _f(x, ctx, cache, state, writes_cache=writes_cache)
                caught.append(f64(x)[:len(toks)])
                return out
            block.forward = wrapped
        plain_core.open(rid)
        plain_core.step([StepItem(rid, toks, [])])
        assert len(caught) == len(streams) == len(models[(name, dtype)][1]["layers"])
        for got_x, want_x in zip(caught, streams):
            assert tt.rel_err(got_x, want_x) < 1e-5


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_a_prompt_then_its_last_tokens_one_by_one(name, dtype, models, reference):
    reqs = make_requests(name)
    steps = tt.schedule_bulk_tail(reqs, tail=45)
    core = make_core(models[(name, dtype)][0], dtype, tt.max_live_tokens(steps))
    got = tt.run_schedule(core, steps)
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lolulorn-decode {name} {dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(5, 2, 17, 3, 48, 2, 31, 7), (2, 2, 2, 3), (1, 64, 1, 16, 2)])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_portions_of_changing_size(name, dtype, sizes, models, reference):
    reqs = make_requests(name)
    if sizes[0] == 2:
        reqs = dict(list(reqs.items())[:3])
    steps = tt.schedule_portions(reqs, sizes)
    core = make_core(models[(name, dtype)][0], dtype, tt.max_live_tokens(steps), page_size=8 if sizes[0] == 1 else 16)
    got = tt.run_schedule(core, steps)
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lolulorn-portions {name} {dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed,max_live,page_size", [(0, 4, 16), (1, 3, 8), (2, 2, 24)])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype, seed, max_live, page_size, models, reference):
    """Up to `max_live` requests at a time, portions of some beside single tokens of others, in a pool and with state slots
    just large enough: what a finished request gives back is used by the next."""
    base = make_requests(name)
    reqs = {f"{rid}#{k}": toks for k in range(2) for rid, toks in base.items()}
    ref = {f"{rid}#{k}": reference[(name, dtype)][rid] for k in range(2) for rid in base}
    steps = tt.schedule_mixed(reqs, seed=seed, max_live=max_live)
    core = make_core(models[(name, dtype)][0], dtype, None, page_size=page_size, max_requests=max_live, num_pages=tt.max_live_pages(steps, page_size))
    got = tt.run_schedule(core, steps)
    check_logits(got, reqs, ref, dtype, f"lolulorn-mixed {name} {dtype}")
    core.manager.check()
    assert not core.manager.groups or core.manager.pages_in_use() == 0
    assert core.step_fn.graph_replays > 0  # the decode-only steps of the tail were replayed from graphs


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mix", "recurrent"])
def test_long_decoding_from_the_first_token(name, dtype, models, reference):
    rid, toks = list(make_requests(name).items())[-1]
    reqs = {rid: toks}
    steps = tt.schedule_bulk_tail(reqs, tail=len(toks))
    core = make_core(models[(name, dtype)][0], dtype, tt.max_live_tokens(steps))
    got = tt.run_schedule(core, steps)
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lolulorn-long {name} {dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_trace_program(dtype, models, reference, tmp_path):
    name = "odd"
    reqs = make_requests(name)
    steps = tt.schedule_mixed(reqs, seed=5, max_live=4)
    got = tt.run_trace_program(models[(name, dtype)][0], dtype, steps, str(tmp_path), tt.max_live_tokens(steps), CONFIGS[name][0]["vocab"])
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lolulorn-trace {dtype}")


def draw_config(seed):
    """A geometry drawn from the seed: every size, constant and count, the layers' kinds and order, who reads whose keys."""
    rng = np.random.default_rng(4000 + seed)
    pick = lambda *options: options[int(rng.integers(len(options)))]  # noqa: E731
    width = pick(40, 48, 64, 96, 104, 160)

    def feed_forward():
        kind = pick(None, "dense", "moe", "moe")
        if kind == "dense":
            return dense(pick(8, 20, 24, 40, 56))
        if kind == "moe":
            count = pick(1, 2, 3, 4)
            per = pick(1, 2, 3, 4)
            keep = int(rng.integers(1, count + 1))
            return moe(pick(8, 12, 24), count * per, int(rng.integers(1, keep * per + 1)), groups=pick(None, (1, 1)) if count == 1 else (count, keep))
        return None

    def mask():
        return pick(None, (int(rng.integers(1, 120)), pick(0, 1, 3, 19, 50)))

    layers, owners = [], []
    for i in range(int(rng.integers(2, 7))):
        kind = pick("attention", "attention", "delta", "gla")
        if kind == "attention":
            if owners and rng.random() < 0.5:
                j = owners[int(rng.integers(len(owners)))]
                of = layers[j]["mixer"]
                m = dict(of, heads=of["kv_heads"] * pick(1, 2, 4), kv_from=j)
                m.pop("mask", None)
                own = mask()
                if own:
                    m["mask"] = {"size": own[0], "keep_first": own[1]}
            else:
                kv, dim = pick(1, 2, 3), pick(4, 8, 10, 16, 24, 32)
                dims = 2 * int(rng.integers(1, dim // 2 + 1))
                rot = pick(None, (dims, pick(10.0, 500.0, 5e5)), (dims, pick(10.0, 10000.0), pick(1.5, 2.0, 8.0)))
                m = att(kv * pick(1, 2, 4), kv, dim, pick(dim, dim, 4, 12, 40), mask=mask(), rot=rot, scale=pick(None, 0.3, 1.0 if dim <= 8 else 0.4))
                owners.append(i)
        elif kind == "delta":
            kv = pick(1, 2, 3)
            m = delta(kv * pick(1, 2, 3), kv, pick(4, 8, 10, 16, 36), pick(4, 8, 12, 33, 72), pick(1, 2, 3, 4, 6))
        else:
            m = gla(pick(1, 2, 3, 4), pick(4, 8, 10, 16, 36), pick(4, 8, 12, 33, 72), pick(1.0, 4.0, 20.0), pick(1, 4, 16, 20))
        layers.append(layer(kind, m, feed_forward()))
    return config(pick(97, 256, 500), width, pick(1e-5, 1e-6, 1e-3), layers, scale=pick(2.0, 5.0, 12.0)), pick(8, 16, 24)


# (seeds whose rows do not magnify: half a unit in the last place of a 32-bit number, put on every sublayer's input in the twin, moves no
# logit by more than 1e-6 of its row's largest)
@pytest.mark.parametrize("seed", [0, 1, 4, 5, 6, 8, 9, 10, 11, 12, 14, 15, 16, 19, 20, 21])
def test_drawn_geometries_whole_and_mixed(seed, tmp_path):
    cfg, page_size = draw_config(seed)
    reqs = {f"g{i}": tt.random_tokens(seed * 10 + i, n, cfg["vocab"]) for i, n in enumerate([1, 19, 77, 150, 260])}
    for dtype in DTYPES:
        d = str(tmp_path / f"m_{dtype}")
        raw, t = write_model(d, cfg, 100 + seed, dtype)
        ref = {rid: plain.forward(raw, t, toks) for rid, toks in reqs.items()}
        steps = tt.schedule_whole(reqs)
        core = make_core(d, dtype, tt.max_live_tokens(steps), page_size=page_size)
        check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lolulorn-drawn seed {seed} whole {dtype}", family="lolulorn-drawn", tol=TOL_DRAWN)
        steps = tt.schedule_mixed(reqs, seed=seed, max_live=3)
        core = make_core(d, dtype, None, page_size=page_size, max_requests=3, num_pages=tt.max_live_pages(steps, page_size))
        check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lolulorn-drawn seed {seed} mixed {dtype}", family="lolulorn-drawn", tol=TOL_DRAWN)
        core.manager.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_real_widths_in_long_steps(dtype, tmp_path):
    """Heads of 64 and 128, a width of 512, prompts of hundreds of tokens in one step and in mixed batches: the tiles of the large
    products, the matrix-core attention that jumps from the kept positions to the window, recurrences in segments, the experts'
    large tiles, the choice a wave a token."""
    cfg = config(1000, 512, 1e-5, [
        layer("delta", delta(8, 4, 64, 128, 4), moe(128, 16, 4, groups=(4, 2))),
        layer("attention", att(8, 2, 64, 64, mask=(128, 6), rot=(32, 10000.0, 4.0)), dense(1024)),
        layer("gla", gla(4, 128, 64, 16.0, 32), moe(64, 8, 2)),
        layer("attention", att(4, 2, 128, 128, mask=(200, 150), rot=(64, 5e5)), dense(768)),
        layer("attention", att(16, 2, 64, 64, mask=(256, 3), rot=(32, 10000.0, 4.0), kv_from=1), moe(96, 6, 2, groups=(3, 2))),
    ], scale=3.0)
    d = str(tmp_path / "m")
    raw, t = write_model(d, cfg, 31, dtype)
    reqs = {f"r{i}": tt.random_tokens(900 + i, n, raw["vocab"]) for i, n in enumerate([330, 700, 45])}
    ref = {rid: plain.forward(raw, t, toks) for rid, toks in reqs.items()}
    steps = tt.schedule_whole(reqs)
    core = make_core(d, dtype, tt.max_live_tokens(steps))
    check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lolulorn-wide whole {dtype}", family="lolulorn-wide")
    steps = tt.schedule_mixed(reqs, seed=3, max_live=3, portions=(2, 130, 64, 300, 17))
    core = make_core(d, dtype, None, max_requests=3, num_pages=tt.max_live_pages(steps, 16))
    check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lolulorn-wide mixed {dtype}", family="lolulorn-wide")
    core.manager.check()


def generate_greedy(raw, t, prompt, n_new):
    toks = list(prompt)
    for _ in range(n_new):
        toks.append(int(np.argmax(plain.forward(raw, t, toks)[-1])))
    return toks[len(prompt):]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mix", "odd"])
def test_greedy_generation_through_the_entry_point(name, dtype, models):
    """Engine.generate: the scheduler batches the prompts in portions beside decoding requests, in a pool that does not hold
    them all at once (requests are preempted and computed again, their slots' state starting over); each token is the twin's
    greedy choice given the tokens so far."""
    from liyab_amd import Engine, SamplingParams

    d, raw, t = models[(name, dtype)]
    prompts = [tt.random_tokens(70 + i, n, raw["vocab"]) for i, n in enumerate([1, 13, 64, 100, 7])]
    n_new = 12
    engine = Engine(d, dtype=dtype, page_size=16, num_pages=14, max_num_seqs=3, max_batched_tokens=48, prefill_chunk=24)
    engine.stop_at_eos = False
    results = engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=n_new))
    for prompt, res in zip(prompts, results):
        assert len(res.tokens) == n_new
        ref = plain.forward(raw, t, prompt + res.tokens[:-1])
        for i, tok in enumerate(res.tokens):
            row = ref[len(prompt) - 1 + i]
            slack = (1e-5 if dtype == "float32" else 5e-2) * np.abs(row).max()
            assert row[tok] >= row.max() - slack, f"token {i} of prompt length {len(prompt)}: {tok} vs {int(np.argmax(row))}"
        if dtype == "float32":
            assert res.tokens == generate_greedy(raw, t, prompt, n_new)
    engine.core.manager.check()


def test_command_line(models):
    d, raw, tensors = models[("mix", "float32")]
    prompt = tt.random_tokens(90, 11, raw["vocab"])
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "liyab-cli"), "-m", d, "-p", ",".join(map(str, prompt)), "-n", "6",
                        "--temp", "0", "--dtype", "float32", "--json", "--phases"], capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    turn = [json.loads(l) for l in p.stdout.splitlines() if l.startswith("{")][1]
    assert turn["tokens"] == generate_greedy(raw, tensors, prompt, 6)
    assert set(turn["phases_ms"]) == {"embed", "scored_attention", "gated_delta", "gated_linear_attention", "routed_ffn", "gated_ffn", "lm_head"}
