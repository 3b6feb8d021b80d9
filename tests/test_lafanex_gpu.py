"""Lafanex through the engine against its plain twin (`plain_lafanex.py`): each mechanism alone, then whole models of
several geometries under every way of cutting and batching the work, in 32-bit and in bfloat16 (needs the GPU). The
geometries differ from each other in every size and in the order of their layers; one has sizes no kernel tiles evenly,
one nothing but recurrences (no cache at all), one nothing but attention, one a single plain stream, one the values that other geometries
happen to share or make one (one stream, one head, one tap, one state, one expert, a loop run once)."""

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_lafanex as plain
import trace_tools as tt
from conftest import ROOT, TOL
from plain_gpt2 import read_model

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
# float32: the largest difference of a row relative to its largest |logit|, as for the other models.
# bfloat16, against the twin in float64 with the same rounded matrices: the root mean square of a row's difference over
# that of the row's logits, both with their means taken off; a fault in a mechanism makes it about 1.
TOL_B = {"float32": TOL["float32"], "bfloat16": 3e-2}
TOL_DRAWN = 1e-1
KEPT_32BIT = (".conv", ".A_log", ".hc1.mix", ".hc2.mix")  # 2-D tensors that the engine keeps in 32 bits


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
def att(heads, kv_heads, dim, vdim, rot=None, scale=None):
    """rot = (dims, base)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5}
    if rot:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
    return m


def scan(inner, state, dt_rank, conv):
    return {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, limit, experts, top, identity=0, scale=1.0, shared=None):
    """shared = (ff, limit)."""
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top, "identity": identity, "scale": scale}}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def layer(kind, m, mlp=None):
    return {"type": kind, "mixer": m, "mlp": mlp}


def config(vocab, width, eps, layers, streams=None, loop=None):
    out = {"architecture": "Lafanex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if streams:
        out["streams"] = streams
    if loop:
        out["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return out


CONFIGS = {
    # every kind of layer and feed-forward; the middle layers three times over; a shared expert of the experts' own form and one of another
    "mix": (config(300, 96, 1e-5, [
        layer("mamba1", scan(72, 12, 6, 3), moe(24, 1.2, 8, 3, identity=3, scale=2.0, shared=(24, 1.2))),
        layer("attention", att(6, 2, 24, 16, rot=(12, 10000.0)), dense(80)),
        layer("mamba1", scan(128, 9, 4, 4), None),
        layer("attention", att(4, 1, 16, 24, rot=(16, 500.0), scale=0.6), moe(32, 2.0, 5, 2, identity=1, scale=1.5, shared=(40, 0.8))),
        layer("mamba1", scan(64, 16, 8, 2), dense(64)),
    ], streams=3, loop=(1, 3, 3)), 61),
    # sizes that no kernel tiles evenly; two taps; more choices than experts with tensors
    "odd": (config(211, 100, 1e-6, [
        layer("attention", att(3, 3, 10, 6, rot=(6, 777.0)), moe(13, 0.7, 5, 4, identity=2, scale=0.8, shared=(13, 0.7))),
        layer("mamba1", scan(37, 5, 3, 2), moe(9, 3.0, 3, 4, identity=4, scale=3.0)),
        layer("attention", att(5, 1, 6, 10, rot=(2, 30.0)), None),
        layer("mamba1", scan(50, 27, 11, 6), dense(30)),
    ], streams=2, loop=(0, 2, 2)), 72),
    # recurrences only: no cache at all; one tap (no history), many states, one state
    "recurrent": (config(128, 64, 1e-5, [
        layer("mamba1", scan(160, 16, 4, 1), moe(32, 1.0, 4, 1, identity=1, shared=(24, 1.0))),
        layer("mamba1", scan(64, 40, 24, 4), None),
        layer("mamba1", scan(100, 1, 1, 5), dense(40)),
    ], streams=4), 63),
    # attention only (no state at all): heads of 64 and 128, values wider and narrower than keys, no turn, the last layer twice over
    "keys": (config(150, 64, 1e-5, [
        layer("attention", att(1, 1, 64, 64, rot=(64, 10000.0)), dense(48)),
        layer("attention", att(2, 1, 128, 8, rot=(32, 1e6)), None),
        layer("attention", att(8, 4, 8, 24), moe(16, 1.5, 4, 4, scale=0.5)),
        layer("attention", att(4, 2, 32, 32, rot=(4, 20.0), scale=0.4), moe(16, 1.5, 4, 2, identity=4, shared=(16, 1.5))),
    ], streams=2, loop=(3, 4, 2)), 64),
    # one plain stream
    "plain": (config(170, 80, 1e-4, [
        layer("attention", att(4, 2, 16, 16, rot=(8, 100.0)), moe(24, 1.0, 6, 2, identity=2, scale=1.7, shared=(16, 2.5))),
        layer("mamba1", scan(96, 8, 5, 4), dense(56)),
    ], loop=(0, 2, 2)), 65),
    # what other geometries share or make one
    "ones": (config(128, 72, 1e-5, [
        layer("attention", att(1, 1, 16, 16, rot=(16, 100.0)), moe(24, 1.0, 1, 1, scale=1.0)),
        layer("mamba1", scan(72, 1, 1, 1), moe(16, 1.0, 1, 2, identity=1, shared=(16, 1.0))),
        layer("attention", att(2, 1, 8, 8, rot=(8, 1.0), scale=1.0), dense(24)),
    ], streams=1, loop=(1, 2, 1)), 66),
}
LENGTHS = {"mix": [1, 2, 23, 70, 131, 260], "odd": [3, 40, 97, 200], "recurrent": [1, 50, 140, 230], "keys": [2, 65, 150, 300], "plain": [2, 33, 90, 170], "ones": [4, 5, 66, 150]}


def weigh_all(cfg):
    """The same model with routers that weigh every output: in bfloat16 a rounding ahead of a router whose candidates lie a
    rounding apart takes another expert than the twin, and the row then differs by far more than any rounding. The choice
    itself is compared in 32-bit throughout, and in bfloat16 where the router is run alone."""
    cfg = json.loads(json.dumps(cfg))
    for entry in cfg["layers"]:
        mlp = entry["mlp"]
        if mlp is not None and mlp["kind"] == "moe":
            mlp["router"]["top"] = mlp["router"]["experts"] + mlp["router"]["identity"]
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
            d = str(tmp_path_factory.mktemp(f"lafanex_{name}_{dtype}"))
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

        self.raw = config(50, width, eps, [entry], streams=2)
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
@pytest.mark.parametrize("m", [att(4, 2, 24, 16, rot=(12, 10000.0)), att(3, 3, 10, 6, rot=(6, 777.0)), att(2, 1, 128, 48, rot=(32, 2e4)), att(8, 4, 8, 8, rot=(8, 20.0)),
                               att(1, 1, 64, 64, rot=(64, 1e6), scale=0.3), att(5, 1, 6, 10, rot=(2, 3.0)), att(6, 3, 80, 96)])
def test_attention_alone_in_portions(dtype, m):
    """Turned pairs and unit heads without weights, one in the softmax's denominator, grouped keys, keys and values of their own
    widths, from portion to portion down to single tokens; a second request finds pages that were used before."""
    p = _Layer(dtype, layer("attention", m), width=72)
    rng = np.random.default_rng(3)
    for k, portions in enumerate(PORTIONS + ((130,), (100, 2, 90))):
        x, xs = _inputs(p, rng, sum(portions))
        want = plain.attention(xs, p.t, "l0.mix.", m, np.arange(len(xs), dtype=np.float64), p.eps)
        got = _mixer_alone(p, x, portions, rid=f"a{k}")
        assert tt.rel_err(got, want) < MIXER_TOL[dtype], (m, portions[:4])


def _marked_layer(dtype, H, G, D, V, width, page_size, scale=1.0):
    """An attention layer whose queries and keys see two channels only: a row large in channel 0 has queries and keys along one
    entry of a head (behind the turned ones), a row large in channel 1 along another, so that rows of the first kind attend to each other
    with nearly all their weight (a head's length is fixed, only its direction can mark one)."""
    q, kk = torch.zeros(H * D, width), torch.zeros(G * D, width)
    for h in range(H):
        q[h * D + 12, 0] = q[h * D + 13, 1] = 1.0
    for g in range(G):
        kk[g * D + 12, 0] = kk[g * D + 13, 1] = 1.0
    m = att(H, G, D, V, rot=(8, 10000.0), scale=scale)
    return m, _Layer(dtype, layer("attention", m), width=width, tensors={"l0.mix.q": q, "l0.mix.k": kk}, page_size=page_size)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page_size", [8, 16, 64])
def test_a_marked_key_far_away_and_at_the_pages_borders(dtype, page_size):
    """One earlier row matches the last query and holds values of its own: at the very start, on either side of pages' borders, far
    back, beside the query. In one prompt, in portions, and decoded token by token."""
    H, G, D, V, width, n = 4, 2, 16, 8, 48, 420
    m, p = _marked_layer(dtype, H, G, D, V, width, page_size)
    pos = np.arange(n, dtype=np.float64)
    last = n - 1
    places = {0, 1, page_size - 1, page_size, 2 * page_size - 1, 2 * page_size, last - 1, last - page_size, (last // page_size) * page_size - 1, (last // page_size) * page_size, 200}
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
        want = plain.attention(rounded(x), p.t, "l0.mix.", m, pos, p.eps)
        without = plain.attention(rounded(blind), p.t, "l0.mix.", m, pos, p.eps)
        assert np.abs(want[last] - without[last]).max() / np.abs(want).max() > 0.2, j
        for k, portions in enumerate(((n,), (n - 40,) + (1,) * 40, (100, 2, 150, 37, 2, n - 291))):
            got = _mixer_alone(p, x, portions, rid=f"k{case}_{k}")
            assert tt.rel_err(got, want) < (2e-5 if dtype == "float32" else 3e-2), (j, portions[:3])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D", [(4, 2, 16), (2, 2, 64), (2, 1, 128)])
def test_one_in_the_softmaxs_denominator(dtype, H, G, D):
    """Queries that no key matches: every score is far below zero, the one in the denominator takes nearly all the weight and the
    result all but vanishes, where a softmax without it would give a mean of the values. Beside queries whose scores are around zero."""
    width, V, n = 48, 16, 150
    q, kk = torch.zeros(H * D, width), torch.zeros(G * D, width)
    for h in range(H):
        q[h * D + D - 1, 0] = 1.0
    for g in range(G):
        kk[g * D + D - 1, 1] = 1.0
    m = att(H, G, D, V, rot=(D // 2, 1000.0), scale=6.0 / D)
    p = _Layer(dtype, layer("attention", m), width=width, tensors={"l0.mix.q": q, "l0.mix.k": kk}, page_size=16)
    rng = np.random.default_rng(4)
    x = rand(rng, n, width)
    x[:, 0], x[:, 1] = 2.0, -2.0  # score -6 at every key
    x[40:60, 0] = 0.0  # queries of length zero: scores of zero
    xs = f64(x.to(torch.bfloat16).float() if dtype == "bfloat16" else x)
    want = plain.attention(xs, p.t, "l0.mix.", m, np.arange(n, dtype=np.float64), p.eps)
    assert np.abs(want[:30]).max() < 0.1 * np.abs(want[40:60]).max()
    for k, portions in enumerate(((n,), (70, 2, 38) + (1,) * 40, (1,) * n)):
        got = _mixer_alone(p, x, portions, rid=f"s{k}")
        assert np.abs(got - want).max() < (2e-5 if dtype == "float32" else 3e-2) * np.abs(want).max()
        # a vanishing row is right by itself, not only beside the large ones
        assert np.abs(got[:10] - want[:10]).max() < (2e-4 if dtype == "float32" else 6e-2) * np.abs(want[:10]).max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", [scan(96, 16, 6, 4), scan(37, 5, 3, 2), scan(64, 1, 1, 1), scan(130, 24, 16, 3), scan(200, 40, 9, 5), scan(72, 100, 40, 4), scan(320, 8, 24, 7)])
def test_the_selective_scan_alone_in_portions(dtype, m):
    """The states and the convolution's last inputs travel from portion to portion, down to single tokens, and through steps long
    enough for segments; a second request in a slot that was used before starts from zeros whatever the slot holds; one tap
    keeps no inputs."""
    p = _Layer(dtype, layer("mamba1", m), width=72)
    rng = np.random.default_rng(5)
    for k, portions in enumerate(PORTIONS + ((260,), (3, 255, 2), (47, 48, 49, 33, 32, 31))):
        x, xs = _inputs(p, rng, sum(portions))
        got = _mixer_alone(p, x, portions, rid=f"r{k}")
        assert tt.rel_err(got, plain.mamba1(xs, p.t, "l0.mix.", m)) < MIXER_TOL[dtype], (m, portions[:4])


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_requests_of_a_step_walk_their_own_states(dtype):
    """Requests of very different portions in one step (a step in segments holds portions of one segment, of several and of a single
    token): each one's rows are those of its own sequence."""
    from liyab_amd.engine import StepItem

    m = scan(96, 12, 6, 4)
    p = _Layer(dtype, layer("mamba1", m), width=72)
    core, mix = p.core, p.block.mixer
    rng = np.random.default_rng(6)
    takes = {"a": (1, 130, 2, 64), "b": (70, 1, 2, 1), "c": (33, 64, 2, 200)}
    rows = {rid: _inputs(p, rng, sum(t)) for rid, t in takes.items()}
    got = {rid: [] for rid in takes}
    for rid in takes:
        core.open(rid)
    done = dict.fromkeys(takes, 0)
    for k in range(4):
        order = [r for r in (("a", "b", "c"), ("c", "a", "b"), ("b", "c", "a"), ("a", "c", "b"))[k]]
        items = [StepItem(rid, [1] * takes[rid][k], []) for rid in order]
        ctx, lengths = core.step_fn.prepare(items)
        x = torch.cat([rows[rid][0][done[rid]:done[rid] + takes[rid][k]] for rid in order]).to(DEV).to(core.dtype)
        y = torch.empty(x.shape[0], p.width, dtype=torch.float32, device=DEV)
        mix.forward(x, ctx, None, core.storage.state(0), None, out=y)
        core.step_fn.commit(items, lengths)
        at = 0
        for rid in order:
            got[rid].append(f64(y[at:at + takes[rid][k]]))
            at += takes[rid][k]
            done[rid] += takes[rid][k]
    for rid in takes:
        assert tt.rel_err(np.concatenate(got[rid]), plain.mamba1(rows[rid][1], p.t, "l0.mix.", m)) < MIXER_TOL[dtype], rid


def test_the_selective_scan_carries_a_token_far_and_forgets_at_once():
    """States that hardly decay carry one early token to the end of a long sequence; where the step size is large at one token, what
    was before is gone. Whole, in portions and token by token."""
    m, width, n = scan(64, 8, 4, 2), 64, 600
    t = {"l0.mix.A_log": torch.full((64, 8), -7.0), "l0.mix.dt.b": torch.full((64,), -1.0)}
    p = _Layer("float32", layer("mamba1", m), width=width, tensors=t)
    rng = np.random.default_rng(7)
    x = rand(rng, n, width)
    x[5] *= 30.0
    want = plain.mamba1(f64(x), p.t, "l0.mix.", m)
    blind = f64(x)
    blind[5] = 0.0
    assert np.abs(plain.mamba1(blind, p.t, "l0.mix.", m)[-1] - want[-1]).max() > 0.05 * np.abs(want[-1]).max()
    for k, portions in enumerate(((n,), (n - 40,) + (1,) * 40, (100, 2, 150, 37, 2, 107, 202), (1,) * n)):
        assert tt.rel_err(_mixer_alone(p, x, portions, rid=f"f{k}"), want) < 2e-5
    fast = _Layer("float32", layer("mamba1", m), width=width, tensors={"l0.mix.A_log": torch.full((64, 8), 5.0), "l0.mix.dt.b": torch.full((64,), 4.0)})
    x = rand(rng, n, width)
    want = plain.mamba1(f64(x), fast.t, "l0.mix.", m)
    for k, portions in enumerate(((n,), (300, 2, 298))):
        assert tt.rel_err(_mixer_alone(fast, x, portions, rid=f"q{k}"), want) < 2e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,C,rank", [(1, 37, 3), (33, 64, 16), (130, 100, 5), (200, 96, 48), (65, 31, 8), (70, 50, 100)])
def test_step_sizes_keep_their_digits(dtype, n, C, rank):
    """softplus of the product with unrounded rows, down to step sizes a millionth of one: relative to each one's own size."""
    from liyab_amd.kernels import lib

    rng = np.random.default_rng(n)
    ldw = -(-rank // 8) * 8
    low = rand(rng, n, ldw + 4).to(DEV)
    low[:, rank:] = float("nan")  # (what lies behind the rank is not looked at)
    w = torch.zeros(C, ldw, dtype=getattr(torch, dtype), device=DEV)
    w[:, :rank] = rand(rng, C, rank, scale=rank ** -0.5)
    bias = torch.linspace(-14.0, 25.0, C, device=DEV)
    dt = torch.empty(n, C, device=DEV)
    lib.call("liyab_scan_steps", dt.data_ptr(), low.data_ptr(), ldw + 4, w.data_ptr(), ldw, 1 if dtype == "bfloat16" else 0, bias.data_ptr(), n, C, rank,
             torch.cuda.current_stream().cuda_stream)
    want = plain.softplus(f64(low)[:, :rank] @ f64(w)[:, :rank].T + f64(bias))
    assert (np.abs(f64(dt) - want) / want).max() < (2e-5 if dtype == "float32" else 1e-4)


def _ffn_alone(p, x):
    """The feed-forward's result for the rows x, its rows a token and identity entries added up by the streams' update."""
    from liyab_amd.engine import StepItem
    from liyab_amd.kernels import ops

    n = x.shape[0]
    ffn = p.block.ffn
    k = int(getattr(ffn, "rows_a_token", 1))
    y = torch.full((n * k, p.width), float("nan"), dtype=torch.float32, device=DEV)  # (an identity entry's row is not written, and must not be read)
    p.core.open("f")
    ctx, _ = p.core.step_fn.prepare([StepItem("f", [1] * n, [])])
    identity = ffn.forward(x.to(DEV).to(p.core.dtype), ctx, None, out=y)
    total = torch.zeros(n, 1, p.width, dtype=torch.float32, device=DEV)
    ops.streams_update(total, y=y, n_sum=k, identity=identity)
    # added to a stream of its own, as blocks without streams do
    residual = torch.ones(n, p.width, dtype=torch.float32, device=DEV)
    ffn.forward(x.to(DEV).to(p.core.dtype), ctx, residual)
    p.core.close("f")
    assert tt.rel_err(f64(residual) - 1.0, f64(total[:, 0])) < 1e-5
    return f64(total[:, 0])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", [moe(24, 1.2, 8, 3, identity=3, scale=2.0, shared=(24, 1.2)), moe(24, 1.2, 8, 3, identity=3, scale=2.0, shared=(24, 0.4)), moe(13, 0.7, 5, 4, identity=2, shared=(13, 0.7)),
                               moe(32, 2.0, 5, 2, identity=1, scale=1.5, shared=(40, 0.8)), moe(9, 3.0, 3, 4, identity=4, scale=3.0), moe(16, 1.0, 1, 1), moe(16, 1.0, 1, 2, identity=1, shared=(16, 1.0)),
                               moe(8, 1.5, 80, 6, identity=5, scale=2.5, shared=(64, 9.0)), moe(16, 50.0, 4, 4, scale=0.3, shared=(16, 50.0)), moe(8, 0.5, 2, 1, identity=9)])
def test_experts_beside_identity_experts_and_a_shared_one_alone(dtype, m):
    """Who is chosen, with which weight, and the sum over experts with tensors, identity experts and the shared one, for few rows (one
    workgroup routes and lists, the small tiles, the shared expert as one more entry) and many; the twin's router reads the same
    rounded rows, so the choice is compared in bfloat16 too. Limits that cut and limits that do not."""
    p = _Layer(dtype, layer("attention", att(1, 1, 8, 8), m), width=72)
    ffn = p.block.ffn
    assert ffn.shared_listed == (m.get("shared") is not None and m["shared"] == m["expert"])
    for n in (1, 9, 64, 65, 300):
        x, xs = _inputs(p, np.random.default_rng(9 + n), n, scale=1.5)
        want = plain.routed_feed_forward(xs, p.t, "l0.mlp.", m)
        assert tt.rel_err(_ffn_alone(p, x), want) < MIXER_TOL[dtype], (m, n)


def _choice(z, correction, top, identity=0, scale=1.0, extra=False, block=None):
    from liyab_amd.kernels import ops

    block = block or ops.GROUPED_ROWS
    n, E = z.shape[0], z.shape[1] - (1 if extra else 0)
    rows_a_token, listed = top + (1 if extra else 0), E - identity + (1 if extra else 0)
    tiles = ops.moe_tiles(n * rows_a_token, listed, block)
    ids = torch.empty(n * rows_a_token, dtype=torch.int32, device=DEV)
    w = torch.empty(n * rows_a_token, dtype=torch.float32, device=DEV)
    rows = torch.empty(tiles * block, dtype=torch.int32, device=DEV)
    tile_group = torch.empty(tiles, dtype=torch.int32, device=DEV)
    ops.moe_route(z.to(DEV).contiguous(), top, ids, w, rows, tile_group, block=block, scores="softmax_all", correction=correction.to(DEV), scale=scale, identity=identity, extra=extra)
    ids_h, rows_h = ids.cpu().numpy(), rows.cpu().numpy()
    assert sorted(rows_h[rows_h >= 0].tolist()) == np.flatnonzero(ids_h >= 0).tolist()  # every entry with tensors is listed once, in a tile of its expert
    for place in np.flatnonzero(rows_h >= 0):
        assert int(tile_group[place // block]) == ids_h[rows_h[place]]
    return ids_h.reshape(n, rows_a_token), f64(w).reshape(n, rows_a_token)


def test_choices_worked_by_hand():
    """The choice goes by the corrected score, the weight is the score itself times the scale; an identity output gets no list; every
    token's own entry comes last, weighted by its own logit."""
    p = np.array([[0.5, 0.1, 0.05, 0.15, 0.2]])
    z = torch.from_numpy(np.log(p)).float()
    ids, w = _choice(z, torch.zeros(5), 3, identity=1, scale=2.0)
    assert ids.tolist() == [[0, -1, 3]] and np.abs(w - [[1.0, 0.4, 0.3]]).max() < 1e-6
    ids, w = _choice(z, torch.tensor([-1.0, 0.0, 0.3, 0.0, 0.0]), 2, identity=2)
    assert ids.tolist() == [[2, -1]] and np.abs(w - [[0.05, 0.2]]).max() < 1e-6
    # corrections below every score: still the largest of what is left, and negative choice scores are no bar
    ids, w = _choice(z, torch.tensor([-9.0, -9.5, -9.2, -9.9, -12.0]), 4)
    assert ids.tolist() == [[0, 2, 1, 3]]
    # equal scores: the lower number first
    ids, _ = _choice(torch.zeros(70, 6), torch.zeros(6), 3, identity=4)
    assert (ids == [0, 1, -1]).all()
    from liyab_amd.kernels import ops

    ids, w = _choice(torch.cat([z, torch.tensor([[0.7]])], dim=1).repeat(40, 1), torch.zeros(5), 2, identity=1, scale=3.0, extra=True, block=ops.SKINNY_ROWS)
    assert (ids == [0, -1, 4]).all() and np.abs(w - [1.5, 0.6, plain.logistic(0.7)]).max() < 1e-6
    # logits far from zero
    ids, w = _choice(z + 300.0, torch.zeros(5), 1, scale=1.0)
    assert ids.tolist() == [[0]] and np.abs(w - 0.5).max() < 1e-4


@pytest.mark.parametrize("n,E,top,identity", [(1, 9, 3, 2), (64, 130, 7, 30), (65, 40, 5, 0), (500, 18, 4, 3)])
def test_choices_of_many_tokens(n, E, top, identity):
    rng = np.random.default_rng(n)
    z, c = rand(rng, n, E, scale=2.0), rand(rng, E, scale=0.1)
    ids, w = _choice(z, c, top, identity=identity, scale=1.3)
    chosen, weights = plain.route(f64(z), f64(c), top, 1.3)
    assert (ids == np.where(chosen < E - identity, chosen, -1)).all() and np.abs(w - weights).max() < 1e-6


@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("S", [1, 2, 3, 4, 5, 8])
@pytest.mark.parametrize("d,n_sum", [(72, 1), (70, 3), (1030, 2), (2048, 1), (4100, 2)])
def test_the_streams_update_alone(out_dtype, S, d, n_sum):
    """The streams from the old ones (a matrix that is not symmetric shows its direction), the sum of a token's rows with identity
    entries among them, the next norm of a combination of the new streams; entering, reading gathered rows, one plain stream; widths
    that a thread's registers hold and not, even and odd ones."""
    from liyab_amd.kernels import ops

    rng = np.random.default_rng(S * 10000 + d)
    n, eps = 5, 1e-5
    x, y, e = rand(rng, n, S, d), rand(rng, n * n_sum, d), rand(rng, n, d)
    mix, add, take, w = rand(rng, S, S), rand(rng, S), rand(rng, S), rand(rng, d, scale=0.2, mean=1.0)
    h = rand(rng, n, d).to(out_dtype)
    ids = torch.from_numpy(rng.integers(-1, 2, n * n_sum).astype(np.int32))
    weights = rand(rng, n * n_sum)

    def normed(streams, comb, weight):
        u = np.einsum("s,nsd->nd", comb, streams)
        return plain.unit(u, eps) * (1.0 if weight is None else weight)

    ys = f64(y).reshape(n, n_sum, d)
    tol = 2e-5 if out_dtype == torch.float32 else 1e-2
    for identity in (False, True):
        rows = np.where((ids.numpy().reshape(n, n_sum) < 0)[..., None], f64(weights).reshape(n, n_sum, 1) * f64(h)[:, None, :], ys) if identity else ys
        total = rows.sum(axis=1)
        want = np.einsum("st,nsd->ntd", f64(mix), f64(x)) + f64(add)[None, :, None] * total[:, None, :]
        xd, out = x.to(DEV), h.to(DEV)  # (the rows that were routed lie where the next ones go)
        yd = y.clone()
        if identity:
            yd[ids < 0] = float("nan")
        entries = ops.IdentityEntries(ids.to(DEV), weights.to(DEV), n_sum, out) if identity else None
        ops.streams_update(xd, y=yd.to(DEV), n_sum=n_sum, identity=entries, mix=mix.to(DEV), add=add.to(DEV), next_norm=(take.to(DEV), w.to(DEV), eps), out=out)
        assert tt.rel_err(f64(xd).reshape(n, -1), want.reshape(n, -1)) < 1e-5
        assert tt.rel_err(f64(out), normed(want, f64(take), f64(w))) < tol
    # one plain sum a stream, nothing read off
    xd = x.to(DEV)
    ops.streams_update(xd, y=y.to(DEV), n_sum=n_sum)
    assert tt.rel_err(f64(xd).reshape(n, -1), (f64(x) + ys.sum(axis=1)[:, None, :]).reshape(n, -1)) < 1e-5
    # entering: all streams are the rows, and the first norm of them; then gathered rows are read off the plain sum
    out = torch.empty(n, d, dtype=out_dtype, device=DEV)
    ops.streams_update(xd, enter=e.to(DEV), next_norm=(take.to(DEV), w.to(DEV), eps), out=out)
    assert torch.equal(xd.cpu(), e[:, None, :].expand(n, S, d))
    assert tt.rel_err(f64(out), normed(f64(xd), f64(take), f64(w))) < tol
    xd = x.to(DEV)
    picked = torch.tensor([3, 0, 3], dtype=torch.int32, device=DEV)
    out = torch.empty(3, d, dtype=out_dtype, device=DEV)
    ops.streams_update(xd, next_norm=(None, w.to(DEV), eps), out=out, rows=picked)
    assert tt.rel_err(f64(out), normed(f64(x)[[3, 0, 3]], np.ones(S), f64(w))) < tol and torch.equal(xd.cpu(), x)


@pytest.mark.parametrize("dtype", DTYPES)
def test_connections_that_single_a_stream_out(dtype, tmp_path):
    """A sublayer that reads the second stream alone and gives to the first alone, and a mix that moves each stream to the next: a
    direction read the wrong way round, or new streams where old ones belong, changes the logits by much."""
    from liyab_amd.weights.safetensors_io import write_safetensors

    cfg = config(90, 48, 1e-5, [layer("attention", att(2, 1, 16, 8, rot=(8, 100.0)), dense(32)), layer("mamba1", scan(40, 4, 3, 3), moe(16, 1.0, 4, 4, identity=1, shared=(16, 1.0)))],
                 streams=3, loop=(0, 2, 2))
    d = str(tmp_path / "m")
    write_model(d, cfg, 3, dtype)
    raw, t = read_model(d)
    step = np.array([[0.0, 1.0, 0.0], [0.0, 0.0, 1.0], [1.0, 0.0, 0.0]])
    for i in range(2):
        for q in (1, 2):
            t[f"l{i}.hc{q}.in"], t[f"l{i}.hc{q}.out"], t[f"l{i}.hc{q}.mix"] = np.array([0.0, 1.0, 0.0]), np.array([1.0, 0.0, 0.25]), step
    write_safetensors(os.path.join(d, "model.safetensors"), {k: torch.from_numpy(np.ascontiguousarray(v)).float() for k, v in t.items()}, {})
    t = twin_tensors(t, dtype)
    reqs = {f"c{i}": tt.random_tokens(30 + i, n, 90) for i, n in enumerate([1, 40, 150])}
    ref = {rid: plain.forward(raw, t, toks) for rid, toks in reqs.items()}
    turned = {k: (v.T if k.endswith((".hc1.mix", ".hc2.mix")) else v) for k, v in t.items()}
    assert np.abs(plain.forward(raw, turned, reqs["c2"]) - ref["c2"]).max() > 0.1 * np.abs(ref["c2"]).max()
    for steps in (tt.schedule_whole(reqs), tt.schedule_portions(reqs, (2, 5, 1, 9)), tt.schedule_mixed(reqs, seed=2, max_live=3)):
        core = make_core(d, dtype, None, page_size=8, max_requests=3, num_pages=tt.max_live_pages(steps, 8))
        check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lafanex-connections {dtype}", family="lafanex-connections")
        core.manager.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_each_pass_of_a_loop_has_a_cache_and_state_of_its_own(dtype, models):
    """Two passes over the same weights hold pages and slots apart, and a layer's device tensors are shared by its passes."""
    core = make_core(models[("mix", dtype)][0], dtype, 64)
    blocks = core.model.blocks
    assert len(blocks) == 9 and blocks[1].mixer.in_weight.data_ptr() == blocks[3].mixer.in_weight.data_ptr() == blocks[5].mixer.in_weight.data_ptr()
    assert blocks[2].mixer.out_weight.data_ptr() == blocks[4].mixer.out_weight.data_ptr()
    assert len({core.storage.layer(i).k.data_ptr() for i in (1, 3, 5, 7)}) == 4
    assert len({core.storage.state(i).data_ptr() for i in (0, 2, 4, 6, 8)}) == 5


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
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lafanex-whole {name} {dtype}")
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
                caught.append(f64(x)[:len(toks)].sum(axis=1))
                return out
            block.forward = wrapped
        plain_core.open(rid)
        plain_core.step([StepItem(rid, toks, [])])
        assert len(caught) == len(streams) == len(plain.runs(models[(name, dtype)][1]))
        for got_x, want_x in zip(caught, streams):
            assert tt.rel_err(got_x, want_x) < 1e-5


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_a_prompt_then_its_last_tokens_one_by_one(name, dtype, models, reference):
    reqs = make_requests(name)
    steps = tt.schedule_bulk_tail(reqs, tail=45)
    core = make_core(models[(name, dtype)][0], dtype, tt.max_live_tokens(steps))
    got = tt.run_schedule(core, steps)
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lafanex-decode {name} {dtype}")


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
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lafanex-portions {name} {dtype}")


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
    check_logits(got, reqs, ref, dtype, f"lafanex-mixed {name} {dtype}")
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
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lafanex-long {name} {dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_trace_program(dtype, models, reference, tmp_path):
    name = "odd"
    reqs = make_requests(name)
    steps = tt.schedule_mixed(reqs, seed=5, max_live=4)
    got = tt.run_trace_program(models[(name, dtype)][0], dtype, steps, str(tmp_path), tt.max_live_tokens(steps), CONFIGS[name][0]["vocab"])
    check_logits(got, reqs, reference[(name, dtype)], dtype, f"lafanex-trace {dtype}")


def draw_config(seed):
    """A geometry drawn from the seed: every size, constant and count, the layers' kinds and order, what is looped."""
    rng = np.random.default_rng(7000 + seed)
    pick = lambda *options: options[int(rng.integers(len(options)))]  # noqa: E731
    width = pick(40, 48, 64, 96, 104, 160)

    def feed_forward():
        kind = pick(None, "dense", "moe", "moe")
        if kind == "dense":
            return dense(pick(8, 20, 24, 40, 56))
        if kind == "moe":
            experts, identity, ff, limit = pick(1, 2, 3, 5, 8), pick(0, 0, 1, 2, 4), pick(8, 12, 24), pick(0.5, 1.0, 3.0)
            return moe(ff, limit, experts, int(rng.integers(1, experts + identity + 1)), identity=identity, scale=pick(1.0, 0.5, 1.5), shared=pick(None, (ff, limit), (16, 0.8)))
        return None

    layers = []
    for i in range(int(rng.integers(2, 6))):
        if pick("attention", "mamba1") == "attention":
            kv, dim = pick(1, 2, 3), pick(4, 8, 10, 16, 24, 32)
            rot = pick(None, (2 * int(rng.integers(1, dim // 2 + 1)), pick(10.0, 500.0, 5e5)), (dim, 1e4))
            layers.append(layer("attention", att(kv * pick(1, 2, 4), kv, dim, pick(dim, dim, 4, 12, 40), rot=rot, scale=pick(None, 0.3, 1.0 if dim <= 8 else 0.4)), feed_forward()))
        else:
            layers.append(layer("mamba1", scan(pick(24, 40, 64, 75, 130), pick(1, 4, 7, 16, 24, 33), pick(1, 3, 8, 16), pick(1, 2, 3, 4, 6)), feed_forward()))
    start = int(rng.integers(0, len(layers)))
    loop = pick(None, (start, int(rng.integers(start + 1, len(layers) + 1)), pick(1, 2, 3)))
    return config(pick(97, 256, 500), width, pick(1e-5, 1e-6, 1e-3), layers, streams=pick(None, 1, 2, 3, 4, 6), loop=loop), pick(8, 16, 24)


@pytest.mark.parametrize("seed", range(16))
def test_drawn_geometries_whole_and_mixed(seed, tmp_path):
    cfg, page_size = draw_config(seed)
    reqs = {f"g{i}": tt.random_tokens(seed * 10 + i, n, cfg["vocab"]) for i, n in enumerate([1, 19, 77, 150, 260])}
    for dtype in DTYPES:
        d = str(tmp_path / f"m_{dtype}")
        raw, t = write_model(d, cfg, 100 + seed, dtype)
        ref = {rid: plain.forward(raw, t, toks) for rid, toks in reqs.items()}
        steps = tt.schedule_whole(reqs)
        core = make_core(d, dtype, tt.max_live_tokens(steps), page_size=page_size)
        check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lafanex-drawn seed {seed} whole {dtype}", family="lafanex-drawn", tol=TOL_DRAWN)
        steps = tt.schedule_mixed(reqs, seed=seed, max_live=3)
        core = make_core(d, dtype, None, page_size=page_size, max_requests=3, num_pages=tt.max_live_pages(steps, page_size))
        check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lafanex-drawn seed {seed} mixed {dtype}", family="lafanex-drawn", tol=TOL_DRAWN)
        core.manager.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_real_widths_in_long_steps(dtype, tmp_path):
    """Heads of 64 and 128, a width of 512, prompts of hundreds of tokens in one step and in mixed batches: the tiles of the large
    products, the matrix-core attention with the fixed sink, the scan in segments, the experts' large tiles beside the shared expert's own
    products, the choice a wave a token."""
    cfg = config(1000, 512, 1e-5, [
        layer("mamba1", scan(1024, 16, 32, 4), moe(128, 3.0, 16, 3, identity=4, scale=2.0, shared=(128, 3.0))),
        layer("attention", att(8, 2, 64, 64, rot=(64, 10000.0)), dense(1024)),
        layer("mamba1", scan(768, 24, 48, 3), dense(768)),
        layer("attention", att(4, 2, 128, 128, rot=(64, 5e5)), moe(64, 1.5, 8, 2, identity=1, shared=(192, 2.0))),
    ], streams=2, loop=(1, 3, 2))
    d = str(tmp_path / "m")
    raw, t = write_model(d, cfg, 31, dtype)
    reqs = {f"r{i}": tt.random_tokens(900 + i, n, raw["vocab"]) for i, n in enumerate([330, 700, 45])}
    ref = {rid: plain.forward(raw, t, toks) for rid, toks in reqs.items()}
    steps = tt.schedule_whole(reqs)
    core = make_core(d, dtype, tt.max_live_tokens(steps))
    check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lafanex-wide whole {dtype}", family="lafanex-wide")
    steps = tt.schedule_mixed(reqs, seed=3, max_live=3, portions=(2, 130, 64, 300, 17))
    core = make_core(d, dtype, None, max_requests=3, num_pages=tt.max_live_pages(steps, 16))
    check_logits(tt.run_schedule(core, steps), reqs, ref, dtype, f"lafanex-wide mixed {dtype}", family="lafanex-wide")
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
    assert set(turn["phases_ms"]) == {"embed", "scored_attention", "selective_scan", "routed_ffn", "gated_ffn", "lm_head"}
