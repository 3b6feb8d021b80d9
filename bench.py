"""Decode and prefill throughput of the engine on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch 8] [--size small|medium|large|xl|wide] [--layers L]
    python bench.py --sequences 1,2,4,8 [-n 128]     # together against in turns, and whether replies are the same
    python bench.py --prefill-tokens 512,2048,8192   # prefill tokens a second per length
    python bench.py --workload medium16|xl64         # the continuous-batching and the batch-64 workloads of the larger sizes
    python bench.py --link-floor                     # what one dependent kernel of a replayed graph costs at least
    python bench.py --product 4096,4096,16384,8,15   # one product in tiles of 128 x 128 and of 256 x 256
    python bench.py --design bokulix|mofulix|dopilorn|larulorn|lolulorn|lafanex [--design-sizes small,medium,xl] [--layers L] [--phases]   # that design beside GPT-2 (dopilorn, larulorn: beside Mofulix; lolulorn, lafanex: beside Larulorn) at equal sizes

The default run has GPT-2 small's layer sizes (12 layers, width 768, 12 heads
of 64, feed-forward 3072, vocabulary 50257, 1024 positions) with random
weights in bfloat16, a batch of 8 requests with 512-token prompts decoding
towards 1,024 tokens. A step is one decode step of the whole engine loop:
scheduler, model step, sampling, tokens back on the host. It prints one JSON
line: decoded tokens a second, the prefill of 2,048 tokens (two prompts of
1,024), the decode step's share of the HBM roofline (bytes it has to read:
every weight once and the live requests' cache, over its time), and decoding
at batch 1 and 64. Token ids are seeded synthetic ones; no dataset is used.
The reference measures the same way: tokens a second beside a ceiling from
the bytes a decoded token must read (src/core/model_bytes.h:1-5,
docs/guide/development.md:115-122) and prefill over synthetic ids
(tools/liyab_bench.cpp:87-169).
"""

import argparse
import json
import os
import sys
import tempfile
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

HBM_PEAK_GBS = 8000.0  # MI355X, published
MFMA_PEAK = {"bf16": 2.5e15, "fp32": 157.3e12}

SMALL = {"architectures": ["GPT2LMHeadModel"], "model_type": "gpt2", "n_layer": 12, "n_embd": 768, "n_head": 12,
         "n_inner": 3072, "vocab_size": 50257, "n_positions": 1024, "layer_norm_epsilon": 1e-5,
         "activation_function": "gelu_new", "tie_word_embeddings": True}
# GPT-2's other sizes, for --size: the layer sizes and, with them, the number of layers
# ("wide": no GPT-2 of anybody's, but the architecture at layer sizes where a decode step is bound by the weights' bytes, not by
# its chain of kernels: 403 MB of matrices a layer; run it with --layers 8 or so)
WEIGHT_SEEDS = {"small": 10, "medium": 20, "large": 25, "xl": 30, "wide": 40}
SIZES = {"small": {}, "medium": {"n_layer": 24, "n_embd": 1024, "n_head": 16, "n_inner": 4096},
         "large": {"n_layer": 36, "n_embd": 1280, "n_head": 20, "n_inner": 5120},
         "xl": {"n_layer": 48, "n_embd": 1600, "n_head": 25, "n_inner": 6400},
         "wide": {"n_layer": 32, "n_embd": 4096, "n_head": 32, "n_inner": 16384}}


def weight_bytes(cfg, elt):
    d, F, V, L = cfg["n_embd"], cfg["n_inner"], cfg["vocab_size"], cfg["n_layer"]
    matrices = L * (3 * d * d + d * d + 2 * d * F) + V * d  # the tied table is read once, as the head
    vectors = L * (3 * d + d + F + d + 4 * d) + 2 * d  # biases and norm vectors, float32
    return matrices * elt + vectors * 4


def kv_bytes_per_position(cfg, elt):
    return 2 * cfg["n_layer"] * cfg["n_embd"] * elt


def prefill_flops(cfg, prompt_lens, logit_rows):
    d, F, V, L = cfg["n_embd"], cfg["n_inner"], cfg["vocab_size"], cfg["n_layer"]
    n = sum(prompt_lens)
    flops = 2.0 * n * L * (3 * d * d + d * d + 2 * d * F)
    for t in prompt_lens:
        flops += L * 2.0 * d * t * (t + 1)  # q.k and p.v over the causal half
    return flops + 2.0 * logit_rows * d * V


def make_engine(model_dir, dtype, batch, ctx, page_size=64, prefill_chunk=1024, batch_invariant=False, phases=False):
    from liyab_amd import Engine

    pages = batch * (-(-ctx // page_size)) + 4
    return Engine(model_dir, dtype=dtype, page_size=page_size, num_pages=pages, max_num_seqs=max(batch, 2),
                  max_batched_tokens=max(2048, batch), prefill_chunk=prefill_chunk, ctx=ctx, batch_invariant=batch_invariant,
                  phases=phases)


def decode_run(engine, cfg, batch, prompt_len, steps, warmup, seed=11, step_bytes=None):
    """(tokens/s, ms/step, bytes/step) over `steps` decode steps of `batch` requests. `step_bytes(contexts, steps,
    elt)`: the bytes a timed step has to read, for a design whose bytes are not GPT-2's."""
    import numpy as np
    import torch

    from liyab_amd import SamplingParams

    rng = np.random.default_rng(seed)
    engine.stop_at_eos = False
    for i in range(batch):
        prompt = rng.integers(0, cfg.get("vocab_size", cfg.get("vocab")), prompt_len).tolist()
        # (requests that go on for some steps past the timed ones: a request about to reach its last
        # token is waited for, not run ahead of, and that wait is no part of a decode step)
        engine.add_request(prompt, SamplingParams(temperature=0.0, max_tokens=steps + warmup + 8), rid=f"b{batch}-{i}")
    while any(r.remaining > 1 or not r.generated for r in engine.scheduler.running) or engine.scheduler.waiting:
        engine.step()  # prompts, until every request is decoding
    for _ in range(warmup):
        engine.step()
    contexts = [r.computed for r in engine.scheduler.running]
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        engine.step()
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    elt = 2 if engine.core.dtype == torch.bfloat16 else 4
    # each timed step s reads the cache of positions [0, context + s] of every request
    kv_positions = sum(c * steps + steps * (steps + 1) // 2 for c in contexts)
    if step_bytes is not None:
        bytes_per_step = step_bytes(contexts, steps, elt)
    else:
        bytes_per_step = weight_bytes(cfg, elt) + kv_positions * kv_bytes_per_position(cfg, elt) / max(steps, 1)
    for r in list(engine.scheduler.running):
        engine.abort(r.rid)
    return batch * steps / dt, dt * 1e3 / max(steps, 1), bytes_per_step


def workload_run(engine, cfg, prompts, params_of, label):
    """A whole workload through the engine's loop: requests arrive together, prompts go in portions
    beside decoding requests. Returns generated tokens a second, all tokens (prompt and generated)
    a second, and the share of the HBM roofline: the bytes every step has to read (each weight
    once, and the cache of the positions its requests hold) over the whole time."""
    import torch

    elt = 2 if engine.core.dtype == torch.bfloat16 else 4
    w_bytes, kv_pos = weight_bytes(cfg, elt), kv_bytes_per_position(cfg, elt)
    engine.stop_at_eos = False
    rids = [engine.add_request(p, params_of(i), rid=f"{label}-{i}") for i, p in enumerate(prompts)]
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    steps = bytes_read = 0
    while engine.has_unfinished():
        before = engine.core.step_fn.steps
        engine.step()
        if engine.core.step_fn.steps > before:
            h = engine.core.step_fn.last_context.host
            bytes_read += w_bytes + kv_pos * sum(f + q for f, q in zip(h.first_pos, h.q_lens))
            steps += 1
    engine.flush()
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    results = [engine.result(r) for r in rids]
    for r in rids:
        engine.release(r)
    generated = sum(len(r.tokens) for r in results)
    prompt_tokens = sum(len(p) for p in prompts)
    return {"generated_tok_s": round(generated / dt, 1), "all_tok_s": round((generated + prompt_tokens) / dt, 1),
            "seconds": round(dt, 4), "steps": steps, "ms_per_step": round(dt * 1e3 / max(steps, 1), 4),
            "generated": generated, "prompt_tokens": prompt_tokens,
            "preemptions": sum(r.stats.preemptions for r in results),
            "roofline_frac": round(bytes_read / dt / 1e9 / HBM_PEAK_GBS, 4)}, [r.tokens for r in results]


def product_run(M, N, K, tiles, device="cuda:0", reps=30):
    """One product a[M, K] . w[N, K]^T + bias in bfloat16 (outputs bfloat16), as the tiled matrix-core
    kernel runs it in the tiles named (0: the kernel's own choice; 2 and 6: 64 x 64, 8: 128 x 128,
    15: 256 x 256): microseconds and TFLOP/s each."""
    import torch

    from liyab_amd.kernels import ops

    dev = torch.device(device)
    a = torch.randn(M, K, device=dev).bfloat16()
    w = (torch.randn(N, K, device=dev) * 0.02).bfloat16()
    bias = torch.randn(N, device=dev)
    out = torch.empty(M, N, dtype=torch.bfloat16, device=dev)
    runs = []
    for tile in tiles:
        for _ in range(3):
            ops.gemm_mfma_dl(a, w, bias, out=out, tile=tile)
        torch.cuda.synchronize()
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        e0.record()
        for _ in range(reps):
            ops.gemm_mfma_dl(a, w, bias, out=out, tile=tile)
        e1.record()
        torch.cuda.synchronize()
        us = e0.elapsed_time(e1) / reps * 1e3
        runs.append({"tile": tile, "us": round(us, 1), "tflops": round(2.0 * M * N * K / us / 1e6, 1)})
    return {"metric": "one product, bfloat16", "M": M, "N": N, "K": K, "runs": runs}


def link_floor(device="cuda:0", links=100):
    """What a dependent kernel costs at least inside a replayed graph, measured with the library's
    own kernels: a chain of kernels that each write one word (the distance from one kernel's end
    to the next one's start), and a chain of norms over 8 rows of 768 in which each reads what the
    one before wrote (a boundary, a first read of fresh data, a few hundred cycles of work, a write)."""
    import torch

    from liyab_amd.kernels import ops

    dev = torch.device(device)
    one = torch.zeros(64, dtype=torch.int32, device=dev)
    a = torch.randn(8, 768, device=dev)
    b = torch.empty_like(a)
    w, bias = torch.ones(768, device=dev), torch.zeros(768, device=dev)
    out = {}
    for name, body in (("a kernel that writes one word", lambda i: ops.fill_(one[:1], i)),
                       ("a norm of 8 rows of 768 that reads the one before", lambda i: ops.layernorm(b if i % 2 == 0 else a, a if i % 2 == 0 else b, w, bias, 1e-5))):
        for i in range(3):
            body(i)
        torch.cuda.synchronize()
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g):
            for i in range(links):
                body(i)
        best = float("inf")
        for _ in range(6):
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            e0.record()
            g.replay()
            e1.record()
            e1.synchronize()
            best = min(best, e0.elapsed_time(e1))
        out[name] = round(best * 1e3 / links, 3)
    return {"metric": "microseconds a dependent kernel of a replayed graph", "links": links, "us_per_link": out}


def copy_bandwidth(device="cuda:0", mbytes=1024, repeat=5):
    """GB/s of a device-to-device copy of `mbytes` (bytes read plus bytes written over the best
    time): what this machine's memory gives a plain stream, beside the published peak that the
    roofline shares are taken against (the reference measures its read ceiling the same way,
    tools/liyab_bench.cpp:1-9)."""
    import torch

    n = mbytes * (1 << 20) // 4
    a = torch.empty(n, dtype=torch.float32, device=device).normal_()
    b = torch.empty_like(a)
    best = float("inf")
    for _ in range(repeat + 1):
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        e0.record()
        b.copy_(a)
        e1.record()
        e1.synchronize()
        best = min(best, e0.elapsed_time(e1))
    return 2.0 * n * 4 / (best * 1e-3) / 1e9


def prefill_run(engine, cfg, prompt_lens, repeat=5, seed=12):
    """Best of `repeat`: (tokens/s, ms) of one step that holds the whole prompts."""
    import numpy as np
    import torch

    from liyab_amd.engine import StepItem

    rng = np.random.default_rng(seed)
    prompts = [rng.integers(0, cfg.get("vocab_size", cfg.get("vocab")), n) for n in prompt_lens]  # arrays of ids, as the scheduler hands portions over
    best = float("inf")
    for it in range(repeat + 2):
        for i in range(len(prompts)):
            engine.core.open(f"p{i}")
        items = [StepItem(f"p{i}", p, [len(p) - 1]) for i, p in enumerate(prompts)]
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        engine.core.step(items)
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        for i in range(len(prompts)):
            engine.core.close(f"p{i}")
        if it >= 2:
            best = min(best, dt)
    n = sum(prompt_lens)
    return n / best, best * 1e3


def ttft_run(engine, cfg, prompt_len=512, repeat=6, seed=14):
    """An idle engine and one prompt: milliseconds until step() has launched everything (the host's
    share), the step's kernels on the device (events around it), and until the first token is on the
    host; best of `repeat`, prompts of prompt_len - 0, 1, 2, ... tokens. First with everything the
    engine knows of earlier steps forgotten before each prompt, so that its step is launched kernel by
    kernel (`first_sight_*`: a size the engine has not seen); then as they come: the prompts' steps are
    padded to one size, captured after three sights and replayed (`ms`, `host_ms`, `device_ms`)."""
    import numpy as np
    import torch

    from liyab_amd import SamplingParams

    rng = np.random.default_rng(seed)
    engine.stop_at_eos = False

    def one(length):
        prompt = rng.integers(0, cfg["vocab_size"], length).tolist()
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        rid = engine.add_request(prompt, SamplingParams(temperature=0.0, max_tokens=1))
        e0.record()
        engine.step()
        e1.record()
        t1 = time.perf_counter()
        while engine.has_unfinished():
            engine.step()
        engine.flush()
        t2 = time.perf_counter()
        torch.cuda.synchronize()
        engine.release(rid)
        return (t1 - t0) * 1e3, e0.elapsed_time(e1), (t2 - t0) * 1e3

    out = {"prompt_len": prompt_len}
    for label, forget in (("first_sight_", True), ("", False)):
        best = [float("inf")] * 3
        for it in range(repeat + 4):
            if forget:
                engine.core.step_fn.forget_graphs()
            got = one(prompt_len - it % 8)
            if it >= 4:
                best = [min(a, b) for a, b in zip(best, got)]
        out.update({label + "host_ms": round(best[0], 4), label + "device_ms": round(best[1], 4), label + "ms": round(best[2], 4)})
    return out


def sequences_run(engine, cfg, counts, prompt_len, n_new, seed=13):
    """Several sequences generated together against the same sequences one after the other, as
    the reference's liyab-seq-bench reports them (tools/liyab_seq_bench.cpp:1-32): total tokens
    a second both ways, the gain, and whether every reply equals its reply alone. Greedy, and
    with a seeded temperature."""
    import numpy as np
    import torch

    from liyab_amd import SamplingParams

    rng = np.random.default_rng(seed)
    engine.stop_at_eos = False
    out = []
    for count in counts:
        prompts = [rng.integers(0, cfg["vocab_size"], prompt_len).tolist() for _ in range(count)]
        for name, make in (("greedy", lambda i: SamplingParams(temperature=0.0, max_tokens=n_new)),
                           ("temperature 0.8", lambda i: SamplingParams(temperature=0.8, top_k=40, top_p=0.95, seed=100 + i, max_tokens=n_new))):
            for _ in range(2):  # the second run replays captured graphs
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                together = engine.generate(prompts, [make(i) for i in range(count)])
                torch.cuda.synchronize()
                t_together = time.perf_counter() - t0
                t0 = time.perf_counter()
                alone = [engine.generate([p], [make(i)])[0] for i, p in enumerate(prompts)]
                torch.cuda.synchronize()
                t_turns = time.perf_counter() - t0
            total = sum(len(r.tokens) for r in together)
            out.append({"sequences": count, "sampling": name, "together_tok_s": round(total / t_together, 1),
                        "in_turns_tok_s": round(total / t_turns, 1), "gain": round(t_turns / t_together, 2),
                        "same": all(a.tokens == b.tokens for a, b in zip(together, alone))})
    return {"metric": "sequences together against in turns", "prompt_len": prompt_len, "new_tokens": n_new, "runs": out}


# -- Bokulix beside GPT-2 at equal sizes ------------------------------------------------------------------
# Layers that resemble real ones: GPT-2 small's, medium's and XL's widths, head counts and feed-forward widths; the
# Bokulix of each has the same width, layers, heads (of 64, values of 64), vocabulary and positions, a cached row
# of 128, a window that covers the context (so that attention walks as many keys), four taps, and experts whose
# chosen ones together are as wide as GPT-2's feed-forward (top x ff = n_inner). (A cached row wider than 128 is
# taken by the plain attention kernel in prompts: the matrix-core prefill kernel holds heads up to 128.)
BOKULIX_SHAPES = {"small": {"rank": 128, "experts": 8, "top": 2}, "medium": {"rank": 128, "experts": 16, "top": 2},
                  "xl": {"rank": 128, "experts": 16, "top": 4}}


def bokulix_config(gpt2_cfg, shape):
    d, H, F, L = gpt2_cfg["n_embd"], gpt2_cfg["n_head"], gpt2_cfg["n_inner"], gpt2_cfg["n_layer"]
    hd = d // H
    entry = {"type": "latent_attention",
             "mixer": {"heads": H, "dim": hd, "vdim": hd, "kv_rank": shape["rank"], "scale": hd ** -0.5, "mask": {"size": gpt2_cfg["n_positions"]}},
             "mlp": {"kind": "moe", "expert": {"ff": F // shape["top"]}, "router": {"experts": shape["experts"], "top": shape["top"]}}}
    return {"architecture": "Bokulix", "vocab": gpt2_cfg["vocab_size"], "width": d, "max_positions": gpt2_cfg["n_positions"],
            "norm": {"eps": 1e-5}, "canon": {"taps": 4}, "layers": [json.loads(json.dumps(entry)) for _ in range(L)]}


def bokulix_step_bytes(cfg, batch):
    """The bytes a decode step of `batch` tokens has to read: every matrix of the mixers, gates and routers once, the
    experts that tokens choose (as many distinct ones as uniform choices make on average), the head, and the cached rows
    inside each request's window."""
    def step_bytes(contexts, steps, elt):
        d, V = cfg["width"], cfg["vocab"]
        total = V * d * elt
        for entry in cfg["layers"]:
            m, mlp = entry["mixer"], entry["mlp"]
            H, D, Vd, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
            total += ((H * D + R + H * Vd) * d + H * D * R + H * Vd * R + d * H * Vd + d * d) * elt
            if mlp is not None:
                E, top, F = mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"]
                chosen = E * (1.0 - (1.0 - top / E) ** batch)
                total += (d * d + E * d) * elt + chosen * 3 * F * d * elt
            window = (m.get("mask") or {}).get("size", 0)
            seen = sum(sum(min(c + s + 1, window) if window else c + s + 1 for s in range(steps)) for c in contexts) / max(steps, 1)
            total += seen * R * elt
        return total
    return step_bytes


def bokulix_prefill_flops(cfg, prompt_lens, logit_rows):
    d, V, n = cfg["width"], cfg["vocab"], sum(prompt_lens)
    flops = 2.0 * logit_rows * d * V
    for entry in cfg["layers"]:
        m, mlp = entry["mixer"], entry["mlp"]
        H, D, Vd, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
        flops += 2.0 * n * ((H * D + R + H * Vd) * d + H * D * R + H * Vd * R + d * H * Vd + d * d)
        window = (m.get("mask") or {}).get("size", 0)
        for t in prompt_lens:
            keys = sum(min(i + 1, window) if window else i + 1 for i in range(t))
            flops += 4.0 * H * R * keys  # scores and weighted rows against the cached rows
        if mlp is not None:
            E, top, F = mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"]
            flops += 2.0 * n * (d * d + E * d + top * 3 * F * d)
    return flops


# -- Mofulix beside GPT-2 at equal sizes --------------------------------------------------------------------
# The Mofulix of each size has GPT-2's width, layers, vocabulary and head count (heads of 64 everywhere), its layers
# taking turns as gated attention (as many key heads as query heads, so that attention reads what GPT-2's reads), wkv,
# and attention with a bias by distance beside a state space (heads of 64 with a state of 64, four taps); the gated
# feed-forward is two thirds as wide as GPT-2's, which makes its three matrices as large as GPT-2's two.
def mofulix_config(gpt2_cfg):
    d, H, F, L = gpt2_cfg["n_embd"], gpt2_cfg["n_head"], gpt2_cfg["n_inner"], gpt2_cfg["n_layer"]
    hd = d // H
    ff = max(64, F * 2 // 3 // 64 * 64)
    mlp = {"kind": "dense", "ff": ff, "limit": 7.0}
    kinds = [
        {"type": "attention", "mixer": {"heads": H, "kv_heads": H, "dim": hd, "vdim": hd, "scale": hd ** -0.5, "softcap": 30.0,
                                        "rot": {"dims": hd, "base": 10000.0, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}},
        {"type": "wkv", "mixer": {"heads": H, "dim": hd, "decay_rank": 64}},
        {"type": "parallel", "mixer": {"left": {"heads": H, "kv_heads": H, "dim": hd, "vdim": hd, "scale": hd ** -0.5, "bias_max": 128, "bias_rows": 32,
                                                "q_temp": {"coef": 0.1, "every": 512}},
                                       "right": {"heads": H, "vdim": hd, "state": 64, "groups": 1, "conv": 4, "norm_groups": 1}}},
    ]
    layers = [dict(json.loads(json.dumps(kinds[i % 3])), mlp=dict(mlp)) for i in range(L)]
    return {"architecture": "Mofulix", "vocab": gpt2_cfg["vocab_size"], "width": d, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5},
            "max_positions": gpt2_cfg["n_positions"], "layers": layers}


def _mofulix_layer_weights(entry, d):
    """Matrix elements of a layer (what a step reads of it), and of them those of products (2 flops an element a token)."""
    m, kind = entry["mixer"], entry["type"]
    n = 3 * entry["mlp"]["ff"] * d if entry.get("mlp") else 0
    if kind == "attention":
        H, G, D = m["heads"], m["kv_heads"], m["dim"]
        n += (H * D + G * D + H * D) * d + d * H * D
    elif kind == "wkv":
        HD, R = m["heads"] * m["dim"], m.get("decay_rank", 16)
        n += 4 * HD * d + R * d + HD * R + d * HD
    else:
        a, b = m["left"], m["right"]
        n += (a["heads"] * a["dim"] + a["kv_heads"] * (a["dim"] + a["vdim"])) * d + d * a["heads"] * a["vdim"]
        inner = b["heads"] * b["vdim"]
        n += (2 * inner + 2 * b["groups"] * b["state"] + b["heads"]) * d + d * inner
    return n


def mofulix_step_bytes(cfg, batch):
    """The bytes a decode step has to read: every matrix once, the head, the cached keys and values of the attention layers,
    and the 32-bit state of the recurrent ones (read and written) a request."""
    def step_bytes(contexts, steps, elt):
        d, V = cfg["width"], cfg["vocab"]
        total = V * d * elt
        seen = sum(sum(c + s + 1 for s in range(steps)) for c in contexts) / max(steps, 1)
        for entry in cfg["layers"]:
            m = entry["mixer"]
            total += _mofulix_layer_weights(entry, d) * elt
            if entry["type"] == "attention":
                total += seen * 2 * m["kv_heads"] * m["dim"] * elt
            elif entry["type"] == "wkv":
                total += len(contexts) * 2 * m["heads"] * m["dim"] * m["dim"] * 4
            else:
                a, b = m["left"], m["right"]
                total += seen * a["kv_heads"] * (a["dim"] + a["vdim"]) * elt + len(contexts) * 2 * b["heads"] * b["vdim"] * b["state"] * 4
        return total
    return step_bytes


def mofulix_prefill_flops(cfg, prompt_lens, logit_rows):
    d, V, n = cfg["width"], cfg["vocab"], sum(prompt_lens)
    flops = 2.0 * logit_rows * d * V
    pairs = sum(t * (t + 1) / 2 for t in prompt_lens)
    for entry in cfg["layers"]:
        m = entry["mixer"]
        flops += 2.0 * n * _mofulix_layer_weights(entry, d)
        if entry["type"] == "attention":
            flops += 2.0 * pairs * m["heads"] * 2 * m["dim"]
        elif entry["type"] == "wkv":
            flops += n * m["heads"] * 6.0 * m["dim"] * m["dim"]  # a token: the state's update and its read, a head
        else:
            a, b = m["left"], m["right"]
            flops += 2.0 * pairs * a["heads"] * (a["dim"] + a["vdim"]) + n * b["heads"] * 6.0 * b["vdim"] * b["state"]
    return flops



# -- Dopilorn beside Mofulix at equal sizes -------------------------------------------------------------------
# The Dopilorn of each size has GPT-2's width, layers, vocabulary and head count; its layers take turns as a delta-rule recurrence
# (heads of 64, a decay of rank 64), attention in two maps a head (maps of 32, values of 64, as many key heads as query heads, a
# convolution of four taps on the projections, a window as long as the context, so that each map walks every key) and latent
# attention (heads of 64 over cached rows of 128, as Bokulix's: the matrix-core kernel for prompts holds rows up to 128; queries through
# a latent of half the width); two norms and
# two convolutions of four taps a layer; a feed-forward of two matrices as wide as GPT-2's. It stands beside Mofulix, the engine's
# other design of parallel layers that mixes recurrences with attention.
def dopilorn_config(gpt2_cfg):
    d, H, F, L = gpt2_cfg["n_embd"], gpt2_cfg["n_head"], gpt2_cfg["n_inner"], gpt2_cfg["n_layer"]
    hd = d // H
    mlp = {"kind": "dense", "ff": F}
    kinds = [
        {"type": "general_delta", "mixer": {"heads": H, "dim": hd, "decay_rank": 64}},
        {"type": "attention", "mixer": {"heads": H, "kv_heads": H, "dim": hd // 2, "vdim": hd, "scale": (hd // 2) ** -0.5, "diff": 0.5, "conv": 4,
                                        "mask": {"size": gpt2_cfg["n_positions"]}}},
        {"type": "latent_attention", "mixer": {"heads": H, "dim": hd, "vdim": hd, "kv_rank": 128, "q_rank": d // 2 // 64 * 64,
                                               "scale": hd ** -0.5}},
    ]
    layers = [dict(json.loads(json.dumps(kinds[i % 3])), mlp=dict(mlp)) for i in range(L)]
    return {"architecture": "Dopilorn", "vocab": gpt2_cfg["vocab_size"], "width": d, "norm": {"eps": 1e-5}, "canon": {"taps": 4}, "logit_softcap": 30.0,
            "max_positions": gpt2_cfg["n_positions"], "layers": layers}


def _dopilorn_layer_weights(entry, d):
    """Matrix elements of a layer (what a step reads of it; all of them are products' operands, 2 flops an element a token)."""
    m, kind = entry["mixer"], entry["type"]
    n = 2 * entry["mlp"]["ff"] * d if entry.get("mlp") else 0
    H, D = m["heads"], m["dim"]
    if kind == "general_delta":
        R = m.get("decay_rank", 16)
        n += 5 * H * D * d + R * d + H * D * R + d * H * D
    elif kind == "attention":
        G, V = m.get("kv_heads", H), m.get("vdim", D)
        n += (2 * H * D + 2 * G * D + G * V) * d + d * H * V
    else:
        V, R, Q = m["vdim"], m["kv_rank"], m["q_rank"]
        n += (Q + R + H) * d + H * D * Q + H * (D + V) * R + d * H * V
    return n


def dopilorn_step_bytes(cfg, batch):
    """The bytes a decode step has to read: every matrix once, the head, the cached rows inside the windows (two planes of keys
    and one of values, padded to one width; one latent row), and the 32-bit state of the recurrent layers (read and written)."""
    def step_bytes(contexts, steps, elt):
        d, V = cfg["width"], cfg["vocab"]
        total = V * d * elt
        for entry in cfg["layers"]:
            m = entry["mixer"]
            total += _dopilorn_layer_weights(entry, d) * elt
            if entry["type"] == "general_delta":
                total += len(contexts) * 2 * m["heads"] * m["dim"] * m["dim"] * 4
            elif entry["type"] == "attention":
                window = (m.get("mask") or {}).get("size", 0)
                seen = sum(sum(min(c + s + 1, window) if window else c + s + 1 for s in range(steps)) for c in contexts) / max(steps, 1)
                P = -(-max(m["dim"], m.get("vdim", m["dim"])) // 8) * 8
                total += seen * 3 * m.get("kv_heads", m["heads"]) * P * elt
            else:
                seen = sum(sum(c + s + 1 for s in range(steps)) for c in contexts) / max(steps, 1)
                total += seen * m["kv_rank"] * elt
        return total
    return step_bytes


def dopilorn_prefill_flops(cfg, prompt_lens, logit_rows):
    d, V, n = cfg["width"], cfg["vocab"], sum(prompt_lens)
    flops = 2.0 * logit_rows * d * V
    for entry in cfg["layers"]:
        m = entry["mixer"]
        flops += 2.0 * n * _dopilorn_layer_weights(entry, d)
        if entry["type"] == "general_delta":
            flops += n * m["heads"] * 8.0 * m["dim"] * m["dim"]  # a token: what the key sees, the state's update, its read, a head
        elif entry["type"] == "attention":
            window = (m.get("mask") or {}).get("size", 0)
            pairs = sum(sum(min(i + 1, window) if window else i + 1 for i in range(t)) for t in prompt_lens)
            flops += 2.0 * pairs * m["heads"] * 2 * (m["dim"] + m.get("vdim", m["dim"]))
        else:
            pairs = sum(t * (t + 1) / 2 for t in prompt_lens)
            flops += 2.0 * pairs * m["heads"] * 2 * m["kv_rank"]
    return flops


# -- Larulorn beside Mofulix at equal sizes -------------------------------------------------------------------
# The Larulorn of each size has GPT-2's width, layers, vocabulary and head count (heads of 64 everywhere); its layers take turns as
# attention with a sink and biases (as many key heads as query heads, turned halves on a ramp, values mixed with the first layer's)
# over a clamped feed-forward as Mofulix's, gated attention beside a gated linear recurrence as wide as the model (a part a head, four
# taps) over the same feed-forward, and attention again over eight experts of a quarter of GPT-2's inner width in four groups of which
# two stay, two experts a token, beside a shared expert of that width. It stands beside Mofulix, the engine's other design that mixes
# recurrences with attention under a clamped feed-forward.
def larulorn_config(gpt2_cfg):
    d, H, F, L = gpt2_cfg["n_embd"], gpt2_cfg["n_head"], gpt2_cfg["n_inner"], gpt2_cfg["n_layer"]
    hd = d // H
    ff = max(64, F * 2 // 3 // 64 * 64)
    dense = {"kind": "dense", "ff": ff, "limit": 7.0}
    moe = {"kind": "moe", "expert": {"ff": F // 4}, "router": {"experts": 8, "top": 2, "groups": {"count": 4, "keep": 2}}, "shared": {"ff": F // 4}}
    rot = {"dims": hd, "base": 10000.0, "scaling": {"factor": 8.0, "original": 8192, "fast": 32.0, "slow": 1.0}}
    own = {"heads": H, "kv_heads": H, "dim": hd, "vdim": hd, "scale": hd ** -0.5, "rot": rot, "v_mix": True}
    kinds = [
        {"type": "attention", "mixer": own, "mlp": dense},
        {"type": "parallel", "mixer": {"left": {"heads": H, "kv_heads": H, "dim": hd, "vdim": hd, "scale": hd ** -0.5, "rot": {"dims": hd, "base": 10000.0}},
                                       "right": {"width": d, "blocks": H, "conv": 4}, "left_scale": 0.75, "right_scale": 1.25}, "mlp": dense},
        {"type": "attention", "mixer": own, "mlp": moe},
    ]
    return {"architecture": "Larulorn", "vocab": gpt2_cfg["vocab_size"], "width": d, "norm": {"eps": 1e-5}, "logit_scale": 1.0,
            "max_positions": gpt2_cfg["n_positions"], "layers": [json.loads(json.dumps(kinds[i % 3])) for i in range(L)]}


def _larulorn_layer_weights(entry, d, per_token=True):
    """Matrix elements of a layer that a token's products read (2 flops an element a token); with `per_token` False, those a decode
    step of many requests reads at most (every expert)."""
    m, mlp = entry["mixer"], entry.get("mlp")
    n = 0
    if mlp and mlp["kind"] == "dense":
        n += 3 * mlp["ff"] * d
    elif mlp:
        r = mlp["router"]
        n += r["experts"] * d + (r["top"] if per_token else r["experts"]) * 2 * mlp["expert"]["ff"] * d + 2 * (mlp.get("shared") or {"ff": 0})["ff"] * d
    a = m if entry["type"] == "attention" else m["left"]
    n += (a["heads"] * a["dim"] + a["kv_heads"] * (a["dim"] + a["vdim"])) * d + d * a["heads"] * a["vdim"]
    if entry["type"] == "parallel":
        W, B = m["right"]["width"], m["right"]["blocks"]
        n += a["heads"] * a["vdim"] * d + 3 * W * d + 2 * W * (W // B)
    return n


def larulorn_step_bytes(cfg, batch):
    """The bytes a decode step has to read: every matrix a token of the batch can take (min(batch * top, experts) experts), the head, the
    cached keys and values, and the 32-bit state of the recurrent layers (read and written) a request."""
    def step_bytes(contexts, steps, elt):
        d, V = cfg["width"], cfg["vocab"]
        total = V * d * elt
        seen = sum(sum(c + s + 1 for s in range(steps)) for c in contexts) / max(steps, 1)
        for entry in cfg["layers"]:
            m, mlp = entry["mixer"], entry.get("mlp")
            n = _larulorn_layer_weights(entry, d, per_token=True)
            if mlp and mlp["kind"] == "moe":
                r = mlp["router"]
                n += (min(len(contexts) * r["top"], r["experts"]) - r["top"]) * 2 * mlp["expert"]["ff"] * d
            total += n * elt
            a = m if entry["type"] == "attention" else m["left"]
            total += seen * a["kv_heads"] * (a["dim"] + a["vdim"]) * elt
            if entry["type"] == "parallel":
                total += len(contexts) * 2 * m["right"]["width"] * m["right"]["conv"] * 4
        return total
    return step_bytes


def larulorn_prefill_flops(cfg, prompt_lens, logit_rows):
    d, V, n = cfg["width"], cfg["vocab"], sum(prompt_lens)
    flops = 2.0 * logit_rows * d * V
    pairs = sum(t * (t + 1) / 2 for t in prompt_lens)
    for entry in cfg["layers"]:
        m = entry["mixer"]
        a = m if entry["type"] == "attention" else m["left"]
        flops += 2.0 * n * _larulorn_layer_weights(entry, d) + 2.0 * pairs * a["heads"] * (a["dim"] + a["vdim"])
    return flops


# The Lolulorn of each size has GPT-2's width, layers, vocabulary and head count (heads of 64 everywhere); its layers take turns as a gated
# delta rule (half as many query/key heads as value heads where the number is even, four taps) over a gated feed-forward two thirds as wide
# as GPT-2's, gated linear attention (a decay of rank 16) over eight gated experts of a quarter of GPT-2's inner width in four groups of
# which two stay, two a token, and attention under a window of half the positions behind which four first positions stay visible, over the
# same dense feed-forward; every second attention layer reads the keys and values of the one before it. It stands beside Larulorn, the
# engine's closest design: attention and recurrences, one sublayer after the other with a norm behind each, experts chosen among groups.
def lolulorn_config(gpt2_cfg):
    d, H, F, L = gpt2_cfg["n_embd"], gpt2_cfg["n_head"], gpt2_cfg["n_inner"], gpt2_cfg["n_layer"]
    hd = d // H
    dense = {"kind": "dense", "ff": max(64, F * 2 // 3 // 64 * 64)}
    moe = {"kind": "moe", "expert": {"ff": F // 4}, "router": {"experts": 8, "top": 2, "groups": {"count": 4, "keep": 2}}}
    attention = {"heads": H, "kv_heads": H, "dim": hd, "vdim": hd, "scale": hd ** -0.5, "mask": {"size": gpt2_cfg["n_positions"] // 2, "keep_first": 4},
                 "rot": {"dims": hd, "base": 10000.0, "scaling": {"factor": 4.0}}}
    layers = []
    for i in range(L):
        if i % 3 == 0:
            layers.append({"type": "delta", "mixer": {"heads": H, "kv_heads": H // 2 if H % 2 == 0 else H, "dim": hd, "vdim": hd, "conv": 4}, "mlp": dense})
        elif i % 3 == 1:
            layers.append({"type": "gla", "mixer": {"heads": H, "dim": hd, "vdim": hd, "tau": 16.0, "decay_rank": 16}, "mlp": moe})
        else:
            layers.append({"type": "attention", "mixer": dict(attention, **({"kv_from": i - 3} if i % 6 == 5 else {})), "mlp": dense})
    return {"architecture": "Lolulorn", "vocab": gpt2_cfg["vocab_size"], "width": d, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5},
            "max_positions": gpt2_cfg["n_positions"], "layers": json.loads(json.dumps(layers))}


def _lolulorn_layer_weights(entry, d, experts=None):
    """Matrix elements of a layer that a token's products read (2 flops an element a token), with `experts` experts in place of a token's own."""
    m, mlp = entry["mixer"], entry.get("mlp")
    n = 0
    if mlp and mlp["kind"] == "dense":
        n += 3 * mlp["ff"] * d
    elif mlp:
        n += mlp["router"]["experts"] * d + (experts or mlp["router"]["top"]) * 3 * mlp["expert"]["ff"] * d
    H, D, V = m["heads"], m["dim"], m["vdim"]
    n += d * H * V
    if entry["type"] == "attention":
        n += H * D * d + (0 if "kv_from" in m else m["kv_heads"] * (D + V) * d)
    elif entry["type"] == "delta":
        n += (2 * m["kv_heads"] * D + 2 * H * V + 2 * H) * d
    else:
        n += (2 * H * D + 2 * H * V + m["decay_rank"]) * d + H * D * m["decay_rank"]
    return n


def lolulorn_step_bytes(cfg, batch):
    """The bytes a decode step has to read: every matrix a token of the batch can take (min(batch * top, experts) experts), the head, the
    cached keys and values inside each request's window, and the 32-bit state of the recurrent layers (read and written) a request."""
    def step_bytes(contexts, steps, elt):
        d, V = cfg["width"], cfg["vocab"]
        total = V * d * elt
        for entry in cfg["layers"]:
            m, mlp = entry["mixer"], entry.get("mlp")
            r = mlp["router"] if mlp and mlp["kind"] == "moe" else None
            total += _lolulorn_layer_weights(entry, d, min(len(contexts) * r["top"], r["experts"]) if r else None) * elt
            if entry["type"] == "attention":
                reach = m["mask"]["size"] + m["mask"]["keep_first"]
                seen = sum(sum(min(c + s + 1, reach) for s in range(steps)) for c in contexts) / max(steps, 1)
                total += seen * m["kv_heads"] * (m["dim"] + m["vdim"]) * elt
            else:
                total += len(contexts) * 2 * m["heads"] * m["dim"] * m["vdim"] * 4
                if entry["type"] == "delta":
                    total += len(contexts) * m["conv"] * (2 * m["kv_heads"] * m["dim"] + m["heads"] * m["vdim"]) * 4
        return total
    return step_bytes


def lolulorn_prefill_flops(cfg, prompt_lens, logit_rows):
    d, V, n = cfg["width"], cfg["vocab"], sum(prompt_lens)
    flops = 2.0 * logit_rows * d * V
    for entry in cfg["layers"]:
        m = entry["mixer"]
        flops += 2.0 * n * _lolulorn_layer_weights(entry, d)
        if entry["type"] == "attention":
            reach = m["mask"]["size"] + m["mask"]["keep_first"]
            flops += 2.0 * sum(min(i + 1, reach) for t in prompt_lens for i in range(t)) * m["heads"] * (m["dim"] + m["vdim"])
        else:
            flops += n * m["heads"] * m["dim"] * m["vdim"] * (8.0 if entry["type"] == "delta" else 5.0)  # (the recurrence token by token)
    return flops


# The Lafanex of each size has GPT-2's width, layers, vocabulary and head count, and two residual streams; its layers take turns as attention
# (as many key heads as query heads, whole heads turned) over a gated feed-forward two thirds as wide as GPT-2's, a selective scan twice as wide as the
# model (16 states a channel, a rank of a sixteenth of the width, four taps) over the same feed-forward, and attention again over eight gated experts of a
# quarter of GPT-2's inner width and two identity experts, two a token, beside a shared expert of that width. It stands beside Larulorn, the engine's
# closest design: attention with sinks and a recurrence a channel, a norm before each sublayer, experts beside a shared one.
def lafanex_config(gpt2_cfg):
    d, H, F, L = gpt2_cfg["n_embd"], gpt2_cfg["n_head"], gpt2_cfg["n_inner"], gpt2_cfg["n_layer"]
    hd = d // H
    dense = {"kind": "dense", "ff": max(64, F * 2 // 3 // 64 * 64)}
    expert = {"ff": F // 4, "limit": 7.0}
    moe = {"kind": "moe", "expert": expert, "router": {"experts": 8, "top": 2, "identity": 2, "scale": 2.5}, "shared": expert}
    attention = {"heads": H, "kv_heads": H, "dim": hd, "vdim": hd, "scale": hd ** -0.5, "rot": {"dims": hd, "base": 10000.0}}
    kinds = [{"type": "attention", "mixer": attention, "mlp": dense},
             {"type": "mamba1", "mixer": {"inner": 2 * d, "state": 16, "dt_rank": max(8, d // 16), "conv": 4}, "mlp": dense},
             {"type": "attention", "mixer": attention, "mlp": moe}]
    return {"architecture": "Lafanex", "vocab": gpt2_cfg["vocab_size"], "width": d, "streams": 2, "norm": {"eps": 1e-5}, "max_positions": gpt2_cfg["n_positions"],
            "layers": [json.loads(json.dumps(kinds[i % 3])) for i in range(L)]}


def _lafanex_layer_weights(entry, d, experts=None):
    """Matrix elements of a layer that a token's products read (2 flops an element a token), with `experts` experts in place of a token's own
    (an identity expert, which has none, taken as one with)."""
    m, mlp = entry["mixer"], entry.get("mlp")
    n = 0
    if mlp and mlp["kind"] == "dense":
        n += 3 * mlp["ff"] * d
    elif mlp:
        r = mlp["router"]
        n += (r["experts"] + r["identity"] + 1) * d + (experts or r["top"]) * 3 * mlp["expert"]["ff"] * d + 3 * mlp["shared"]["ff"] * d
    if entry["type"] == "attention":
        return n + (m["heads"] * m["dim"] + m["kv_heads"] * (m["dim"] + m["vdim"])) * d + d * m["heads"] * m["vdim"]
    W = m["inner"]
    return n + 3 * W * d + (2 * m["dt_rank"] + 2 * m["state"]) * W


def lafanex_step_bytes(cfg, batch):
    """The bytes a decode step has to read: every matrix a token of the batch can take (min(batch * top, experts) experts), the head, the
    cached keys and values, and the 32-bit state of the recurrent layers (read and written) a request."""
    def step_bytes(contexts, steps, elt):
        d, V = cfg["width"], cfg["vocab"]
        total = V * d * elt
        seen = sum(sum(c + s + 1 for s in range(steps)) for c in contexts) / max(steps, 1)
        for entry in cfg["layers"]:
            m, mlp = entry["mixer"], entry.get("mlp")
            r = mlp["router"] if mlp and mlp["kind"] == "moe" else None
            total += _lafanex_layer_weights(entry, d, min(len(contexts) * r["top"], r["experts"]) if r else None) * elt
            if entry["type"] == "attention":
                total += seen * m["kv_heads"] * (m["dim"] + m["vdim"]) * elt
            else:
                total += len(contexts) * 4 * m["inner"] * (2 * m["state"] + m["conv"]) + 4 * m["inner"] * m["state"]
        return total
    return step_bytes


def lafanex_prefill_flops(cfg, prompt_lens, logit_rows):
    d, V, n = cfg["width"], cfg["vocab"], sum(prompt_lens)
    flops = 2.0 * logit_rows * d * V
    pairs = sum(t * (t + 1) / 2 for t in prompt_lens)
    for entry in cfg["layers"]:
        m = entry["mixer"]
        flops += 2.0 * n * _lafanex_layer_weights(entry, d)
        if entry["type"] == "attention":
            flops += 2.0 * pairs * m["heads"] * (m["dim"] + m["vdim"])
        else:
            flops += n * m["inner"] * m["state"] * 7.0  # (the recurrence token by token)
    return flops


DESIGNS = {"bokulix": (lambda gpt2, size: bokulix_config(gpt2, BOKULIX_SHAPES[size]), bokulix_step_bytes, bokulix_prefill_flops),
           "mofulix": (lambda gpt2, size: mofulix_config(gpt2), mofulix_step_bytes, mofulix_prefill_flops),
           "dopilorn": (lambda gpt2, size: dopilorn_config(gpt2), dopilorn_step_bytes, dopilorn_prefill_flops),
           "larulorn": (lambda gpt2, size: larulorn_config(gpt2), larulorn_step_bytes, larulorn_prefill_flops),
           "lolulorn": (lambda gpt2, size: lolulorn_config(gpt2), lolulorn_step_bytes, lolulorn_prefill_flops),
           "lafanex": (lambda gpt2, size: lafanex_config(gpt2), lafanex_step_bytes, lafanex_prefill_flops)}
BESIDE = {"dopilorn": "mofulix", "larulorn": "mofulix", "lolulorn": "larulorn", "lafanex": "larulorn"}  # the engine's closest model, where that is not GPT-2


def design_run(args):
    """A design and GPT-2 side by side at each of the named sizes: a prefill of 2,048 tokens (two prompts of 1,024) with its
    share of the matrix peak, and decode steps at batch 1, 8 and 64 with their share of the HBM roofline."""
    from liyab_amd.weights import write_random_model

    make_config, step_bytes_of, flops_of = DESIGNS[args.design]
    short = "bf16" if args.dtype == "bfloat16" else "fp32"
    runs = []
    for size in args.design_sizes.split(","):
        gpt2 = dict(SMALL, **SIZES[size])
        if args.layers:
            gpt2["n_layer"] = args.layers
        beside = BESIDE.get(args.design, "gpt2")
        designs = {beside: gpt2 if beside == "gpt2" else DESIGNS[beside][0](gpt2, size), args.design: make_config(gpt2, size)}
        if args.design_only:
            del designs[beside]
        ctx = gpt2["n_positions"]
        k = max(16, min(args.steps, 128, ctx - args.prompt - 16))
        for name, cfg in designs.items():
            with tempfile.TemporaryDirectory() as d:
                write_random_model(d, cfg, WEIGHT_SEEDS[size], dtype="bfloat16" if short == "bf16" else "float32")
                engine = make_engine(d, args.dtype, 64, ctx, page_size=args.page_size, phases=args.phases)
                lens = [1024, 1024]
                ptps, pms = prefill_run(engine, cfg, lens)
                flops = DESIGNS[name][2](cfg, lens, 2) if name != "gpt2" else prefill_flops(cfg, lens, 2)
                run = {"design": name, "size": size, "layers": gpt2["n_layer"],
                       "prefill": {"tokens": 2048, "tok_s": round(ptps, 1), "ms": round(pms, 4), "gflop": round(flops / 1e9, 1),
                                   "frac_of_matrix_peak": round(flops / (pms * 1e-3) / MFMA_PEAK[short], 4)}}
                if args.phases:
                    run["prefill"]["phases_ms"] = {n: round(v / 7, 4) for n, v in engine.phases_ms(reset=True).items()}  # (prefill_run steps 7 times)
                for b in (1, 8, 64):
                    bytes_fn = DESIGNS[name][1](cfg, b) if name != "gpt2" else None
                    t, ms, nbytes = decode_run(engine, cfg, b, args.prompt, k, 4, step_bytes=bytes_fn)
                    run[f"decode_b{b}"] = {"tok_s": round(t, 1), "ms_per_step": round(ms, 4), "mbytes_per_step": round(nbytes / 1e6, 1),
                                           "frac_of_hbm_peak": round(nbytes / (ms * 1e-3) / 1e9 / HBM_PEAK_GBS, 4)}
                    if args.phases:
                        # the run's prompts went through the same timer: the same prompts alone are taken off
                        whole = engine.phases_ms(reset=True)
                        decode_run(engine, cfg, b, args.prompt, 0, 0, step_bytes=bytes_fn)
                        prompts = engine.phases_ms(reset=True)
                        run[f"decode_b{b}"]["phases_ms"] = {n: round(max(v - prompts.get(n, 0.0), 0.0) / (k + 4), 4) for n, v in whole.items()}
                runs.append(run)
                del engine
    print(json.dumps({"metric": f"{args.design.capitalize()} beside {BESIDE.get(args.design, 'GPT-2').capitalize() if args.design in BESIDE else 'GPT-2'} at equal layer sizes: prefill of 2,048 tokens and decode steps", "dtype": short,
                      "data": "synthetic", "page_size": args.page_size, "prompt_len": args.prompt, "runs": runs}))
    return 0


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=504)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--size", default="small", choices=sorted(SIZES), help="GPT-2 small's sizes (the default), medium's, large's or XL's; or layers of width 4,096")
    ap.add_argument("--layers", type=int, default=0, help="fewer layers than the configuration has, if needed")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--prompt", type=int, default=512)
    ap.add_argument("--positions", type=int, default=0, help="a longer context than the size's own (the position table grows), e.g. 8192 with --prompt 7000")
    ap.add_argument("--no-points", action="store_true", help="skip the batch 1 / 64 points and the prefill")
    ap.add_argument("--prefill-only", action="store_true", help="run only the prefill of 2,048 tokens (for profiling)")
    ap.add_argument("--prefill-tokens", default="", help="e.g. 512,2048,8192: best-of-5 prefill tokens a second per length, "
                    "in prompts of up to 1,024 tokens (the reference's liyab-bench --prefill --tokens)")
    ap.add_argument("--sequences", default="", help="e.g. 1,2,4: that many sequences together against one after the other "
                    "(the reference's liyab-seq-bench): tokens a second both ways and whether every reply equals its reply alone")
    ap.add_argument("-n", type=int, default=128, help="tokens generated per sequence with --sequences")
    ap.add_argument("--workload", default="", choices=["", "medium16", "xl64"],
                    help="medium16: GPT-2 medium's sizes, 16 requests with prompts of 64 to 1,023 tokens, portions of 256, 128 greedy "
                         "tokens each; xl64: GPT-2 XL's sizes, 64 requests with prompts of 256 tokens decoding to 1,024, greedy and at temperature 1")
    ap.add_argument("--page-size", type=int, default=64, help="positions a cache page (default 64; the engine's own default is 16)")
    ap.add_argument("--batch-invariant", action="store_true", help="kernels chosen from sizes and positions only (reproducible bfloat16 replies)")
    ap.add_argument("--product", default="", help="M,N,K[,tile,...]: time one bfloat16 product in the tiled kernel's tiles (0: its own choice, 6: 64 x 64, 8: 128 x 128, 15: 256 x 256)")
    ap.add_argument("--link-floor", action="store_true", help="measure what one dependent kernel of a replayed graph costs at least")
    ap.add_argument("--phases", action="store_true", help="device milliseconds per phase of the forward pass (embed, attention, dense_ffn, lm_head) a decode step "
                    "and a prefill of 2,048 tokens, as the reference's command line prints them (tools/liyab_cli.cpp:198-211); steps run kernel by kernel, without graphs")
    ap.add_argument("--design", default="", choices=["", "bokulix", "mofulix", "dopilorn", "larulorn", "lolulorn", "lafanex"],
                    help="bokulix, mofulix: that design beside GPT-2 at equal layer sizes (prefill and decode, both with their rooflines); "
                         "dopilorn, larulorn: beside Mofulix, lolulorn, lafanex: beside Larulorn, the engine's closest model")
    ap.add_argument("--design-only", action="store_true", help="with --design: skip the GPT-2 run (for profiling)")
    ap.add_argument("--design-sizes", default="small,medium,xl", help="the sizes --design runs (of small, medium, xl)")
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} is not supported")
        return 2
    import torch

    from liyab_amd.weights import write_random_model

    if args.product:
        sizes = [int(x) for x in args.product.split(",")]
        print(json.dumps(product_run(sizes[0], sizes[1], sizes[2], sizes[3:] or [0])))
        return 0
    if args.link_floor:
        print(json.dumps(link_floor()))
        return 0
    if args.design:
        return design_run(args)
    if args.workload:
        args.size = "medium" if args.workload == "medium16" else "xl"
    cfg = dict(SMALL, **SIZES[args.size])
    full_layers = cfg["n_layer"]
    if args.layers:
        cfg["n_layer"] = args.layers
    if args.positions:
        cfg["n_positions"] = args.positions
    ctx = cfg["n_positions"]
    steps = max(1, min(args.steps, ctx - args.prompt - args.warmup))
    short = "bf16" if args.dtype == "bfloat16" else "fp32"
    with tempfile.TemporaryDirectory() as d:
        write_random_model(d, cfg, WEIGHT_SEEDS[args.size], dtype="bfloat16" if short == "bf16" else "float32")
        slots = max(args.batch, 64 if not args.no_points else args.batch)
        if args.prefill_tokens:
            slots = max(slots, max(-(-int(x) // ctx) for x in args.prefill_tokens.split(",")))
        if args.workload:
            import numpy as np

            from liyab_amd import SamplingParams

            layers_note = {"n_layer": cfg["n_layer"], "n_layer_full": full_layers}
            if args.workload == "medium16":
                # the continuous-batching workload at GPT-2 medium's sizes: 16 requests, prompt lengths uniform in [64, 1024) and ids
                # from seed 21, continuously batched with portions of 256, 128 greedy tokens each (capped at the positions)
                rng = np.random.default_rng(21)
                lens = rng.integers(64, 1024, 16).tolist()
                prompts = [rng.integers(0, cfg["vocab_size"], n).tolist() for n in lens]
                engine = make_engine(d, args.dtype, 16, ctx, page_size=args.page_size, prefill_chunk=256, batch_invariant=args.batch_invariant)
                engine.warmup()
                runs = {}
                for rep in range(2):  # the second run finds its recurring shapes captured
                    runs["greedy"], _ = workload_run(engine, cfg, prompts, lambda i: SamplingParams(temperature=0.0, max_tokens=128), f"m{rep}")
                print(json.dumps({"metric": "GPT-2 medium sizes: 16 requests, prompts of 64 to 1,023 tokens in portions of 256, 128 greedy tokens each",
                                  "dtype": short, "data": "synthetic", "page_size": args.page_size, **layers_note,
                                  "prompt_lens": lens, "runs": runs}))
            else:
                # the batch-64 workload at GPT-2 XL's sizes: 64 requests, prompts of 256 ids from seed 31, decoding to 1,024
                # positions, greedy and at temperature 1
                rng = np.random.default_rng(31)
                prompts = [rng.integers(0, cfg["vocab_size"], 256).tolist() for _ in range(64)]
                engine = make_engine(d, args.dtype, 64, ctx, page_size=args.page_size, prefill_chunk=256, batch_invariant=args.batch_invariant)
                engine.warmup()
                runs = {}
                n_new = ctx - 256 + 1
                for name, make in (("greedy", lambda i: SamplingParams(temperature=0.0, max_tokens=n_new)),
                                   ("temperature 1.0", lambda i: SamplingParams(temperature=1.0, top_k=0, top_p=1.0, seed=1000 + i, max_tokens=n_new))):
                    runs[name], _ = workload_run(engine, cfg, prompts, make, name[:1])
                print(json.dumps({"metric": "GPT-2 XL sizes: 64 requests, prompts of 256 tokens decoding to 1,024 positions",
                                  "dtype": short, "data": "synthetic", "page_size": args.page_size, **layers_note, "runs": runs}))
            return 0
        engine = make_engine(d, args.dtype, slots, ctx, page_size=args.page_size, batch_invariant=args.batch_invariant)
        if args.prefill_tokens:
            runs = []
            for total in [int(x) for x in args.prefill_tokens.split(",")]:
                lens = [ctx] * (total // ctx) + ([total % ctx] if total % ctx else [])
                ptps, pms = prefill_run(engine, cfg, lens)
                flops = prefill_flops(cfg, lens, len(lens))
                runs.append({"tokens": total, "prompts": len(lens), "value": round(ptps, 1), "ms": round(pms, 4),
                             "frac": round(flops / (pms * 1e-3) / MFMA_PEAK[short], 4)})
            print(json.dumps({"metric": f"prefill tok/s (GPT-2 {args.size} sizes)", "dtype": short, "runs": runs}))
            return 0
        if args.sequences:
            print(json.dumps(sequences_run(engine, cfg, [int(x) for x in args.sequences.split(",")], args.prompt, args.n)))
            return 0
        if args.phases:
            timed = make_engine(d, args.dtype, max(args.batch, 2), ctx, page_size=args.page_size, batch_invariant=args.batch_invariant, phases=True)
            k = min(steps, 64)
            decode_run(timed, cfg, args.batch, args.prompt, 4, 2)  # every kernel has run once
            timed.phases_ms(reset=True)
            tps, ms, _ = decode_run(timed, cfg, args.batch, args.prompt, k, 0, seed=12)
            whole = timed.phases_ms(reset=True)  # the prompts of the run, too: taken off below
            prefill_run(timed, cfg, [1024, 1024], repeat=1)
            prefill = timed.phases_ms(reset=True)
            per = lambda table, n: {name: round(v / n, 4) for name, v in table.items()}  # noqa: E731
            # the prompts of the decode run went through the same timer: one step of `batch` prompts of args.prompt tokens
            timed.phases_ms(reset=True)
            decode_run(timed, cfg, args.batch, args.prompt, 0, 0, seed=12)
            prompts_only = timed.phases_ms(reset=True)
            decode = {name: max(whole.get(name, 0.0) - prompts_only.get(name, 0.0), 0.0) for name in whole}
            print(json.dumps({"metric": f"device ms per phase (GPT-2 {args.size} sizes, {short}; steps launched kernel by kernel)",
                              "decode_step": {"batch": args.batch, "steps": k, "phases_ms": per(decode, k), "ms_per_step_wall": round(ms, 4)},
                              "prefill_2048": {"phases_ms": per(prefill, 3)}}))
            return 0
        if args.prefill_only:
            ptps, pms = prefill_run(engine, cfg, [1024, 1024], repeat=20)
            print(json.dumps({"prefill": {"value": round(ptps, 1), "tokens": 2048, "ms": round(pms, 4)}}))
            return 0
        tps, ms, bytes_per_step = decode_run(engine, cfg, args.batch, args.prompt, steps, args.warmup)
        achieved = bytes_per_step / (ms * 1e-3) / 1e9
        out = {
            "metric": f"decode tok/s (GPT-2 {args.size} sizes, batch {args.batch}, {args.prompt}-token prompts decoding to {ctx})",
            "value": round(tps, 1), "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": args.warmup,
            "ms_per_step": round(ms, 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
            "dtype": short, "data": "synthetic",
            "config": {"model": f"gpt2-{args.size}-sizes-random-weights", "n_layer": cfg["n_layer"], "n_layer_full": full_layers,
                       "n_embd": cfg["n_embd"], "n_head": cfg["n_head"], "head_dim": cfg["n_embd"] // cfg["n_head"],
                       "n_inner": cfg["n_inner"], "vocab_size": cfg["vocab_size"], "n_positions": cfg["n_positions"],
                       "global_batch": args.batch, "seq_len": ctx, "prompt_len": args.prompt, "page_size": args.page_size,
                       "batch_invariant": bool(args.batch_invariant),
                       "weights_seed": WEIGHT_SEEDS[args.size], "ids_seed": 11, "parallelism": "single-gpu"},
            "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                         "frac": round(achieved / HBM_PEAK_GBS, 4)},
        }
        if not args.no_points:
            out["roofline"]["measured_copy"] = round(copy_bandwidth(), 1)  # a 1 GiB device-to-device copy on this machine, GB/s
        if not args.no_points:
            lens = [1024, 1024]
            ptps, pms = prefill_run(engine, cfg, lens)
            flops = prefill_flops(cfg, lens, len(lens))
            out["prefill"] = {"value": round(ptps, 1), "tokens": sum(lens), "ms": round(pms, 4),
                              "frac": round(flops / (pms * 1e-3) / MFMA_PEAK[short], 4)}
            out["ttft"] = ttft_run(engine, cfg, min(args.prompt, ctx - 16))
            # every point over at least 64 steps after at least 3 of its own shape, whatever --steps says: fewer do
            # not outlast the first sight of a shape (an eager run, then a capture)
            points = {}
            k, w = min(max(steps, 64), 256, ctx - args.prompt - 8), max(args.warmup, 3)
            for b in (1, 64):
                t, pms_b, pbytes = decode_run(engine, cfg, b, args.prompt, k, w)
                points[f"decode_b{b}"] = round(t, 1)
                points[f"decode_b{b}_ms_per_step"] = round(pms_b, 4)
                points[f"decode_b{b}_mbytes_per_step"] = round(pbytes / 1e6, 1)
                points[f"decode_b{b}_roofline_frac"] = round(pbytes / (pms_b * 1e-3) / 1e9 / HBM_PEAK_GBS, 4)
            points["steps_per_point"] = k
            if args.page_size != 16:
                # the headline batch again with pages of 16 positions, the engine's own default
                small_pages = make_engine(d, args.dtype, args.batch, ctx, page_size=16, batch_invariant=args.batch_invariant)
                t, pms_b, _ = decode_run(small_pages, cfg, args.batch, args.prompt, k, w)
                points[f"decode_b{args.batch}_page16"] = round(t, 1)
                points[f"decode_b{args.batch}_page16_ms_per_step"] = round(pms_b, 4)
                del small_pages
            # the headline batch in the engine's two other modes: replies that do not depend on the batch, and the 32-bit path
            others = []
            if not args.batch_invariant and short == "bf16":
                others.append((f"decode_b{args.batch}_batch_invariant", args.dtype, True))
            if short == "bf16":
                others.append((f"decode_b{args.batch}_fp32", "float32", False))
            del engine
            for name, dtype, invariant in others:
                other = make_engine(d, dtype, args.batch, ctx, page_size=args.page_size, batch_invariant=invariant)
                t, pms_b, _ = decode_run(other, cfg, args.batch, args.prompt, k, w)
                points[name] = round(t, 1)
                points[name + "_ms_per_step"] = round(pms_b, 4)
                del other
            out["points"] = points
    print(json.dumps(out))
    return 0


if __name__ == "__main__":
    sys.exit(main())
