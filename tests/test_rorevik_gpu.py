"""Rorevik on the GPU: bin/trace_run as a child process (whole prompts, decoded tails, portions down to two
tokens, mixed batches in a pool of the live peak with four slots) in float32 and bfloat16 against the plain model,
with weights made so that single keys, the cap on the scores, the positions, the convolutions' taps, the states' memory,
channels that forget at once and channels that do not, and every factor and bias carry the result; every layer run's residual stream; long
decoding through captured graphs with a slot used again; generation through the Python entry point and the
command line."""
import os
import subprocess
import sys

import pytest
import torch

from tests.plain import rorevik_plain as plain
from tests.rorevik_util import (CONFIGS, PAGE_SIZES, delta, layer, make_model_dir, parallel, plain_logits, read, residual_streams, run_tool,
                                sharpen)
from tests.tiny import random_tokens
from tests.trace_util import ROOT, TraceBuilder, changing_portions, check_dumps, mixed, tail_one_by_one, whole

pytestmark = pytest.mark.gpu

# About five times the worst error seen.  Sharpened scores, gates and decays turn the rounding of their bfloat16 inputs
# into tenths of the largest logit: the bfloat16 runs sharpen less and pin gross faults, what is exact is pinned by the
# float32 runs.
TOL = {"float32": 1.5e-4, "bfloat16": 1e-1}
SHARP = {"float32": 2.0, "bfloat16": 0.5}
GENTLE = {"float32": (), "bfloat16": (".g1", ".g2", ".a1", ".a2", ".in")}
LENGTHS = {"a": 70, "b": 45, "c": 100, "d": 33, "e": 64, "f": 1, "g": 2}


def all_ways_trace(requests, tail=32):
    tb = TraceBuilder()
    names = list(requests)
    whole(tb, names[0] + "#whole", requests[names[0]])
    whole(tb, names[2] + "#whole", requests[names[2]])
    tail_one_by_one(tb, names[1] + "#tail", requests[names[1]], tail=tail)
    changing_portions(tb, names[2] + "#cut", requests[names[2]], seed=1)
    changing_portions(tb, names[4] + "#cut", requests[names[4]], seed=2)
    mixed(tb, {rid + "#mix": t for rid, t in requests.items()}, seed=5)
    return tb


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "A/default page", "B", "C", "D"])
def test_trace_gpu(tmp_path, which, dtype):
    which, default_page = which[0], len(which) > 1
    d = make_model_dir(tmp_path, which, dtype=torch.bfloat16)
    sharpen(d, SHARP[dtype], skip=GENTLE[dtype])
    vocab = CONFIGS[which]["vocab"]
    requests = {rid: random_tokens(n, vocab, 10 + i) for i, (rid, n) in enumerate(LENGTHS.items())}
    tb = all_ways_trace(requests)
    out = str(tmp_path / "out")
    run_tool(d, dtype, out, tb, page_size=None if default_page else PAGE_SIZES[which])
    worst = check_dumps(out, tb, plain_logits(d, requests), TOL[dtype])
    print(f"trace {which} {dtype}: worst relative error {worst:.3g}, pool {tb.max_tokens} tokens")


# every form of the kernels by size: head sizes of the attention, state channels and value channels of the state space
# (16 bytes at a time or not), key channels and sharing of the delta rule
KINDS = {
    "attention of 32, 16 state channels": layer(parallel(6, 6, 32, 32, 0.2, 3.0, 100.0, 32, 2, 32, 16, 2, 4, 1), 40),
    "attention of 160, 100 state channels": layer(parallel(4, 2, 160, 96, 0.08, 8.0, 1e4, 80, 3, 20, 100, 1, 3, 5), None),
    "attention of 128, 128 state channels": layer(parallel(8, 2, 128, 128, 0.08, 5.0, 1e4, 64, 8, 64, 128, 2, 4, 4), 24),
    "attention of 256, 256 state channels": layer(parallel(2, 1, 256, 64, 0.06, 1.0, 1e4, 256, 1, 40, 256, 1, 5, 1), None),
    "attention of 64, values of 200": layer(parallel(8, 1, 64, 200, 0.12, 4.0, 50.0, 2, 2, 200, 24, 1, 2, 8), 40, 0.5),
    "odd sizes": layer(parallel(7, 7, 31, 45, 0.15, 2.0, 1e4, 30, 7, 13, 19, 7, 7, 13, 0.3, -0.8), 33),
    "delta heads of 64": layer(delta(4, 4, 64, 64, 4, 16, 16), 40),
    "delta heads of 256": layer(delta(2, 1, 256, 32, 3, 9, 50), None),
    "delta heads of 16, values of 256": layer(delta(6, 2, 16, 256, 8, 24, 24), 24),
    "odd delta heads": layer(delta(9, 3, 31, 29, 9, 7, 3), 33, 4.0),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", list(KINDS))
def test_models_of_one_kind_of_layer(tmp_path, kind, dtype):
    spec = {"architecture": "Rorevik", "vocab": 90, "width": 76, "max_positions": 120, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.0}, "layers": [KINDS[kind]] * 2,
            "loop": {"start": 1, "stop": 2, "times": 2}}
    d = make_model_dir(tmp_path, "one", dtype=torch.bfloat16, config=spec)
    sharpen(d, SHARP[dtype], skip=GENTLE[dtype])
    requests = {rid: random_tokens(n, 90, 10 + i) for i, (rid, n) in enumerate(LENGTHS.items())}
    tb = all_ways_trace(requests)
    out = str(tmp_path / "out")
    run_tool(d, dtype, out, tb, page_size=16)
    worst = check_dumps(out, tb, plain_logits(d, requests), TOL[dtype])
    print(f"trace of {kind}, {dtype}: worst relative error {worst:.3g}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", list(CONFIGS))
def test_every_layer_run_follows_the_plain_model_gpu(tmp_path, which, dtype):
    """The residual stream after every block that runs: a whole prompt, then the same prompt in two portions and three
    single tokens through the caches and the state rows (so the first run that goes wrong is named)."""
    from litellmengine_amd.cache import CacheManager
    from litellmengine_amd.engine import ModelRunner, StepEntry
    from litellmengine_amd.models import load_model

    d = make_model_dir(tmp_path, which, dtype=torch.bfloat16)
    sharpen(d, SHARP[dtype], skip=GENTLE[dtype])
    tokens = random_tokens(70, CONFIGS[which]["vocab"], 3)
    want = residual_streams(d, tokens)
    model = load_model(d, dtype)
    cache = CacheManager(model, page_size=PAGE_SIZES[which], num_pages=40, max_requests=2, dtype=model.ctx.dtype, device=model.ctx.device)
    runner = ModelRunner(model, cache, use_graphs=False)
    seen = []
    for b in model.blocks:
        def wrapped(hidden, delta, step, layer_cache, next_norm=None, inner=b.forward):
            out = inner(hidden, delta, step, layer_cache, next_norm=next_norm)
            seen.append(hidden.double().cpu() + (out.total() if hasattr(out, "total") else out).double().cpu())
            return out
        b.forward = wrapped
    tol = 2e-4 if dtype == "float32" else 6e-2
    for cuts in ([70], [40, 27, 1, 1, 1]):
        slot, at = runner.admit(), 0
        for n in cuts:
            seen.clear()
            runner.step([StepEntry(slot, tokens[at : at + n], [])])
            assert len(seen) == len(want)
            for i, (got, ref) in enumerate(zip(seen, want)):
                err = (got - ref[at : at + n]).abs().max() / ref.abs().max()
                assert err < tol, f"layer run {i}, tokens {at}..{at + n}: {float(err):.3g}"
            at += n
        runner.release(slot)
    for b in model.blocks:
        del b.forward  # (the wrappers hold the model in a cycle)


PEAK = {"float32": (4.0, 1.5e-4), "bfloat16": (1.0, 2e-1)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B"])
def test_trace_with_single_keys_standing_out(tmp_path, which, dtype):
    """Requests of hundreds of tokens whose attentions pick out single keys (near and hundreds back, at the borders of
    pages) under the cap, and whose states remember for hundreds of tokens in some heads and channels; the last 110 tokens
    of one request are decoded one by one."""
    d = make_model_dir(tmp_path, which, seed=5, dtype=torch.bfloat16)
    factor, tol = PEAK[dtype]
    sharpen(d, factor, memory=1.6, skip=GENTLE[dtype])
    vocab = CONFIGS[which]["vocab"]
    requests = {"p": random_tokens(300, vocab, 41), "q": random_tokens(170, vocab, 42),
                "r": random_tokens(230, vocab, 43), "s": random_tokens(90, vocab, 44)}
    tb = TraceBuilder()
    whole(tb, "p#whole", requests["p"])
    tail_one_by_one(tb, "p#tail", requests["p"], tail=110)
    changing_portions(tb, "r#cut", requests["r"], seed=3)
    mixed(tb, {rid + "#mix": t for rid, t in requests.items()}, seed=6)
    out = str(tmp_path / "out")
    run_tool(d, dtype, out, tb, page_size=PAGE_SIZES[which])
    worst = check_dumps(out, tb, plain_logits(d, requests), tol)
    print(f"peaked trace {which} {dtype}: worst relative error {worst:.3g}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_in_a_batch_with_slots_used_again(tmp_path, dtype):
    """Three requests decode 150 tokens each side by side (captured graphs), the shortest ends and its
    slot, pages and state rows go to a newcomer whose prompt runs beside the others' single tokens."""
    d = make_model_dir(tmp_path, "B", seed=9, dtype=torch.bfloat16)
    sharpen(d, SHARP[dtype], memory=1.6, skip=GENTLE[dtype])
    vocab = CONFIGS["B"]["vocab"]
    requests = {rid: random_tokens(n, vocab, 60 + i) for i, (rid, n) in enumerate({"a": 170, "b": 200, "c": 230, "n": 90}.items())}
    tb = TraceBuilder()
    tb.step([(r, requests[r][: len(requests[r]) - 150], [0]) for r in "abc"])
    live, at = ["a", "b", "c"], {r: len(requests[r]) - 150 for r in "abc"}
    at["n"] = 0
    for i in range(150):
        entries, end = [], []
        for r in list(live):
            n = 40 if r == "n" and at[r] == 0 else 1
            entries.append((r, requests[r][at[r] : at[r] + n], [n - 1]))
            at[r] += n
            if at[r] == len(requests[r]):
                end.append(r)
                live.remove(r)
        tb.step(entries, end)
        if i == 20:
            live.remove("a")
            tb.steps[-1]["end"].append("a")
            tb.live.pop("a")
            live.append("n")
    out = str(tmp_path / "out")
    run_tool(d, dtype, out, tb, page_size=16, max_requests=3)
    worst = check_dumps(out, tb, plain_logits(d, requests), 1.5e-4 if dtype == "float32" else 1.5e-1)
    print(f"long decoding {dtype}: worst relative error {worst:.3g}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_many_requests_decode_side_by_side(tmp_path, dtype):
    """Twenty-one requests of unequal lengths decode forty tokens each (one graph replayed; batches of sixteen and more run
    the two mixers' chains on two streams), some of them ending early, so that the batch passes that size on its way
    down: every row of every step against the plain model."""
    d = make_model_dir(tmp_path, "B", seed=11, dtype=torch.bfloat16)
    sharpen(d, SHARP[dtype], memory=1.6, skip=GENTLE[dtype])
    vocab = CONFIGS["B"]["vocab"]
    heads = {f"r{i}": 3 + 2 * i for i in range(21)}  # tokens ahead of the decoding
    tails = {r: 40 if i % 3 else 15 + i for i, r in enumerate(heads)}
    requests = {r: random_tokens(heads[r] + tails[r], vocab, 90 + i) for i, r in enumerate(heads)}
    tb = TraceBuilder()
    tb.step([(r, requests[r][: heads[r]], [heads[r] - 1]) for r in heads])
    live, at = list(heads), dict(heads)
    while live:
        entries, end = [], []
        for r in list(live):
            entries.append((r, [requests[r][at[r]]], [0]))
            at[r] += 1
            if at[r] == len(requests[r]):
                end.append(r)
                live.remove(r)
        tb.step(entries, end)
    out = str(tmp_path / "out")
    run_tool(d, dtype, out, tb, page_size=16, max_requests=21)
    worst = check_dumps(out, tb, plain_logits(d, requests), 1.5e-4 if dtype == "float32" else 1e-1)
    print(f"many side by side {dtype}: worst relative error {worst:.3g}")


@pytest.mark.parametrize("which", ["A", "B"])
def test_greedy_generation_through_the_entry_point(tmp_path, which):
    from litellmengine_amd.entrypoints.generate import generate

    d = make_model_dir(tmp_path, which, dtype=torch.bfloat16)
    sharpen(d, 1.5)
    cfg, w = read(d)
    prompts = [random_tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate((1, 7, 23, 60))]
    want = [plain.greedy(cfg, w, p, 12) for p in prompts]
    assert generate(d, prompts, max_tokens=12, dtype="float32", page_size=PAGE_SIZES[which]) == want
    # portions, and a pool in which requests are preempted and recomputed
    assert generate(d, prompts, max_tokens=12, dtype="float32", page_size=8, prefill_chunk=16,
                    max_tokens_per_step=24, num_pages=14) == want


def test_command_line_generates(tmp_path):
    d = make_model_dir(tmp_path, "B", dtype=torch.bfloat16)
    sharpen(d, 1.5)
    cfg, w = read(d)
    prompt = random_tokens(19, cfg["vocab"], 80)
    want = plain.greedy(cfg, w, prompt, 10)
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "litellmengine"), "--model", d, "--input-ids",
                           ",".join(map(str, prompt)), "--max-tokens", "10", "--temperature", "0", "--dtype", "float32"],
                          text=True, capture_output=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    lines = proc.stdout.split("\n")
    got = [int(t) for t in lines[lines.index("New token ids:") + 1].replace(" ", "").split(",")]
    assert got == want
