"""Telulorn on the CPU: the plain implementation's mechanisms against what their equations say, the configuration
and checkpoint, and the engine (cache, state rows, step, scheduler, trace replay) with substitute kernels against
the plain model."""
import copy
import json
import math
import os

import pytest
import torch

from litellmengine_amd.cache import CacheManager
from litellmengine_amd.config import ConfigError, TelulornConfig, architecture_of, load_config
from litellmengine_amd.engine import LLMEngine, ModelRunner, StepEntry
from litellmengine_amd.models import load_model, looped_plan
from litellmengine_amd.parts import CacheSpec, GatedAttention, KVCacheSpec, RotaryInterleaved, geometric_slopes
from litellmengine_amd.weights.loader import WeightError
from tests.plain import telulorn_plain as plain
from tests.telulorn_util import (CONFIGS, PAGE_SIZES, make_model_dir, plain_logits, read, residual_streams, run_tool, sharpen)
from tests.tiny import random_tokens
from tests.torch_ops import TorchOps
from tests.trace_util import TraceBuilder, changing_portions, check_dumps, mixed, tail_one_by_one, whole


def rnd(shape, seed, scale=1.0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


# -- the plain mechanisms -------------------------------------------------------------------------------
def test_plain_chunks_and_kept_windows():
    m = plain.chunk_mask(11, 4)
    for i in range(11):
        assert m[i].nonzero().flatten().tolist() == list(range(i // 4 * 4, i + 1))
    m = plain.kept_window_mask(12, 3, 2)
    for i in range(12):
        assert m[i].nonzero().flatten().tolist() == sorted(set(range(min(2, i + 1))) | set(range(max(0, i - 2), i + 1)))
    assert torch.equal(plain.kept_window_mask(9, 4, 0), plain.kept_window_mask(9, 4, 0) & (torch.arange(9).view(-1, 1) - torch.arange(9) < 4))


def test_plain_slopes_and_distance_bias():
    assert torch.allclose(plain.head_slopes(8), torch.tensor([0.5 ** (h + 1) for h in range(8)], dtype=torch.float64))
    assert torch.allclose(plain.head_slopes(3), torch.tensor(geometric_slopes(3), dtype=torch.float64))
    b = plain.distance_bias(6, 4)
    assert float(b[2, 5, 1]) == pytest.approx(4 * 2.0 ** -6) and float(b[:, 3, 3].abs().max()) == 0.0
    # with everything else equal a key twice as far loses that much of its weight
    w = plain.softmax_weights(-plain.distance_bias(5, 1), plain.chunk_mask(5, 5))
    assert torch.allclose(w[0, 4, 1:] / w[0, 4, :-1], torch.full((4,), math.exp(2.0 ** -8), dtype=torch.float64))


def test_plain_mixed_heads_and_gates():
    T, H = 5, 3
    w = torch.softmax(rnd((H, T, T), 1), dim=-1)
    talk = rnd((H, H), 2)
    got = plain.mixed_over_heads(w, talk)
    for h in range(H):
        assert torch.allclose(got[h], sum(float(talk[h, g]) * w[g] for g in range(H)))
    assert torch.equal(plain.mixed_over_heads(w, torch.eye(H, dtype=torch.float64)), w)
    v = rnd((T, 1, 4), 3)  # one value head for all: the mixed sum is the mix of the sums
    assert torch.allclose(plain.heads_values(got, v), torch.einsum("hg,igd->ihd", talk, plain.heads_values(w, v)))


def test_plain_sink_takes_a_share_and_far_scores_do_not_overflow():
    s, sink = rnd((2, 4, 4), 1, 3.0), torch.tensor([0.5, -1.0], dtype=torch.float64)
    mask = plain.chunk_mask(4, 4)
    w = plain.softmax_weights(s, mask, sink)
    e = torch.exp(s).masked_fill(~mask, 0.0)
    assert torch.allclose(w, e / (e.sum(-1, keepdim=True) + torch.exp(sink).view(2, 1, 1)))
    assert float((w.sum(-1) < 1.0).float().mean()) == 1.0
    low = plain.softmax_weights(s - 1000.0, mask, sink)
    assert float(low.abs().max()) < 1e-12 and not bool(torch.isnan(low).any())
    assert torch.allclose(plain.softmax_weights(s, mask).sum(-1), torch.ones(2, 4, dtype=torch.float64))


def test_plain_rotations_keep_norms_depend_on_distances_and_turn_back():
    x, pos = rnd((6, 2, 10), 1), torch.tensor([0, 1, 2, 7, 100, 1000])
    y = plain.turn_pairs(x, pos, 8, 100.0)
    assert torch.equal(y[0], x[0]) and torch.equal(y[..., 8:], x[..., 8:])
    assert torch.allclose((y[..., 0:8:2] ** 2 + y[..., 1:8:2] ** 2), (x[..., 0:8:2] ** 2 + x[..., 1:8:2] ** 2))
    assert torch.allclose(plain.turn_pairs(y, pos, 8, 100.0, sign=-1.0), x)
    a, b = rnd((1, 1, 8), 2), rnd((1, 1, 8), 3)
    dot = lambda i, j: float((plain.turn_pairs(a, torch.tensor([i]), 8, 50.0) * plain.turn_pairs(b, torch.tensor([j]), 8, 50.0)).sum())
    assert dot(9, 4) == pytest.approx(dot(105, 100)) and dot(9, 4) != pytest.approx(dot(9, 5), abs=1e-3)
    # a value turned by j and turned back by i depends on i - j alone
    turn = lambda i, j: plain.turn_pairs(plain.turn_pairs(a, torch.tensor([j]), 8, 50.0), torch.tensor([i]), 8, 50.0, sign=-1.0)
    assert torch.allclose(turn(9, 4), turn(105, 100)) and torch.allclose(turn(33, 33), a)


def test_plain_recurrence_is_a_sum_and_carries_over():
    T, H, d, vd = 7, 2, 3, 4
    q, k, v, alpha = rnd((T, H, d), 1), rnd((T, H, d), 2), rnd((T, H, vd), 3), torch.sigmoid(rnd((T, H, d), 4))
    o = plain.linear_recurrence(q, k, v, alpha)
    for t in range(T):
        want = torch.zeros(H, vd, dtype=torch.float64)
        for s in range(t + 1):
            kept = alpha[s + 1 : t + 1].prod(dim=0)  # the token's own write is not decayed
            want += ((q[t] * k[s] * kept).sum(-1, keepdim=True)) * v[s]
        assert torch.allclose(o[t], want)
    w = {"a1": rnd((2, 5), 5), "a2": rnd((6, 2), 6), "a2.b": rnd((6,), 7, 3.0)}
    h = rnd((4, 5), 8)
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    assert torch.allclose(plain.decays(h, w, "", 16.0), (1 / (1 + torch.exp(-z))) ** (1 / 16.0))
    assert torch.allclose(plain.log_sigmoid(torch.tensor([-800.0, 800.0], dtype=torch.float64)), torch.tensor([-800.0, 0.0], dtype=torch.float64))


def test_plain_order_of_layers():
    runs = plain.layer_runs({"layers": [0] * 5, "loop": {"start": 1, "stop": 3, "times": 3}})
    assert runs == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None), (4, None)]
    assert plain.layer_runs({"layers": [0] * 2}) == [(0, None), (1, None)]
    plan = looped_plan(5, 1, 3, 3)
    assert [(e.block, None if e.inject is None else e.inject.vector) for e in plan] == runs
    assert [e.inject.embedding for e in plan if e.inject] == [False, True, True]
    for bad in ((0, 0, 1), (2, 6, 1), (1, 2, 0)):
        with pytest.raises(ValueError):
            looped_plan(5, *bad)


# -- configuration, parts and checkpoints -----------------------------------------------------------------
def test_config_round_trip_defaults_and_faults():
    for spec in CONFIGS.values():
        cfg = TelulornConfig.from_dict(spec)
        assert TelulornConfig.from_dict(cfg.to_dict()) == cfg
        assert architecture_of(spec).name == "Telulorn"
    base = CONFIGS["A"]

    def changed(path, value):
        d = copy.deepcopy(base)
        at = d
        for key in path[:-1]:
            at = at[key]
        if value is None:
            del at[path[-1]]
        else:
            at[path[-1]] = value
        return d

    cfg = TelulornConfig.from_dict(changed(["loop"], None))
    assert cfg.loop is None and cfg.layers[0].mixer.keep_first == 4 and cfg.layers[1].mlp is None
    assert TelulornConfig.from_dict(changed(["layers", 0, "mixer", "mask"], None)).layers[0].mixer.window is None
    assert TelulornConfig.from_dict(changed(["layers", 0, "mixer", "mask", "keep_first"], None)).layers[0].mixer.keep_first == 0
    assert TelulornConfig.from_dict(changed(["layers", 1, "mixer", "left_scale"], None)).layers[1].mixer.left_scale == 1.0
    for path, value in ((["layers", 0, "type"], "conv"), (["layers", 0, "mixer", "kv_heads"], 4), (["layers", 0, "mixer", "vdim"], 41),
                        (["layers", 0, "mixer", "rot", "dims"], 7), (["layers", 0, "mixer", "rot", "dims"], 26), (["layers", 0, "mixer", "rot"], None),
                        (["layers", 1, "mixer", "right", "tau"], None), (["layers", 1, "mixer", "left", "mask", "size"], 0),
                        (["loop", "stop"], 6), (["loop", "times"], 0), (["layers", 0, "mlp", "kind"], "moe"), (["norm"], None), (["width"], 0),
                        (["layers", 0, "mixer", "mask", "keep_first"], -1)):
        with pytest.raises(ConfigError):
            TelulornConfig.from_dict(changed(path, value))


def test_the_decays_rank_is_read_from_the_checkpoints_shapes(tmp_path):
    d = make_model_dir(tmp_path, "A")
    path = os.path.join(d, "config.json")
    with open(path) as f:
        spec = json.load(f)
    for i in (1, 3, 4):
        del spec["layers"][i]["mixer"]["right"]["decay_rank"]
    with open(path, "w") as f:
        json.dump(spec, f)
    assert [load_config(d).layers[i].mixer.right.decay_rank for i in (1, 3, 4)] == [5, 16, 3]
    tokens = random_tokens(12, 131, 1)
    _, cache, runner = cpu_runner(d, 4, 16)
    got = runner.step([StepEntry(runner.admit(), tokens, [11])])
    assert (got[0].double() - plain_logits(d, {"a": tokens})["a"][11]).abs().max() < 1e-5
    with pytest.raises(ConfigError):
        TelulornConfig.from_dict(spec).with_tensor_shapes({})


def test_checkpoint_faults_are_reported_together(tmp_path):
    from safetensors.torch import load_file, save_file

    d = make_model_dir(tmp_path, "A")
    path = os.path.join(d, "model.safetensors")
    t = load_file(path)
    del t["loop.step"]
    t["l1.mix.left.talk"] = torch.ones(6, 5)
    t["l0.mix.sink"] = torch.ones(3)
    t["l1.mix.left.q.b"] = torch.ones(3)  # the mixed heads' projections have no biases
    save_file(t, path, metadata={"format": "pt"})
    with pytest.raises(WeightError) as e:
        load_model(d, "float32", device="cpu", ops=TorchOps())
    assert all(n in str(e.value) for n in ("loop.step", "l1.mix.left.talk", "l0.mix.sink", "l1.mix.left.q.b"))


def test_what_no_kernel_takes_is_refused_when_the_parts_are_built():
    turn = lambda n: RotaryInterleaved(n, 100.0)
    for bad in (dict(num_q_heads=3), dict(dim=300), dict(rotation=turn(40)), dict(value_rotation=turn(16)), dict(window=4, chunk=4),
                dict(keep_first=3), dict(talk=True, window=4), dict(chunk=4, sinks=True), dict(num_q_heads=256, num_kv_heads=2, talk=True)):
        with pytest.raises(ValueError):
            GatedAttention(**{**dict(prefix="", hidden_size=32, num_q_heads=4, num_kv_heads=2, dim=32, vdim=32, scale=0.2), **bad})
    for bad in (dict(window=3, chunk=3), dict(chunk=0), dict(keep_first=2), dict(window=3, keep_first=-1)):
        with pytest.raises(ValueError):
            KVCacheSpec(2, 32, **bad)


# -- pages behind chunks and behind windows that keep the first tokens ------------------------------------
class _Stub:
    """Something with cache layers, for a CacheManager without a model."""

    def __init__(self, *specs):
        from litellmengine_amd.models import PlanEntry
        from types import SimpleNamespace

        self.blocks = [SimpleNamespace(mixer=SimpleNamespace(cache_spec=lambda s=s: s, state_spec=lambda: None)) for s in specs]
        self.plan = [PlanEntry(i, i) for i in range(len(specs))]

    def cache_layers(self):
        return {i: b.mixer for i, b in enumerate(self.blocks)}


@pytest.mark.parametrize("P", [1, 4, 16])
@pytest.mark.parametrize("kind", ["chunk", "kept"])
def test_pages_that_no_later_query_sees_go_back_and_the_others_stay(P, kind):
    spec = KVCacheSpec(1, 8, chunk=13) if kind == "chunk" else KVCacheSpec(1, 8, 9, keep_first=6)
    m = CacheManager(_Stub(spec), page_size=P, num_pages=60, max_requests=2, dtype=torch.float32, device="cpu")
    g = m.groups[0]
    s, other = m.admit(), m.admit()
    m.extend(other, 5)
    m.commit(other, 5)
    n = 0
    for step in [3, 1, 1, 9, 1, 1, 1, 1, 1, 1, 1, 1, 14, 2, 5, 1, 1]:
        m.extend(s, n + step)
        n += step
        m.commit(s, n)
        # what the next query (position n) sees
        first = n // 13 * 13 if kind == "chunk" else max(0, n - 8)
        needed = {p // P for p in range(first, n)} | ({p // P for p in range(min(6, n))} if kind == "kept" else set())
        held = {i for i, page in enumerate(g.tables[s]) if page >= 0}
        assert needed <= held
        assert held == {i for i in range(-(-n // P)) if i >= first // P or (kind == "kept" and i < -(-6 // P))}
    assert len(set(g.held_pages(s)) & set(g.held_pages(other))) == 0
    m.release(s)
    m.release(other)
    assert g.pool.num_free == 60


def test_a_step_that_did_not_happen_gives_back_what_it_took_behind_a_chunk():
    m = CacheManager(_Stub(KVCacheSpec(1, 8, chunk=8), KVCacheSpec(1, 8, 5, keep_first=3)), page_size=2, num_pages=30, max_requests=1,
                     dtype=torch.float32, device="cpu")
    s = m.admit()
    m.extend(s, 19)
    m.commit(s, 19)
    free = m.free_pages()
    m.extend_many([(s, 29)])
    m.shrink_many([(s, 19)])
    assert m.free_pages() == free
    m.release(s)
    assert m.free_pages() == [30, 30]


def test_a_pool_sized_for_chunks_and_kept_windows_holds_the_longest_step():
    """Pools made from the chunk, the window, the kept tokens and the step budget are enough for every request at once."""
    specs = (KVCacheSpec(1, 8, chunk=13), KVCacheSpec(1, 8, 9, keep_first=6))
    m = CacheManager(_Stub(*specs), page_size=4, num_pages=400, max_requests=3, dtype=torch.float32, device="cpu", max_tokens_per_step=10)
    assert all(g.pool.num_pages < 40 for g in m.groups)
    slots, lens = [m.admit() for _ in range(3)], [0, 0, 0]
    for step in range(60):
        wants = [(s, n + (10 if (step + i) % 3 == 0 else 1)) for i, (s, n) in enumerate(zip(slots, lens))]
        m.extend_many(wants)
        m.commit_many(wants)
        lens = [n for _, n in wants]


def test_cache_specs_tell_masks_apart():
    specs = {KVCacheSpec(2, 32), KVCacheSpec(2, 32, 8), KVCacheSpec(2, 32, 8, keep_first=1), KVCacheSpec(2, 32, chunk=8)}
    assert len(specs) == 4 and [s.span for s in (KVCacheSpec(2, 32), KVCacheSpec(2, 32, chunk=7), KVCacheSpec(2, 32, 5, keep_first=2))] == [None, 7, 5]
    assert isinstance(KVCacheSpec(1, 8), CacheSpec)


# -- the engine with substitute kernels -------------------------------------------------------------------
def cpu_runner(d, page_size, num_pages, max_requests=4):
    model = load_model(d, "float32", device="cpu", ops=TorchOps())
    cache = CacheManager(model, page_size=page_size, num_pages=num_pages, max_requests=max_requests, dtype=torch.float32, device="cpu")
    return model, cache, ModelRunner(model, cache)


@pytest.mark.parametrize("which", list(CONFIGS))
def test_every_layer_run_follows_the_plain_model(tmp_path, which):
    d = make_model_dir(tmp_path, which)
    sharpen(d, 2.0)
    tokens = random_tokens(45, CONFIGS[which]["vocab"], 3)
    want = residual_streams(d, tokens)
    model, cache, runner = cpu_runner(d, PAGE_SIZES[which], 16)
    seen = []
    for b in model.blocks:
        def wrapped(hidden, delta, step, layer_cache, next_norm=None, inner=b.forward):
            out = inner(hidden, delta, step, layer_cache, next_norm=next_norm)
            seen.append(hidden.double() + (out.total() if hasattr(out, "total") else out).double())
            return out
        b.forward = wrapped
    runner.step([StepEntry(runner.admit(), tokens, [])])
    assert len(seen) == len(want) == len(model.plan)
    for i, (got, ref) in enumerate(zip(seen, want)):
        assert (got - ref).abs().max() < 1e-4 * max(1.0, float(ref.abs().max())), f"layer run {i}"
    for b in model.blocks:
        del b.forward  # (the wrappers hold the model in a cycle)


@pytest.mark.parametrize("which", list(CONFIGS))
def test_trace_cpu(tmp_path, which):
    """Whole, with a decoded tail, in portions down to two tokens, and mixed in a pool of the live peak
    with four slots (pages, slots and state rows are used again)."""
    d = make_model_dir(tmp_path, which)
    sharpen(d, 2.0)
    vocab = CONFIGS[which]["vocab"]
    requests = {rid: random_tokens(n, vocab, 20 + i) for i, (rid, n) in enumerate({"a": 50, "b": 45, "c": 70, "d": 33, "f": 1}.items())}
    tb = TraceBuilder()
    whole(tb, "a#whole", requests["a"])
    tail_one_by_one(tb, "b#tail", requests["b"], tail=20)
    changing_portions(tb, "c#cut", requests["c"], seed=1)
    mixed(tb, {rid + "#mix": t for rid, t in requests.items()}, seed=5)
    out = str(tmp_path / "out")
    run_tool(d, "float32", out, tb, page_size=PAGE_SIZES[which], in_process_ops=TorchOps())
    check_dumps(out, tb, plain_logits(d, requests), 1e-4)


def test_every_pass_has_a_cache_and_a_state_of_its_own_zeroed_when_a_slot_is_used_again(tmp_path):
    d = make_model_dir(tmp_path, "A")
    sharpen(d, 2.0)
    cfg, w = read(d)
    model, cache, runner = cpu_runner(d, 4, 12, max_requests=1)
    assert len(model.plan) == 8 and set(cache.states) == {1, 3, 4, 6, 7}  # the parallel layers' runs: blocks 1 and 3 twice, 4 once
    assert sum(len(g.cache_ids) for g in cache.groups) == 8
    first, second = random_tokens(9, 131, 1), random_tokens(6, 131, 2)
    s = runner.admit()
    runner.step([StepEntry(s, first, [])])
    assert all(float(st[s].abs().max()) > 0 for st in cache.states.values())
    assert not torch.equal(cache.states[1][s], cache.states[4][s])  # the same block's two passes
    runner.release(s)
    s2 = runner.admit()
    assert s2 == s and all(float(st[s].abs().max()) == 0 for st in cache.states.values())
    got = runner.step([StepEntry(s2, second, [5])])
    assert (got[0].double() - plain.forward(cfg, w, second)[5]).abs().max() < 1e-5


@pytest.mark.parametrize("which", ["A", "C"])
def test_greedy_generation_through_the_scheduler(tmp_path, which):
    """Requests of unequal lengths batched, prompts in portions, tokens launched ahead of their reading (the loop adds
    the embedding's rows of tokens that only the device knows), then a pool so small that requests are preempted and
    recomputed: the same tokens."""
    d = make_model_dir(tmp_path, which)
    sharpen(d, 1.5)
    cfg, w = read(d)
    prompts = [random_tokens(n, cfg["vocab"], 40 + i) for i, n in enumerate((1, 7, 23, 40))]
    want = [plain.greedy(cfg, w, p, 6) for p in prompts]
    for run_ahead in (False, True):
        model = load_model(d, "float32", device="cpu", ops=TorchOps())
        eng = LLMEngine(model, page_size=8, num_pages=16, max_requests=4, prefill_chunk=16, max_tokens_per_step=24, run_ahead=run_ahead)
        assert eng.generate(prompts, 6) == want
    small = LLMEngine(load_model(d, "float32", device="cpu", ops=TorchOps()), page_size=8, num_pages=8, max_requests=4,
                      prefill_chunk=16, max_tokens_per_step=24, run_ahead=False)
    assert small.generate(prompts, 6) == want
    assert all(g.pool.num_held == 0 for g in small.cache.groups)


def test_what_is_added_between_blocks_reaches_blocks_of_every_arrangement():
    """`Injected.total()`, the plain way to take what enters the stream: a delta of every kind, the vector, the rows."""
    from litellmengine_amd.parts import EmbeddedRows, Injected, PartialSums, ScaledSum

    ops = TorchOps()
    table, ids = rnd((7, 4), 1).float(), torch.tensor([3, 0, 6], dtype=torch.int32)
    vec, x, y = rnd((4,), 2).float(), rnd((3, 4), 3).float(), rnd((3, 4), 4).float()
    rows = table[ids.long()] * 0.5
    again = EmbeddedRows(ids, table, 0.5)
    for delta, plainly in ((None, 0.0), (x, x), (ScaledSum(x, y, 2.0), 2.0 * (x + y)), (PartialSums(torch.stack([x, y])), x + y)):
        assert torch.allclose(Injected(delta, vec, again, ops).total(), plainly + vec + rows)
        assert torch.allclose(Injected(delta, vec, None, ops).total(), plainly + vec)
        hidden = rnd((3, 4), 5).float()
        want = hidden + plainly + rows
        ops.inject_rmsnorm(hidden, delta, None, again, torch.ones(4), 1e-5, torch.float32)
        assert torch.allclose(hidden, want)


def test_a_lost_mechanism_would_show(tmp_path):
    """The measure of the GPU traces with sharpened weights: in the plain model of such weights, a chunk or a window one
    token off, one kept token less, a softmax without its sinks, unmixed heads, values that are not turned, a state that
    forgot what came before the last 60 tokens, or passes without their vectors or without the embedding's rows move the
    logits by far more than the 32-bit tolerance."""
    d = make_model_dir(tmp_path, "B", seed=5, dtype=torch.bfloat16)
    sharpen(d, 2.0, memory=1.6)
    cfg, w = read(d)
    tokens = random_tokens(140, cfg["vocab"], 42)
    base = plain.forward(cfg, w, tokens)
    moved = lambda cfg2, w2: ((plain.forward(cfg2, w2, tokens) - base).abs().max(dim=1).values / base.abs().max())

    def with_mixer(i, path, value):
        c = copy.deepcopy(cfg)
        at = c["layers"][i]["mixer"]
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        return c

    share = lambda m: float((m > 1e-3).float().mean())
    assert share(moved(with_mixer(0, ["left", "mask", "size"], 25), w)) > 0.5
    assert share(moved(with_mixer(1, ["mask", "size"], 47), w)) > 0.4  # (where the lost key is no kept one)
    assert share(moved(with_mixer(1, ["mask", "keep_first"], 32), w)) > 0.3
    assert share(moved(with_mixer(3, ["mask", "keep_first"], 0), w)) > 0.1
    without = lambda change: {n: change(n, t) for n, t in w.items()}
    assert share(moved(cfg, without(lambda n, t: t - 60.0 if n.endswith(".sink") else t))) > 0.9
    assert share(moved(cfg, without(lambda n, t: torch.eye(t.shape[0], dtype=t.dtype) if n.endswith(".talk") else t))) > 0.9
    assert share(moved(cfg, without(lambda n, t: t * 0 if n == "loop.step" else t))) > 0.9
    kept = plain.turn_pairs
    try:
        plain.turn_pairs = lambda x, pos, dims, base_, sign=1.0: x if dims == x.shape[-1] == 64 else kept(x, pos, dims, base_, sign)
        assert share(moved(cfg, w)) > 0.9
    finally:
        plain.turn_pairs = kept
    runs = plain.layer_runs
    try:  # (pass 0's vector, but no embedding rows, ahead of every pass)
        plain.layer_runs = lambda c: [(i, None if t is None else 0) for i, t in runs(c)]
        assert share(moved(cfg, w)) > 0.9
    finally:
        plain.layer_runs = runs
    p = "l2.mix.right."
    h = rnd((140, 128), 3)
    m = cfg["layers"][2]["mixer"]["right"]
    whole_run = plain.gated_linear_attention(h, w, p, m, 1e-6)[-1]
    fresh = plain.gated_linear_attention(h[-60:], w, p, m, 1e-6)[-1]
    assert float((whole_run - fresh).abs().max() / whole_run.abs().max()) > 1e-3
