"""Rorevik on the CPU: the plain implementation's mechanisms against what their equations say, the configuration
and checkpoint, and the engine (cache, state rows, positions, step, scheduler, trace replay) with substitute kernels
against the plain model."""
import copy
import json
import math
import os

import pytest
import torch

from litellmengine_amd.cache import CacheManager
from litellmengine_amd.config import ConfigError, RorevikConfig, architecture_of, load_config
from litellmengine_amd.engine import LLMEngine, ModelRunner, StepEntry
from litellmengine_amd.models import load_model, looped_plan
from litellmengine_amd.parts import (Embedding, GatedAttention, GatedDeltaMixer, GatedMLP, Injected, RMSNorm, RotaryInterleaved, ScaledSum,
                                     SideBySideMixer, StateSpaceMixer)
from litellmengine_amd.weights.loader import WeightError
from tests.plain import rorevik_plain as plain
from tests.rorevik_util import CONFIGS, PAGE_SIZES, make_model_dir, plain_logits, read, residual_streams, run_tool, sharpen
from tests.tiny import random_tokens
from tests.torch_ops import TorchOps
from tests.trace_util import TraceBuilder, changing_portions, check_dumps, mixed, tail_one_by_one, whole


def rnd(shape, seed, scale=1.0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


# -- the plain mechanisms -------------------------------------------------------------------------------
def test_plain_convolution_is_causal_and_its_last_tap_meets_the_token_itself():
    u, taps, bias = rnd((9, 3), 1), rnd((3, 4), 2), rnd((3,), 3)
    y = plain.causal_conv(u, taps, bias)
    for t in range(9):
        for c in range(3):
            assert float(y[t, c]) == pytest.approx(float(bias[c]) + sum(float(taps[c, 3 - b]) * float(u[t - b, c]) for b in range(min(4, t + 1))))
    moved = u.clone()
    moved[5:] += 1.0
    assert torch.equal(plain.causal_conv(moved, taps)[:5], plain.causal_conv(u, taps)[:5])
    assert torch.allclose(plain.causal_conv(u, taps[:, -1:]), u * taps[:, -1])


def test_plain_unit_vectors_norms_and_softplus():
    x = rnd((5, 7), 1)
    assert torch.allclose((plain.unit_vectors(x) ** 2).sum(-1), torch.ones(5, dtype=torch.float64), atol=1e-5)
    assert float(plain.unit_vectors(torch.zeros(1, 7)).abs().max()) == 0.0
    tiny = torch.full((1, 4), 1e-3, dtype=torch.float64)
    assert float(plain.unit_vectors(tiny)[0, 0]) == pytest.approx(1e-3 / math.sqrt(4e-6 + 1e-6))  # (the constant is inside the root)
    assert float(plain.rms_unit(tiny, 1e-6)[0, 0]) == pytest.approx(1e-3 / math.sqrt(1e-6 + 1e-6))
    s = plain.softplus(torch.tensor([-800.0, 0.0, 800.0], dtype=torch.float64))
    assert torch.allclose(s, torch.tensor([0.0, math.log(2.0), 800.0], dtype=torch.float64))


def test_plain_rotations_keep_norms_and_depend_on_distances():
    x, pos = rnd((6, 2, 10), 1), torch.tensor([0, 1, 2, 7, 100, 1000])
    y = plain.turn_pairs(x, pos, 8, 100.0)
    assert torch.equal(y[0], x[0]) and torch.equal(y[..., 8:], x[..., 8:])
    assert torch.allclose((y[..., 0:8:2] ** 2 + y[..., 1:8:2] ** 2), (x[..., 0:8:2] ** 2 + x[..., 1:8:2] ** 2))
    a, b = rnd((1, 1, 8), 2), rnd((1, 1, 8), 3)
    dot = lambda i, j: float((plain.turn_pairs(a, torch.tensor([i]), 8, 50.0) * plain.turn_pairs(b, torch.tensor([j]), 8, 50.0)).sum())
    assert dot(9, 4) == pytest.approx(dot(105, 100)) and dot(9, 4) != pytest.approx(dot(9, 5), abs=1e-3)


def test_plain_capped_scores_and_causal_weights():
    s = torch.tensor([-1000.0, -1.0, 0.0, 0.01, 1.0, 1000.0], dtype=torch.float64)
    c = plain.capped(s, 4.0)
    assert float(c.abs().max()) <= 4.0 and float(c[0]) == -4.0 and float(c[3]) == pytest.approx(0.01, rel=1e-4)
    assert torch.all(c[1:] > c[:-1])
    w = plain.causal_softmax(rnd((2, 5, 5), 1, 3.0))
    assert torch.allclose(w.sum(-1), torch.ones(2, 5, dtype=torch.float64)) and torch.equal(w, w.tril()) and float(w[0, 0, 0]) == 1.0
    # under the cap the best of two keys weighs e^(2 cap) times the worst, whatever their scores
    two = plain.causal_softmax(plain.capped(torch.tensor([[[0.0, 0.0], [500.0, -500.0]]], dtype=torch.float64), 1.5))
    assert float(two[0, 1, 0] / two[0, 1, 1]) == pytest.approx(math.exp(3.0))


def test_plain_delta_rule_corrects_forgets_by_channel_and_carries_over():
    T, H, d, vd = 6, 2, 4, 3
    k = torch.eye(4, dtype=torch.float64)[[0, 1, 2, 0, 3, 1]].view(T, 1, d).repeat(1, H, 1)
    v, q = rnd((T, H, vd), 1), rnd((T, H, d), 2)
    one, g1 = torch.ones(T, H, dtype=torch.float64), torch.ones(T, H, d, dtype=torch.float64)
    reads = lambda key: torch.eye(4, dtype=torch.float64)[key].view(1, 1, d).repeat(T, H, 1)
    o = plain.delta_recurrence(reads(0), k, v, one, g1)  # whole corrections, nothing forgotten
    assert torch.allclose(o[:3], v[:1].repeat(3, 1, 1)) and torch.allclose(o[3:], v[3:4].repeat(3, 1, 1))
    g = g1.clone()
    g[..., 0], g[..., 1] = 0.5, 0.25
    o = plain.delta_recurrence(reads(1), k, v, one, g)
    assert torch.allclose(o[1], v[1]) and torch.allclose(o[3], v[1] * 0.25 ** 2)  # the token's own write is not decayed
    half = plain.delta_recurrence(reads(0), k, v, 0.5 * one, g1)
    assert torch.allclose(half[3], 0.5 * v[0] + 0.5 * (v[3] - 0.5 * v[0]))
    # a run in two: the second starts from the first one's state
    beta, g = torch.sigmoid(rnd((T, H), 3)), torch.sigmoid(rnd((T, H, d), 4))
    kk = plain.unit_vectors(rnd((T, H, d), 5))
    S = torch.zeros(H, d, vd, dtype=torch.float64)
    for t in range(T):
        S = torch.diag_embed(g[t]) @ S
        S = S + kk[t].unsqueeze(-1) @ (beta[t].view(H, 1, 1) * (v[t].unsqueeze(1) - kk[t].unsqueeze(1) @ S))
    want = (q[-1].unsqueeze(1) @ S).squeeze(1)
    assert torch.allclose(plain.delta_recurrence(q, kk, v, beta, g)[-1], want)


def test_plain_channel_decays():
    w = {"a1": rnd((2, 5), 5), "a2": rnd((6, 2), 6), "dt_bias": rnd((6,), 7, 3.0), "A_log": rnd((2,), 9)}
    h = rnd((4, 5), 8)
    z = (h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]
    got = plain.channel_decays(h, w, "", 2, 3)
    for head in range(2):
        want = (1 + torch.exp(z[:, 3 * head : 3 * head + 3])) ** -torch.exp(w["A_log"][head])
        assert torch.allclose(got[:, head], want)


def test_plain_state_space_recurrence_is_a_sum_with_a_skip():
    T, H, vd, N = 7, 2, 3, 4
    x, B, C, dt = rnd((T, H, vd), 1), rnd((T, H, N), 2), rnd((T, H, N), 3), torch.rand(T, H, dtype=torch.float64)
    rate, D = torch.tensor([0.3, 2.0], dtype=torch.float64), torch.tensor([0.7, -1.0], dtype=torch.float64)
    y = plain.ssd_recurrence(x, B, C, dt, rate, D)
    for t in range(T):
        want = D.view(H, 1) * x[t]
        for s in range(t + 1):
            kept = torch.exp(-rate * dt[s + 1 : t + 1].sum(dim=0))  # the token's own write is not decayed
            want = want + (kept * dt[s] * (C[t] * B[s]).sum(-1)).view(H, 1) * x[s]
        assert torch.allclose(y[t], want)


def test_plain_gated_norm_goes_part_by_part_with_the_gate_first():
    y, z, w = rnd((3, 12), 1), rnd((3, 12), 2), rnd((12,), 3)
    got = plain.gated_group_norm(y, z, w, 3, 1e-5)
    a = y * z / (1 + torch.exp(-z))
    for p in range(3):
        part = a[:, 4 * p : 4 * p + 4]
        assert torch.allclose(got[:, 4 * p : 4 * p + 4], part / torch.sqrt((part ** 2).mean(-1, keepdim=True) + 1e-5) * w[4 * p : 4 * p + 4])
    assert not torch.allclose(got, plain.gated_group_norm(y, z, w, 1, 1e-5))


def test_plain_clamped_feed_forward_and_first_rows():
    w = {n: rnd(s, i) for i, (n, s) in enumerate({"gate": (4, 5), "gate.b": (4,), "up": (4, 5), "up.b": (4,), "down": (5, 4), "down.b": (5,)}.items())}
    h = rnd((6, 5), 9, 3.0)
    g, u = torch.clamp(h @ w["gate"].T + w["gate.b"], max=0.8), torch.clamp(h @ w["up"].T + w["up.b"], -0.8, 0.8)
    want = (g / (1 + torch.exp(-1.702 * g)) * (1 + u)) @ w["down"].T + w["down.b"]
    assert torch.allclose(plain.clamped_ff(h, w, "", 0.8), want)
    assert float(torch.min(h @ w["gate"].T + w["gate.b"])) < -0.8  # (the gate is not clamped from below)
    cfg = {"embedding": {"scale": 3.0}, "norm": {"eps": 1e-5}}
    e = {"embed": rnd((4, 6), 1), "pos": rnd((9, 6), 2), "embed.norm": rnd((6,), 3)}
    x = plain.embedded(cfg, e, [2, 2, 0])
    for t, tok in enumerate([2, 2, 0]):
        row = 3.0 * e["embed"][tok] + e["pos"][t]
        assert torch.allclose(x[t], row / torch.sqrt((row ** 2).mean() + 1e-5) * e["embed.norm"])
    assert not torch.allclose(x[0], x[1])


def test_plain_order_of_layers():
    assert plain.layer_runs({"layers": [0] * 5, "loop": {"start": 1, "stop": 3, "times": 3}}) == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    assert plain.layer_runs({"layers": [0] * 2}) == [0, 1]
    plan = looped_plan(5, 1, 3, 3, inject=False)
    assert [e.block for e in plan] == [0, 1, 2, 1, 2, 1, 2, 3, 4] and all(e.inject is None for e in plan)


# -- configuration, parts and checkpoints -----------------------------------------------------------------
def test_config_round_trip_defaults_and_faults():
    for spec in CONFIGS.values():
        cfg = RorevikConfig.from_dict(spec)
        assert RorevikConfig.from_dict(cfg.to_dict()) == cfg
        assert architecture_of(spec).name == "Rorevik"
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

    cfg = RorevikConfig.from_dict(changed(["loop"], None))
    assert cfg.loop is None and cfg.layers[1].mlp is None and cfg.layers[4].mixer.left.rot_dims == 0
    assert RorevikConfig.from_dict(changed(["embedding"], None)).embedding_scale == 1.0
    assert RorevikConfig.from_dict(changed(["layers", 1, "mixer", "left", "softcap"], None)).layers[1].mixer.left.softcap is None
    assert RorevikConfig.from_dict(changed(["layers", 1, "mixer", "right_scale"], None)).layers[1].mixer.right_scale == 1.0
    assert RorevikConfig.from_dict(changed(["layers", 1, "mixer", "right", "groups"], None)).layers[1].mixer.right.groups == 1
    assert RorevikConfig.from_dict(changed(["layers", 0, "mixer", "kv_heads"], None)).layers[0].mixer.kv_heads == 6
    for path, value in ((["layers", 0, "type"], "conv"), (["layers", 0, "mixer", "kv_heads"], 4), (["layers", 0, "mixer", "conv"], 0),
                        (["layers", 0, "mixer", "conv"], None), (["layers", 1, "mixer", "left", "rot", "dims"], 7),
                        (["layers", 1, "mixer", "left", "rot", "dims"], 22), (["layers", 1, "mixer", "left", "rot", "base"], None),
                        (["layers", 1, "mixer", "left", "softcap"], 0.0), (["layers", 1, "mixer", "right", "groups"], 4),
                        (["layers", 1, "mixer", "right", "norm_groups"], 7), (["layers", 1, "mixer", "right", "state"], None),
                        (["loop", "stop"], 6), (["loop", "times"], 0), (["layers", 0, "mlp", "kind"], "moe"), (["layers", 0, "mlp", "limit"], None),
                        (["layers", 0, "mlp", "limit"], -1.0), (["norm"], None), (["width"], 0), (["max_positions"], None),
                        (["layers", 0, "mixer", "decay_rank"], 0)):
        with pytest.raises(ConfigError):
            RorevikConfig.from_dict(changed(path, value))


def test_the_inner_ranks_are_read_from_the_checkpoints_shapes(tmp_path):
    d = make_model_dir(tmp_path, "A")
    path = os.path.join(d, "config.json")
    with open(path) as f:
        spec = json.load(f)
    for i in (0, 2):
        del spec["layers"][i]["mixer"]["decay_rank"], spec["layers"][i]["mixer"]["gate_rank"]
    with open(path, "w") as f:
        json.dump(spec, f)
    assert [(load_config(d).layers[i].mixer.decay_rank, load_config(d).layers[i].mixer.gate_rank) for i in (0, 2)] == [(5, 7), (16, 1)]
    tokens = random_tokens(12, 131, 1)
    _, cache, runner = cpu_runner(d, 4, 16)
    got = runner.step([StepEntry(runner.admit(), tokens, [11])])
    assert (got[0].double() - plain_logits(d, {"a": tokens})["a"][11]).abs().max() < 1e-5
    with pytest.raises(ConfigError):
        RorevikConfig.from_dict(spec).with_tensor_shapes({})


def test_checkpoint_faults_are_reported_together(tmp_path):
    from safetensors.torch import load_file, save_file

    d = make_model_dir(tmp_path, "A")
    path = os.path.join(d, "model.safetensors")
    t = load_file(path)
    del t["pos"], t["head"]
    t["l1.mix.right.conv"] = torch.ones(6, 5)
    t["l0.mix.dt_bias"] = torch.ones(6)
    t["l1.mix.left.q.b"] = torch.ones(3)  # the projections have no biases
    save_file(t, path, metadata={"format": "pt"})
    with pytest.raises(WeightError) as e:
        load_model(d, "float32", device="cpu", ops=TorchOps())
    assert all(n in str(e.value) for n in ("pos", "head", "l1.mix.right.conv", "l0.mix.dt_bias", "l1.mix.left.q.b"))


def test_what_no_kernel_takes_is_refused_when_the_parts_are_built():
    ssd = dict(prefix="", hidden_size=32, heads=4, vdim=8, state=8, groups=2, taps=3, norm_groups=2, norm_eps=1e-5)
    for bad in (dict(groups=3), dict(vdim=300), dict(state=0), dict(state=257), dict(taps=0), dict(norm_groups=5)):
        with pytest.raises(ValueError):
            StateSpaceMixer(**{**ssd, **bad})
    dlt = dict(prefix="", hidden_size=32, heads=4, kv_heads=2, dim=8, vdim=8, taps=3, norm_eps=1e-5, decay_rank=3, gate_rank=2,
               names=("q", "k", "v", "b", "a1", "a2", "A_log", "dt_bias", "g1", "g2", "norm", "o"))
    GatedDeltaMixer(**dlt)
    for bad in (dict(gate_rank=None), dict(decay_rank=0), dict(dim=300), dict(kv_heads=3)):
        with pytest.raises(ValueError):
            GatedDeltaMixer(**{**dlt, **bad})
    att = dict(prefix="", hidden_size=32, num_q_heads=4, num_kv_heads=2, dim=32, vdim=32, scale=0.2, gated=False, softcap=3.0)
    GatedAttention(**att)
    for bad in (dict(softcap=0.0), dict(softcap=-1.0), dict(out_scale=0.5), dict(chunk=4), dict(talk=True),
                dict(value_rotation=RotaryInterleaved(32, 100.0))):
        with pytest.raises(ValueError):
            GatedAttention(**{**att, **bad})
    for bad in (dict(activation="clamp"), dict(limit=2.0), dict(activation="clamp", limit=0.0)):
        with pytest.raises(ValueError):
            GatedMLP("", 32, 64, **bad)
    with pytest.raises(ValueError):
        Embedding("embed", 10, 8, positions_name="pos")
    with pytest.raises(ValueError):
        SideBySideMixer(StateSpaceMixer(**ssd), StateSpaceMixer(**{**ssd, "prefix": "b."}), left_scale=1.0)


def test_sums_with_a_factor_each_and_a_bias_on_the_way():
    a, b, bias = rnd((3, 4), 1).float(), rnd((3, 4), 2).float(), rnd((4,), 3).float()
    assert torch.allclose(ScaledSum(a, b, 0.5, 2.0).total(), 0.5 * a + 2.0 * b)
    assert torch.allclose(ScaledSum(a, b, 0.5).total(), 0.5 * (a + b)) and torch.allclose(ScaledSum(a, None, 0.5).total(), 0.5 * a)
    ops = TorchOps()
    inner = Injected(a, bias, None, ops)
    assert torch.allclose(Injected(inner, bias, None, ops).total(), a + 2 * bias)
    from types import SimpleNamespace
    norm = RMSNorm("n", 4, 1e-5)
    norm.bind({"n": torch.ones(4)}, SimpleNamespace(dtype=torch.float32, device="cpu", ops=ops))
    hidden = rnd((3, 4), 5).float()
    rows = torch.tensor([2, 0], dtype=torch.int32)
    want = plain.rms_unit((hidden + a + bias)[[2, 0]].double(), 1e-5)
    assert torch.allclose(norm.forward(hidden.clone(), inner, rows=rows).double(), want, atol=1e-6)
    want = plain.rms_unit((hidden + 0.5 * a + 2.0 * b).double(), 1e-5)
    assert torch.allclose(norm.forward(hidden.clone(), ScaledSum(a, b, 0.5, 2.0)).double(), want, atol=1e-6)


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
    assert len(model.plan) == 8 and set(cache.states) == set(range(8))  # every mixer keeps a state
    assert sum(len(g.cache_ids) for g in cache.groups) == 5  # the parallel layers' runs: blocks 1 and 3 twice, 4 once
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


def test_a_request_ends_where_the_positions_end(tmp_path):
    """As many tokens as there are positions run, one more is refused before anything has changed; the scheduler refuses a
    request that could grow past them."""
    spec = {**CONFIGS["C"], "max_positions": 20}
    d = make_model_dir(tmp_path, "short", config=spec)
    sharpen(d, 1.0)
    tokens = random_tokens(20, 77, 1)
    model, cache, runner = cpu_runner(d, 8, 16)
    assert model.max_positions == 20
    s, other = runner.admit(), runner.admit()
    runner.step([StepEntry(s, tokens[:18], [])])
    free = cache.free_pages()
    with pytest.raises(ValueError):
        runner.step([StepEntry(other, tokens[:5], [4]), StepEntry(s, [1, 2, 3], [2])])
    assert cache.free_pages() == free and cache.length(s) == 18 and cache.length(other) == 0
    got = runner.step([StepEntry(s, tokens[18:], [1])])
    assert (got[0].double() - plain_logits(d, {"a": tokens})["a"][19]).abs().max() < 1e-5
    with pytest.raises(ValueError):
        runner.step([StepEntry(s, [1], [0])])
    eng = LLMEngine(model, page_size=8, num_pages=16, max_requests=2, run_ahead=False)
    with pytest.raises(ValueError):
        eng.add_request(tokens[:15], 7)  # 15 + 6 cached tokens
    assert len(eng.generate([tokens[:15]], 6)[0]) == 6
    r = eng.add_request(tokens[:10], 4, keep_session=True)
    eng.run_until_finished()
    with pytest.raises(ValueError):
        eng.append_input_tokens(r, tokens[:5], 4)
    eng.append_input_tokens(r, tokens[:3], 4)
    eng.run_until_finished()
    assert r.finished


@pytest.mark.parametrize("which", ["A", "C"])
def test_greedy_generation_through_the_scheduler(tmp_path, which):
    """Requests of unequal lengths batched, prompts in portions, tokens launched ahead of their reading (the first rows are
    made of tokens that only the device knows), then a pool so small that requests are preempted and recomputed: the
    same tokens."""
    d = make_model_dir(tmp_path, which)
    sharpen(d, 1.5)
    cfg, w = read(d)
    prompts = [random_tokens(n, cfg["vocab"], 40 + i) for i, n in enumerate((1, 7, 23, 40))]
    want = [plain.greedy(cfg, w, p, 6) for p in prompts]
    for run_ahead in (False, True):
        model = load_model(d, "float32", device="cpu", ops=TorchOps())
        eng = LLMEngine(model, page_size=8, num_pages=24, max_requests=4, prefill_chunk=16, max_tokens_per_step=24, run_ahead=run_ahead)
        assert eng.generate(prompts, 6) == want
    small = LLMEngine(load_model(d, "float32", device="cpu", ops=TorchOps()), page_size=8, num_pages=8, max_requests=4,
                      prefill_chunk=16, max_tokens_per_step=24, run_ahead=False)
    assert small.generate(prompts, 6) == want
    assert all(g.pool.num_held == 0 for g in small.cache.groups)


def test_a_lost_mechanism_would_show(tmp_path):
    """The measure of the GPU traces with sharpened weights: in the plain model of such weights, scores without their cap,
    positions one off, a rotation left out, a state or a convolution that forgot what came before, channels that forget
    alike, a skip, a bias, a gate or a factor left out, or a norm over other parts move the logits by far more than the
    32-bit tolerance."""
    d = make_model_dir(tmp_path, "B", seed=5, dtype=torch.bfloat16)
    sharpen(d, 2.0, memory=1.6)
    cfg, w = read(d)
    tokens = random_tokens(120, cfg["vocab"], 42)
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
    assert share(moved(with_mixer(0, ["left", "softcap"], 1e9), w)) > 0.8
    assert share(moved(with_mixer(0, ["left", "rot", "dims"], 30), w)) > 0.8
    assert share(moved(with_mixer(0, ["right", "norm_groups"], 1), w)) > 0.9
    assert share(moved(with_mixer(2, ["right_scale"], 1.0), w)) > 0.9
    without = lambda change: {n: change(n, t) for n, t in w.items()}
    assert share(moved(cfg, without(lambda n, t: torch.roll(t, 1, 0) if n == "pos" else t))) > 0.9
    assert share(moved(cfg, without(lambda n, t: t * 0 if n.endswith(".D") else t))) > 0.9
    assert share(moved(cfg, without(lambda n, t: t * 0 if n.endswith("conv.b") else t))) > 0.9
    assert share(moved(cfg, without(lambda n, t: t * 0 if n.endswith("down.b") else t))) > 0.9
    assert share(moved(cfg, without(lambda n, t: t * 0 if n.endswith(".g2") else t))) > 0.9
    for attr, other in (("unit_vectors", lambda x: x), ("causal_conv", lambda u, taps, bias=None: u * taps[:, -1] + (0 if bias is None else bias))):
        kept = getattr(plain, attr)
        try:
            setattr(plain, attr, other)
            assert share(moved(cfg, w)) > 0.9, attr
        finally:
            setattr(plain, attr, kept)
    kept = plain.channel_decays
    try:
        plain.channel_decays = lambda *a: kept(*a).mean(-1, keepdim=True).expand_as(kept(*a))
        assert share(moved(cfg, w)) > 0.9
    finally:
        plain.channel_decays = kept
    h = rnd((120, 128), 3)
    for run in (lambda t: plain.mamba2(t, w, "l0.mix.right.", cfg["layers"][0]["mixer"]["right"], 1e-6),
                lambda t: plain.channel_delta(t, w, "l1.mix.", cfg["layers"][1]["mixer"], 1e-6)):
        whole_run, fresh = run(h)[-1], run(h[-60:])[-1]  # a state that forgot what came before the last 60 tokens
        assert float((whole_run - fresh).abs().max() / whole_run.abs().max()) > 1e-3
