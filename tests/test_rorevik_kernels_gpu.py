"""The kernels that Rorevik added (first rows from an embedding, position vectors and a norm; attention with capped
scores; the delta rule's walk with a decay per key channel, its decays and gates through narrow middles, its
convolution that moves the state on; Mamba-2's convolution, recurrence and gated norm; the clamped gate; sums of two
parts with a factor each), each alone against its plain torch form (tests/torch_ops.py), in float32 and bfloat16, at
sizes that are no powers of two."""
import pytest
import torch

from litellmengine_amd.parts.base import Injected, ScaledSum
from tests.test_kezasun_kernels_gpu import batch, ints, ops, rnd, tol
from tests.test_telulorn_kernels_gpu import paged_setup
from tests.torch_ops import TorchOps, v_pages

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
REF = TorchOps(torch.float64)


def close(got, want, limit, what=""):
    err = float((got.double() - want.double()).abs().max())
    assert err < limit, (what, err)


# -- the first rows ------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [72, 50, 256, 2048, 9000])
def test_embedding_norm(dtype, H):
    o = ops()
    V, P, N = 40, 17, 6
    table, pos = rnd((V, H), dtype, 1), rnd((P, H), dtype, 2)
    ids, positions = ints([3, 39, 0, 7, 7, 21]), ints([0, 16, 5, 3, 4, 1])
    w, nw = 1.0 + rnd((H,), torch.float32, 3, 0.1), (1.0 + rnd((H,), torch.float32, 4, 0.1)).to(dtype)
    for args in ((7.5, positions, pos, w, 1e-5, nw, 1e-6), (1.0, positions, pos, None, 0.0, nw, 1e-5), (0.3, None, None, w, 1e-5, None, 0.0)):
        want = REF.embedding_norm(ids, table, *args, dtype)
        got = o.embedding_norm(ids, table, *args, dtype)
        assert got[0].dtype == torch.float32
        close(got[0], want[0], 2e-5)
        assert (got[1] is None) == (want[1] is None)
        if got[1] is not None:
            assert got[1].dtype == dtype
            close(got[1], want[1], tol(dtype, 5))
    # ids below zero stand for what the step before left on the device
    feedback, seqs, slots = ints([11, 39, 5]), ints([0, 0, 1, 1, 1, 1]), ints([2, 1])
    ids = ints([-1, 3, -1, 7, 7, 21])
    args = (2.0, positions, pos, w, 1e-5, nw, 1e-6, dtype, feedback, seqs, slots)
    close(o.embedding_norm(ids, table, *args)[0], REF.embedding_norm(ids, table, *args)[0], 2e-5)
    same = ints([5, 3, 39, 7, 7, 21])
    assert torch.equal(o.embedding_norm(ids, table, *args)[0], o.embedding_norm(same, table, *args[:8])[0])


# -- sums -----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [72, 50, 4096])
def test_two_parts_with_a_factor_each_and_a_bias_beside_the_delta(dtype, H):
    o = ops()
    a, b, bias = rnd((7, H), dtype, 1), rnd((7, H), torch.float32, 2), rnd((H,), torch.float32, 3)
    w = 1.0 + rnd((H,), torch.float32, 4, 0.1)
    hidden, rows = rnd((7, H), torch.float32, 5), ints([6, 0, 3])
    want_h, got_h = hidden.clone(), hidden.clone()
    want = REF.scaled_add_rmsnorm(want_h, a, b, 0.6, w, 1e-5, dtype, mult_b=-1.7)
    got = o.scaled_add_rmsnorm(got_h, a, b, 0.6, w, 1e-5, dtype, mult_b=-1.7)
    close(got_h, want_h, 1e-5)
    close(got, want, tol(dtype, 4))
    close(got_h, hidden + ScaledSum(a, b, 0.6, -1.7).total(), 1e-5)
    got = o.scaled_add_rmsnorm(got_h, a, b, 0.6, w, 1e-5, dtype, rows, mult_b=-1.7)
    close(got, REF.scaled_add_rmsnorm(want_h.clone(), a, b, 0.6, w, 1e-5, dtype, rows, mult_b=-1.7), tol(dtype, 4))
    for delta in (a, None, ScaledSum(a, b, 0.6, 0.9), Injected(a, bias, None, o)):
        want_h, got_h = hidden.clone(), hidden.clone()
        want = REF.inject_rmsnorm(want_h, delta, bias, None, w, 1e-5, dtype)
        got = o.inject_rmsnorm(got_h, delta, bias, None, w, 1e-5, dtype)
        close(got_h, want_h, 1e-5)
        close(got, want, tol(dtype, 4))
        some = o.inject_rmsnorm(hidden, delta, bias, None, w, 1e-5, dtype, rows)  # some rows, nothing written
        close(some, want[rows.long()], tol(dtype, 4))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F", [20, 64, 100, 1024])
def test_clamped_gate(dtype, F):
    o = ops()
    z, b = rnd((9, 2 * F), dtype, 1, 3.0), rnd((2 * F,), dtype, 2)
    for limit in (0.7, 2.0, 7.0):
        for bias in (b, None):
            close(o.bias_act(z, "clamp", True, bias=bias, limit=limit), REF.bias_act(z, "clamp", True, bias=bias, limit=limit), tol(dtype, 20))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,K,F", [(1, 64, 40), (8, 2048, 8192), (16, 1024, 96), (5, 72, 50), (31, 256, 64), (40, 128, 64), (3, 50, 24), (9, 4096, 12288)])
def test_clamped_gate_behind_its_product(dtype, M, K, F):
    """One launch with the activation in its epilogue where there are few rows, the product and the activation elsewhere."""
    o = ops()
    x, w, b = rnd((M, K), dtype, 1), rnd((2 * F, K), dtype, 2, K ** -0.5), rnd((2 * F,), dtype, 3)
    for limit, bias in ((0.6, b), (3.0, None)):
        close(o.gate_up_clamped(x, w, bias, limit), REF.gate_up_clamped(x, w, bias, limit), tol(dtype, 4))


# -- attention with capped scores ---------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nq,nkv,D,P", [(6, 2, 64, 16), (4, 4, 32, 16), (8, 1, 96, 32), (5, 5, 128, 16), (2, 1, 256, 16), (3, 1, 160, 16), (6, 3, 40, 8)])
@pytest.mark.parametrize("cap,window", [(5.0, None), (0.8, None), (20.0, 70)])
def test_capped_attention(dtype, nq, nkv, D, P, cap, window):
    """Whole prompts, portions after a past, single tokens; scores far beyond the cap and near zero; with sinks."""
    o = ops()
    q, kv, table, slots, cu, kv_lens, seqs, most = paged_setup(dtype, [1, 40, 3, 1, 70], [200, 0, 90, 66, 130], nq, nkv, D, P, 3)
    for sinks in (None, rnd((nq,), torch.float32, 8)):
        want = REF.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, window, 0.6, sinks=sinks, softcap=cap)
        got = o.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, window, 0.6, 1, 70, most, sinks=sinks, softcap=cap)
        close(got, want, tol(dtype))
    without = REF.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, window, 0.6)
    assert (REF.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, window, 0.6, softcap=cap).double() - without.double()).abs().max() > 0.01


@pytest.mark.parametrize("dtype", DTYPES)
def test_capped_attention_in_key_splits_every_form_and_beside_kept_keys(dtype):
    o = ops()
    for q_lens, pasts in (([1], [3000]), ([20], [3000]), ([1, 1], [2500, 900]), ([600], [0])):
        for D in (64, 128):
            q, kv, table, slots, cu, kv_lens, seqs, most = paged_setup(dtype, q_lens, pasts, 4, 1, D, 16, 7)
            want = REF.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, None, 0.25, softcap=3.0)
            for form in ((0, 1, 2, 3) if dtype == torch.bfloat16 and max(q_lens) > 4 else (0,)):
                o.force_prefill_form = form
                try:
                    got = o.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, None, 0.25, min(q_lens), max(q_lens), most, softcap=3.0)
                finally:
                    o.force_prefill_form = 0
                close(got, want, tol(dtype), (q_lens, D, form))
    q, kv, table, slots, cu, kv_lens, seqs, most = paged_setup(dtype, [1, 30], [200, 90], 4, 2, 64, 16, 7)
    want = REF.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, 50, 0.4, softcap=2.0, keep_first=9)
    close(o.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, 50, 0.4, 1, 30, most, softcap=2.0, keep_first=9), want, tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("q_len", [1, 30])
def test_a_far_key_under_the_cap(dtype, q_len):
    """One key's score is far above the cap: it weighs e^cap against the others' e^-cap, no more."""
    o = ops()
    D, P, past, cap = 64, 16, 500, 4.0
    for place in (0, P - 1, P, 300):
        q, kv, table, slots, cu, kv_lens, seqs, most = paged_setup(dtype, [q_len], [past], 2, 1, D, P, 5)
        q[-1, 0] = 1.0
        kv[:, 0] = -1.0  # every key but one: a score of -D
        kv[int(table[int(slots[0]), place // P]), 0, :, place % P, :] = 1.0
        v_pages(kv)[:] = 0.0
        v_pages(kv)[int(table[int(slots[0]), place // P]), :, :, place % P] = 1.0
        got = o.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, None, 1.0, q_len, q_len, most, softcap=cap)
        n = past + q_len - 1  # other keys of the last query
        share = 1.0 / (1.0 + n * torch.exp(torch.tensor(-2.0 * cap)).item())
        close(got[-1, :D], torch.full((D,), share).cuda(), 0.01)


# -- the delta rule with a decay per key channel --------------------------------------------------------
@pytest.mark.parametrize("H,dim,vdim,RA,RG,N", [(3, 24, 20, 5, 7, 9), (1, 100, 12, 16, 1, 1), (4, 64, 64, 24, 24, 130), (2, 8, 33, 40, 17, 67),
                                                (5, 17, 9, 33, 50, 64), (2, 256, 40, 128, 64, 300)])
def test_low_rank_gates(H, dim, vdim, RA, RG, N):
    o = ops()
    up = lambda n: -(-n // 16) * 16
    pad = lambda t, n: torch.nn.functional.pad(t, (0, n - t.shape[1])).contiguous()
    h4 = -(-H // 4) * 4
    low = torch.cat([pad(rnd((N, H), torch.float32, 1), h4), pad(rnd((N, RA), torch.float32, 2), up(RA)), pad(rnd((N, RG), torch.float32, 3), up(RG))], 1)
    a2, g2 = pad(rnd((H * dim, RA), torch.float32, 4, 0.7), up(RA)), pad(rnd((H * vdim, RG), torch.float32, 5), up(RG))
    a_log, dt_bias = rnd((H,), torch.float32, 6), rnd((H * dim,), torch.float32, 7, 4.0)
    want = REF.low_rank_gates(low, h4, a2, a_log, dt_bias, dim, h4 + up(RA), g2)
    got = o.low_rank_gates(low, h4, a2, a_log, dt_bias, dim, h4 + up(RA), g2)
    close(got[0], want[0], 2e-6)
    close(got[1], want[1], 2e-5)
    alone, none = o.low_rank_gates(low, h4, a2, a_log, dt_bias, dim)
    assert none is None and torch.equal(alone, got[0])


@pytest.mark.parametrize("H,G,dim,vdim,q_lens", [(6, 2, 24, 20, [5, 1, 1, 30]), (1, 1, 100, 12, [17, 1]), (4, 4, 64, 64, [1, 1, 1]),
                                                 (2, 1, 256, 40, [70]), (4, 1, 8, 100, [3, 9]), (3, 3, 128, 16, [1, 26]), (4, 2, 32, 24, [40, 1, 33, 2])])
def test_delta_walk_with_a_decay_per_channel(H, G, dim, vdim, q_lens):
    o = ops()
    seq_slots, cu, token_seq, N = batch(q_lens)
    unit = lambda t, heads: torch.nn.functional.normalize(t.view(N, heads, dim), dim=-1).reshape(N, heads * dim).contiguous()
    q, k = unit(rnd((N, G * dim), torch.float32, 1), G) * dim ** -0.5, unit(rnd((N, G * dim), torch.float32, 2), G)
    v, ba = rnd((N, H * vdim), torch.float32, 3), rnd((N, H + 3), torch.float32, 4, 2.0)
    decay = torch.sigmoid(rnd((N, H * dim), torch.float32, 5, 3.0))
    wide = rnd((9, H * vdim * dim + 11), torch.float32, 7, 0.3)
    got_state, want_state = wide.clone(), wide.clone()
    want = REF.delta_scan(q, k, v, ba, None, None, want_state, H, G, dim, vdim, seq_slots, cu, decay=decay)
    got = o.delta_scan(q, k, v, ba, None, None, got_state, H, G, dim, vdim, seq_slots, cu, decay=decay)
    close(got, want, 2e-5)
    close(got_state, want_state, 2e-5)
    s = len(q_lens) - 1  # the last request in pieces of 1, 2, 3, ... tokens
    lo, hi = int(cu[s]), int(cu[s + 1])
    st, rows, at, n = wide.clone(), [], lo, 1
    while at < hi:
        n = min(n, hi - at)
        cut = [t[at : at + n].contiguous() for t in (q, k, v, ba)]
        rows.append(o.delta_scan(*cut, None, None, st, H, G, dim, vdim, ints([int(seq_slots[s])]), ints([0, n]), decay=decay[at : at + n].contiguous()))
        at += n
        n += 1
    close(torch.cat(rows), got[lo:hi], 1e-6)
    close(st[int(seq_slots[s])], got_state[int(seq_slots[s])], 1e-6)


def test_every_channel_forgets_at_its_own_rate():
    """Keys are single channels: what was written under channel i is read back times the product of i's decays."""
    o = ops()
    dim, vdim, N = 32, 16, 20
    k = torch.zeros((N, dim)).cuda()
    k[0, 3], k[1, 7] = 1.0, 1.0
    q = torch.zeros((N, dim)).cuda()
    q[2:, 3], q[2:, 7] = 1.0, 0.0
    q[11:, 3], q[11:, 7] = 0.0, 1.0
    v = rnd((N, vdim), torch.float32, 2)
    decay = torch.ones((N, dim)).cuda()
    decay[:, 3], decay[:, 7] = 0.5, 0.9
    ba = torch.full((N, 1), 40.0).cuda()
    state = torch.zeros((2, vdim * dim)).cuda()
    got = o.delta_scan(q, k, v, ba, None, None, state, 1, 1, dim, vdim, ints([1]), ints([0, N]), decay=decay)
    for t in range(2, N):
        close(got[t], v[0] * 0.5 ** t if t < 11 else v[1] * 0.9 ** (t - 1), 1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("J", [2, 3, 4, 8])
def test_delta_convolution_moves_the_state_on_with_single_tokens(dtype, J):
    o = ops()
    G, H, dim, vdim = 2, 4, 24, 20
    cols = 2 * G * dim + H * vdim
    seq_slots, cu, token_seq, N = batch([1, 1, 1])
    u, taps, wide = rnd((N, cols), dtype, 1), rnd((cols, J), torch.float32, 2, 0.5), rnd((9, 13 + (J - 1) * cols), torch.float32, 3)
    a, b = wide.clone(), wide.clone()
    want = o.delta_conv(u, taps, a[:, 13:], token_seq, cu, seq_slots, G, dim, H, vdim, 1e-6, dim ** -0.5)
    o.conv_state_update(u, a[:, 13:], J - 1, cu, seq_slots)
    assert o.can_advance_conv(J, 1) and not o.can_advance_conv(J, 2) and not o.can_advance_conv(9, 1)
    got = o.delta_conv(u, taps, b[:, 13:], token_seq, cu, seq_slots, G, dim, H, vdim, 1e-6, dim ** -0.5, advance=True)
    assert all(torch.equal(x, y) for x, y in zip(got, want)) and torch.equal(a, b) and not torch.equal(a, wide)


@pytest.mark.parametrize("dtype", DTYPES)
def test_delta_output_norm_with_a_sigmoid_gate_in_32_bit(dtype):
    o = ops()
    for H, vdim in ((6, 20), (1, 256), (5, 100)):
        x, gate = rnd((9, H * vdim), torch.float32, 1, 3.0), rnd((9, H * vdim), torch.float32, 2, 2.0)
        w = 1.0 + rnd((vdim,), torch.float32, 3, 0.1)
        got = o.delta_out_norm(x, gate, w, 1e-5, H, vdim, act="sigmoid", out_dtype=dtype)
        assert got.dtype == dtype
        close(got, REF.delta_out_norm(x, gate, w, 1e-5, H, vdim, act="sigmoid", out_dtype=dtype), tol(dtype, 4))


# -- Mamba-2 --------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,J,q_lens", [(100, 3, [5, 1, 1, 2]), (300, 1, [7, 1]), (40, 4, [1, 1, 1]), (77, 6, [40, 3]), (64, 9, [12, 1, 30]),
                                        (1000, 4, [700, 1, 37, 2, 560]), (50, 2, [1, 9, 2])])
def test_ssd_convolution(dtype, C, J, q_lens):
    """Columns in the middle of a row, state rows that are columns of a wider one, more taps than the runs take; the
    state moves on; the same tokens one by one give the same rows."""
    o = ops()
    seq_slots, cu, token_seq, N = batch(q_lens)
    u, taps, bias = rnd((N, C + 12), dtype, 1), rnd((C, J), torch.float32, 2, 0.5), rnd((C,), torch.float32, 3)
    wide = rnd((9, 13 + max(1, J - 1) * C), torch.float32, 4)
    a, b = wide.clone(), wide.clone()
    for bb in (bias, None):
        a, b = wide.clone(), wide.clone()
        want = REF.ssd_conv(u, 7, taps, bb, a[:, 13:], token_seq, cu, seq_slots)
        got = o.ssd_conv(u, 7, taps, bb, b[:, 13:], token_seq, cu, seq_slots, single=max(q_lens) == 1)
        close(got, want, 2e-5)
        close(a, b, 1e-7)
    st, rows = wide.clone(), []
    n0 = min(q_lens[0], 40)
    for t in range(n0):
        rows.append(o.ssd_conv(u[t : t + 1].contiguous(), 7, taps, None, st[:, 13:], ints([0]), ints([0, 1]), seq_slots[:1].contiguous(), single=True))
    close(torch.cat(rows), got[:n0], 1e-6)
    if n0 == q_lens[0]:
        close(st[int(seq_slots[0])], b[int(seq_slots[0])], 1e-7)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,K,H,C,J", [(1, 50, 3, 40, 4), (8, 2048, 64, 700, 4), (5, 100, 7, 77, 1), (70, 128, 12, 64, 3), (3, 64, 4, 64, 9), (200, 72, 1, 300, 2)])
def test_step_sizes_made_beside_the_convolution(dtype, N, K, H, C, J):
    o = ops()
    u, taps, state = rnd((N, C), dtype, 1), rnd((C, J), torch.float32, 2, 0.5), rnd((N + 1, max(1, J - 1) * C), torch.float32, 3)
    x, w = rnd((N, K), dtype, 4), rnd((H, K), dtype, 5)
    where = (ints(list(range(N))), ints(list(range(N + 1))), ints(list(range(N))[::-1]))
    a, b = state.clone(), state.clone()
    want = REF.ssd_conv(u, 0, taps, None, a, *where, x=x, dt_w=w)
    got = o.ssd_conv(u, 0, taps, None, b, *where, single=True, x=x, dt_w=w)
    close(got[0], want[0], 2e-5)
    close(got[1], want[1], 1e-4 * max(1.0, K ** 0.5 / 8))
    close(a, b, 1e-7)
    assert torch.equal(o.ssd_conv(u, 0, taps, None, state.clone(), *where, single=True), got[0])


def ssd_case(H, G, vdim, n, q_lens, seed=1, steep=1.0):
    seq_slots, cu, token_seq, N = batch(q_lens)
    c = rnd((N, H * vdim + 2 * G * n), torch.float32, seed)
    dt_in = rnd((N, H + 2), torch.float32, seed + 1, 1.5)
    dt_bias, a_log, D = rnd((H,), torch.float32, seed + 2), rnd((H,), torch.float32, seed + 3, steep) - 1.0, rnd((H,), torch.float32, seed + 4)
    wide = rnd((9, H * vdim * n + 12), torch.float32, seed + 5, 0.5)
    return c, dt_in, dt_bias, a_log, D, wide, seq_slots, cu


@pytest.mark.parametrize("H,G,vdim,n,q_lens", [
    (6, 2, 20, 24, [5, 1, 1, 30]), (1, 1, 12, 100, [17, 1]), (4, 4, 64, 64, [1, 1, 1]), (2, 1, 40, 256, [70]), (4, 1, 100, 8, [3, 200]),
    (3, 3, 16, 128, [1, 26, 64, 65]), (4, 2, 24, 48, [40, 1, 133, 2, 32, 33]), (8, 1, 64, 128, [300]), (5, 1, 33, 17, [130, 31]),
    (2, 2, 256, 16, [129]), (16, 4, 32, 32, [257, 1, 1, 63]), (2, 1, 48, 192, [90])])
def test_ssd_recurrence(H, G, vdim, n, q_lens):
    """From states that are not zero: requests that are walked beside requests that are cut into chunks, whose last
    chunk is whole, nearly empty or nearly whole; then a request in pieces gives the same rows and the same state."""
    o = ops()
    c, dt_in, dt_bias, a_log, D, wide, seq_slots, cu = ssd_case(H, G, vdim, n, q_lens)
    par = (dt_bias, a_log, D)
    got_state, want_state = wide.clone(), wide.clone()
    want = REF.ssd_scan(c, dt_in, *par, want_state, H, G, vdim, n, seq_slots, cu)
    got = o.ssd_scan(c, dt_in, *par, got_state, H, G, vdim, n, seq_slots, cu, min(q_lens), max(q_lens))
    scale = max(1.0, float(want.abs().max()))
    close(got, want, 4e-6 * scale)
    close(got_state, want_state, 4e-6 * max(1.0, float(want_state.abs().max())))
    assert torch.equal(got_state[:, H * vdim * n:], wide[:, H * vdim * n:])  # what lies behind the matrices stays
    s = max(range(len(q_lens)), key=lambda i: q_lens[i])  # the longest request in pieces
    lo, hi = int(cu[s]), int(cu[s + 1])
    st, rows, at = wide.clone(), [], lo
    for size in [1, 2, 31, 32, 33, 64, 2, 66] * 4:
        m = min(size, hi - at)
        if m == 0:
            break
        rows.append(o.ssd_scan(c[at : at + m].contiguous(), dt_in[at : at + m].contiguous(), *par, st, H, G, vdim, n,
                               ints([int(seq_slots[s])]), ints([0, m]), m, m))
        at += m
    close(torch.cat(rows), got[lo:at], 4e-6 * scale)
    # bounds that are not known choose the same results
    again = wide.clone()
    close(o.ssd_scan(c, dt_in, *par, again, H, G, vdim, n, seq_slots, cu), got, 1e-6 * scale)
    close(again, got_state, 1e-6 * scale)


def test_ssd_neighbours_deep_in_a_chunk_behind_a_steep_drop():
    """One token wipes the state (a step size of thousands); its followers hardly decay: their weights among each other
    are as exact as if the drop had not been."""
    o = ops()
    H, vdim, n, N = 2, 32, 32, 64
    c, dt_in, dt_bias, a_log, D, wide, seq_slots, cu = ssd_case(H, 1, vdim, n, [N])
    a_log, dt_bias = torch.full((H,), 3.0).cuda(), torch.zeros(H).cuda()
    dt_in = torch.full((N, H + 2), -6.0).cuda()
    dt_in[10] = 400.0
    want = REF.ssd_scan(c, dt_in, dt_bias, a_log, D, wide.clone(), H, 1, vdim, n, seq_slots, cu)
    got = o.ssd_scan(c, dt_in, dt_bias, a_log, D, wide.clone(), H, 1, vdim, n, seq_slots, cu, N, N)
    err = (got.double() - want.double()).abs().max(dim=1).values / want.abs().max(dim=1).values.double()
    assert err.max() < 1e-5, err  # (one float for the sums: 2e-4)


def test_ssd_heads_that_share_a_workgroup():
    o = ops()
    c, dt_in, dt_bias, a_log, D, wide, seq_slots, cu = ssd_case(12, 2, 24, 40, [150, 90])
    args = (c, dt_in, dt_bias, a_log, D)
    want = REF.ssd_scan(*args, wide.clone(), 12, 2, 24, 40, seq_slots, cu)
    kept = o.ssd_heads_a_group
    for k in (1, 2, 3, 6):
        o.ssd_heads_a_group = lambda *a: k
        try:
            close(o.ssd_scan(*args, wide.clone(), 12, 2, 24, 40, seq_slots, cu, 90, 150), want, 4e-6 * max(1.0, float(want.abs().max())), k)
        finally:
            o.ssd_heads_a_group = kept
    assert o.ssd_heads_a_group(64, 8, 1) == 1 and o.ssd_heads_a_group(64, 8, 10 ** 6) == 8


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("inner,groups", [(120, 1), (120, 5), (96, 2), (4096, 1), (4096, 8), (9000, 1), (60, 60)])
def test_ssd_gated_norm(dtype, inner, groups):
    o = ops()
    y, u, w = rnd((7, inner), torch.float32, 1, 2.0), rnd((7, inner + 9), dtype, 2), 1.0 + rnd((inner,), torch.float32, 3, 0.1)
    close(o.ssd_gate_norm(y, u, 4, w, 1e-5, groups), REF.ssd_gate_norm(y, u, 4, w, 1e-5, groups), tol(dtype, 8))
