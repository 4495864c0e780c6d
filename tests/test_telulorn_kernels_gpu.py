"""The kernels that Telulorn added (what enters the stream between two blocks with the norm behind it, rotations in
neighbouring pairs with rotated values and the turn back under an element-wise gate, windows that keep the first
keys in every attention kernel, attention whose heads' weights are mixed, gated linear attention), each alone
against its plain torch form (tests/torch_ops.py), in float32 and bfloat16, at sizes that are no powers of two."""
import pytest
import torch

from litellmengine_amd.parts.base import EmbeddedRows, PartialSums, ScaledSum
from tests.test_kezasun_kernels_gpu import batch, ints, ops, rnd, tol
from tests.test_kezasun_kernels_gpu import paged_setup as kezasun_paged_setup
from tests.torch_ops import TorchOps, v_pages

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
REF = TorchOps(torch.float64)


def paged_setup(*args):
    """q, pages, block table, slots, first rows, lengths, requests of the tokens, longest length (of scrambled pages)."""
    *arrays, _, most = kezasun_paged_setup(*args)
    return (*arrays, most)


# -- what enters the stream between two blocks --------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [40, 250, 1000, 9000])
@pytest.mark.parametrize("kind", ["nothing", "delta", "pair", "sums"])
def test_inject_rmsnorm(dtype, H, kind):
    """A block's result of every kind, a vector for all rows, and the embedding's rows once more (among them one
    whose id the step before has left on the device); each alone and together."""
    o = ops()
    N, V = 6, 11
    hidden = rnd((N, H), torch.float32, 2, 3.0)
    vec = rnd((H,), torch.float32, 3)
    table = rnd((V, H), dtype, 4)
    ids, seqs, slots, feedback = ints([3, 0, -1, 10, 3, -1]), ints([0, 0, 1, 2, 2, 2]), ints([2, 0, 1]), ints([7, 5, 1])
    w = 1.0 + rnd((H,), torch.float32, 5, 0.1)
    delta = {"nothing": None, "delta": rnd((N, H), dtype, 6), "pair": ScaledSum(rnd((N, H), dtype, 7), rnd((N, H), torch.float32, 8), 1.0),
             "sums": PartialSums(rnd((3, N, H), torch.float32, 9))}[kind]
    for vector in (None, vec):
        for again in (None, EmbeddedRows(ids, table, 1.5, feedback, seqs, slots)):
            want_h, got_h = hidden.clone(), hidden.clone()
            want = REF.inject_rmsnorm(want_h, delta, vector, again, w, 1e-5, dtype)
            got = o.inject_rmsnorm(got_h, delta, vector, again, w, 1e-5, dtype)
            assert (got_h.double() - want_h.double()).abs().max() < 4e-6
            assert got.dtype == dtype and (got.double() - want.double()).abs().max() < tol(dtype, 4)
            if kind == "nothing" and vector is None and again is None:
                assert torch.equal(got_h, hidden)


# -- rotations in pairs, rotated values, the turn back under the gate ----------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nq,nkv,dim,vdim,rot,D,bias,turn_values", [(6, 2, 24, 40, 8, 64, True, True), (4, 4, 64, 64, 64, 64, True, True),
                                                                    (3, 1, 48, 16, 2, 64, False, True), (8, 2, 31, 33, 0, 64, False, False),
                                                                    (1, 1, 96, 96, 48, 96, True, True), (5, 5, 7, 5, 6, 32, True, False)])
def test_pair_rotation_cache_write_and_turn_back(dtype, nq, nkv, dim, vdim, rot, D, bias, turn_values):
    o = ops()
    P, pages = 16, 9
    # a run of tokens side by side in a page, a run that begins in the middle, scattered places, one that is not written
    slots = list(range(32, 40)) + list(range(83, 99)) + [3, 17, 18, 79, -1, 0, 33 + 80, 120, 121]
    N = len(slots)
    where = [700 + i for i in range(24)] + [0, 1, 2, 5, 9, 100000, 11, 3, 4]
    slots, pos = ints(slots), ints(where)
    used = nq * dim + nkv * (dim + vdim)
    u = rnd((N, used + nq * vdim), dtype, 1)
    b = rnd((used,), dtype, 2, 0.5) if bias else None
    freq = lambda n: torch.pow(torch.tensor(1e4, dtype=torch.float64), -torch.arange(n // 2, dtype=torch.float64) * 2 / max(n, 1)).float().cuda()
    cs = o.rope_table(pos, freq(rot)) if rot else None
    vcs = o.rope_table(pos, freq(vdim)) if turn_values else None
    kv_got = torch.full((pages, 2, nkv, P, D), 7.0, dtype=dtype).cuda()
    kv_want = kv_got.clone()
    want = REF.pair_rope_write(u, b, slots, cs, vcs, kv_want, nq, nkv, dim, vdim)
    got = o.pair_rope_write(u, b, slots, cs, vcs, kv_got, nq, nkv, dim, vdim)
    assert got.shape == (N, nq, D) and (got.double() - want.double()).abs().max() < tol(dtype, 4)
    assert (kv_got.double() - kv_want.double()).abs().max() < tol(dtype, 4)
    if dim < D:
        assert float(got[:, :, dim:].abs().max()) == 0.0
    a = rnd((N, nq * D), dtype, 5)
    want = REF.turn_back_gate(a, u, used, nq, vdim, vcs, 0.7)
    got = o.turn_back_gate(a, u, used, nq, vdim, vcs, 0.7)
    assert got.shape == (N, nq * vdim) and (got.double() - want.double()).abs().max() < tol(dtype, 2)
    if turn_values:  # a value turned by its position and turned back by the same position is itself
        kv = torch.zeros((pages, 2, nkv, P, D), dtype=torch.float32).cuda()
        uf = u.float()
        o.pair_rope_write(uf, None, slots, None if cs is None else cs, vcs, kv, nq, nkv, dim, vdim)
        row = v_pages(kv)[int(slots[3]) // P, :, :, int(slots[3]) % P]  # [nkv, D]
        back = o.turn_back_gate(row.reshape(1, -1).contiguous(), torch.full((1, nkv * vdim), 60.0).cuda(), 0, nkv, vdim,
                                vcs[3:4].contiguous(), 1.0)
        assert (back.view(nkv, vdim) - uf[3, nq * dim + nkv * dim : used].view(nkv, vdim)).abs().max() < 1e-5


# -- windows that keep the first keys -----------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,P,nq,nkv", [(64, 16, 6, 2), (96, 16, 3, 3), (128, 32, 8, 2), (48, 8, 4, 1), (32, 16, 40, 2), (160, 16, 2, 1)])
@pytest.mark.parametrize("window,keep", [(33, 4), (70, 20), (16, 65), (5, 1)])
def test_attention_with_kept_first_keys(dtype, D, P, nq, nkv, window, keep):
    """Prompts whole, portions after a past, single tokens, all in one step: the first keys just inside and just
    outside, overlapping the window, and beyond it; with sinks."""
    o = ops()
    q, kv, table, slots, cu, kv_lens, seqs, most = paged_setup(dtype, [1, 40, 3, 1, 70], [200, 0, 90, 66, 130], nq, nkv, D, P, 3)
    sinks = rnd((nq,), torch.float32, 8)
    want = REF.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, window, 0.2, sinks=sinks, keep_first=keep)
    got = o.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, window, 0.2, 1, 70, most, sinks=sinks, keep_first=keep)
    assert (got.double() - want.double()).abs().max() < tol(dtype)
    without = REF.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, window, 0.2, sinks=sinks)
    assert (want.double() - without.double()).abs().max() > 0.02


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("q_len", [1, 30])
def test_the_last_kept_key_and_the_first_that_is_not(dtype, q_len):
    """One key's score stands out: as the last kept key it takes all the weight, one further it is not seen."""
    o = ops()
    D, P, window, keep = 64, 16, 40, 18
    past = 400
    for place, seen in ((0, True), (keep - 1, True), (keep, False), (past + q_len - 1 - window, False)):
        q, kv, table, slots, cu, kv_lens, seqs, most = paged_setup(dtype, [q_len], [past], 2, 1, D, P, 5)
        page, off = int(table[int(slots[0]), place // P]), place % P
        kv[page, 0, :, off, :] = (q[-1, 0].float() * 4).to(dtype)
        v_pages(kv)[page, :, :, off] = 9.0
        got = o.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, window, 0.3, q_len, q_len, most, keep_first=keep)
        want = REF.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, window, 0.3, keep_first=keep)
        assert (got.double() - want.double()).abs().max() < tol(dtype, 10)
        assert bool(got[-1, :D].float().mean() > 8.0) == seen, place


def test_key_splits_with_kept_first_keys():
    """A decode batch and a short portion behind a long past whose window is cut into key splits."""
    o = ops()
    for q_lens, pasts in (([1], [3000]), ([20], [3000]), ([1, 1], [2500, 900])):
        for dtype in DTYPES:
            q, kv, table, slots, cu, kv_lens, seqs, most = paged_setup(dtype, q_lens, pasts, 4, 1, 64, 16, 7)
            want = REF.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, 2048, 0.25, keep_first=100)
            got = o.paged_attention(q, kv, table, slots, cu, kv_lens, seqs, 2048, 0.25, min(q_lens), max(q_lens), most, keep_first=100)
            assert (got.double() - want.double()).abs().max() < tol(dtype)


# -- heads' weights mixed -------------------------------------------------------------------------------
def talking_case(dtype, q_lens, pasts, H, G, D, P, seed=3):
    q, kv, table, slots, cu, kv_lens, seqs, most = paged_setup(dtype, q_lens, pasts, H, G, D, P, seed)
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], dtype=torch.float32).cuda()
    talk = rnd((H, H), torch.bfloat16, seed + 1, 0.5).float()
    return (q, kv, table, slots, cu, kv_lens, seqs), most, slopes, talk


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,P", [(8, 4, 64, 16), (6, 2, 32, 16), (1, 1, 128, 32), (12, 3, 96, 16), (16, 16, 64, 16), (16, 2, 128, 16),
                                     (20, 5, 64, 48), (32, 8, 128, 16), (32, 1, 32, 16), (3, 3, 160, 16), (40, 8, 32, 16), (5, 1, 48, 8)])
@pytest.mark.parametrize("chunk", [None, 24, 100])
def test_talking_attention(dtype, H, G, D, P, chunk):
    """Whole prompts, portions after a past that begin and end in the middle of a chunk, single tokens (the first of
    a chunk, the last of one): heads of every number the kernels tell apart, pages larger and smaller."""
    o = ops()
    args, most, slopes, talk = talking_case(dtype, [1, 37, 2, 1, 61, 1], [100, 0, 47, 99, 130, 0], H, G, D, P)
    want = REF.talking_attention(*args, chunk, 0.2, slopes, talk)
    got = o.talking_attention(*args, chunk, 0.2, slopes, talk, 1, 61, most)
    err = (got.double() - want.double()).abs().max()
    assert err < tol(dtype, max(1.0, float(want.double().abs().max()))), float(err)
    # single tokens alone, and without a distance bias
    args, most, slopes, talk = talking_case(dtype, [1, 1, 1], [190, 23, 24], H, G, D, P, 9)
    want = REF.talking_attention(*args, chunk, 0.2, None, talk)
    got = o.talking_attention(*args, chunk, 0.2, None, talk, 1, 1, most)
    assert (got.double() - want.double()).abs().max() < tol(dtype, max(1.0, float(want.double().abs().max())))


@pytest.mark.parametrize("dtype", DTYPES)
def test_both_forms_of_the_prompt_kernel_and_long_chunks(dtype):
    o = ops()
    for H, G, q_lens, pasts, chunk in ((16, 4, [700, 300], [0, 250], 256), (32, 8, [600], [333], 512), (16, 4, [1, 1], [3000, 1900], 2048)):
        args, most, slopes, talk = talking_case(dtype, q_lens, pasts, H, G, 64, 16, 11)
        want = REF.talking_attention(*args, chunk, 0.15, slopes, talk)
        got = o.talking_attention(*args, chunk, 0.15, slopes, talk, min(q_lens), max(q_lens), most)
        assert (got.double() - want.double()).abs().max() < tol(dtype, max(1.0, float(want.double().abs().max())))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("q_len", [1, 20])
def test_a_chunks_first_key_and_the_one_before_it(dtype, q_len):
    """One key stands out for one head only: the heads that listen to that head read its value, the others do not;
    the key before the chunk's first is nobody's."""
    o = ops()
    H, G, D, P, chunk, past = 8, 2, 64, 16, 120, 300
    pos = past + q_len - 1
    first = pos // chunk * chunk
    for place, seen in ((first, True), (first - 1, False), (pos, True)):
        q, kv, table, slots, cu, kv_lens, seqs, most = paged_setup(dtype, [q_len], [past], H, G, D, P, 5)
        # head 5 alone looks for the key of its group (1) at `place`, and its value is in group 0 as well
        q[-1] *= 0.05
        q[-1, 5] = 2.0
        page, off = int(table[int(slots[0]), place // P]), place % P
        kv[page, 0, 1, off, :] = 1.0
        v_pages(kv)[page, :, :, off] = 50.0
        talk = torch.zeros((H, H)).cuda()
        talk[2, 5] = 1.0  # head 2 (group 0) listens to head 5 alone, head 6 to head 0
        talk[6, 0] = 1.0
        args = (q, kv, table, slots, cu, kv_lens, seqs)
        got = o.talking_attention(*args, chunk, 0.3, None, talk, q_len, q_len, most)
        want = REF.talking_attention(*args, chunk, 0.3, None, talk)
        assert (got.double() - want.double()).abs().max() < tol(dtype, 50)
        heads = got[-1].float().view(H, D).mean(1)
        assert bool(heads[2] > 45.0) == seen and abs(float(heads[6])) < 5.0 and float(heads[[0, 1, 3, 4, 5, 7]].abs().max()) == 0.0


# -- gated linear attention -----------------------------------------------------------------------------
@pytest.mark.parametrize("N,R,C,tau", [(5, 16, 40, 16.0), (1, 3, 300, 1.0), (70, 40, 257, 2.5)])
def test_gla_decay(N, R, C, tau):
    o = ops()
    low, a2, b = rnd((N, R), torch.float32, 1, 3.0), rnd((R, C), torch.float32, 2, 3.0), rnd((C,), torch.float32, 3, 5.0)
    b[:2] = torch.tensor([3000.0, -3000.0])  # one that never forgets, one that forgets almost at once
    got, want = o.gla_decay(low, a2, b, tau), REF.gla_decay(low, a2, b, tau)
    assert (got.double() - want.double()).abs().max() < 2e-5
    assert float(got[:, 0].min()) == 1.0 and float(got[:, 1].max()) < 1e-3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dim,vdim,q_lens", [(3, 24, 20, [5, 1, 1, 30]), (1, 100, 12, [17, 1]), (4, 64, 64, [1, 1, 1]), (2, 256, 40, [70]),
                                               (4, 8, 100, [3, 9]), (2, 128, 256, [1, 26]), (2, 16, 33, [200, 1, 139]), (1, 48, 128, [300, 130, 2])])
def test_gla_scan(dtype, H, dim, vdim, q_lens):
    """From states that are not zero, portions beside single tokens, in one walk and in pieces; then the first
    request's tokens in smaller portions give the same rows and the same state as in one go."""
    o = ops()
    slots, cu, seqs, N = batch(q_lens)
    cols = 2 * H * (dim + vdim)
    u = rnd((N, cols), dtype, 1)
    decay = torch.sigmoid(rnd((N, H * dim), torch.float32, 2, 2.0) + 1.0)
    norm_w = 1.0 + rnd((vdim,), torch.float32, 3, 0.2)
    wide = rnd((9, H * dim * vdim + 7), torch.float32, 4, 0.5)
    got_state, want_state = wide.clone(), wide[:, : H * dim * vdim].clone()
    want = REF.gla_scan(u, decay, dim ** -0.5, norm_w, 1e-5, want_state, H, dim, vdim, slots, cu)
    got = o.gla_scan(u, decay, dim ** -0.5, norm_w, 1e-5, got_state[:, : H * dim * vdim], H, dim, vdim, slots, cu, max(q_lens))
    big = float(want.double().abs().max())
    assert (got.double() - want.double()).abs().max() < tol(dtype, max(1.0, big))
    assert (got_state[:, : H * dim * vdim] - want_state).abs().max() < 2e-4 * float(want_state.abs().max())
    assert torch.equal(got_state[:, H * dim * vdim :], wide[:, H * dim * vdim :])  # columns behind belong to somebody else
    n0, st, rows, at = q_lens[0], wide.clone(), [], 0
    for n in [2, 1, 3, 70, 1] + [5] * 60:
        n = min(n, n0 - at)
        if n <= 0:
            break
        part, args = slice(at, at + n), (ints([int(slots[0])]), ints([0, n]))
        rows.append(o.gla_scan(u[part].contiguous(), decay[part].contiguous(), dim ** -0.5, norm_w, 1e-5, st[:, : H * dim * vdim], H,
                               dim, vdim, args[0], args[1], n))
        at += n
    assert (torch.cat(rows).double() - got[:n0].double()).abs().max() < tol(dtype, max(1.0, big))
    assert (st[int(slots[0])] - got_state[int(slots[0])]).abs().max() < 2e-4 * float(want_state.abs().max())
    from litellmengine_amd.csrc import build

    assert build.load_library("gla").lle_gla_piece() == o.GLA_PIECE


def test_gla_channels_that_never_forget_and_that_forget_at_once():
    """A decay of one keeps the first token's write for three hundred tokens, a decay of nothing keeps only the
    newest; both in pieces."""
    o = ops()
    dim, vdim, N = 4, 8, 300
    u = torch.zeros((N, 2 * (dim + vdim))).cuda()
    u[:, 0], u[:, 1] = 1.0, 1.0  # q reads channels 0 and 1
    u[0, dim] = 1.0  # the first token writes channel 0, every token channel 1
    u[:, dim + 1] = 1.0
    u[:, 2 * dim : 2 * dim + vdim] = torch.arange(N).float().cuda()[:, None] * 0.01 + 1.0
    u[0, 2 * dim : 2 * dim + vdim] = torch.arange(vdim).float().cuda() * 10.0
    u[:, 2 * dim + vdim :] = 30.0  # gates wide open: silu(30) = 30
    decay = torch.zeros((N, dim)).cuda()
    decay[:, 0] = 1.0
    state = torch.zeros((2, dim * vdim)).cuda()
    got = o.gla_scan(u, decay, 1.0, torch.ones(vdim).cuda(), 1e-6, state, 1, dim, vdim, ints([1]), ints([0, N]), N)
    want = u[0, 2 * dim : 2 * dim + vdim] + u[-1, 2 * dim : 2 * dim + vdim]
    assert (state[1].view(dim, vdim)[:2].sum(0) - want).abs().max() < 1e-4
    want = want / (want * want).mean().sqrt() * 30.0
    assert (got[-1] - want).abs().max() < 1e-3
    assert float(state[0].abs().max()) == 0.0
