"""Pizunex on the GPU against the plain implementation (tests/plain_pizunex.py): each new mechanism's kernels alone, with
inputs made so that a window that is one token off, a cap in the wrong place, a wrong key head, a lost state or a decay on
the wrong token shows; then whole models of six small configurations in 32-bit and in bfloat16: whole prompts, portions,
token by token, unequal batches, slots and pages used again, long decoding, the first tokens, and greedy generation through
the pipeline; and configurations drawn from a seed."""
import pytest
import torch

import plain_pizunex as P
from pizunex_cases import CONFIGS, model_folder, plain_logits, plain_model, tokens_for
from helpers import assert_logits_close

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
DEV = "cuda:0"
F64 = torch.float64


@pytest.fixture(scope="module", autouse=True)
def need_gpu():
    if not torch.cuda.is_available():
        pytest.skip("no GPU")


def engine(name, dtype, max_tokens=1024, max_slots=None):
    from synaptix_amd import Engine
    return Engine.load(model_folder(name), dtype=dtype, max_tokens=max_tokens, max_slots=max_slots)


def dev(t, dtype=torch.float32):
    return t.to(device=DEV, dtype=dtype).contiguous()


def ints(xs):
    return torch.tensor(list(xs), dtype=torch.int32, device=DEV)


def randn(g, *shape):
    return torch.randn(*shape, generator=g, dtype=F64)


class Step:
    """The device arrays of a step over sequences (slot, tokens cached before, new tokens)."""

    def __init__(self, seqs):
        self.slots, self.past, self.new = zip(*seqs)
        starts = [0]
        for n in self.new:
            starts.append(starts[-1] + n)
        self.seq_start, self.seq_past, self.seq_slot = ints(starts), ints(self.past), ints(self.slots)
        self.tok_seq = ints(b for b, n in enumerate(self.new) for _ in range(n))
        self.tok_pos = ints(p + i for p, n in zip(self.past, self.new) for i in range(n))
        self.N = starts[-1]


def paged(rows_by_head, dtype, n_pages, order):
    """rows_by_head [T, heads, n] into pages [n_pages, heads, 64, n] at the pages `order` names."""
    T, Hh, n = rows_by_head.shape
    pages = torch.zeros((n_pages, Hh, 64, n), dtype=torch.float64)
    for t in range(T):
        pages[order[t // 64], :, t % 64] = rows_by_head[t]
    return pages.to(dtype)


# ----------------------------------------------------------------------------- the delta rule with one decay a head
def delta_inputs(g, T, H, K, D, E, log_rate=-4.0):
    """(fused rows [q | k | v], step and decay inputs, bias, log rates) with decays near one, and the cell's inputs."""
    qkv, ba = randn(g, T, 2 * K * D + H * E), randn(g, T, 2 * H)
    bias, a_log = randn(g, H), log_rate + 0.5 * randn(g, H)
    return qkv.float().double(), ba.float().double(), bias.float().double(), a_log.float().double()


def delta_want(qkv, ba, bias, a_log, H, K, D, E, state=None):
    T = qkv.shape[0]
    q, k, v = qkv[:, :K * D], qkv[:, K * D:2 * K * D], qkv[:, 2 * K * D:]
    q = (P.unit(q.reshape(T, K, D)) * D ** -0.5).repeat_interleave(H // K, 1)
    k = P.unit(k.reshape(T, K, D)).repeat_interleave(H // K, 1)
    beta = torch.sigmoid(ba[:, :H])
    decay = torch.exp(-torch.exp(a_log) * torch.nn.functional.softplus(ba[:, H:] + bias))
    return P.delta_cell(q, k, v.reshape(T, H, E), beta, decay, state)


@pytest.mark.parametrize("H,K,D,E", [(4, 2, 16, 24), (3, 3, 7, 5), (6, 1, 40, 70), (2, 2, 64, 33), (8, 4, 128, 16), (2, 1, 130, 18),
                                     (1, 1, 256, 12), (5, 5, 33, 64), (4, 1, 100, 40)])
def test_the_scan_in_portions_from_states_in_given_rows(H, K, D, E):
    """Three sequences of unequal lengths, in portions of 17, 1 and the rest (16 tokens a chunk: a chunk and one, one,
    several), one of them behind a state that is already there, in rows 4, 0 and 2 of six; rows of nobody stay as they are;
    then one token each from where the portions ended, token by token and through the chunks."""
    from synaptix_amd.kernels import ops
    g = torch.Generator().manual_seed(H + D)
    lens, rows = [70, 18, 41], [4, 0, 2]
    seqs = [delta_inputs(g, n + 3, H, K, D, E) for n in lens]
    bias, a_log = seqs[0][2], seqs[0][3]
    start = [None, None, 0.3 * randn(g, H, D, E)]
    want = [delta_want(s[0], s[1], bias, a_log, H, K, D, E, st) for s, st in zip(seqs, start)]
    state = torch.zeros(6, H, D, E, device=DEV)
    state[[1, 3, 5]] = 7.5
    state[2] = dev(start[2])
    got = [[] for _ in lens]

    def run(cuts, chunked):
        st = Step([(r, a, b - a) for r, (a, b) in zip(rows, cuts)])
        qkv = torch.cat([s[0][a:b] for s, (a, b) in zip(seqs, cuts)])
        ba = torch.cat([s[1][a:b] for s, (a, b) in zip(seqs, cuts)])
        pad = dev(torch.cat([ba, randn(g, ba.shape[0], 3)], 1))                 # (columns of longer rows)
        out = torch.empty((st.N, H * E), device=DEV)
        ops.head_delta_scan(dev(qkv), pad, pad[:, H:], dev(bias), dev(a_log), D ** -0.5, 1e-6, state, st.seq_start, st.seq_slot,
                            out, H, K, D, E, chunked=chunked)
        at = 0
        for i, (a, b) in enumerate(cuts):
            got[i].append(out[at:at + b - a].cpu().double())
            at += b - a

    run([(0, 17)] * 3, True)
    run([(17, 18)] * 3, True)
    run([(18, 70), (18, 19), (18, 41)], True)
    run([(70, 71), (19, 20), (41, 42)], False)
    run([(71, 72), (20, 21), (42, 43)], True)
    for i in range(3):
        o = torch.cat(got[i])
        w = want[i][0][:o.shape[0]].reshape(o.shape[0], H * E)
        assert float((o - w).abs().max()) < 2e-5 * max(1.0, float(w.abs().max())), f"sequence {i}"
    assert bool((state[[1, 3, 5]] == 7.5).all()), "rows of nobody"
    ends = [72, 21, 43]
    for i, n in enumerate(ends):
        _, S = delta_want(seqs[i][0][:n], seqs[i][1][:n], bias, a_log, H, K, D, E, start[i])
        assert float((state[rows[i]].cpu().double() - S).abs().max()) < 2e-5 * max(1.0, float(S.abs().max())), f"state of {i}"


@pytest.mark.parametrize("chunked", [True, False])
def test_a_token_far_back_still_counts(chunked):
    """A value written 150 tokens ago, read with its key by the last token: most of the result is that value (the plain cell
    says so first), through nine chunk borders and a portion's border."""
    from synaptix_amd.kernels import ops
    H, K, D, E, T = 2, 1, 32, 16, 151
    g = torch.Generator().manual_seed(4)
    qkv, ba, bias, a_log = delta_inputs(g, T, H, K, D, E, log_rate=-8.0)
    qkv[:, 31] = qkv[:, D + 31] = 0.0           # the last key value belongs to the far token alone
    qkv[0, D:2 * D] = 0.0
    qkv[0, D + 31] = 5.0
    qkv[T - 1, :D] = 0.0
    qkv[T - 1, 31] = 5.0
    ba[0, :H] = 8.0
    want, _ = delta_want(qkv, ba, bias, a_log, H, K, D, E)
    far = qkv[0, 2 * K * D:].view(H, E) * D ** -0.5
    assert float((want[-1] - far).abs().max()) < 0.2 * float(far.abs().max())
    state = torch.zeros(2, H, D, E, device=DEV)
    last = None
    cuts = [(0, 90), (90, T)] if chunked else [(t, t + 1) for t in range(T)]
    for a, b in cuts:
        st = Step([(0, a, b - a)])
        out = torch.empty((b - a, H * E), device=DEV)
        d = dev(ba[a:b])
        ops.head_delta_scan(dev(qkv[a:b]), d, d[:, H:], dev(bias), dev(a_log), D ** -0.5, 1e-6, state, st.seq_start, st.seq_slot,
                            out, H, K, D, E, chunked=chunked)
        last = out[-1].cpu().double().view(H, E)
    assert float((last - want[-1]).abs().max()) < 1e-6


def test_keys_that_repeat_and_decays_that_end_a_chunk():
    """Chunks whose keys are nearly one key and whose steps are nearly one (every token replaces what the one before wrote:
    the chunk's triangular system is far from the identity), with the sign turned at times, and decays down to zero in the
    middle of chunks."""
    from synaptix_amd.kernels import ops
    H, K, D, E, T = 4, 2, 48, 20, 100
    g = torch.Generator().manual_seed(9)
    qkv, ba, bias, a_log = delta_inputs(g, T, H, K, D, E)
    base = randn(g, 1, 2 * K * D)
    sign = torch.where(torch.rand(T, 1, generator=g, dtype=F64) < 0.3, -1.0, 1.0)
    qkv[:, :2 * K * D] = sign * base + 0.02 * qkv[:, :2 * K * D]
    ba[:, :H] = 5.0
    ba[37, H:] = ba[64, H:] = 3e4           # (the decay underflows to zero)
    qkv = qkv.float().double()
    want, S = delta_want(qkv, ba, bias, a_log, H, K, D, E)
    state = torch.zeros(1, H, D, E, device=DEV)
    st = Step([(0, 0, T)])
    out = torch.empty((T, H * E), device=DEV)
    d = dev(ba)
    ops.head_delta_scan(dev(qkv), d, d[:, H:], dev(bias), dev(a_log), D ** -0.5, 1e-6, state, st.seq_start, st.seq_slot, out, H, K,
                        D, E, chunked=True)
    assert float((out.cpu().double() - want.reshape(T, -1)).abs().max()) < 2e-5
    assert float((state[0].cpu().double() - S).abs().max()) < 2e-5 * max(1.0, float(S.abs().max()))


def test_many_sequences_in_one_step():
    """So many (sequence, head) pairs that a workgroup takes two groups of columns; sequences of 1 to 50 tokens in rows in
    another order than the step's; a negative slot takes the last row."""
    from synaptix_amd.kernels import ops
    H, K, D, E = 16, 8, 24, 40
    g = torch.Generator().manual_seed(2)
    lens = [1, 50, 16, 17, 33, 2, 15] * 5 + [32]
    B = len(lens)
    rows = torch.randperm(B, generator=g).tolist()
    seqs = [delta_inputs(g, n, H, K, D, E) for n in lens]
    bias, a_log = seqs[0][2], seqs[0][3]
    state = torch.zeros(B + 1, H, D, E, device=DEV)
    st = Step([(r, 0, n) for r, n in zip(rows, lens)])
    st.seq_slot[3] = -1
    ba = dev(torch.cat([s[1] for s in seqs]))
    out = torch.empty((st.N, H * E), device=DEV)
    ops.head_delta_scan(dev(torch.cat([s[0] for s in seqs])), ba, ba[:, H:], dev(bias), dev(a_log), D ** -0.5, 1e-6, state,
                        st.seq_start, st.seq_slot, out, H, K, D, E, chunked=True)
    at = 0
    for i, n in enumerate(lens):
        w, S = delta_want(seqs[i][0], seqs[i][1], bias, a_log, H, K, D, E)
        assert float((out[at:at + n].cpu().double() - w.reshape(n, -1)).abs().max()) < 2e-5, f"sequence {i} of {n} tokens"
        row = B if i == 3 else rows[i]
        assert float((state[row].cpu().double() - S).abs().max()) < 2e-5, f"state of sequence {i}"
        at += n
    assert float(state[rows[3]].abs().max()) == 0.0


def test_gate_as_silu_behind_the_heads_norm():
    from synaptix_amd.kernels import ops
    g = torch.Generator().manual_seed(5)
    N, H, E = 21, 3, 70
    o, gate, gain = randn(g, N, H, E), 2.0 * randn(g, N, H * E + 5), 1.0 + 0.3 * randn(g, E)
    want = P.over_rms(o, 1e-5) * gain * P.silu(gate[:, :H * E].reshape(N, H, E))
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 3e-2)):
        out = torch.empty((N, H * E), dtype=dtype, device=DEV)
        gd = dev(gate)
        ops.head_norm_gate(dev(o.reshape(N, H * E)), dev(gain.repeat(H)), 1e-5, gd, out, H, E, silu=True)
        assert float((out.cpu().double() - want.reshape(N, -1)).abs().max()) < tol * max(1.0, float(want.abs().max()) / 4)


# ----------------------------------------------------------------------------- attention
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh,nk,D,every,rot", [(4, 2, 16, 16, 0), (6, 6, 12, 1, 0), (3, 1, 10, 61, 4), (8, 4, 64, 7, 0), (40, 8, 96, 64, 0), (64, 4, 128, 30, 0)])
def test_intake_with_norms_over_all_heads_a_temperature_and_keys_as_values(nh, nk, D, every, rot, dtype):
    """Norms over the whole query and the whole key projection (heads of unlike sizes: a norm a head would show), values
    that are the keys before their norm, a temperature that steps between the tokens; pages over a border."""
    from synaptix_amd.kernels import ops
    from synaptix_amd.parts import RotaryInterleaved
    g = torch.Generator().manual_seed(nh + D)
    st = Step([(0, 60, 10), (1, 0, 3)])
    width = (nh + nk) * D
    rows = randn(g, st.N, width + 4)
    rows[:, :D] *= 5.0                                    # the first query head and the last key head are large
    rows[:, width - D:width] *= 3.0
    qg, kg = 1.0 + 0.3 * randn(g, nh * D), 1.0 + 0.3 * randn(g, nk * D)
    q, k = P.rms_norm(rows[:, :nh * D], qg, 1e-5), P.rms_norm(rows[:, nh * D:width], kg, 1e-5)
    f = P.rates(300.0, rot)[0] if rot else torch.zeros(0, dtype=F64)
    turn = lambda x, n: torch.cat([P.rotate_pairs(x.reshape(st.N, n, D)[:10], f, first=60), P.rotate_pairs(x.reshape(st.N, n, D)[10:], f)])
    temp = P.temperature(70, 0.7, every)
    pos = [60 + i for i in range(10)] + [0, 1, 2]
    q, k = turn(q, nh) * temp[pos][:, None, None], turn(k, nk)
    v = rows[:, nh * D:width].reshape(st.N, nk, D)
    qo = torch.empty((st.N, nh * D), dtype=dtype, device=DEV)
    kp = torch.zeros((4, nk, 64, D), dtype=dtype, device=DEV)
    vp = torch.zeros((4, nk, D, 64), dtype=dtype, device=DEV)
    table = ints([2, 0, 1, 3]).view(2, 2)
    how = dict(rotation=RotaryInterleaved(300.0, rot, 128).tables(DEV), pairs=True, q_temp=(0.7, every))
    ops.window_intake(dev(rows), None, qo, kp, vp, table, st.tok_seq, st.tok_pos, dev(qg), dev(kg), 1e-5, nh, nk, D, D,
                      norm_whole=True, values_are_keys=True, **how)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    for got, want, what in [(qo.view(st.N, nh, D), q, "queries")]:
        assert float((got.cpu().double() - want).abs().max()) < tol * max(1.0, float(want.abs().max())), what
    for n, (page, slot) in enumerate([(2, 60), (2, 61), (2, 62), (2, 63)] + [(0, i) for i in range(6)] + [(1, 0), (1, 1), (1, 2)]):
        assert float((kp[page, :, slot].cpu().double() - k[n]).abs().max()) < tol * max(1.0, float(k.abs().max())), f"key of token {n}"
        assert float((vp[page, :, :, slot].cpu().double() - v[n]).abs().max()) < tol * max(1.0, float(v.abs().max())), f"value of token {n}"
    # norms a head (one gain for all) with the same temperature and values: the other kernel
    one_q, one_k = qg[:D], kg[:D]
    q1 = turn(P.rms_norm(rows[:, :nh * D].reshape(st.N, nh, D), one_q, 1e-5), nh) * temp[pos][:, None, None]
    ops.window_intake(dev(rows), None, qo, kp, vp, table, st.tok_seq, st.tok_pos, dev(one_q), dev(one_k), 1e-5, nh, nk, D, D,
                      values_are_keys=True, **how)
    assert float((qo.view(st.N, nh, D).cpu().double() - q1).abs().max()) < tol * max(1.0, float(q1.abs().max()))
    assert float((vp[1, :, :, 2].cpu().double() - v[12]).abs().max()) < tol * max(1.0, float(v.abs().max()))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("window", [1, 2, 37, 63, 64, 65, 130, None])
@pytest.mark.parametrize("cap", [6.0, None])
def test_cap_distance_bias_and_every_edge_of_a_window(window, cap, dtype):
    """Keys are one-hot in their position (modulo the key size) and queries are long, so that a query gives nearly all its
    weight to the visible keys of one residue, the nearest of them first (the bias): a window that is one token off, a cap
    behind the bias instead of before it, or a slope of the wrong head changes the result by its own size.  All queries at
    once (prompts: in bf16 the tiles on the matrix cores), a second piece that starts inside a page, and single queries at
    the borders of pages and windows, over pages in a shuffled order."""
    from synaptix_amd.kernels import ops
    H, G, D, T = 4, 2, 16, 200
    g = torch.Generator().manual_seed(3)
    k = torch.zeros(T, G, D, dtype=F64)
    q = torch.zeros(T, H, D, dtype=F64)
    for t in range(T):
        for gg in range(G):
            k[t, gg, (t + gg) % D] = 1.0
        for h in range(H):
            q[t, h, (t - 1 - 3 * h) % D] = 9.0           # head h looks 1 + 3 h back (and at what shares that residue)
    q = q + 0.1 * randn(g, T, H, D)
    v = randn(g, T, G, D)
    q, k, v = [x.to(dtype).double() for x in (q, k, v)]
    slopes = P.linear_slopes(H)
    want = P.attend(q, k, v, 1.0, P.window_mask(T, window), cap, slopes).reshape(T, H * D)
    order = [3, 0, 2, 1]
    kp, vp = paged(k, dtype, 5, order).to(DEV), paged(v, dtype, 5, order).transpose(2, 3).contiguous().to(DEV)
    qd, table = dev(q.reshape(T, H * D), dtype), ints(order).view(1, 4)
    how = dict(window=window or 0, slopes=dev(slopes), softcap=cap or 0.0)
    tol = 2e-4 if dtype == torch.float32 else 4e-2

    def run(first, n, tiles=False):
        st = Step([(0, first, n)])
        out = torch.empty((n, H * D), dtype=dtype, device=DEV)
        if tiles:
            ops.window_attention_prefill_bf16(qd[first:first + n], kp, vp, table, st.seq_start, st.seq_past, out, 1.0, H, G, D, D, **how)
        else:
            ops.window_attention(qd[first:first + n], kp, vp, table, st.tok_seq, st.tok_pos, out, 1.0, H, G, D, D, **how)
        return float((out.cpu().double() - want[first:first + n]).abs().max())

    assert run(0, T) < tol, "every query, one wave a (token, head)"
    if dtype == torch.bfloat16:
        assert run(0, T, tiles=True) < tol, "every query, tiles on the matrix cores"
        assert run(70, T - 70, tiles=True) < tol, "a second piece that starts inside a page, in tiles"
        assert run(0, 3, tiles=True) < tol, "the first three tokens, in tiles"
    assert run(70, T - 70) < tol, "a second piece that starts inside a page"
    for t in sorted({T - 1, 130, 129, 128, 65, 64, 63, 37, 36, 2, 1, 0}):
        assert run(t, 1) < tol, f"the single query at {t}"
    # the bias and the cap are not nothing, nor is their order
    assert float((P.attend(q, k, v, 1.0, P.window_mask(T, window), cap).reshape(T, -1) - want).abs().max()) > 0.1 or window in (1, 2)
    if cap is not None and window not in (1, 2):
        assert float((P.attend(q, k, v, 1.0, P.window_mask(T, window), None, slopes).reshape(T, -1) - want).abs().max()) > 0.1


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_one_far_key_among_hundreds(dtype):
    """One query and one key are scaled so that this key's score stands out among 700 in spite of the bias: the result is
    that key's value where the query's window holds it and another where it does not: the first key that a window still
    holds and the one that it has just lost, in a prompt and alone."""
    from synaptix_amd.kernels import ops
    H, G, D, T = 2, 1, 32, 700
    g = torch.Generator().manual_seed(5)
    q, k, v = 0.3 * randn(g, T, H, D), 0.3 * randn(g, T, G, D), randn(g, T, G, D)
    order = list(range(11))
    slopes = torch.tensor([2.0 ** -6, 2.0 ** -9], dtype=F64)
    for far, at, window, cap, seen in [(3, 699, None, None, True), (100, 699, 600, 40.0, True), (99, 699, 600, 40.0, False),
                                       (636, 699, 64, 40.0, True), (635, 699, 64, 40.0, False), (640, 640, 1, 40.0, True),
                                       (63, 127, 65, None, True), (62, 127, 65, None, False)]:
        qq, kk = q.clone(), k.clone()
        kk[far] = 0.0
        kk[far, 0, 5] = 6.0
        qq[at, :, 5] = 8.0
        qq, kk, vv = [x.to(dtype).double() for x in (qq, kk, v)]
        want = P.attend(qq, kk, vv, 1.0, P.window_mask(T, window), cap, slopes)[at].reshape(1, H * D)
        near = float((want.view(H, D) - vv[far, 0]).abs().max())
        assert (near < 1e-2) == seen, (far, at, window, near)
        kp, vp = paged(kk, dtype, 11, order).to(DEV), paged(vv, dtype, 11, order).transpose(2, 3).contiguous().to(DEV)
        how = dict(window=window or 0, softcap=cap or 0.0, slopes=dev(slopes))
        tol = 2e-4 if dtype == torch.float32 else 4e-2
        qd = dev(qq[:at + 1].reshape(at + 1, H * D), dtype)
        for first, what in ((at, "alone"), (0, "in a prompt")):
            st = Step([(0, first, at + 1 - first)])
            out = torch.empty((at + 1 - first, H * D), dtype=dtype, device=DEV)
            ops.window_attention(qd[first:], kp, vp, ints(order).view(1, 11), st.tok_seq, st.tok_pos, out, 1.0, H, G, D, D, **how)
            assert float((out[-1:].cpu().double() - want).abs().max()) < tol, (what, far, at, window)
        if dtype == torch.bfloat16:
            out = torch.empty((at + 1, H * D), dtype=dtype, device=DEV)
            ops.window_attention_prefill_bf16(qd, kp, vp, ints(order).view(1, 11), st.seq_start, st.seq_past, out, 1.0, H, G, D, D, **how)
            assert float((out[-1:].cpu().double() - want).abs().max()) < tol, ("prompt in tiles", far, at, window)


# ----------------------------------------------------------------------------- latent attention, the norm of columns
def test_norm_of_the_first_columns_of_longer_rows():
    from synaptix_amd.kernels import ops
    g = torch.Generator().manual_seed(6)
    for N, D in ((1, 24), (9, 130), (300, 96), (8, 257), (5, 1536), (3, 2048), (2, 2100)):
        x, gain = randn(g, N, D + 11), 1.0 + 0.3 * randn(g, D)
        want = P.rms_norm(x[:, :D], gain, 1e-5)
        xd = dev(x)
        for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2e-2)):
            out = torch.empty((N, D), dtype=dtype, device=DEV)
            ops.rmsnorm_rows(xd[:, :D], dev(gain), 1e-5, out)
            assert float((out.cpu().double() - want).abs().max()) < tol * float(want.abs().max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_latent_intake_from_two_products_equals_one(dtype):
    """The queries in rows of their own and the latent in columns of other rows: the same pages and queries as from one
    fused row, with a stretched rotation whose factor acts on both."""
    from synaptix_amd.kernels import ops
    from synaptix_amd.parts import RotaryScaledInterleaved
    H, D, R, C = 3, 10, 6, 16
    g = torch.Generator().manual_seed(7)
    st = Step([(0, 61, 6), (1, 0, 2)])
    nq = H * (D + R)
    rows, gain = randn(g, st.N, nq + C + R), 1.0 + 0.3 * randn(g, C)
    pos = RotaryScaledInterleaved(300.0, R, 128, factor=4.0, original=64, fast=8.0, slow=1.0)
    cos, sin = pos.tables(DEV)
    table = ints([2, 0, 1, 3]).view(2, 2)
    got = []
    for split in (False, True):
        qn = torch.zeros((st.N, H * D), dtype=dtype, device=DEV)
        qf = torch.zeros((st.N, H * (C + R)), dtype=dtype, device=DEV)
        kp = torch.zeros((4, 1, 64, C + R), dtype=dtype, device=DEV)
        vp = torch.zeros((4, 1, C, 64), dtype=dtype, device=DEV)
        down = dev(torch.cat([randn(g, st.N, 5), rows[:, nq:]], 1))[:, 5:] if split else None
        ops.latent_intake(dev(rows[:, :nq]) if split else dev(rows), dev(gain), 1e-5, cos, sin, qn, qf, kp, vp, table, st.tok_seq,
                          st.tok_pos, H, D, R, C, 66, down=down)
        got.append((qn, qf, kp, vp))
    for a, b in zip(*got):
        assert torch.equal(a, b)
    f, mult = P.rates(300.0, R, {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0})
    turned = torch.cat([P.rotate_pairs(rows[:6, nq + C:], f, mult, first=61), P.rotate_pairs(rows[6:, nq + C:], f, mult)])
    tol = 1e-4 if dtype == torch.float32 else 3e-2
    k = got[0][2]
    for n, (page, slot) in enumerate([(2, 61), (2, 62), (2, 63), (0, 0), (0, 1), (0, 2), (1, 0), (1, 1)]):
        assert float((k[page, 0, slot, C:].cpu().double() - turned[n]).abs().max()) < tol


# ----------------------------------------------------------------------------- the squared relu as an epilogue
@pytest.mark.parametrize("M", [1, 3, 8, 9, 16, 20, 40, 64, 65, 130, 300, 600, 1100])
@pytest.mark.parametrize("N,K,keep_rows", [(256, 128, False), (48, 64, False), (48, 64, True), (40, 72, True), (33, 20, True), (512, 256, False)])
def test_squared_relu_inside_every_product(M, N, K, keep_rows):
    from synaptix_amd.kernels import ops
    from synaptix_amd.parts import Matrix, linear
    g = torch.Generator().manual_seed(M + N)
    x, w = randn(g, M, K).to(torch.bfloat16).double(), (0.2 * randn(g, N, K)).to(torch.bfloat16).double()
    want = torch.relu(x @ w.T).pow(2)
    assert float((want == 0).double().mean()) > 0.3
    scale = float(want.abs().max())
    m = Matrix(dev(w, torch.bfloat16), keep_rows=keep_rows)
    for out_dtype, tol in ((torch.bfloat16, 1e-2), (torch.float32, 1e-5)):
        got = linear(dev(x, torch.bfloat16), m, out_dtype, point="relu_squared")
        assert got.dtype == out_dtype and float((got.cpu().double() - want).abs().max()) < tol * scale, (M, N, K, out_dtype)
    got = linear(dev(x), Matrix(dev(w), keep_rows=True), torch.float32, point="relu_squared")
    assert float((got.cpu().double() - want).abs().max()) < 1e-5 * scale
    if M <= 16 and m.packed is not None:       # behind a norm's unfinished rows: the row's factor first, then the square
        ss = torch.rand(M, 4, generator=torch.Generator().manual_seed(M)) + 0.5
        inv = torch.rsqrt(ss.double().sum(1) / K + 1e-5)[:, None]
        out = torch.empty((M, N), dtype=torch.float32, device=DEV)
        ops.gemm_packed(dev(x, torch.bfloat16), m.packed, out, row_scale=(dev(ss), K, 1e-5), point="relu_squared")
        want2 = torch.relu((x @ w.T) * inv).pow(2)
        assert float((out.cpu().double() - want2).abs().max()) < 1e-4 * float(want2.abs().max())


def test_an_activation_over_partial_sums_is_refused():
    from synaptix_amd.kernels import ops
    x, w = torch.zeros(4, 2048, dtype=torch.bfloat16, device=DEV), torch.zeros(64, 2048, dtype=torch.bfloat16, device=DEV)
    out = torch.empty(2, 4, 64, device=DEV)
    with pytest.raises(ops.KernelError):
        ops.gemm(x, w, out, point="relu_squared")
    with pytest.raises(ops.KernelError):
        ops.gemm_packed(x, ops.pack_weight(w), out, point="relu_squared")
    with pytest.raises(ops.KernelError):
        ops.gemm(x, w, out[0], point="cube")


# ----------------------------------------------------------------------------- whole models

NAMES = ["P", "Q", "R", "S", "T", "U"]


def lengths(name):
    return {"P": [1, 2, 21, 64, 65, 150], "Q": [3, 70, 71, 129, 140], "R": [5, 64, 66, 200], "S": [1, 2, 3, 66, 90],
            "T": [2, 17, 100, 130], "U": [1, 33, 71, 140]}[name]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts(name, dtype):
    eng = engine(name, dtype)
    for i, n in enumerate(lengths(name)):
        toks = tokens_for(name, n, 100 + i)
        s = eng.acquire()
        got = eng.step([(s, toks)], want="all")
        assert_logits_close(got, plain_logits(name, toks), dtype, f"{name} {dtype} {n} tokens whole", sharp=True)
        eng.release(s)
    eng.cache.check()


@pytest.mark.parametrize("name", NAMES)
def test_the_residual_after_every_layer_in_float32(name):
    """The model's layer runs one after another (a block that runs twice counts twice): the residual rows that each leaves,
    read from the engine's own pass."""
    from synaptix_amd.parts import as_delta
    toks = tokens_for(name, 70, 3)
    want = plain_model(name).residuals(toks)
    eng = engine(name, "float32")
    got = []
    for block in eng.model.blocks:
        inner = block.forward

        def spy(resid, pending, ctx, cache, owner=True, inner=inner):
            out = inner(resid, pending, ctx, cache, owner)
            delta = as_delta(out)
            got.append(resid.clone() + (delta.sum(0) if delta.dim() == 3 else delta))      # (partial sums not yet added)
            return out
        block.forward = spy
    eng.step([(eng.acquire(), toks)], want="last")
    assert len(got) == len(want)
    for i, (a, b) in enumerate(zip(got, want)):
        assert float((a.cpu().double() - b).abs().max()) < 1e-4 * max(1.0, float(b.abs().max())), f"after layer {i}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_portions_of_several_sizes(name, dtype):
    """A prompt in portions of 2, 1, 3, 17, 64 and 2 tokens and the rest: every portion starts from the pages, the states
    and the convolutions' inputs that the earlier ones left (inside a page, inside a chunk of the scan, at a page's border,
    inside and beyond the first window)."""
    toks = tokens_for(name, 230, 7)
    want = plain_logits(name, toks)
    eng = engine(name, dtype)
    s, at, got = eng.acquire(), 0, []
    for n in [2, 1, 3, 17, 64, 2, 41, 100]:
        got.append(eng.step([(s, toks[at:at + n])], want="all"))
        at += n
    assert at == len(toks)
    assert_logits_close(torch.cat(got), want, dtype, f"{name} {dtype} in portions", sharp=True)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,head,n", [("P", 30, 130), ("Q", 1, 160), ("R", 50, 160), ("S", 3, 90), ("T", 35, 100), ("U", 60, 150)])
def test_prompt_then_token_by_token(name, head, n, dtype):
    """Decoding long enough that every window passes over decoded tokens and over a page's border."""
    toks = tokens_for(name, n, 21)
    want = plain_logits(name, toks)
    eng = engine(name, dtype)
    s = eng.acquire()
    got = [eng.step([(s, toks[:head])], want="all")]
    for t in toks[head:]:
        got.append(eng.step([(s, [t])], want="last"))
    assert_logits_close(torch.cat(got), want, dtype, f"{name} {dtype} token by token", sharp=True)
    eng.release(s)
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_unequal_batches_and_slots_used_again(name, dtype):
    """Requests of unequal lengths start together and are decoded together, the shorter ones ending earlier; then other
    requests take the slots, state rows and pages that came free (the cache has room for little more than one batch), in
    another order: each request's logits equal the plain model's for that request alone."""
    reqs = {f"r{i}": tokens_for(name, n + 9, 300 + i) for i, n in enumerate(lengths(name))}
    ids = list(reqs)
    eng = engine(name, dtype, max_tokens=64 * 9, max_slots=3)
    for batch in (ids[:3], (ids[3:] + ids[:1])[:3], list(reversed(ids))[:3]):
        slots = {r: eng.acquire() for r in batch}
        head = {r: max(1, len(reqs[r]) - 9 - 3 * i) for i, r in enumerate(batch)}
        got = {r: [] for r in batch}
        out = eng.step([(slots[r], reqs[r][:head[r]]) for r in batch], want="all")
        at = 0
        for r in batch:
            got[r].append(out[at:at + head[r]])
            at += head[r]
        fed, live = dict(head), list(batch)
        while live:
            out = eng.step([(slots[r], [reqs[r][fed[r]]]) for r in live], want="last")
            for i, r in enumerate(live):
                got[r].append(out[i:i + 1])
                fed[r] += 1
            for r in [r for r in live if fed[r] == len(reqs[r])]:
                eng.release(slots[r])
                live.remove(r)
        for r in batch:
            assert_logits_close(torch.cat(got[r]), plain_logits(name, reqs[r]), dtype, f"{name} {dtype} {r} in a batch",
                                sharp=True)
        eng.cache.check()
    assert eng.cache.free_slots == 3


@pytest.mark.parametrize("dtype", DTYPES)
def test_prompts_and_single_tokens_in_one_step(dtype):
    """A step that brings a prompt's portion to one sequence and one token each to two others, as the scheduler mixes them."""
    for name in ("P", "R"):
        reqs = [tokens_for(name, n, 40 + n) for n in (90, 60, 75)]
        want = [plain_logits(name, r) for r in reqs]
        eng = engine(name, dtype)
        slots = [eng.acquire() for _ in reqs]
        eng.step([(slots[0], reqs[0][:50]), (slots[1], reqs[1][:57])], want=None)
        out = eng.step([(slots[0], reqs[0][50:51]), (slots[2], reqs[2][:33]), (slots[1], reqs[1][57:58])], want="all")
        assert_logits_close(out[:1], want[0][50:51], dtype, f"{name} single beside a prompt", sharp=True)
        assert_logits_close(out[1:34], want[2][:33], dtype, f"{name} prompt beside singles", sharp=True)
        assert_logits_close(out[34:], want[1][57:58], dtype, f"{name} second single", sharp=True)
        out = eng.step([(slots[2], reqs[2][33:75]), (slots[0], reqs[0][51:90])], want="last")
        assert_logits_close(out, torch.stack([want[2][74], want[0][89]]), dtype, f"{name} both went on", sharp=True)


@pytest.mark.parametrize("seed", list(range(8000, 8020)))
def test_configurations_drawn_from_a_seed(seed):
    """Layer kinds, orders, head counts, sizes, windows, caps, temperatures, rotations and shared tensors drawn from a seed
    (the cases above are chosen; these are not): a prompt whole, then requests of unequal lengths cut at unequal places and
    decoded together, 3 to 20 of them, against the plain model for each alone; every fourth one also in bfloat16."""
    import random
    from pizunex_cases import random_model
    from synaptix_amd import Engine
    cfg, folder, plain = random_model(seed)
    rng = random.Random(seed + 1)
    g = torch.Generator().manual_seed(seed)
    T = rng.choice([70, 150, 250])
    lens = [T, 9, T // 2] + [rng.randint(2, T) for _ in range(rng.choice([0, 3, 6, 17]))]
    toks = [torch.randint(0, cfg.vocab, (n,), generator=g).tolist() for n in lens]
    want = [plain.logits(t) for t in toks]
    for dtype in DTYPES if seed % 4 == 0 else DTYPES[:1]:
        eng = Engine.load(folder, dtype=dtype, max_tokens=8192, max_slots=32)
        s = eng.acquire()
        assert_logits_close(eng.step([(s, toks[0])], want="all"), want[0], dtype, f"seed {seed} whole", sharp=True)
        eng.release(s)
        slots = [eng.acquire() for _ in toks]
        cut = [min(max(1, len(t) - 12 - 3 * (i % 5)), len(t)) for i, t in enumerate(toks)]
        out = eng.step([(s, t[:k]) for s, t, k in zip(slots, toks, cut)], want="all")
        got, at = [[] for _ in toks], 0
        for i, k in enumerate(cut):
            got[i].append(out[at:at + k])
            at += k
        fed, live = list(cut), [i for i in range(len(toks)) if cut[i] < len(toks[i])]
        while live:
            out = eng.step([(slots[i], [toks[i][fed[i]]]) for i in live], want="last")
            for j, i in enumerate(live):
                got[i].append(out[j:j + 1])
                fed[i] += 1
            live = [i for i in live if fed[i] < len(toks[i])]
        for i in range(len(toks)):
            assert_logits_close(torch.cat(got[i]), want[i], dtype, f"seed {seed} {dtype} request {i} of {len(toks)}", sharp=True)
        eng.cache.check()


def test_windows_give_their_pages_back():
    """A long sequence in a cache that holds far fewer tokens than it has (the configuration has windows and states only)."""
    toks = tokens_for("U", 500, 12)
    want = plain_logits("U", toks)
    eng = engine("U", "float32", max_tokens=64 * 5, max_slots=1)
    s = eng.acquire()
    got = [eng.step([(s, toks[:40])], want="all")]
    for at in range(40, 460, 60):
        got.append(eng.step([(s, toks[at:at + 60])], want="all"))
    for t in toks[460:]:
        got.append(eng.step([(s, [t])], want="last"))
    assert_logits_close(torch.cat(got), want, "float32", "500 tokens through 5 pages", sharp=True)
    eng.release(s)
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_first_tokens(dtype):
    """Sequences of one and two tokens, and every position up to the windows and a little more, one by one."""
    for name in ("P", "S", "T"):
        if name == "S" and dtype != "float32":
            # (a first token's read-out is its value times k . q, brought to one size by the norm behind it: with keys of six
            # values k . q may be next to nothing, and the rounding of the norms' outputs alone then moves the logits by a third)
            continue
        eng = engine(name, dtype)
        toks = tokens_for(name, 45, 77)
        want = plain_logits(name, toks)
        for n in (1, 2):
            s = eng.acquire()
            assert_logits_close(eng.step([(s, toks[:n])], want="all"), plain_logits(name, toks[:n]), dtype,
                                f"{name} {dtype} first {n}", sharp=True)
            eng.release(s)
        s = eng.acquire()
        got = [eng.step([(s, [t])], want="last") for t in toks]
        assert_logits_close(torch.cat(got), want, dtype, f"{name} {dtype} from the first token one by one", sharp=True)


def test_long_decoding_in_float32():
    """400 tokens one by one: the window passes many times, the temperature climbs, the states are carried throughout."""
    toks = tokens_for("P", 400, 5)
    want = plain_logits("P", toks)
    eng = engine("P", "float32", max_tokens=512, max_slots=1)
    s = eng.acquire()
    got = [eng.step([(s, toks[:2])], want="all")]
    for t in toks[2:]:
        got.append(eng.step([(s, [t])], want="last"))
    assert_logits_close(torch.cat(got), want, "float32", "400 tokens one by one", sharp=True)


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_pipeline(dtype):
    """Pipeline.generate_batch (the scheduler, slots, captured decode steps, the sampler) against greedy decoding with the
    plain model; in bfloat16 a token may differ where the two best logits are close, then the plain model's logits for the
    generated sequence must say so."""
    import synaptix_amd
    name = "R"
    pipe = synaptix_amd.load(model_folder(name), dtype="f32" if dtype == "float32" else "bf16", max_seq=512)
    prompts = [tokens_for(name, n, 900 + n) for n in (3, 70, 20)]
    outs, stats = pipe.generate_batch(prompts, synaptix_amd.GenerationConfig(max_new_tokens=12, temperature=0.0))
    assert stats.new_tokens == 36
    for prompt, out in zip(prompts, outs):
        assert len(out.tokens) == 12 and out.finish_reason == "length"
        logits = plain_logits(name, prompt + out.tokens)
        for i, tok in enumerate(out.tokens):
            row = logits[len(prompt) - 1 + i]
            best = int(row.argmax())
            if dtype == "float32":
                assert tok == best or float(row[best] - row[tok]) < 1e-4
            else:
                assert tok == best or float(row[best] - row[tok]) < 0.05 * float(row.abs().max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["P", "R", "T"])
def test_decode_steps_replayed_from_a_graph(name, dtype):
    """Captured decode steps (three rows wide in a graph of four: one row is padding) with eager work of another sequence
    between the replays; every replay against the plain model."""
    eng = engine(name, dtype, max_tokens=64 * 12)
    assert eng.graph_ok
    reqs = [tokens_for(name, n, 60 + n) for n in (90, 20, 140)]
    other = tokens_for(name, 60, 4)
    want = [plain_logits(name, r) for r in reqs]
    heads = [len(r) - 12 for r in reqs]
    slots = [eng.acquire() for _ in reqs]
    eng.step([(s, r[:h]) for s, r, h in zip(slots, reqs, heads)], want=None)
    runner = eng.decode_runner(3, 256)
    assert runner.rows == 4
    extra = eng.acquire()
    for i in range(12):
        _, lg = runner.step(slots, [r[h + i] for r, h in zip(reqs, heads)])
        for j in range(3):
            assert_logits_close(lg[j:j + 1].clone(), want[j][heads[j] + i:heads[j] + i + 1], dtype,
                                f"{name} {dtype} replay {i} row {j}", sharp=True)
        got = eng.step([(extra, other[5 * i:5 * i + 5])], want="last")        # an eager prompt portion in between
        assert_logits_close(got, plain_logits(name, other)[5 * i + 4:5 * i + 5], dtype, f"{name} {dtype} eager between replays",
                            sharp=True)
    eng.cache.check()


def test_short_prompt_steps_replayed_from_a_graph():
    """bfloat16 prompt steps of a few tokens go through captured graphs with padding rows (an extra sequence on the spare
    page and state row); portions of a prompt one after another, each from what the last one left."""
    name = "R"
    eng = engine(name, "bfloat16")
    assert eng.graph_ok and eng.prompt_graphs
    toks = tokens_for(name, 120, 8)
    want = plain_logits(name, toks)
    s, at = eng.acquire(), 0
    for n in (10, 10, 30, 10, 40, 20):
        got = eng.step([(s, toks[at:at + n])], want="last")
        at += n
        assert_logits_close(got, want[at - 1:at], "bfloat16", f"prompt portion ending at {at} through a graph", sharp=True)
    assert any(k[0] == "prompt" for k in eng._runners), "no prompt step was replayed from a graph"


def test_command_line_and_trace_replay_as_a_user_starts_them(tmp_path):
    """`random` writes a model folder from a configuration file, `run` generates from it, and bin/trace_run replays steps
    over it (prompts of unequal lengths together, then single tokens, a request that ends early, its slot used again by a
    later request) in both types; the logits against the plain model."""
    import json
    import os
    import subprocess
    import sys
    from helpers import ROOT, run_trace

    cfg_file = tmp_path / "config.json"
    cfg_file.write_text(json.dumps(CONFIGS["P"]))
    folder = str(tmp_path / "model")
    env = dict(os.environ, PYTHONPATH=ROOT)
    subprocess.run([sys.executable, "-m", "synaptix_amd", "random", str(cfg_file), folder, "--seed", "3"], check=True,
                   env=env, cwd=ROOT, timeout=300)
    plain = P.PlainPizunex.from_folder(folder)
    prompt = tokens_for("P", 9, 1)
    run = subprocess.run([sys.executable, "-m", "synaptix_amd", "run", folder, "--prompt-ids", ",".join(map(str, prompt)),
                          "--max-tokens", "4", "--temperature", "0", "--compute-dtype", "f32"], check=True, env=env, cwd=ROOT,
                         timeout=300, capture_output=True, text=True)
    assert run.stdout.strip() or run.stderr.strip()
    a, b, c = tokens_for("P", 70, 2), tokens_for("P", 5, 3), tokens_for("P", 30, 4)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:66], "want": [0, 65]}, {"id": "b", "tokens": b[:3], "want": [2]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[66:67], "want": [0]}, {"id": "b", "tokens": b[3:4], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[67:68], "want": []}, {"id": "b", "tokens": b[4:5], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[68:69], "want": [0]}], "end": []},
             {"step": 4, "entries": [{"id": "c", "tokens": c, "want": [0, 29]}], "end": ["c"]},
             {"step": 5, "entries": [{"id": "a", "tokens": a[69:70], "want": [0]}], "end": ["a"]}]
    la, lb, lc = plain.logits(a), plain.logits(b), plain.logits(c)
    want = {0: torch.stack([la[0], la[65], lb[2]]), 1: torch.stack([la[66], lb[3]]), 2: lb[4:5], 3: la[68:69],
            4: torch.stack([lc[0], lc[29]]), 5: la[69:70]}
    for dtype in DTYPES:
        out = run_trace(folder, dtype, steps, 256, str(tmp_path / f"out_{dtype}"))
        assert sorted(out) == sorted(want)
        for k, w in want.items():
            assert_logits_close(out[k], w, dtype, f"trace step {k} in {dtype}", sharp=True)
