"""Sunosun on the GPU against the plain implementation (tests/plain_sunosun.py): each new mechanism's kernels alone, with
inputs made so that a lost state, a decay on the wrong token or channel, a missing sink, a wrong group or an addition in the
wrong pass shows; then whole models of six small configurations in 32-bit and in bfloat16: whole prompts, portions, token by
token, unequal batches, slots and pages used again, long decoding, the first tokens, and greedy generation through the
pipeline; and configurations drawn from a seed."""
import math

import pytest
import torch

import plain_sunosun as P
from sunosun_cases import CONFIGS, model_folder, plain_logits, plain_model, tokens_for
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


# ----------------------------------------------------------------------------- gated linear attention
def gla_inputs(g, T, H, D, E, rank, z_mean=4.0, z_std=1.0):
    """(projection rows [q | k | v | gate | middle] with columns beside them, a2, bias): decays near one by default."""
    rows = randn(g, T, 2 * H * D + 2 * H * E + rank + 3).float().double()
    a2 = (z_std * rank ** -0.5 * randn(g, H * D, rank)).float().double()
    return rows, a2, (z_mean + 0.5 * randn(g, H * D)).float().double()


def gla_columns(rows, H, D, E, rank):
    at, out = 0, []
    for n in (H * D, H * D, H * E, H * E, rank):
        out.append(rows[:, at:at + n])
        at += n
    return out


def gla_want(rows, a2, bias, H, D, E, tau, state=None):
    T, rank = rows.shape[0], a2.shape[1]
    q, k, v, _, mid = gla_columns(rows, H, D, E, rank)
    alpha = P.decays(mid @ a2.T + bias, tau).view(T, H, D)
    o, S = P.gla_cell(q.reshape(T, H, D) * D ** -0.5, k.reshape(T, H, D), v.reshape(T, H, E), alpha, state)
    return o.reshape(T, H * E), S


def gla_scan(rows, a2, bias, tau, state, st, H, D, E):
    from synaptix_amd.kernels import ops
    q, k, v, _, mid = gla_columns(rows, H, D, E, a2.shape[1])
    out = torch.empty((st.N, H * E), device=DEV)
    ops.gated_linear_scan(q, k, v, mid, dev(a2.T), dev(bias), D ** -0.5, tau, state, st.seq_start, st.seq_slot, out, H, D, E)
    return out


def gla_step(rows, a2, bias, tau, state, st, H, D, E, gain, eps, out):
    from synaptix_amd.kernels import ops
    q, k, v, gate, mid = gla_columns(rows, H, D, E, a2.shape[1])
    ops.gated_linear_step(q, k, v, mid, dev(a2.T), dev(bias), D ** -0.5, tau, state, st.seq_start, st.seq_slot, dev(gain), eps,
                          gate, out, H, D, E)


@pytest.mark.parametrize("H,D,E,rank", [(4, 16, 24, 4), (3, 7, 5, 1), (2, 64, 33, 16), (8, 128, 16, 20), (2, 130, 18, 70), (1, 256, 12, 130),
                                        (5, 33, 64, 3), (4, 100, 40, 16), (1, 1, 1, 2), (2, 20, 512, 8), (2, 48, 510, 8), (3, 12, 300, 5)])
def test_gated_linear_attention_in_portions_from_states_in_given_rows(H, D, E, rank):
    """Three sequences of unequal lengths, in portions of 17, 2 and the rest (16 tokens a chunk: a chunk and one, two,
    several), one of them behind a state that is already there, in rows 4, 0 and 2 of six; rows of nobody stay as they are;
    then single tokens with the heads' norm and gate, into columns of longer rows."""
    g = torch.Generator().manual_seed(H + D)
    tau, lens, rows = 8.0, [70, 19, 41], [4, 0, 2]
    _, a2, bias = gla_inputs(g, 1, H, D, E, rank)
    seqs = [gla_inputs(g, n + 2, H, D, E, rank)[0] for n in lens]
    start = [None, None, 0.3 * randn(g, H, D, E)]
    want = [gla_want(s, a2, bias, H, D, E, tau, st)[0] for s, st in zip(seqs, start)]
    state = torch.zeros(6, H, D, E, device=DEV)
    state[[1, 3, 5]] = 7.5
    state[2] = dev(start[2])
    got = [[] for _ in lens]
    for cuts in ([(0, 17)] * 3, [(17, 19)] * 3, [(19, 70), None, (19, 41)]):
        on = [i for i in range(3) if cuts[i] is not None]
        st = Step([(rows[i], cuts[i][0], cuts[i][1] - cuts[i][0]) for i in on])
        out, at = gla_scan(dev(torch.cat([seqs[i][cuts[i][0]:cuts[i][1]] for i in on])), a2, bias, tau, state, st, H, D, E), 0
        for i in on:
            n = cuts[i][1] - cuts[i][0]
            got[i].append(out[at:at + n].cpu().double())
            at += n
    for i in range(3):
        o = torch.cat(got[i])
        w = want[i][:lens[i]]
        assert float((o - w).abs().max()) < 2e-5 * max(1.0, float(w.abs().max())), f"sequence {i}"
    gain = (1.0 + 0.3 * randn(g, H * E)).float().double()
    st = Step([(r, n, 1) for r, n in zip(rows, lens)])
    for k in range(2):
        x = torch.stack([s[n + k] for s, n in zip(seqs, lens)])
        gate = gla_columns(x, H, D, E, rank)[3]
        o = P.rms_norm(torch.stack([w[n + k] for w, n in zip(want, lens)]).view(3, H, E), None, 1e-5).reshape(3, H * E)
        w = o * gain * gate * torch.sigmoid(gate)
        for dtype, tol in ((torch.float32, 3e-5),) if k == 0 else ((torch.bfloat16, 1e-2),):
            long = torch.full((3, H * E + 9), 3.0, dtype=dtype, device=DEV)
            gla_step(dev(x), a2, bias, tau, state, st, H, D, E, gain, 1e-5, long[:, 4:4 + H * E])
            assert float((long[:, 4:4 + H * E].cpu().double() - w).abs().max()) < tol * max(1.0, float(w.abs().max())), dtype
            assert bool((long[:, :4] == 3.0).all() and (long[:, 4 + H * E:] == 3.0).all())
    assert bool((state[[1, 3, 5]] == 7.5).all()), "rows of nobody"
    for i, n in enumerate(lens):
        _, S = gla_want(seqs[i][:n + 2], a2, bias, H, D, E, tau, start[i])
        assert float((state[rows[i]].cpu().double() - S).abs().max()) < 2e-5 * max(1.0, float(S.abs().max())), f"state of {i}"


@pytest.mark.parametrize("single", [False, True])
def test_a_token_far_back_still_counts(single):
    """A value written 150 tokens ago in a key channel of its own, read by the last token: most of the result is that value
    (the plain cell says so first), through nine chunk borders and a portion's border."""
    H, D, E, rank, tau, T = 2, 32, 16, 4, 16.0, 151
    g = torch.Generator().manual_seed(4)
    rows, a2, bias = gla_inputs(g, T, H, D, E, rank)
    a2[31::D], bias[31::D] = 0.0, 9.0
    q, k, v, _, _ = gla_columns(rows, H, D, E, rank)
    q[:, 31::D] = k[:, 31::D] = 0.0              # the last channel belongs to the far token alone
    k[0, 31::D] = 5.0
    q[T - 1] = 0.0
    q[T - 1, 31::D] = 5.0
    want, _ = gla_want(rows, a2, bias, H, D, E, tau)
    far = v[0] * 25.0 * D ** -0.5
    assert float((want[-1] - far).abs().max()) < 0.01 * float(far.abs().max())
    state = torch.zeros(2, H, D, E, device=DEV)
    if single:
        gain = torch.ones(H * E, dtype=F64)
        for t in range(T):
            out = torch.empty((1, H * E), device=DEV)
            gla_step(dev(rows[t:t + 1]), a2, bias, tau, state, Step([(0, t, 1)]), H, D, E, gain, 1e-6, out)
        gate = gla_columns(rows, H, D, E, rank)[3][-1:]
        want = P.rms_norm(want[-1:].view(1, H, E), None, 1e-6).view(1, H * E) * gate * torch.sigmoid(gate)
    else:
        for a, b in ((0, 90), (90, T)):
            out = gla_scan(dev(rows[a:b]), a2, bias, tau, state, Step([(0, a, b - a)]), H, D, E)[-1:]
    assert float((out[-1].cpu().double() - want[-1]).abs().max()) < 2e-5 * float(want[-1].abs().max())


@pytest.mark.parametrize("z_mean,z_std,tau", [(-3.0, 3.0, 1.0), (-60.0, 30.0, 1.0), (-300.0, 100.0, 0.5), (0.0, 8.0, 1.0), (14.0, 2.0, 16.0),
                                              (0.0, 1.0, 16.0), (40.0, 10.0, 2.0), (-20.0, 0.5, 4.0)])
def test_decays_from_nothing_to_one(z_mean, z_std, tau):
    """Channels that forget everything at once beside others that keep everything, decays whose product underflows within a
    chunk (the sums are then taken term by term), and decays that differ from one in the last digits only."""
    H, D, E, rank, T = 3, 40, 20, 6, 75
    g = torch.Generator().manual_seed(int(abs(z_mean)) + 1)
    rows, a2, bias = gla_inputs(g, T, H, D, E, rank, z_mean, z_std)
    bias[::3] = 20.0
    a2[::3] = 0.0
    want, S = gla_want(rows, a2, bias, H, D, E, tau)
    state = torch.zeros(1, H, D, E, device=DEV)
    got = gla_scan(dev(rows[:70]), a2, bias, tau, state, Step([(0, 0, 70)]), H, D, E).cpu().double()
    assert float((got - want[:70]).abs().max()) < 3e-5 * float(want.abs().max())
    gain = torch.ones(H * E, dtype=F64)
    for t in range(70, T):
        out = torch.empty((1, H * E), device=DEV)
        gla_step(dev(rows[t:t + 1]), a2, bias, tau, state, Step([(0, t, 1)]), H, D, E, gain, 1e-6, out)
        gate = gla_columns(rows, H, D, E, rank)[3][t:t + 1]
        w = P.rms_norm(want[t].view(1, H, E), None, 1e-6).view(1, H * E) * gate * torch.sigmoid(gate)
        assert float((out.cpu().double() - w).abs().max()) < 1e-4 * float(w.abs().max())
    assert float((state[0].cpu().double() - S).abs().max()) < 3e-5 * float(S.abs().max())


def test_decays_next_to_one_over_thousands_of_tokens():
    """2,000 tokens with decays of 1 - 1e-5 .. 1 - 1e-3: an error that leaned one way in every token's logarithm would add up."""
    H, D, E, rank, tau, T = 1, 16, 16, 2, 4.0, 2000
    g = torch.Generator().manual_seed(3)
    rows, a2, bias = gla_inputs(g, T, H, D, E, rank, 7.5, 0.3)
    want, S = gla_want(rows, a2, bias, H, D, E, tau)
    state = torch.zeros(1, H, D, E, device=DEV)
    got = gla_scan(dev(rows), a2, bias, tau, state, Step([(0, 0, T)]), H, D, E).cpu().double()
    assert float((got - want).abs().max()) < 3e-5 * float(want.abs().max())
    assert float((state[0].cpu().double() - S).abs().max()) < 3e-5 * float(S.abs().max())


def test_many_sequences_of_one_to_fifty_tokens_in_one_step():
    """Chunks of 36 sequences side by side, some of one token, in a wide value size (two groups of columns a workgroup)."""
    H, D, E, rank, tau = 6, 24, 128, 8, 16.0
    g = torch.Generator().manual_seed(12)
    _, a2, bias = gla_inputs(g, 1, H, D, E, rank)
    lens = [1 + (i * 17) % 50 for i in range(36)]
    seqs = [gla_inputs(g, n, H, D, E, rank)[0] for n in lens]
    state = torch.zeros(37, H, D, E, device=DEV)
    out = gla_scan(dev(torch.cat(seqs)), a2, bias, tau, state, Step([(35 - i, 0, n) for i, n in enumerate(lens)]), H, D, E)
    at = 0
    for i, n in enumerate(lens):
        want, S = gla_want(seqs[i], a2, bias, H, D, E, tau)
        assert float((out[at:at + n].cpu().double() - want).abs().max()) < 2e-5 * float(want.abs().max()), f"sequence {i}"
        assert float((state[35 - i].cpu().double() - S).abs().max()) < 2e-5 * float(S.abs().max()), f"state of {i}"
        at += n
    assert bool((state[36] == 0).all())


def test_unfit_calls_are_refused():
    from synaptix_amd.kernels import ops
    H, D, E, rank = 2, 8, 8, 4
    rows = torch.zeros(4, 2 * H * D + 2 * H * E + rank, device=DEV)
    q, k, v, gate, mid = gla_columns(rows, H, D, E, rank)
    st, state, out = Step([(0, 0, 4)]), torch.zeros(1, H, D, E, device=DEV), torch.empty(4, H * E, device=DEV)
    a2, bias = torch.zeros(rank, H * D, device=DEV), torch.zeros(H * D, device=DEV)
    ok = dict(a2=a2, a_bias=bias, q_scale=1.0, tau=1.0, state=state, seq_start=st.seq_start, seq_slot=st.seq_slot, out=out, n_heads=H,
              dim=D, vdim=E)
    ops.gated_linear_scan(q, k, v, mid, **ok)
    for bad in (dict(a2=a2[:, 1:].contiguous()), dict(a_bias=bias[1:]), dict(state=state[:, :, :7].contiguous()), dict(dim=300), dict(out=out.double()),
                dict(scratch=lambda n, k: torch.empty(3, device=DEV))):
        with pytest.raises(ops.KernelError):
            ops.gated_linear_scan(q, k, v, mid, **dict(ok, **bad))
    with pytest.raises(ops.KernelError):
        ops.gated_linear_scan(q, k.contiguous(), v, mid, **ok)           # columns of other rows


# ----------------------------------------------------------------------------- attention: unequal sizes, the sink of one, a factor
@pytest.mark.parametrize("H,G,D,E", [(4, 1, 48, 16), (6, 3, 16, 64), (3, 1, 10, 14), (2, 2, 128, 32), (8, 2, 96, 48)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_attention_without_positions_into_columns_of_longer_rows(H, G, D, E, dtype):
    """150 queries over pages in a shuffled order, all at once and then three single tokens: biases on q, k and v, values of
    another size than keys, one added to every softmax's denominator (scores of the first heads are so low that the sink
    takes nearly everything), a factor on the results, and columns of longer rows on both sides; one far key stands out."""
    from synaptix_amd.kernels import ops
    T, N0 = 150, 147
    g = torch.Generator().manual_seed(H * D + E)
    rows = randn(g, T, H * D + G * D + G * E)
    bias = 0.5 * randn(g, H * D + G * D + G * E)
    rows[5, H * D:H * D + G * D] *= 6.0                       # a key that stands out for whoever looks its way
    scale = 1.5 * D ** -0.5
    x = (rows + bias).to(dtype).double() if dtype == torch.bfloat16 else rows + bias
    q, k, v = x[:, :H * D].reshape(T, H, D), x[:, H * D:H * D + G * D].reshape(T, G, D), x[:, H * D + G * D:].reshape(T, G, E)
    mask = torch.arange(T)[None, :] <= torch.arange(T)[:, None]
    want = torch.stack([P.softmax_one((q[:, h] @ k[:, h // (H // G)].T) * scale, mask) @ v[:, h // (H // G)] for h in range(H)], 1)
    want = 0.6 * want.reshape(T, H * E)
    no_sink = torch.stack([torch.softmax(((q[:, h] @ k[:, h // (H // G)].T) * scale).masked_fill(~mask, -math.inf), -1)
                           @ v[:, h // (H // G)] for h in range(H)], 1).reshape(T, H * E) * 0.6
    assert float((want - no_sink).abs().max()) > 0.1 * float(want.abs().max())
    order = [4, 1, 3]
    kp = torch.zeros((6, G, 64, D), dtype=dtype, device=DEV)
    vp = torch.zeros((6, G, E, 64), dtype=dtype, device=DEV)
    table, long = ints(order + [0]).view(1, 4), dev(torch.cat([rows, randn(g, T, 5)], 1))
    tol = 3e-5 if dtype == torch.float32 else 1.5e-2
    for a, b in [(0, N0)] + [(t, t + 1) for t in range(N0, T)]:
        st = Step([(0, a, b - a)])
        qo = torch.empty((b - a, H * D), dtype=dtype, device=DEV)
        ops.window_intake(long[a:b, :rows.shape[1]], dev(bias), qo, kp, vp, table, st.tok_seq, st.tok_pos, None, None, 0.0, H, G, D, E)
        wide = torch.full((b - a, H * E + 8), 2.0, dtype=dtype, device=DEV)
        o = wide[:, 4:4 + H * E]
        fns = [lambda: ops.window_attention(qo, kp, vp, table, st.tok_seq, st.tok_pos, o, scale, H, G, D, E, sink_one=True, out_scale=0.6)]
        if dtype == torch.bfloat16 and ops.window_prefill_takes(D, E) and b - a > 1:
            fns.append(lambda: ops.window_attention_prefill_bf16(qo, kp, vp, table, st.seq_start, st.seq_past, o, scale, H, G, D, E,
                                                                 sink_one=True, out_scale=0.6))
        for fn in fns:
            o.fill_(0.0)
            fn()
            assert float((o.cpu().double() - want[a:b]).abs().max()) < tol * max(1.0, float(want.abs().max())), (a, b)
            assert bool((wide[:, :4] == 2.0).all() and (wide[:, 4 + H * E:] == 2.0).all())


# ----------------------------------------------------------------------------- the embedding's pass
@pytest.mark.parametrize("V,W", [(64, 96), (50, 72), (33, 41), (48, 1024)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_sinusoidal_positions_in_the_embeddings_pass(V, W, dtype):
    """Rows of a table (plain, and in fragment order where the sizes allow it) times a scale plus the sinusoid of the rows'
    positions, near 0 and far away, and a copy of the rows."""
    from synaptix_amd.models import TokenEmbedding
    g = torch.Generator().manual_seed(W)
    table = randn(g, V, W).to(torch.bfloat16).double()
    pos = [0, 1, 2, 63, 64, 1000, 4095, 65535, 1000003]
    ids = torch.randint(0, V, (len(pos),), generator=g).tolist()
    e = TokenEmbedding("e", V, W, scale=3.5, sinusoid_base=10000.0)
    e.load(lambda n: dev(table, dtype))
    keep = torch.empty((len(pos), W), device=DEV)
    got = e.forward(ints(ids), ints(pos), keep)
    want = 3.5 * table[ids]
    for r, p in enumerate(pos):
        for c in range(W):
            ang = p * 10000.0 ** (-2.0 * (c // 2) / W)
            want[r, c] += math.sin(ang) if c % 2 == 0 else math.cos(ang)
    assert float((got.cpu().double() - want).abs().max()) < 2e-6
    assert torch.equal(got, keep)
    plain = TokenEmbedding("e", V, W)
    plain.load(lambda n: dev(table, dtype))
    assert torch.equal(plain.forward(ints(ids)).cpu().double(), table[ids])


# ----------------------------------------------------------------------------- what a pass adds to the residual
@pytest.mark.parametrize("W", [64, 72, 41, 4096, 5000, 9000, 17000])
def test_rows_and_a_vector_beside_the_terms_of_a_residual_sum(W):
    from synaptix_amd.kernels import ops
    g = torch.Generator().manual_seed(W)
    N = 5
    x, rows, vec, gain = randn(g, N, W), randn(g, N, W), randn(g, W), 1.0 + 0.2 * randn(g, W)
    a, b, scale, gate = randn(g, 6, N, W), randn(g, N, W), randn(g, W), randn(g, N, 3)
    gd = dev(gate)
    for terms, add in (([], 0), ([(dev(a), None, None)], a.sum(0)),
                       ([(dev(a), dev(scale), None), (dev(b), None, gd[:, 2:])], a.sum(0) * scale + b * torch.sigmoid(gate[:, 2:]))):
        for r, v in ((rows, vec), (None, vec), (rows, None), (None, None)):
            if r is None and v is None and not terms:
                continue
            summed = x + add + (0 if r is None else r) + (0 if v is None else v)
            for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2e-2)):
                resid, out = dev(x), torch.empty((N, W), dtype=dtype, device=DEV)
                ops.add_scaled_rmsnorm(resid, terms, dev(gain), 1e-6, out, add_rows=None if r is None else dev(r),
                                       add_vec=None if v is None else dev(v))
                assert float((resid.cpu().double() - summed).abs().max()) < 1e-5
                want = P.rms_norm(summed, gain, 1e-6)
                assert float((out.cpu().double() - want).abs().max()) < tol * float(want.abs().max())
                pick = ints([3, 0])
                few, resid = torch.empty((2, W), dtype=dtype, device=DEV), dev(x)
                ops.add_scaled_rmsnorm(resid, terms, dev(gain), 1e-6, few, pick, None if r is None else dev(r), None if v is None else dev(v))
                assert float((few.cpu().double() - want[[3, 0]]).abs().max()) < tol * float(want.abs().max()) and torch.equal(resid, dev(x))


@pytest.mark.parametrize("W,M", [(256, 1), (256, 8), (64, 5)])
def test_a_norm_adds_a_pass_inputs_whatever_the_last_sublayer_left(W, M):
    """RmsNorm behind InjectedDelta around nothing, a tensor, partial sums, several terms, and a product that has not been
    run (which the norm runs with the additions in its epilogue)."""
    from synaptix_amd.parts import RmsNorm, InjectedDelta, SummedDeltas, Matrix, as_rows
    from synaptix_amd.parts.linear import DeferredProduct
    g = torch.Generator().manual_seed(W + M)
    norm = RmsNorm("n", W, 1e-6)
    gain = (1.0 + 0.2 * randn(g, W)).to(torch.bfloat16).double()
    norm.load(lambda n: dev(gain, torch.bfloat16))
    x, rows, vec, d, parts = randn(g, M, W), randn(g, M, W), randn(g, W), randn(g, M, W), randn(g, 3, M, W)
    h, w = randn(g, M, 96).to(torch.bfloat16).double(), (0.1 * randn(g, W, 96)).to(torch.bfloat16).double()
    m = Matrix(dev(w, torch.bfloat16))
    assert m.packed is not None
    for inner, add in ((None, 0.0), (dev(d), d), (dev(parts), parts.sum(0)), (SummedDeltas([dev(parts), dev(d)]), parts.sum(0) + d),
                       (DeferredProduct(dev(h, torch.bfloat16), m), h @ w.T)):
        for r in (rows, None):
            resid = dev(x)
            out = as_rows(norm.add_apply(resid, InjectedDelta(inner, None if r is None else dev(r), dev(vec), (M, W)), torch.bfloat16))
            summed = x + add + vec + (0 if r is None else r)
            assert float((resid.cpu().double() - summed).abs().max()) < 2e-5
            want = P.rms_norm(summed, gain, 1e-6)
            assert float((out.cpu().double() - want).abs().max()) < 2e-2 * float(want.abs().max())
            total = InjectedDelta(inner, None if r is None else dev(r), dev(vec), (M, W)).run()
            assert float((total.cpu().double() - (summed - x)).abs().max()) < 2e-5


# ----------------------------------------------------------------------------- the cap on the logits
@pytest.mark.parametrize("M", [1, 5, 8, 9, 40, 300])
@pytest.mark.parametrize("N,K,keep_rows", [(256, 128, False), (48, 96, False), (41, 72, True), (512, 256, False)])
def test_a_soft_cap_behind_an_output_matrix(M, N, K, keep_rows):
    from synaptix_amd.parts import Matrix, linear
    g = torch.Generator().manual_seed(M + N)
    x, w = randn(g, M, K).to(torch.bfloat16).double(), randn(g, N, K).to(torch.bfloat16).double()
    z = x @ w.T
    for cap in (3.0, 40.0):
        want = cap * torch.tanh(z / cap)
        got = linear(dev(x, torch.bfloat16), Matrix(dev(w, torch.bfloat16), keep_rows=keep_rows), torch.float32, point=("softcap", cap))
        assert float((got.cpu().double() - want).abs().max()) < 2e-5 * cap
        got = linear(dev(x), Matrix(dev(w), keep_rows=True), torch.float32, point=("softcap", cap))
        assert float((got.cpu().double() - want).abs().max()) < 2e-5 * cap


def test_a_cap_that_is_none_or_in_the_wrong_place_is_refused():
    from synaptix_amd.kernels import ops
    from synaptix_amd.parts import Matrix, linear
    x, w = torch.zeros(40, 64, dtype=torch.bfloat16, device=DEV), torch.zeros(48, 64, dtype=torch.bfloat16, device=DEV)
    with pytest.raises(ops.KernelError):
        ops.gemm(x, w, torch.empty(40, 48, device=DEV), point=("softcap", 3.0))
    with pytest.raises(ops.KernelError):
        linear(x, Matrix(w), torch.float32, point=("softcap", 0.0))
    with pytest.raises(TypeError):
        linear(x, Matrix(w), torch.bfloat16, point=("softcap", 3.0))


# ----------------------------------------------------------------------------- the router and its experts
@pytest.mark.parametrize("N,E,top,groups,keep", [(1, 8, 4, 2, 1), (70, 12, 3, 4, 2), (9, 6, 1, 6, 1), (33, 64, 8, 8, 3), (5, 7, 3, 1, 1), (130, 256, 8, 8, 4),
                                                 (20, 10, 10, 5, 5), (12, 4, 2, 4, 2)])
def test_a_router_of_sigmoids_whose_groups_score_by_their_two_best(N, E, top, groups, keep):
    """Exact choice; corrections that leave every choice score negative (a group that is shut out counts as minus infinity,
    not as 0) or reorder everything; weights from the scores alone."""
    from synaptix_amd.kernels import ops
    g = torch.Generator().manual_seed(N + E)
    z = (1.5 * randn(g, N, E)).float().double()
    for corr in (torch.zeros(E, dtype=F64), -2.0 + 0.3 * randn(g, E), 1.5 * randn(g, E)):
        corr = corr.float().double()
        ids = torch.empty((N, top), dtype=torch.int32, device=DEV)
        wt = torch.empty((N, top), device=DEV)
        ops.route_scores(dev(torch.cat([z, randn(g, N, 5)], 1))[:, :E], dev(corr), ids, wt, groups, keep, True, 1.7, sigmoid=True,
                         group_two=True, renorm_eps=1e-20)
        want_ids, want_wt = P.route(z, corr, top, groups, keep, 1.7)
        order = torch.argsort(ids.cpu().long(), 1)
        want_order = torch.argsort(want_ids, 1)
        assert torch.equal(ids.cpu().long().gather(1, order), want_ids.gather(1, want_order))
        assert float((wt.cpu().double().gather(1, order) - want_wt.gather(1, want_order)).abs().max()) < 1e-5
    # scores so low that their sum is nothing beside the 1e-20 in the denominator: weights of 0, not of 1 / top
    ops.route_scores(torch.full((N, E), -80.0, device=DEV), None, ids, wt, groups, keep, True, 1.7, sigmoid=True, group_two=True,
                     renorm_eps=1e-20)
    assert float(wt.abs().max()) < 1e-10


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W,F,E,top,groups,keep,S", [(64, 32, 8, 3, 4, 2, 48), (96, 20, 6, 2, 1, 1, None), (128, 128, 4, 4, 2, 2, 64), (128, 64, 16, 2, 4, 1, 32)])
def test_experts_that_square_a_relu_beside_a_gated_shared_one(W, F, E, top, groups, keep, S, dtype):
    from synaptix_amd.parts import RoutedExperts, UngatedMlp, as_delta
    g = torch.Generator().manual_seed(W + F)
    w = {"router": 0.3 * randn(g, E, W), "correction": -1.5 + 0.2 * randn(g, E)}
    for e in range(E):
        w.update({f"e{e}.up": 0.2 * randn(g, F, W), f"e{e}.down": 0.2 * randn(g, W, F)})
    if S is not None:
        w.update({"shared.sg": 0.4 * randn(g, 1, W), "shared.up": 0.2 * randn(g, S, W), "shared.down": 0.2 * randn(g, W, S)})
    w = {n: t.to(torch.bfloat16).double() for n, t in w.items()}
    ff = RoutedExperts("", W, F, E, top, "relu_squared", router="scores", score="sigmoid", group_score="two", n_groups=groups,
                       keep_groups=keep, renorm=True, renorm_eps=1e-20, route_scale=1.7,
                       shared=None if S is None else UngatedMlp("shared.", W, S), shared_gate=None if S is None else "shared.sg")
    assert set(ff.tensor_specs()) == set(w)
    ff.load(lambda n: dev(w[n], dtype))
    c = {"router": {"experts": E, "top": top, "groups": {"count": groups, "keep": keep}, "scale": 1.7}}
    if S is not None:
        c["shared"] = {"ff": S}
    for N in (1, 5, 70, 300):
        h = randn(g, N, W).to(dtype).double()
        want = P.experts(h, w, "", c)
        got = as_delta(ff.forward(dev(h, dtype), None))
        got = got.sum(0) if got.dim() == 3 else got
        tol = 1e-4 if dtype == torch.float32 else 3e-2
        assert float((got.cpu().double() - want).abs().max()) < tol * max(1.0, float(want.abs().max())), f"{N} rows"


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
    """A prompt in portions of 2, 1, 3, 17, 64 and 2 tokens and the rest: every portion starts from the pages and the
    states that the earlier ones left (inside a page, inside a chunk of the scan, at a page's border)."""
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
    """Decoding over several pages' borders, from prompts that end inside a chunk of the scan and inside a page."""
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


@pytest.mark.parametrize("seed", list(range(9000, 9020)))
def test_configurations_drawn_from_a_seed(seed):
    """Layer kinds, orders, head counts, sizes, groups, loops, caps and factors drawn from a seed
    (the cases above are chosen; these are not): a prompt whole, then requests of unequal lengths cut at unequal places and
    decoded together, 3 to 20 of them, against the plain model for each alone; every fourth one also in bfloat16, there
    without the tokens whose choice of experts is a close call (the 32-bit run has them all)."""
    import random
    from sunosun_cases import random_model, routing_margins
    from synaptix_amd import Engine
    cfg, folder, plain = random_model(seed)
    rng = random.Random(seed + 1)
    g = torch.Generator().manual_seed(seed)
    T = rng.choice([70, 150, 250])
    lens = [T, 9, T // 2] + [rng.randint(2, T) for _ in range(rng.choice([0, 3, 6, 17]))]
    toks = [torch.randint(0, cfg.vocab, (n,), generator=g).tolist() for n in lens]
    want = [plain.logits(t) for t in toks]
    clear = [routing_margins(plain, t) > 0.01 for t in toks] if seed % 4 == 0 else None
    for dtype in DTYPES if seed % 4 == 0 else DTYPES[:1]:
        eng = Engine.load(folder, dtype=dtype, max_tokens=8192, max_slots=32)
        s = eng.acquire()
        keep = [c if dtype == "bfloat16" else torch.ones_like(c) for c in clear] if clear else [slice(None)] * len(toks)
        assert_logits_close(eng.step([(s, toks[0])], want="all").cpu()[keep[0]], want[0][keep[0]], dtype, f"seed {seed} whole", sharp=True)
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
            assert_logits_close(torch.cat(got[i]).cpu()[keep[i]], want[i][keep[i]], dtype,
                                f"seed {seed} {dtype} request {i} of {len(toks)}", sharp=True)
        eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_first_tokens(dtype):
    """Sequences of one and two tokens, and the first 45 positions one by one."""
    for name in ("P", "S", "T"):
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
    """400 tokens one by one: the states are carried throughout, every pass of the looped layers' own."""
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
    plain = P.PlainSunosun.from_folder(folder)
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
