"""Each mechanism of the Tigesun design alone against the plain functions of ``plain_tigesun``, in
32-bit and in bfloat16: the embedding through its norm and the next one; a norm behind a sublayer
that takes in the sublayer's bias; the gated activation behind biases, alone and in the product's
epilogue; a gate and then a norm over parts of a row; the convolutions with a bias (both forms of the kernel, two
steps with a request left out, single tokens); the rotation with stretched frequencies; the latent
attention without a rotated part at its window's edges; the recurrence token by token (cut and
alone the same bits, the plain matrices) and in chunks side by side (long and short sequences in
one step, two steps from the states the first left, every way of dealing heads), a token far back
that a head without decay returns and one with decay has lost, decays that forget everything."""
import math

import pytest
import torch

import plain_tigesun as P
from gpu_util import DEV, rel_err, tol
from zinfer_amd import ops

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]


def _rand(shape, seed, scale=1.0, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * scale).to(dtype)


def _i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


def _starts(lens):
    out = [0]
    for n in lens:
        out.append(out[-1] + n)
    return out


# ------------------------------------------------------------------------------ rows and norms
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("W", [48, 50, 320, 2048, 8192, 8196])
def test_embedding_through_its_norm_and_the_next(dt, W):
    T, V, scale = 9, 31, 1.5
    table = _rand((V, W), 1, 1.0, dt)
    ids = _i32([0, 30, 5, 5, 7, 1, 2, 3, 29])
    ga, gb = 1.0 + _rand((W,), 2, 0.3), 1.0 + _rand((W,), 3, 0.3)
    x = torch.empty((T, W), dtype=torch.float32, device=DEV)
    out = torch.empty((T, W), dtype=dt, device=DEV)
    want = P.rms_norm(table[ids.cpu().long()].double() * scale, ga, 1e-5)
    ops.embed_norm(table.to(DEV), ids, ga.to(DEV), 1e-5, x, scale)
    assert rel_err(x, want) < tol(torch.float32)
    alone = x.clone()
    ops.embed_norm(table.to(DEV), ids, ga.to(DEV), 1e-5, x, scale, gb.to(DEV), 1e-3, out)
    assert torch.equal(x, alone)
    assert rel_err(out, P.rms_norm(want, gb, 1e-3)) < tol(dt)
    # a row does not depend on the rows beside it
    one = torch.empty((1, W), dtype=torch.float32, device=DEV)
    ops.embed_norm(table.to(DEV), ids[3:4].contiguous(), ga.to(DEV), 1e-5, one, scale)
    assert torch.equal(one[0], x[3])


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T", [3, 300])
@pytest.mark.parametrize("W", [48, 50, 320, 2048, 4096, 8192])
def test_norm_behind_a_sublayer_takes_its_bias(dt, T, W):
    y, x, b = _rand((T, W), 1), _rand((T, W), 2), _rand((W,), 3)
    ga, gb = 1.0 + _rand((W,), 4, 0.3), 1.0 + _rand((W,), 5, 0.3)
    want = x.double() + P.rms_norm(y.double() + b.double(), ga, 1e-5)
    got = x.to(DEV).clone()
    ops.norm_rows(y.to(DEV), ga.to(DEV), None, 1e-5, got, False, add=True, x_bias=b.to(DEV))
    assert rel_err(got, want) < tol(torch.float32)
    if ops.norm_add_norm_covers(W):
        both, out = x.to(DEV).clone(), torch.empty((T, W), dtype=dt, device=DEV)
        ops.norm_add_norm(y.to(DEV), ga.to(DEV), None, 1e-5, False, both, gb.to(DEV), None, 1e-6,
                          False, out, y_bias=b.to(DEV))
        assert rel_err(both, want) < tol(torch.float32)
        assert rel_err(out, P.rms_norm(want, gb, 1e-6)) < tol(dt)
        one, o1 = x[1:2].to(DEV).clone(), torch.empty((1, W), dtype=dt, device=DEV)
        ops.norm_add_norm(y[1:2].to(DEV).contiguous(), ga.to(DEV), None, 1e-5, False, one, gb.to(DEV),
                          None, 1e-6, False, o1, y_bias=b.to(DEV))
        assert rel_err(one, want[1:2]) < tol(torch.float32)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("n", [24, 50, 384])
def test_gated_activation_behind_biases(dt, n):
    """Rows of a wider matrix; with biases and without."""
    T = 7
    wide = _rand((T, 2 * n + 8), 1, 1.5, dt)
    b = _rand((2 * n,), 2)
    for bias in (b, None):
        out = torch.empty((T, n), dtype=dt, device=DEV)
        ops.gated_rows(wide.to(DEV)[:, :2 * n], None if bias is None else bias.to(DEV), out, "gelu_tanh")
        x = wide[:, :2 * n].double() + (0 if bias is None else bias.double())
        assert rel_err(out, P.gelu_tanh(x[:, :n]) * x[:, n:]) < tol(dt)


@pytest.mark.parametrize("M", [1, 8, 16, 17, 33, 64, 100, 128, 129, 300, 1000, 2048])
@pytest.mark.parametrize("I,K", [(64, 64), (96, 192), (2048, 512), (8192, 256), (5632, 2048)])
def test_gated_activation_in_the_products_epilogue(M, I, K):
    """Every kernel that the number of rows and the sizes lead to, with biases that differ from
    column to column and without."""
    if M > 300 and I * K > (1 << 20) and (M, I) not in ((2048, 8192), (1000, 5632)):
        pytest.skip("one long product a size")
    a = _rand((M, K), 1, 1.0, torch.bfloat16)
    g, u = _rand((I, K), 2, K ** -0.5, torch.bfloat16), _rand((I, K), 3, K ** -0.5, torch.bfloat16)
    bg, bu = _rand((I,), 4), _rand((I,), 5)
    w = ops.pretile_weight(ops.interleave_gate_up(g, u).to(DEV))
    out = torch.empty((M, I), dtype=torch.bfloat16, device=DEV)
    # (32-bit products on the CPU: 64-bit ones of these sizes take seconds)
    zg, zu = (a.float() @ g.float().T).double(), (a.float() @ u.float().T).double()
    ops.gemm_geglu(a.to(DEV), w, ops.interleave_bias(bg, bu).to(DEV), out)
    assert rel_err(out, P.gelu_tanh(zg + bg.double()) * (zu + bu.double())) < tol(torch.bfloat16)
    ops.gemm_geglu(a.to(DEV), w, None, out)
    assert rel_err(out, P.gelu_tanh(zg) * zu) < tol(torch.bfloat16)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("parts,dv", [(1, 24), (3, 8), (2, 50), (4, 128), (2, 516), (1, 4096), (7, 1),
                                      (1, 9000)])
def test_gate_then_norm_over_parts(dt, parts, dv):
    T, W = 6, parts * dv
    y, gate = _rand((T, W), 1), _rand((T, W + 8), 2, 2.0, dt)
    w = 1.0 + _rand((W,), 3, 0.3)
    out = torch.empty((T, W + 4), dtype=dt, device=DEV)
    ops.gate_norm(y.to(DEV), w.to(DEV), gate.to(DEV)[:, :W], out[:, :W], parts, 1e-5)
    assert rel_err(out[:, :W], P.gated_parts_norm(y, gate[:, :W], w, parts, 1e-5)) < tol(dt)


# ------------------------------------------------------------------------------ convolutions
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("taps,C,pad", [(4, 64, 8), (3, 320, 0), (1, 16, 8), (2, 21, 3), (5, 48, 8),
                                        (8, 40, 16), (4, 4352, 64)])
def test_convolutions_with_a_bias(dt, taps, C, pad):
    """Three requests: whole portions first (one of a single token, one shorter than the taps),
    then one left out and the others swapped with one and many tokens; single tokens; both
    output types; slots out of order."""
    K, b = _rand((C, taps), 1, 0.7), _rand((C,), 2)
    offset, slots, lens, more = 8, [3, 0, 2], [35, 1, 2], [3, 0, 1]
    seqs = [_rand((lens[i] + more[i], C + pad), 30 + i, 1.0, dt) for i in range(3)]
    width = (offset + (taps - 1) * C + 7) // 4 * 4
    state = torch.zeros((4, width), dtype=torch.float32, device=DEV)
    state[:, :offset] = 3.0

    def step(parts, which, out_dt, single=False):
        n = [p.shape[0] for p in parts]
        out = torch.empty((sum(n), C), dtype=out_dt, device=DEV)
        ops.short_conv(torch.cat(parts).to(DEV), K.to(DEV), state, offset, _i32([slots[i] for i in which]),
                       _i32([i for i, m in enumerate(n) for _ in range(m)]), _i32(_starts(n)), out,
                       single_tokens=single, bias=b.to(DEV))
        return out, _starts(n)

    want = [P.silu(P.causal_conv(s[:, :C], K, b)) for s in seqs]
    for out_dt in {torch.float32, dt}:
        state[:, offset:] = 0.0
        out, at = step([seqs[i][:lens[i]] for i in range(3)], [0, 1, 2], out_dt)
        for i in range(3):
            assert rel_err(out[at[i]:at[i + 1]], want[i][:lens[i]]) < tol(out_dt)
        out, at = step([seqs[2][lens[2]:], seqs[0][lens[0]:]], [2, 0], out_dt)
        for j, i in enumerate([2, 0]):
            assert rel_err(out[at[j]:at[j + 1]], want[i][lens[i]:]) < tol(out_dt)
        for i in range(3):
            seen = seqs[i][:lens[i] + more[i], :C].float()
            kept = state[slots[i], offset:offset + (taps - 1) * C].cpu().view(taps - 1, C)
            full = torch.cat([torch.zeros((taps, C)), seen])
            assert torch.equal(kept, full[full.shape[0] - (taps - 1):]), i
        assert float((state[:, :offset] - 3.0).abs().max()) == 0.0
        state[:, offset:] = 0.0
        got = [step([seqs[0][t:t + 1]], [0], out_dt, single=True)[0][0].cpu() for t in range(38)]
        state[:, offset:] = 0.0
        whole, _ = step([seqs[0]], [0], out_dt)
        assert torch.equal(torch.stack(got), whole.cpu())


# ------------------------------------------------------------------------------ rotation and attention
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("d,dims", [(12, 8), (64, 64), (96, 40), (128, 128)])
def test_head_norm_and_stretched_rotation(dt, d, dims):
    from zinfer_amd.config.rotary import leading_rotary
    H, T = 3, 7
    scaling = {"factor": 5.0, "original": 300, "fast": 12.0, "slow": 0.7}
    spec = leading_rotary(700.0, dims, scaling)
    src, g = _rand((T, H * d), 1, 1.0, dt), 1.0 + _rand((d,), 2, 0.3)
    positions = [0, 1, 2, 63, 299, 1500, 3000]
    q = torch.empty((T, H * d), dtype=dt, device=DEV)
    freq = torch.tensor(spec.frequencies, dtype=torch.float64).to(torch.float32).to(DEV)
    ops.project_rows(src.to(DEV), _i32(positions), None, 4, [
        ops.RowSegment(0, H * d, q, gain=g.to(DEV), eps=1e-5, hd=d, per_head=True, rot_dims=dims,
                       freq=freq, mag=spec.magnitude)])
    want = P.rotate(P.rms_norm(src.view(T, H, d), g, 1e-5), torch.tensor(positions),
                    {"dims": dims, "base": 700.0, "scaling": scaling})
    # (an angle is the 32-bit product position * frequency: its error grows with the position)
    assert rel_err(q, want.reshape(T, H * d)) < max(tol(dt), 2e-4)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,R", [(4, 18), (6, 64), (3, 96), (16, 128)])
@pytest.mark.parametrize("window", [1, 7, 33, 96])
def test_latent_attention_at_its_windows_edges(dt, H, R, window):
    """Every query of a prompt of 120 and of a token alone: a latent that points at the query's
    own direction stands at the window's oldest position and one before it; table entries
    before the window are -1 for the token alone."""
    ps, n = 8, 120
    pages = (n + ps - 1) // ps
    g = torch.Generator().manual_seed(window)
    perm = torch.randperm(pages, generator=g).tolist()
    last = n - 1
    for inside in (True, False):
        c = _rand((n, R), 3, 0.3, dt)
        q = _rand((n, H * R), 4, 0.3, dt)
        at = last - window + (1 if inside else 0)
        if at < 0:
            continue
        q[last] = 1.0
        c[at] = 3.0
        rows = torch.zeros((pages * ps, R), dtype=dt)
        rows[:n] = c
        pool = ops.masked_pool_from_rows(rows.view(pages, 1, ps, R)[torch.argsort(torch.tensor(perm))]
                                         .contiguous())
        want = P.attend(q.view(n, H, R).double(), c.view(n, 1, R).double(), c.view(n, 1, R).double(), 0.25,
                        P.seen(n, window))
        for queries in (range(n), [last]):
            queries = list(queries)
            table = list(perm)
            if len(queries) == 1:
                for p in range((last - window + 1) // ps):
                    table[p] = -1
            out = torch.empty((len(queries), H * R), dtype=dt, device=DEV)
            ops.attend_masked(q[queries].to(DEV).contiguous(), None, None, pool.to(DEV), None, None,
                              _i32([table]), _i32([0, len(queries)]), _i32([n]),
                              _i32([0] * len(queries)), out, 0.25, 0.0, window, 0, H, 1, R, R, ps,
                              len(queries), n)
            assert rel_err(out, want[queries]) < max(tol(dt), 1e-4)
            mark = float(out[-1].float().mean())
            assert (mark > 2.0) is inside, (inside, mark)


# ------------------------------------------------------------------------------ the recurrence
def _space_inputs(T, H, G, N, dv, seed, dt=torch.float32):
    return (_rand((T, H * dv + 2 * G * N), seed, 1.0, dt), _rand((T, H), seed + 1))


def _space_weights(H):
    return (torch.linspace(-4.0, 1.0, H), torch.linspace(-3.0, 0.5, H), torch.linspace(-1.0, 1.5, H))


def _space_reference(rows, steps, weights, H, G, N, dv, state=None):
    a_log, bias, skip = weights
    T, I = rows.shape[0], H * dv
    x, B, C = torch.split(rows.double(), [I, G * N, G * N], dim=1)
    y, S = P.state_space(x.reshape(T, H, dv), B.reshape(T, G, N), C.reshape(T, G, N),
                         P.softplus(steps.double() + bias.double()), a_log, skip, state)
    return y.reshape(T, I), S


def _run_space(state, parts, slots, weights, H, G, N, dv, chunked=False, heads=None):
    n = [p[0].shape[0] for p in parts]
    rows = torch.cat([p[0] for p in parts]).to(DEV)
    steps = torch.cat([p[1] for p in parts]).to(DEV)
    a_log, bias, skip = (w.float().to(DEV) for w in weights)
    I = H * dv
    out = torch.empty((sum(n), I), dtype=torch.float32, device=DEV)
    lists = ops.fixed_decay_chunk_lists(n) if chunked else None
    if lists is not None:
        lists = tuple(torch.from_numpy(t).to(DEV) if t.size else None for t in lists)
    ops.state_space(rows[:, :I], rows[:, I:I + G * N], rows[:, I + G * N:], steps, a_log, bias, skip, state,
                    _i32(slots), _i32(_starts(n)), out, H, G, N, dv, lists=lists, heads=heads)
    return out.cpu(), _starts(n)


SHAPES = [(4, 2, 12, 10), (3, 1, 7, 3), (5, 5, 40, 6), (2, 2, 64, 64), (6, 1, 128, 40), (1, 1, 256, 5),
          (7, 7, 1, 1), (4, 1, 200, 33)]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,N,dv", SHAPES)
def test_recurrence_token_by_token(dt, H, G, N, dv):
    """Three sequences of unequal length in one launch against the plain walk; then the same cut
    in two steps, in other slots' company, and token by token: the same bits, and the matrices
    left in the slots are the plain ones."""
    lens = [37, 1, 70]
    size = (ops.state_space_state_size(H, N, dv) + 3) // 4 * 4 + 8
    data = [_space_inputs(n, H, G, N, dv, 40 + 3 * i, dt) for i, n in enumerate(lens)]
    w = _space_weights(H)
    state = torch.zeros((5, size), dtype=torch.float32, device=DEV)
    slots = [4, 1, 2]
    whole, at = _run_space(state, data, slots, w, H, G, N, dv)
    for i, (rows, steps) in enumerate(data):
        want, S = _space_reference(rows, steps, w, H, G, N, dv)
        assert rel_err(whole[at[i]:at[i + 1]], want) < 2e-5
        assert rel_err(ops.state_space_state_matrix(state, H, N, dv)[slots[i]], S) < 2e-5
    assert float(state[[0, 3]].abs().max()) == 0.0
    state2 = torch.zeros_like(state)
    cut = [20, 1, 3]
    first, at1 = _run_space(state2, [(r[:c], s[:c]) for (r, s), c in zip(data, cut)], slots, w, H, G, N, dv)
    second, at2 = _run_space(state2, [(data[2][0][3:], data[2][1][3:]), (data[0][0][20:], data[0][1][20:])],
                             [slots[2], slots[0]], w, H, G, N, dv)
    assert torch.equal(torch.cat([first[at1[0]:at1[1]], second[at2[1]:at2[2]]]), whole[at[0]:at[1]])
    assert torch.equal(first[at1[1]:at1[2]], whole[at[1]:at[2]])
    assert torch.equal(torch.cat([first[at1[2]:at1[3]], second[at2[0]:at2[1]]]), whole[at[2]:at[3]])
    assert torch.equal(state2, state)
    state3 = torch.zeros_like(state)
    rows, steps = data[0]
    got = [_run_space(state3, [(rows[t:t + 1], steps[t:t + 1])], [slots[0]], w, H, G, N, dv)[0][0]
           for t in range(lens[0])]
    assert torch.equal(torch.stack(got), whole[at[0]:at[1]])


@pytest.mark.parametrize("H,G,N,dv", SHAPES + [(8, 2, 64, 32), (4, 2, 128, 96), (3, 3, 24, 64),
                                               (8, 1, 128, 64), (4, 1, 48, 16)])
def test_recurrence_in_chunks(H, G, N, dv):
    """Long and short sequences in one step (portions of one token, under a chunk, a whole
    chunk, several with one token over), then more of each from the states left: against the
    plain walk, for every number of heads a workgroup may take (the same bits)."""
    lens, more = [33, 128, 1, 300, 20, 257], [129, 1, 40, 5, 64, 34]
    size = (ops.state_space_state_size(H, N, dv) + 3) // 4 * 4 + 4
    data = [_space_inputs(n + m, H, G, N, dv, 60 + 3 * i, torch.bfloat16)
            for i, (n, m) in enumerate(zip(lens, more))]
    w, slots = _space_weights(H), [5, 0, 3, 1, 4, 2]
    ref = [_space_reference(r, s, w, H, G, N, dv) for r, s in data]
    seen = None
    for heads in [h for h in (1, 2, 4) if (H // G) % h == 0]:
        state = torch.zeros((7, size), dtype=torch.float32, device=DEV)
        first, at1 = _run_space(state, [(r[:n], s[:n]) for (r, s), n in zip(data, lens)], slots, w, H, G, N,
                                dv, True, heads)
        order = [3, 0, 5, 1, 4, 2]
        second, at2 = _run_space(state, [(data[i][0][lens[i]:], data[i][1][lens[i]:]) for i in order],
                                 [slots[i] for i in order], w, H, G, N, dv, True, heads)
        for i in range(6):
            j = order.index(i)
            got = torch.cat([first[at1[i]:at1[i + 1]], second[at2[j]:at2[j + 1]]])
            assert rel_err(got, ref[i][0]) < 6e-5, (heads, i)
            assert rel_err(ops.state_space_state_matrix(state, H, N, dv)[slots[i]], ref[i][1]) < 6e-5
        assert float(state[6].abs().max()) == 0.0
        if seen is None:
            seen = (first, second, state)
        else:
            assert all(torch.equal(a, b) for a, b in zip(seen, (first, second, state)))


@pytest.mark.parametrize("H,G,N,dv,K", [(4, 2, 12, 10, 72), (64, 1, 128, 64, 2048), (3, 3, 24, 7, 4104)])
def test_step_sizes_formed_where_they_are_used(H, G, N, dv, K):
    """Single tokens of five sequences in bfloat16, from states that are not zero: step sizes from
    the rows they are products of against the same given as numbers."""
    T = 5
    size = ops.state_space_state_size(H, N, dv)
    rows, _ = _space_inputs(T, H, G, N, dv, 3, torch.bfloat16)
    h, w = _rand((T, K), 4, 1.0, torch.bfloat16), _rand((H, K), 5, K ** -0.5, torch.bfloat16)
    weights = [t.to(DEV) for t in _space_weights(H)]
    rows, I, got = rows.to(DEV), H * dv, []
    steps = (h.double() @ w.double().T).float().to(DEV)
    for given in (steps, (h.to(DEV), w.to(DEV))):
        state = _rand((T, size), 6).to(DEV)
        out = torch.empty((T, I), dtype=torch.float32, device=DEV)
        ops.state_space(rows[:, :I], rows[:, I:I + G * N], rows[:, I + G * N:], given, *weights, state,
                        _i32(range(T)), _i32(range(T + 1)), out, H, G, N, dv, single_tokens=True)
        got.append((out, state))
    assert rel_err(got[1][0], got[0][0]) < 2e-5 and rel_err(got[1][1], got[0][1]) < 2e-5


def test_a_token_far_back_is_kept_without_decay_and_lost_with_it():
    """Two heads, 600 tokens.  Token 3 alone writes (step size 1) along channel 0 with values that
    stand out; the last token asks for it.  The head whose decay is 1 to rounding returns them,
    the one that loses a tenth a token has lost them; in one portion, in chunks, and with the
    last 50 tokens alone."""
    H, G, N, dv, T = 2, 1, 16, 8, 600
    rows = torch.zeros((T, H * dv + 2 * N))
    value = torch.arange(1.0, dv + 1.0)
    rows[3, :dv] = rows[3, dv:2 * dv] = value
    rows[3, 2 * dv] = 1.0                                       # B of token 3
    rows[T - 1, 2 * dv + N] = 1.0                               # C of the last
    steps = torch.full((T, H), math.log(math.e - 1.0))          # softplus gives 1
    w = (torch.tensor([-30.0, math.log(-math.log(0.9))]), torch.zeros(H), torch.zeros(H))
    size = ops.state_space_state_size(H, N, dv)
    for dt, chunked in ((torch.float32, False), (torch.bfloat16, True)):
        for cuts in ([T], [T - 50] + [1] * 50, [97, 300, 203]):
            state = torch.zeros((1, size), dtype=torch.float32, device=DEV)
            at = 0
            for n in cuts:
                out, _ = _run_space(state, [(rows[at:at + n].to(dt), steps[at:at + n])], [0], w, H, G, N, dv,
                                    chunked)
                at += n
            assert torch.allclose(out[-1][:dv], value, rtol=1e-4), (dt, cuts)
            assert float(out[-1][dv:].abs().max()) < 1e-20


def test_decays_that_forget_everything_and_step_sizes_of_all_sizes():
    """Rates of exp(8) and step sizes up to 40 beside near zero ones: nothing is divided by a
    decay and nothing overflows; the plain outputs in every form."""
    H, G, N, dv, T = 4, 2, 16, 32, 200
    rows, steps = _space_inputs(T, H, G, N, dv, 5, torch.bfloat16)
    steps = steps * 15.0
    steps[::7] = -40.0
    w = (torch.tensor([8.0, 3.0, -2.0, -9.0]), torch.zeros(H), torch.ones(H))
    want, S = _space_reference(rows, steps, w, H, G, N, dv)
    size = ops.state_space_state_size(H, N, dv)
    for dt, chunked in ((torch.float32, False), (torch.bfloat16, False), (torch.bfloat16, True)):
        state = torch.zeros((1, size), dtype=torch.float32, device=DEV)
        out, _ = _run_space(state, [(rows.to(dt), steps)], [0], w, H, G, N, dv, chunked)
        assert torch.isfinite(out).all() and torch.isfinite(state).all()
        assert rel_err(out, want) < 1e-4
        assert rel_err(ops.state_space_state_matrix(state, H, N, dv)[0], S) < 1e-4
