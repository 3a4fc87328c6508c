"""Each mechanism of the Fumanex design alone against the plain functions of ``plain_fumanex``, in
32-bit and in bfloat16: bias and activation over slices of rows; unit norms and the blend of
values on their way into the cache; attention with kept first positions behind a window and a
bias by distance, every size and the MFMA form (a loud key just inside and just outside the
window and the kept range, far back, at page borders; a bias that points at one distance; pages
between the kept ones and the window gone); the rotation's table; the recurrence with a fixed
decay token by token and in chunks (states in slots, cuts, long and short sequences in one step,
a token far back); the norm a head or a row with either gate."""
import math

import pytest
import torch

import plain_fumanex as P
from gpu_util import DEV, rel_err, tol
from test_lodenex_kernels_gpu import Paged
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


# ------------------------------------------------------------------------------ rows
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T, n, before, tail, ones", [(1, 24, 8, 8, 2), (5, 13, 3, 4, 1),
                                                       (7, 2048, 0, 64, 2), (300, 40, 16, 0, 0)])
def test_bias_act_rows(dt, T, n, before, tail, ones):
    """On a slice of columns, into a slice of columns with ones and zeros behind; what lies
    beside both stays; in place too."""
    wide = _rand((T, before + n + 8), 1, 2.0, dt).to(DEV)
    bias = _rand((n,), 2, 1.0)
    out = torch.full((T, before + n + tail + 8), 9.0, dtype=dt, device=DEV)
    x = wide[:, before:before + n]
    ops.bias_act_rows(x, bias.to(DEV), out[:, before:before + n + tail], "gelu_tanh", tail=tail, ones=ones)
    want = P.gelu_tanh(x.double().cpu() + bias.double())
    assert rel_err(out[:, before:before + n], want) < tol(dt)
    assert bool((out[:, before + n:before + n + ones] == 1.0).all())
    assert bool((out[:, before + n + ones:before + n + tail] == 0.0).all())
    assert bool((out[:, :before] == 9.0).all()) and bool((out[:, before + n + tail:] == 9.0).all())
    rows = x.clone()
    ops.bias_act_rows(rows, None, rows, "silu")
    assert rel_err(rows, P.silu(x.double().cpu())) < tol(dt)


def test_add_row():
    x, b = _rand((9, 50), 3), _rand((50,), 4)
    got = x.to(DEV)
    ops.add_row(got, b.to(DEV))
    assert torch.equal(got.cpu(), x + b)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H, G, d, dv", [(5, 1, 7, 3), (6, 3, 16, 8), (4, 2, 32, 64)])
def test_unit_norms_and_blended_values_into_the_cache(dt, H, G, d, dv):
    """q and k over their root mean square a head (biases first), the values blended with rows
    given apart on their way into the pool, and the same values unblended into rows; a head of
    zeros stays zero, the eps is inside the root."""
    T, ps, eps = 6, 4, 1e-2
    width = (H + G) * d + G * dv
    src = _rand((T, width), 5, 0.4, dt)
    src[2, :d] = 0.0
    bias = _rand((width,), 6, 0.5)
    bias[:d] = 0.0
    first, lam = _rand((T, G * dv), 7, 1.0, dt), 0.625
    slots = [4, 5, 6, 7, 0, 1]
    ones = torch.ones(d, device=DEV)
    q = torch.zeros((T, H * d), dtype=dt, device=DEV)
    rows = torch.zeros((T, G * dv), dtype=dt, device=DEV)
    kp = torch.zeros((3, G * ps * d), dtype=dt, device=DEV)
    vp = torch.zeros((3, G * ps * dv), dtype=dt, device=DEV)
    b = bias.to(DEV)
    bq, bk, bv = (t.contiguous() for t in (b[:H * d], b[H * d:(H + G) * d], b[(H + G) * d:]))
    unit = dict(gain=ones, eps=eps, hd=d, per_head=True)
    ops.project_rows(src.to(DEV), _i32(range(T)), _i32(slots), ps, [
        ops.RowSegment(0, H * d, q, bias=bq, **unit),
        ops.RowSegment(H * d, G * d, kp, bias=bk, pool_heads=G, **unit),
        ops.RowSegment((H + G) * d, G * dv, vp, hd=dv, pool_heads=G, bias=bv,
                       blend=(first.to(DEV), lam)),
        ops.RowSegment((H + G) * d, G * dv, rows, hd=dv, bias=bv)])
    x = src.double() + bias.double()
    want_q = P.unit_rms(x[:, :H * d].view(T, H, d), eps)
    assert rel_err(q.view(T, H, d), want_q) < tol(dt)
    assert float(q[2, :d].abs().max()) == 0.0
    s = torch.tensor(slots)
    got_k = ops.masked_pool_rows(kp, G, ps, d)[s // ps, :, s % ps]
    assert rel_err(got_k, P.unit_rms(x[:, H * d:(H + G) * d].view(T, G, d), eps)) < tol(dt)
    v = x[:, (H + G) * d:].view(T, G, dv)
    assert rel_err(rows.view(T, G, dv), v) < tol(dt)
    got_v = ops.masked_pool_rows(vp, G, ps, dv)[s // ps, :, s % ps]
    assert rel_err(got_v, P.mixed_values(v, first.double().view(T, G, dv), lam)) < tol(dt)


# ------------------------------------------------------------------------------ attention
def _table(rel, far):
    """(the kernels' table, entry n: the bias of distance n) of [buckets, heads]."""
    from zinfer_amd.config.distance import bucket_of_distances
    rows = bucket_of_distances(rel.shape[0], far)
    return ops.distance_table(rel.float()[torch.tensor(rows)].T.contiguous()).to(DEV)


def _plain(q, k, v, H, G, scale, cap, window, keep, sink, rel, far):
    """q [T, H, KW]: the last T positions of a sequence of k [n, G, KW], v [n, G, VW]."""
    n, T = k.shape[0], q.shape[0]
    qq = torch.zeros((n, H, q.shape[2]), dtype=torch.float64)
    qq[n - T:] = q.double()
    m = {"scale": scale, "softcap": cap or None, "bias_max": far}
    s = P.attention_scores(qq, k.double(), m, rel)
    a = P.sink_softmax(s, P.seen(n, window or None, keep), sink)
    o = torch.matmul(a, v.double().repeat_interleave(H // G, dim=1).permute(1, 0, 2))
    return o.permute(1, 0, 2)[n - T:]


def _attend(pg, qs, q_lens, dt, H, scale, cap, window, keep, sink, table, mfma=False, n_splits=None,
            strided=False):
    T = sum(q_lens)
    q = torch.cat(qs).reshape(T, -1).to(DEV)
    out = torch.zeros((T, H * pg.VW + 64), dtype=dt, device=DEV)
    o = out[:, 32:32 + H * pg.VW] if strided else out[:, :H * pg.VW].contiguous()
    at, lens = _i32(_starts(q_lens)), _i32(pg.lens)
    if mfma:
        ops.masked_attention_mfma(q, None, None, pg.k_pool, pg.v_pool, sink.to(DEV), pg.table, at,
                                  lens, o, scale, cap, window, 0, H, pg.G, pg.KW, pg.VW, pg.ps,
                                  max(q_lens), max(pg.lens), n_splits=n_splits, keep=keep,
                                  dist_bias=table)
    else:
        seq = [s for s, n in enumerate(q_lens) for _ in range(n)]
        ops.masked_attention(q, None, None, pg.k_pool, pg.v_pool, sink.to(DEV), pg.table, at, lens,
                             _i32(seq), o, scale, cap, window, 0, H, pg.G, pg.KW, pg.VW, pg.ps,
                             max(pg.lens), keep, table)
    if strided:
        assert float(out[:, :32].abs().max()) == 0.0 and float(out[:, 32 + H * pg.VW:].abs().max()) == 0.0
    return o


CASES = [  # H, G, KW, VW, page, lens, q_lens, cap, window, keep, buckets, far
    (4, 2, 12, 20, 4, [60, 9, 1], [60, 9, 1], 4.0, 7, 3, 8, 20.0),
    (3, 3, 16, 16, 8, [170, 41], [23, 1], 0.0, 9, 0, 12, 40.0),
    (20, 1, 10, 6, 4, [37, 80], [37, 2], 8.0, 1, 1, 2, 3.0),
    (6, 2, 8, 12, 16, [150], [150], 2.5, 0, 0, 32, 100.0),
    (2, 1, 40, 24, 16, [300, 65, 33], [1, 1, 1], 30.0, 50, 70, 6, 500.0),
    (5, 5, 96, 96, 16, [200], [60], 18.0, 37, 16, 32, 60.0),
    (2, 2, 7, 3, 2, [30], [30], 1.5, 5, 9, 4, 11.0),
]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("case", CASES)
def test_attention_against_plain(dt, case):
    H, G, KW, VW, ps, lens, q_lens, cap, window, keep, buckets, far = case
    pg = Paged(lens, G, KW, VW, ps, dt, 3)
    scale = 1.3 / math.sqrt(KW)
    sink, rel = _rand((H,), 5, 1.5), _rand((buckets, H), 8, 1.5)
    table = _table(rel, far)
    qs = [_rand((n, H, KW), 20 + i, 1.0, dt) for i, n in enumerate(q_lens)]
    out = _attend(pg, qs, q_lens, dt, H, scale, cap, window, keep, sink, table)
    want = torch.cat([_plain(q, pg.k[s], pg.v[s], H, G, scale, cap, window, keep, sink, rel, far)
                      for s, q in enumerate(qs)])
    assert rel_err(out.view(-1, H, VW), want) < 2 * tol(dt)
    # into a slice of wider rows, and every sequence alone: the same bits
    assert torch.equal(_attend(pg, qs, q_lens, dt, H, scale, cap, window, keep, sink, table,
                               strided=True), out)
    at = 0
    for s, n in enumerate(q_lens):
        one = Paged([lens[s]], G, KW, VW, ps, dt, 77 + s, k=[pg.k[s]], v=[pg.v[s]])
        alone = _attend(one, [qs[s]], [n], dt, H, scale, cap, window, keep, sink, table)
        assert torch.equal(alone, out[at:at + n])
        at += n


MFMA_CASES = [  # H, G, KW, VW, page, lens, q_lens, cap, window, keep, buckets, far
    (6, 3, 96, 32, 16, [330, 90, 33], [330, 90, 33], 12.0, 50, 5, 32, 100.0),
    (8, 8, 64, 96, 16, [300, 41], [77, 2], 0.0, 100, 33, 8, 200.0),
    (32, 1, 128, 128, 16, [250], [150], 5.0, 40, 64, 32, 128.0),
    (12, 4, 128, 64, 32, [700], [700], 30.0, 0, 0, 32, 300.0),
    (4, 2, 32, 128, 8, [420], [200], 20.0, 31, 1, 16, 35.0),
    (10, 2, 96, 96, 16, [500, 600], [5, 130], 15.0, 257, 100, 2, 9.0),
    (3, 1, 32, 32, 16, [200], [200], 6.0, 1, 40, 32, 64.0),
]


@pytest.mark.parametrize("case", MFMA_CASES)
def test_mfma_attention_against_plain(case):
    """Prompt portions, keys in 1, 2 and 4 parts."""
    H, G, KW, VW, ps, lens, q_lens, cap, window, keep, buckets, far = case
    dt = torch.bfloat16
    pg = Paged(lens, G, KW, VW, ps, dt, 3)
    scale = 1.3 / math.sqrt(KW)
    sink, rel = _rand((H,), 5, 1.5), _rand((buckets, H), 8, 1.5)
    table = _table(rel, far)
    qs = [_rand((n, H, KW), 20 + i, 1.0, dt) for i, n in enumerate(q_lens)]
    want = torch.cat([_plain(q, pg.k[s], pg.v[s], H, G, scale, cap, window, keep, sink, rel, far)
                      for s, q in enumerate(qs)])
    for parts in (1, 2, 4, None):
        out = _attend(pg, qs, q_lens, dt, H, scale, cap, window, keep, sink, table, True, parts,
                      strided=parts == 2)
        assert rel_err(out.reshape(-1, H, VW), want) < 2 * tol(dt), parts


@pytest.mark.parametrize("case", MFMA_CASES)
def test_mfma_decode_steps_against_plain(case):
    """One token a sequence: contexts of many lengths over 1, 2 and 5 workgroups."""
    H, G, KW, VW, ps, _, _, cap, window, keep, buckets, far = case
    dt = torch.bfloat16
    lens = [1, 2, 31, 32, 33, 64, 65, 127, 333, 560]
    pg = Paged(lens, G, KW, VW, ps, dt, 4)
    scale = 1.3 / math.sqrt(KW)
    sink, rel = _rand((H,), 5, 1.5), _rand((buckets, H), 8, 1.5)
    table = _table(rel, far)
    qs = [_rand((1, H, KW), 20 + i, 1.0, dt) for i in range(len(lens))]
    want = torch.cat([_plain(q, pg.k[s], pg.v[s], H, G, scale, cap, window, keep, sink, rel, far)
                      for s, q in enumerate(qs)])
    for blocks in (1, 2, 5, None):
        out = _attend(pg, qs, [1] * len(lens), dt, H, scale, cap, window, keep, sink, table, True, blocks)
        assert rel_err(out.view(-1, H, VW), want) < 2 * tol(dt), blocks


def _planted(n, G, KW, VW, at, dt, seed):
    k, v = _rand((n, G, KW), seed, 0.3, dt), _rand((n, G, VW), seed + 1, 0.3, dt)
    k[at] = 0.0
    k[at, :, 0] = 30.0
    v[at] = 5.0
    return k, v


@pytest.mark.parametrize("form", ["float32", "bfloat16", "mfma"])
@pytest.mark.parametrize("T", [1, 37])
def test_a_loud_key_at_the_edges(form, T):
    """A key that takes nearly all the weight when it is seen: the oldest position a window
    holds and the one before it, the last kept position and the next one, position 0, far back
    without a window, at a page's border; for a token alone and in a prompt's portion."""
    dt = torch.float32 if form == "float32" else torch.bfloat16
    mfma = form == "mfma"
    H, G, KW, VW, ps, n = (4, 2, 64, 32, 16, 333) if mfma else (2, 1, 16, 8, 8, 333)
    q = torch.zeros((T, H, KW), dtype=dt)
    q[:, :, 0] = 1.0
    sink, rel = torch.zeros(H), _rand((8, H), 9, 0.2)
    table = _table(rel, 90.0)
    for name, at, window, keep, seen in (
            ("window_in", n - 50, 50, 7, True), ("window_out", n - 51, 50, 7, False),
            ("kept", 6, 50, 7, True), ("behind_the_kept", 7, 50, 7, False),
            ("first", 0, 50, 1, True), ("first_not_kept", 0, 50, 0, False),
            ("last_of_a_page_kept", 2 * ps - 1, 20, 2 * ps, True),
            ("next_page_not_kept", 2 * ps, 20, 2 * ps, False),
            ("last_of_32_kept", 31, 40, 32, True), ("after_32", 32, 40, 32, False),
            ("far", 3, 0, 0, True), ("own", n - 1, 1, 0, True), ("before_own", n - 2, 1, 0, False),
            ("page_border", n // ps * ps, 15, 3, True)):
        k, v = _planted(n, G, KW, VW, at, dt, 40)
        pg = Paged([n], G, KW, VW, ps, dt, 11, k=[k], v=[v])
        for splits in ((1, 3) if mfma else (None,)):
            out = _attend(pg, [q], [T], dt, H, 1.0, 0.0, window, keep, sink, table, mfma, splits)
            last = out.view(T, H, VW)[-1].float().cpu()
            if seen:
                assert float((last - 5.0).abs().max()) < 0.05, name
            else:
                assert float(last.abs().max()) < 1.5, name
            want = _plain(q, k, v, H, G, 1.0, 0.0, window, keep, sink, rel, 90.0)
            assert rel_err(out.view(T, H, VW), want) < 2 * tol(dt), name


@pytest.mark.parametrize("form", ["float32", "bfloat16", "mfma"])
@pytest.mark.parametrize("T", [1, 29])
def test_a_bias_that_points_at_a_distance(form, T):
    """Keys alike: a bias that is loud in one bucket sends the weight to the keys at that
    bucket's distances, each head to its own; kept positions count from their true places; the
    scale and the cap leave the bias alone."""
    dt = torch.float32 if form == "float32" else torch.bfloat16
    H, G, KW, VW, ps, n, B, far = 4, 1, 32, 32, 8, 150, 8, 64.0
    k = torch.zeros((n, G, KW), dtype=dt)
    v = _rand((n, G, VW), 51, 1.0, dt)
    rel = torch.zeros((B, H))
    for h, b in enumerate((0, 3, 5, 7)):                # distances 0, 3, 8..15, 32 and beyond
        rel[b, h] = 20.0
    q = torch.zeros((T, H, KW), dtype=dt)
    pg = Paged([n], G, KW, VW, ps, dt, 12, k=[k], v=[v])
    sink = torch.full((H,), -30.0)
    out = _attend(pg, [q], [T], dt, H, 1e-3, 0.5, 20, 3, sink, _table(rel, far), form == "mfma")
    last, vv = out.view(T, H, VW)[-1].double().cpu(), v[:, 0].double()
    i = n - 1
    for h, keys in enumerate(([i], [i - 3], list(range(i - 15, i - 7)), [0, 1, 2])):
        assert float((last[h] - vv[keys].mean(0)).abs().max()) < 2e-2, h
    want = _plain(q, k, v, H, G, 1e-3, 0.5, 20, 3, sink, rel, far)
    assert rel_err(out.view(T, H, VW), want) < 2 * tol(dt)


@pytest.mark.parametrize("form", ["float32", "mfma"])
@pytest.mark.parametrize("keep", [0, 3, 9])
def test_pages_between_the_kept_ones_and_the_window_are_not_touched(form, keep):
    """Table entries behind the kept positions' pages and before the window are -1 (the cache
    manager has taken those pages back): no kernel looks them up."""
    dt = torch.float32 if form == "float32" else torch.bfloat16
    H, G, KW, VW, ps, n, window = 4, 2, 32, 32, 4, 161, 9
    rel = _rand((8, H), 3)
    for T in (5, 1):
        pg = Paged([n], G, KW, VW, ps, dt, 13)
        q = _rand((T, H, KW), 1, 1.0, dt)
        args = ([q], [T], dt, H, 0.4, 3.0, window, keep, torch.zeros(H), _table(rel, 40.0), form == "mfma")
        full = _attend(pg, *args)
        first, kept = (n - T - window + 1) // ps, (keep + ps - 1) // ps
        assert first > kept + 8
        pg.table[0, kept:first] = -1
        assert torch.equal(_attend(pg, *args), full)


# ------------------------------------------------------------------------------ the recurrence
def test_rotation_table():
    pos = [0, 1, 63, 64, 999, 3000]
    dims, base = 12, 500.0
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    out = torch.empty((len(pos), dims // 2, 2), dtype=torch.float32, device=DEV)
    ops.rotation_table(_i32(pos), freq.float().to(DEV), 1.5, out)
    z = torch.zeros((len(pos), 1, dims), dtype=torch.float64)
    z[:, :, :dims // 2] = 1.0
    want = P.rotate(z, torch.tensor(pos), dims, base)[:, 0]
    got = out.double().cpu()
    assert float((got[..., 0] - 1.5 * want[:, :dims // 2]).abs().max()) < 1e-3
    assert float((got[..., 1] - 1.5 * want[:, dims // 2:]).abs().max()) < 1e-3
    assert float((got[:3, :, 0] - 1.5 * want[:3, :dims // 2]).abs().max()) < 2e-5


def _decay(g):
    d = torch.tensor(g, dtype=torch.float64)
    lg = torch.tensor([math.log2(x) if x > 0 else -1e30 for x in g], dtype=torch.float64)
    return torch.stack([d, lg]).float().to(DEV)


class Recurrence:
    """Sequences for the recurrence's kernels, and what the plain functions give for them."""

    def __init__(self, H, d, dv, g, lens, dt, silu, dims, base=100.0, starts=None, seed=0):
        self.H, self.d, self.dv, self.g, self.dt = H, d, dv, g, dt
        self.silu, self.dims, self.base = silu, dims, base
        self.k_scale = 0.37
        self.start = starts or [0] * len(lens)
        self.rows = [_rand((n, 2 * H * d + H * dv + 8), seed + 10 + i, 1.0, dt) for i, n in enumerate(lens)]

    def plain(self, i, state=None):
        H, d, dv = self.H, self.d, self.dv
        x = self.rows[i].double()
        q, k, v = x[:, :H * d].view(-1, H, d), x[:, H * d:2 * H * d].view(-1, H, d), \
            x[:, 2 * H * d:2 * H * d + H * dv].view(-1, H, dv)
        if self.silu:
            q, k, v = P.silu(q), P.silu(k), P.silu(v)
        if self.dims:
            p = self.start[i] + torch.arange(x.shape[0])
            q, k = P.rotate(q, p, self.dims, self.base), P.rotate(k, p, self.dims, self.base)
        o, S = P.decayed_sums(q, k * self.k_scale, v, self.g, state)
        return o.reshape(x.shape[0], H * dv), S

    def run(self, parts, state, slots, lists=False):
        """``parts``: (sequence, from, to) of this step."""
        H, d, dv = self.H, self.d, self.dv
        x = torch.cat([self.rows[i][a:b] for i, a, b in parts]).to(DEV)
        lens = [b - a for _, a, b in parts]
        pos = [self.start[i] + p for i, a, b in parts for p in range(a, b)]
        table = None
        if self.dims:
            freq = torch.tensor([self.base ** (-2.0 * j / self.dims) for j in range(self.dims // 2)],
                                dtype=torch.float64).float().to(DEV)
            table = torch.empty((len(pos), self.dims // 2, 2), dtype=torch.float32, device=DEV)
            ops.rotation_table(_i32(pos), freq, 1.0, table)
        packed = None
        if lists:
            made = ops.fixed_decay_chunk_lists(lens)
            packed = None if made is None else tuple(
                torch.from_numpy(t).to(DEV) if t.size else None for t in made)
        out = torch.full((len(pos), H * dv), float("nan"), dtype=torch.float32, device=DEV)
        ops.fixed_decay(x[:, :H * d], x[:, H * d:2 * H * d], x[:, 2 * H * d:2 * H * d + H * dv],
                        _decay(self.g), state, _i32([slots[i] for i, _, _ in parts]),
                        _i32(_starts(lens)), out, H, d, dv, silu=self.silu, table=table,
                        k_scale=self.k_scale, lists=packed)
        return out.cpu(), _starts(lens)

    def pool(self, n):
        return torch.zeros((n, ops.fixed_decay_state_size(self.H, self.d, self.dv) + 4),
                           dtype=torch.float32, device=DEV)


WALKS = [  # H, d, dv, decays, lens, silu, dims
    (3, 20, 12, [0.9, 1.0, 0.0], [21, 1, 40], False, 12),
    (2, 6, 10, [0.75, 0.99], [17, 2, 33], True, 0),
    (1, 1, 1, [0.5], [9, 5], True, 0),
    (4, 8, 16, [0.2, 0.5, 0.9, 0.999], [50], False, 8),
    (2, 64, 100, [0.95, 0.99], [19, 30], False, 16),
    (1, 256, 8, [0.9], [11], True, 0),
    (5, 7, 3, [0.3, 0.6, 0.9, 0.95, 1.0], [26, 26, 1, 4], False, 0),
    (2, 130, 70, [0.97, 0.5], [12, 3], False, 130),
]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("case", WALKS)
def test_fixed_decay_token_by_token(dt, case):
    """Sequences of unequal length in one launch, whole; then in two steps from the states the
    first left, in other slots' company, and one by one: the same bits, the plain matrices."""
    H, d, dv, g, lens, silu, dims = case
    r = Recurrence(H, d, dv, g, lens, dt, silu, dims)
    state = r.pool(len(lens) + 2)
    slots = list(range(len(lens), 0, -1))
    whole = [(i, 0, n) for i, n in enumerate(lens)]
    out, at = r.run(whole, state, slots)
    for i in range(len(lens)):
        want, S = r.plain(i)
        assert rel_err(out[at[i]:at[i + 1]], want) < 2e-5, i
        assert rel_err(ops.fixed_decay_state_matrix(state[slots[i]], H, d, dv), S) < 2e-5, i
    assert float(state[0].abs().max()) == 0.0 and float(state[:, -4:].abs().max()) == 0.0
    again = r.pool(len(lens) + 2)
    cuts = [max(1, n - 1 - i) if n > 1 else 1 for i, n in enumerate(lens)]
    o1, a1 = r.run([(i, 0, c) for i, c in enumerate(cuts)], again, slots)
    rest = [(i, c, lens[i]) for i, c in reversed(list(enumerate(cuts))) if c < lens[i]]
    o2, a2 = r.run(rest, again, slots)
    for i, c in enumerate(cuts):
        assert torch.equal(o1[a1[i]:a1[i + 1]], out[at[i]:at[i] + c])
    for j, (i, c, n) in enumerate(rest):
        assert torch.equal(o2[a2[j]:a2[j + 1]], out[at[i] + c:at[i + 1]])
    assert torch.equal(again, state)


CHUNKS = [  # H, d, dv, decays, lens, silu, dims
    (3, 64, 96, [0.99, 0.6, 1.0], [300, 1, 40, 128], False, 32),
    (2, 32, 64, [0.9, 0.998], [129, 33], True, 0),
    (2, 128, 160, [0.995, 0.0], [257, 32, 64], False, 128),
    (1, 96, 24, [0.9995], [700], True, 0),
    (2, 256, 40, [0.97, 0.999], [150, 90], False, 64),
    (3, 20, 12, [0.9, 1.0, 0.5], [140, 3], False, 12),
    (2, 7, 5, [0.95, 0.99], [200], True, 0),
    (1, 40, 130, [0.98], [131, 2, 2], False, 0),
    (2, 256, 32, [0.9, 0.99], [64], True, 0),
]


@pytest.mark.parametrize("case", CHUNKS)
def test_fixed_decay_in_chunks(case):
    """Long sequences in chunks beside short ones token by token, from states that an earlier
    step left: against the plain sums and against the walk from end to end."""
    H, d, dv, g, lens, silu, dims = case
    r = Recurrence(H, d, dv, g, lens, torch.bfloat16, silu, dims, starts=[3 * i for i in range(len(lens))])
    slots = list(range(len(lens)))
    whole = [(i, 0, n) for i, n in enumerate(lens)]
    walked, chunked = r.pool(len(lens)), r.pool(len(lens))
    out, at = r.run(whole, walked, slots)
    got, _ = r.run(whole, chunked, slots, lists=True)
    for i in range(len(lens)):
        want, S = r.plain(i)
        a, b = at[i], at[i + 1]
        assert rel_err(out[a:b], want) < 2e-5, i
        # (silu's rounding of a value to bfloat16 is an activation's)
        assert rel_err(got[a:b], want) < (4e-3 if silu else 6e-5), (i, rel_err(got[a:b], want))
        m = ops.fixed_decay_state_matrix(chunked[slots[i]], H, d, dv)
        assert rel_err(m, S) < (4e-3 if silu else 6e-5), i
    # in two steps, the second from the first one's states
    if max(lens) > 70:
        two = r.pool(len(lens))
        cut = [n // 2 + 1 for n in lens]
        o1, a1 = r.run([(i, 0, c) for i, c in enumerate(cut)], two, slots, lists=True)
        tails = [(i, c, n) for i, (c, n) in enumerate(zip(cut, lens)) if c < n]
        o2, a2 = r.run(tails, two, slots, lists=True)
        for j, (i, c, n) in enumerate(tails):
            assert rel_err(o2[a2[j]:a2[j + 1]], r.plain(i)[0][c:]) < (4e-3 if silu else 6e-5)


@pytest.mark.parametrize("way", ["walk", "chunks", "single"])
def test_a_token_far_back(way):
    """A loud key 600 tokens back: a head without decay returns its value, a head with one has
    lost it; in a prompt either way and with single tokens behind it."""
    H, d, dv, n = 2, 32, 32, 600
    r = Recurrence(H, d, dv, [1.0, 0.9], [n], torch.bfloat16, False, 0)
    x = r.rows[0]
    x[:, H * d:2 * H * d] = 0.0                         # no keys but the first
    x[0, H * d:2 * H * d] = 1.0
    x[:, :H * d] = 0.0
    x[-1, :H * d] = 1.0
    state = r.pool(1)
    if way == "single":
        r.run([(0, 0, n - 9)], state, [0], lists=True)
        for p in range(n - 9, n):
            out, _ = r.run([(0, p, p + 1)], state, [0])
    else:
        out, _ = r.run([(0, 0, n)], state, [0], lists=way == "chunks")
    last = out[-1].double().view(H, dv)
    v = x[0, 2 * H * d:2 * H * d + H * dv].double().view(H, dv)
    assert rel_err(last[0], v[0] * d * r.k_scale) < 1e-4
    assert float(last[1].abs().max()) < 1e-20


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H, dv, heads, gate", [(3, 12, 3, "silu"), (4, 10, 1, "sigmoid"),
                                                 (2, 64, 2, "silu"), (8, 128, 1, "sigmoid"),
                                                 (5, 3, 1, "silu"), (7, 101, 1, "sigmoid")])
def test_norm_and_gate(dt, H, dv, heads, gate):
    """A norm a head without a gain and one over the whole row with a gain, either gate, gate and
    output as slices of wider rows."""
    T, eps = 9, 1e-3
    o = _rand((T, H * dv), 1, 2.0)
    wide = _rand((T, H * dv + 24), 2, 1.5, dt).to(DEV)
    g = wide[:, 8:8 + H * dv]
    gain = 1 + _rand((H * dv,), 3, 0.3) if heads == 1 else None
    out = torch.full((T, H * dv + 16), 5.0, dtype=dt, device=DEV)
    ops.head_norm_gate(o.to(DEV), None if gain is None else gain.to(DEV), g, out[:, 8:8 + H * dv],
                       heads, eps, gate_kind=gate)
    n = P.unit_rms(o.view(T, H, dv), eps).reshape(T, -1) if gain is None else P.rms_norm(o, gain, eps)
    z = g.double().cpu()
    want = n * (P.silu(z) if gate == "silu" else P.sigmoid(z))
    assert rel_err(out[:, 8:8 + H * dv], want) < tol(dt)
    assert bool((out[:, :8] == 5.0).all()) and bool((out[:, 8 + H * dv:] == 5.0).all())
