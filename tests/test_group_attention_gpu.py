"""GPU: grouped attention with windows and sinks, kernel by kernel against the double-precision oracle: keys
that decide the answer just inside and just outside the window and at page borders, head counts and sizes off
the tiles, splits, listed rows, tiles of portions."""
import numpy as np
import pytest

from oracle import layer_stack as ls

pytestmark = pytest.mark.gpu


def t(a, gpu, dtype=None):
    import torch

    x = torch.from_numpy(np.ascontiguousarray(a)).to(gpu)
    return x if dtype is None else x.to(dtype)


def host(x):
    import torch

    return x.to(torch.float64).cpu().numpy()


def attend(q, k, v, scale, lo, n, sink):
    """One row: q [heads, d], k and v [keys, heads, d]; sees keys lo .. n - 1."""
    s = np.einsum("hd,jhd->hj", q, k[lo:n]) * scale
    p = ls.softmax_with_sink(s, np.ones(s.shape, bool), sink)
    return np.einsum("hj,jhd->hd", p, v[lo:n])


class Case:
    """Requests on scattered pages; `spikes` maps (request, key) to a score every query of the request gives it."""

    def __init__(self, rng, gpu, dtype, heads, kv, dim, ps, lens, spikes=()):
        self.heads, self.kv, self.dim, self.ps, self.lens = heads, kv, dim, ps, lens
        need = [-(-n // ps) for n in lens]
        perm = rng.permutation(sum(need) + 3)
        begin = np.concatenate([[0], np.cumsum(need)])
        self.pages, self.begin = t(perm.astype(np.int32), gpu), begin[:-1].astype(np.int32)
        pool = rng.standard_normal(((sum(need) + 3) * ps, kv, 2, dim))
        axis = np.zeros(dim)
        axis[dim // 3] = 1.0
        self.axis = axis
        for r, n in enumerate(lens):
            for j in range(n):
                slot = perm[begin[r] + j // ps] * ps + j % ps
                pool[slot, :, 0, dim // 3] = spikes[(r, j)] if (r, j) in dict(spikes) else 0.0
                if (r, j) in dict(spikes):
                    pool[slot, :, 1] = 2.0 + 0.25 * np.arange(kv)[:, None]
        self.pool = t(pool.reshape(-1, kv, 2 * dim), gpu, dtype)
        hp = host(self.pool).reshape(-1, kv, 2, dim)
        self.kvs = [np.concatenate([hp[p * ps:(p + 1) * ps] for p in perm[begin[r]:begin[r + 1]]]) for r in range(len(lens))]

    def queries(self, rng, rows, gpu, dtype):
        q = rng.standard_normal((rows, self.heads, self.dim))
        q[:, :, self.dim // 3] = 1.0
        return t(q, gpu, dtype)

    def want(self, r, q, n, scale, window, sink, out_scale):
        src = np.arange(self.heads) // (self.heads // self.kv)
        kv = self.kvs[r][:, src]
        return attend(q, kv[:, :, 0], kv[:, :, 1], scale, max(0, n - window) if window else 0, n, sink) * out_scale


SHAPES = [(6, 1, 96, 64), (8, 2, 32, 16), (5, 5, 64, 16), (40, 1, 128, 48), (3, 1, 256, 16), (14, 2, 192, 32)]


@pytest.mark.parametrize("heads,kv,dim,ps", SHAPES)
@pytest.mark.parametrize("window,sink", [(0, 0.0), (37, 1.0), (64, 1.0), (1, 1.0), (33, 0.0), (300, 2.5)])
@pytest.mark.parametrize("kind", ["bf16", "bf16_plain", "f32_plain"])
def test_decode_rows(gpu, heads, kv, dim, ps, window, sink, kind):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(heads + window)
    dt = torch.float32 if kind == "f32_plain" else torch.bfloat16
    lens = [1, 2, 31, 32, 33, 64, 65, 290, 700]
    # the key just outside each window would win everything, the one just inside takes a good share
    spikes = {(r, n - window - 1): 60.0 for r, n in enumerate(lens) if window and n > window}
    spikes.update({(r, n - window): 4.0 for r, n in enumerate(lens) if window and n >= window})
    c = Case(rng, gpu, dt, heads, kv, dim, ps, lens, spikes)
    q = c.queries(rng, len(lens), gpu, dt)
    scale = 1.3 / np.sqrt(dim)
    ld_o = -(-heads * dim // 128) * 128
    form = "rows" if kind == "bf16" else "plain"
    for bound in (max(lens), 1024):
        o = host(ops.group_attn(form, q, c.pool, c.pages, t(c.begin, gpu), t(np.array(lens, np.int32), gpu), ps, scale, window, sink, 0.75,
                                ld_o, max_kv_len=bound))
        qh = host(q)
        for r, n in enumerate(lens):
            want = c.want(r, qh[r], n, scale, window, sink, 0.75)
            assert np.abs(o[r, :heads * dim].reshape(heads, dim) - want).max() < (2e-5 if kind == "f32_plain" else 1.5e-2), (r, n)
        assert (o[:, heads * dim:] == 3.0).all()
    if form == "rows":   # some rows only, in another order: the others are not touched
        pick = np.array([7, 2, 8], np.int32)
        o = host(ops.group_attn(form, q, c.pool, c.pages, t(c.begin, gpu), t(np.array(lens, np.int32), gpu), ps, scale, window, sink, 0.75,
                                rows=t(pick, gpu)))
        for r in range(len(lens)):
            if r in pick:
                assert np.abs(o[r].reshape(heads, dim) - c.want(r, qh[r], lens[r], scale, window, sink, 0.75)).max() < 1.5e-2
            else:
                assert (o[r] == 3.0).all()


@pytest.mark.parametrize("heads,kv,dim,ps", SHAPES)
@pytest.mark.parametrize("window,sink", [(0, 1.0), (37, 1.0), (64, 0.0), (1, 1.0), (130, 1.0)])
@pytest.mark.parametrize("half", [0, 1])
def test_portions_in_tiles(gpu, heads, kv, dim, ps, window, sink, half):
    """Two requests' portions: a whole prompt, and the last tokens of a longer one; spikes at the windows' edges of
    some rows."""
    import torch
    from pie_amd import ops

    if dim > 128 and not half:
        pytest.skip("heads this wide take half tiles only")
    rng = np.random.default_rng(heads + window)
    dt = torch.bfloat16
    total, start = [150, 333], [0, 200]
    spikes = {(0, 40): 5.0, (1, 250): 5.0, (1, 150): 5.0, (0, 0): 4.0}
    c = Case(rng, gpu, dt, heads, kv, dim, ps, total, spikes)
    rows = [(r, j) for r in range(2) for j in range(start[r], total[r])]
    q = c.queries(rng, len(rows), gpu, dt)
    lens = np.array([j + 1 for _, j in rows], np.int32)
    per = ops.group_attn_tile_rows(heads, kv, half)
    tiles, first = [], 0
    for r in range(2):
        n = total[r] - start[r]
        tiles += [(first + i, min(per, n - i)) for i in range(0, n, per)]
        first += n
    scale = 1.3 / np.sqrt(dim)
    o = host(ops.group_attn("tiles", q, c.pool, c.pages, t(np.array([c.begin[r] for r, _ in rows], np.int32), gpu), t(lens, gpu), ps, scale, window,
                            sink, 1.25, tiles=t(np.array(tiles[::-1], np.int32), gpu), half=half))
    qh = host(q)
    near = {e + d for _, e in spikes for d in ([0, window - 1, window, 1] if window else [0])}
    for i, (r, j) in enumerate(rows):
        if i % 13 == 0 or j in near or j == total[r] - 1:
            want = c.want(r, qh[i], j + 1, scale, window, sink, 1.25)
            assert np.abs(o[i].reshape(heads, dim) - want).max() < 2.5e-2, (r, j)


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("heads,kv,dim,rot,biased,normed,own_values", [
    (6, 1, 96, 96, True, True, False), (3, 3, 40, 24, True, True, False), (4, 2, 64, 32, False, True, True), (2, 1, 300, 100, True, False, False),
    (5, 1, 24, 0, False, False, False), (2, 2, 256, 128, True, True, True)])
def test_query_and_key_preparation(gpu, bf, heads, kv, dim, rot, biased, normed, own_values):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(dim)
    dt = torch.bfloat16 if bf else torch.float32
    N, dimp, q_off = 37, -(-dim // 32) * 32, 8
    k_off = q_off + -(-heads * dim // 8) * 8
    v_off = k_off + -(-kv * dim // 8) * 8
    ld = -(-(v_off + kv * dim) // 16) * 16
    fused = t(rng.standard_normal((N, ld)), gpu, dt)
    qb, kb = rng.standard_normal(heads * dim).astype(np.float32), rng.standard_normal(kv * dim).astype(np.float32)
    qn, kn = (rng.uniform(0.5, 1.5, dim).astype(np.float32) for _ in range(2))
    pos = rng.integers(0, 5000, N).astype(np.int32)
    slots = rng.permutation(64)[:N].astype(np.int64)
    slots[5] = -1   # (a row without a place in the cache)
    spec = dict(dims=rot, base=10000.0)
    table = ops.rotary_table(t(pos, gpu), t(ls.rotation_frequencies(spec)[0], gpu), 1.0) if rot else None
    pool = t(np.full((64, kv, 2 * dimp), 7.0), gpu, dt)
    opt = lambda on, a: t(a, gpu) if on else None
    q = host(ops.group_attn_prep(fused, q_off, k_off, v_off if own_values else -1, opt(biased, qb), opt(biased, kb), opt(normed, qn), opt(normed, kn),
                                 table, rot, t(slots, gpu), pool, heads, kv, dim, dimp, 1e-5))
    f, p = host(fused), host(pool)
    rq = f[:, q_off:q_off + heads * dim].reshape(N, heads, dim) + (qb.reshape(heads, dim) if biased else 0)
    rk = f[:, k_off:k_off + kv * dim].reshape(N, kv, dim) + (kb.reshape(kv, dim) if biased else 0)
    turn = lambda x: ls.rotate_halves(x, pos, spec) if rot else x
    wq, wk = turn(ls.rms_norm(rq, qn, 1e-5) if normed else rq), turn(ls.rms_norm(rk, kn, 1e-5) if normed else rk)
    wv = f[:, v_off:v_off + kv * dim].reshape(N, kv, dim) if own_values else rk
    tol = 2.5e-2 if bf else 2e-5
    assert np.abs(q[..., :dim] - wq).max() < tol and (q[..., dim:] == 0).all()
    for n in range(N):
        if slots[n] < 0:
            continue
        row = p[slots[n]]
        assert np.abs(row[:, :dim] - wk[n]).max() < tol and np.abs(row[:, dimp:dimp + dim] - wv[n]).max() < tol
        assert (row[:, dim:dimp] == 0).all() and (row[:, dimp + dim:] == 0).all()
    untouched = np.setdiff1d(np.arange(64), slots)
    assert (p[untouched] == 7.0).all()
