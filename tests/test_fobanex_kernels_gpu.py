"""GPU: the kernels of layers whose sublayers share a norm — joined residuals, gated products with biases and clamps,
expert groups, norms over whole projections, gates on attention outputs — against double-precision statements."""
import numpy as np
import pytest

from oracle import layer_stack as ls
from test_group_attention_gpu import Case, host, t

pytestmark = pytest.mark.gpu


def rule(g, u, limit=np.inf, alpha=1.0, shift=0.0):
    g, u = np.minimum(g, limit), np.clip(u, -limit, limit)
    return g / (1.0 + np.exp(-alpha * g)) * (u + shift)


@pytest.mark.parametrize("M", [1, 2, 4, 7, 16, 40, 64, 130])
@pytest.mark.parametrize("form", ["gemv", "skinny", "tiled", "splitk", "f32"])
@pytest.mark.parametrize("kind", ["biased", "clamped", "both"])
def test_gated_products(gpu, M, form, kind):
    import torch
    from pie_amd import ops

    if form == "gemv" and M > 4:
        pytest.skip("up to four rows")
    rng = np.random.default_rng(M)
    K, N = 1024, 272
    act = t(rng.standard_normal((M, K)), gpu, torch.float32 if form == "f32" else torch.bfloat16)
    w = t(rng.standard_normal((N, K)) * 2 / np.sqrt(K), gpu, torch.bfloat16)
    bias = rng.standard_normal(N).astype(np.float32)
    dev = t(bias, gpu)
    par = dict(limit=1.25, alpha=1.702, shift=1.0) if kind != "biased" else {}
    got = host(ops.linear_glu(form, act, w, ops.glu(dev if kind != "clamped" else None, **par)))
    x = host(act) @ host(w).T + (bias if kind != "clamped" else 0.0)
    want = rule(x[:, 0::2], x[:, 1::2], **par)
    err = np.abs(got - want) / (1.0 + np.abs(want))
    assert err.max() < (1e-4 if form == "f32" else 2.5e-2) and err.mean() < (1e-5 if form == "f32" else 3e-3)


@pytest.mark.parametrize("experts,top,groups,keep", [(9, 3, 3, 2), (64, 8, 8, 3), (12, 4, 1, 1), (6, 6, 2, 2), (1, 1, 1, 1), (200, 17, 5, 1),
                                                     (512, 40, 64, 20)])
@pytest.mark.parametrize("T", [1, 5, 16, 17, 100])
def test_routes_are_chosen_inside_the_kept_groups(gpu, experts, top, groups, keep, T):
    from pie_amd import ops

    rng = np.random.default_rng(experts + T)
    ld = -(-experts // 16) * 16
    z = rng.standard_normal((T, ld)).astype(np.float32) * 2.0
    z[:, experts:] = 50.0   # (columns that pad the product belong to no expert)
    idx, weight, offsets, token, pos = (host(x) for x in ops.moe_route_groups(t(z, gpu), experts, top, groups, keep, 2.5))
    idx, offsets, token, pos = (x.astype(int) for x in (idx, offsets, token, pos))
    want = ls.route(z[:, :experts].astype(np.float64), dict(experts=experts, top=top, scale=2.5, groups=dict(count=groups, keep=keep)))
    got = np.zeros_like(want)
    np.put_along_axis(got, idx, weight, axis=1)
    assert np.allclose(got, want, rtol=1e-5, atol=1e-7) and all(len(set(r)) == top for r in idx)
    assert offsets[0] == 0 and offsets[-1] == T * top and np.array_equal(np.diff(offsets), np.bincount(idx.ravel(), minlength=experts))
    assert sorted(pos.ravel()) == list(range(T * top))
    for n in range(T):
        for k in range(top):
            assert token[pos[n, k]] == n and offsets[idx[n, k]] <= pos[n, k] < offsets[idx[n, k] + 1]


def test_equal_probabilities_go_to_the_lowest_group_and_expert(gpu):
    from pie_amd import ops

    z = np.zeros((3, 16), np.float32)
    z[1, [3, 7, 11]] = 2.0
    z[2, 15] = 1.0
    idx, weight, *_ = (host(x) for x in ops.moe_route_groups(t(z, gpu), 16, 3, 4, 2, 1.0))
    assert idx[0].tolist() == [0, 1, 2] and sorted(idx[1].tolist()) == [0, 3, 7] and idx[2].tolist() == [15, 0, 1]


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("T,E,top,K,N", [(1, 5, 2, 128, 64), (9, 5, 2, 256, 96), (120, 3, 2, 128, 160), (70, 17, 4, 384, 32)])
def test_grouped_products(gpu, bf, T, E, top, K, N):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(T)
    dt = torch.bfloat16 if bf else torch.float32
    act, w = t(rng.standard_normal((T, K)), gpu, dt), t(rng.standard_normal((E, N, K)) * 2 / np.sqrt(K), gpu, torch.bfloat16)
    z = rng.standard_normal((T, 32)).astype(np.float32)
    idx, _, offsets, token, pos = ops.moe_route_groups(t(z, gpu), E, top, 1, 1, 1.0)
    plain = host(ops.moe_grouped_glu(act, token, offsets, w, T * top, None))
    gated = host(ops.moe_grouped_glu(act, token, offsets, w, T * top, ops.glu(None, 0.75, 1.702, 1.0)))
    a, wh, idx, pos = host(act), host(w), host(idx).astype(int), host(pos).astype(int)
    for n in range(T):
        for k in range(top):
            x = wh[idx[n, k]] @ a[n]
            assert np.abs(plain[pos[n, k]] - x).max() < (5e-2 if bf else 1e-4)
            assert np.abs(gated[pos[n, k]] - rule(x[0::2], x[1::2], 0.75, 1.702, 1.0)).max() < (5e-2 if bf else 1e-4)


@pytest.mark.parametrize("T,E,top,K,N", [(1, 5, 2, 128, 64), (1, 1, 1, 64, 16), (9, 5, 2, 256, 96), (120, 3, 2, 128, 160), (70, 17, 4, 384, 32),
                                         (700, 2, 1, 192, 272), (300, 130, 8, 64, 128), (257, 70, 1, 128, 48)])
@pytest.mark.parametrize("block_rows", [0, 64, 128, 256])
def test_grouped_products_in_blocks_of_routes(gpu, T, E, top, K, N, block_rows):
    """Blocks of one expert's routes, over row-major and tile-major weights; some experts without routes, some with many
    blocks, more experts than a wave has lanes."""
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(T + E)
    act, w = t(rng.standard_normal((T, K)), gpu, torch.bfloat16), t(rng.standard_normal((E, N, K)) * 2 / np.sqrt(K), gpu, torch.bfloat16)
    ld = -(-E // 16) * 16
    z = (rng.standard_normal((T, ld)) + (np.arange(ld) % 3 == 1) * 2.0).astype(np.float32)   # (an uneven choice)
    idx, _, offsets, token, pos = ops.moe_route_groups(t(z, gpu), E, top, 1, 1, 1.0)
    wt = ops.repack_mfma_tiles(ops.WeightView("bf16", w.reshape(E * N, K), None, 0, E * N, K)).data.reshape(E, N, K)
    glu = ops.glu(None, 0.75, 1.702, 1.0)
    a, wh, idx, pos = host(act), host(w), host(idx).astype(int), host(pos).astype(int)
    want = np.zeros((T * top, N), np.float32)
    for e in range(E):
        n, k = np.nonzero(idx == e)
        want[pos[n, k]] = a[n] @ wh[e].T
    sorted_act = act[torch.as_tensor(host(token).astype(np.int64), device=gpu)].contiguous()
    for weights, tiled in ((w, False), (wt, True)):
        plain = host(ops.moe_grouped_glu(act, token, offsets, weights, T * top, None, block_rows, tiled))
        assert np.abs(plain - want).max() < 5e-2
        assert np.array_equal(plain, host(ops.moe_grouped_glu(sorted_act, None, offsets, weights, T * top, None, block_rows, tiled)))
        gated = host(ops.moe_grouped_glu(act, token, offsets, weights, T * top, glu, block_rows, tiled))
        assert np.abs(gated - rule(want[:, 0::2], want[:, 1::2], 0.75, 1.702, 1.0)).max() < 5e-2


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("width,ld,rows,top", [(96, 128, 5, 3), (75, 128, 9, 1), (2048, 2048, 3, 8), (4098, 4224, 2, 5), (9000, 9088, 2, 2), (256, 256, 600, 4),
                                               (4096, 4096, 3, 11), (4104, 4224, 520, 9)])
def test_residual_join(gpu, bf, width, ld, rows, top):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(width)
    dt, eps = torch.bfloat16 if bf else torch.float32, 1e-3
    y, y2, ry = (t(rng.standard_normal((n, ld)), gpu, dt) for n in (rows, rows, rows * top))
    pos = rng.permutation(rows * top).reshape(rows, top).astype(np.int32)
    weight, add, nw = (rng.uniform(0.5, 1.5, s).astype(np.float32) for s in ((rows, top), width, width))
    table, toks = t(rng.standard_normal((11, width)), gpu, torch.bfloat16), np.array([i % 13 for i in range(rows)], np.int32)
    routes = (ry, t(pos, gpu), t(weight, gpu))
    mix = np.einsum("nk,nkw->nw", weight, host(ry)[pos])[:, :width]
    emb = host(table)[np.where(toks < 11, toks, 0)]
    for use in ("all", "start", "dense", "mixture"):
        x0 = rng.standard_normal((rows, ld)).astype(np.float32)
        x = t(x0, gpu)
        kw, want = {}, np.zeros((rows, width))
        if use in ("all", "dense", "mixture"):
            kw["y"] = y
            want = want + x0[:, :width] + host(y)[:, :width]
        if use in ("all", "dense"):
            kw.update(y2=y2, add=t(add, gpu))
            want = want + host(y2)[:, :width] + add
        if use in ("all", "mixture"):
            kw["routes"] = routes
            want = want + mix
        if use in ("all", "start"):
            kw.update(tokens=t(toks, gpu), table=table, table_scale=2.5)
            want = want + 2.5 * emb
        xa = host(ops.residual_join(x, width, eps, dt, read_x=use != "start", next_weight=None if use == "dense" else t(nw, gpu), **kw))
        assert np.abs(host(x)[:, :width] - want).max() < 2e-5 and np.array_equal(host(x)[:, width:], x0[:, width:])
        out = want if use == "dense" else ls.rms_norm(want, nw, eps)
        assert np.abs(xa[:, :width] - out).max() < (4e-2 if bf else 2e-5) and (xa[:, width:] == 0).all()


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("heads,kv,dim,vdim,rot,adjacent,normed,own_values", [
    (6, 2, 64, 64, 16, True, True, True), (3, 3, 40, 24, 40, True, True, True), (4, 2, 32, 32, 20, True, False, False), (2, 1, 300, 120, 100, True, True, True),
    (5, 1, 18, 30, 18, True, True, True), (2, 2, 24, 24, 12, False, True, False), (5, 1, 24, 24, 0, True, True, False), (40, 8, 128, 128, 64, True, True, True),
    (64, 2, 256, 256, 128, True, True, False)])
def test_preparation_with_norms_over_whole_projections(gpu, bf, heads, kv, dim, vdim, rot, adjacent, normed, own_values):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(dim + heads)
    dt = torch.bfloat16 if bf else torch.float32
    N, dimp, q_off = 37, -(-max(dim, vdim) // 32) * 32, 8
    k_off = q_off + -(-heads * dim // 8) * 8
    v_off = k_off + -(-kv * dim // 8) * 8
    ld = -(-(v_off + kv * vdim) // 16) * 16
    fused = rng.standard_normal((N, ld))
    fused[3] *= 20.0   # (a long row is normed as a whole)
    fused = t(fused, gpu, dt)
    qn, kn = (rng.uniform(0.5, 1.5, n * dim).astype(np.float32) for n in (heads, kv))
    pos, slots = rng.integers(0, 5000, N).astype(np.int32), rng.permutation(64)[:N].astype(np.int64)
    slots[5] = -1   # (a row without a place in the cache)
    spec = dict(dims=rot, base=10000.0)
    table = ops.rotary_table(t(pos, gpu), t(ls.rotation_frequencies(spec)[0], gpu), 1.0) if rot else None
    pool = t(np.full((64, kv, 2 * dimp), 7.0), gpu, dt)
    opt = lambda a: t(a, gpu) if normed else None
    q = host(ops.group_attn_prep_joint(fused, q_off, k_off, v_off if own_values else -1, opt(qn), opt(kn), table, rot, adjacent, t(slots, gpu), pool, heads,
                                       kv, dim, vdim, dimp, 1e-5))
    f, p = host(fused), host(pool)
    rq, rk = f[:, q_off:q_off + heads * dim], f[:, k_off:k_off + kv * dim]
    rv = f[:, v_off:v_off + kv * vdim] if own_values else rk
    if normed:
        rq, rk = ls.rms_norm(rq, qn, 1e-5), ls.rms_norm(rk, kn, 1e-5)
    turn = lambda x: (ls.rotate_pairs if adjacent else ls.rotate_halves)(x, pos, spec) if rot else x
    wq, wk, wv = turn(rq.reshape(N, heads, dim)), turn(rk.reshape(N, kv, dim)), rv.reshape(N, kv, vdim)
    tol = lambda want: (1e-2 if bf else 1e-5) * max(1.0, np.abs(want).max())
    assert np.abs(q[..., :dim] - wq).max() < tol(wq) and (q[..., dim:] == 0).all()
    for n in range(N):
        if slots[n] < 0:
            continue
        row = p[slots[n]]
        assert np.abs(row[:, :dim] - wk[n]).max() < tol(wk[n]) and np.abs(row[:, dimp:dimp + vdim] - wv[n]).max() < tol(wv[n])
        assert (row[:, dim:dimp] == 0).all() and (row[:, dimp + vdim:] == 0).all()
    assert (p[np.setdiff1d(np.arange(64), slots)] == 7.0).all()


@pytest.mark.parametrize("heads,kv,dim,ps", [(6, 2, 64, 16), (5, 5, 96, 64), (40, 1, 128, 16), (4, 2, 192, 32)])
@pytest.mark.parametrize("form", ["rows", "splits", "tiles", "plain", "f32"])
def test_gates_on_grouped_attention(gpu, heads, kv, dim, ps, form):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(heads)
    dt = torch.float32 if form == "f32" else torch.bfloat16
    lens = [1, 33, 64, 700] if form == "splits" else [90, 33]
    c = Case(rng, gpu, dt, heads, kv, dim, ps, lens)
    rows = [(0, j) for j in range(90)] if form == "tiles" else list(enumerate(n - 1 for n in lens))
    q = c.queries(rng, len(rows), gpu, dt)
    ld_gate, off = heads * dim + 24, 8
    fused = t(rng.standard_normal((len(rows), ld_gate)) * 3, gpu, dt)
    gate = fused[:, off:]   # (columns of wider rows)
    table = np.array([j + 1 for _, j in rows], np.int32)
    begin = np.array([c.begin[r] for r, _ in rows], np.int32)
    kw = {}
    if form == "tiles":
        per = ops.group_attn_tile_rows(heads, kv, 1)
        kw = dict(tiles=t(np.array([(i, min(per, 90 - i)) for i in range(0, 90, per)], np.int32), gpu), half=1)
    o = host(ops.group_attn({"splits": "rows", "f32": "plain"}.get(form, form), q, c.pool, c.pages, t(begin, gpu), t(table, gpu), ps, dim ** -0.5, gate=gate, **kw))
    g = ls.sigmoid(host(fused)[:, off:off + heads * dim]).reshape(len(rows), heads, dim)
    qh = host(q)
    for i, (r, j) in enumerate(rows):
        want = c.want(r, qh[i], j + 1, dim ** -0.5, 0, 0.0, 1.0) * g[i]
        assert np.abs(o[i].reshape(heads, dim) - want).max() < (2e-5 if form == "f32" else 2.5e-2), (r, j)


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("M,heads,C,K", [(1, 3, 32, 64), (20, 5, 64, 128), (70, 2, 96, 32)])
def test_gates_on_per_head_products(gpu, bf, M, heads, C, K):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(M)
    dt = torch.bfloat16 if bf else torch.float32
    act, gate = t(rng.standard_normal((M, heads, K)), gpu, dt), t(rng.standard_normal((M, heads * C + 8)) * 2, gpu, dt)
    w = t(rng.standard_normal((heads, C, K)) / np.sqrt(K), gpu, torch.bfloat16)
    got = host(ops.head_linear(act, w, gate=gate))
    want = np.einsum("mhk,hck->mhc", host(act), host(w)) * ls.sigmoid(host(gate)[:, :heads * C]).reshape(M, heads, C)
    assert np.abs(got - want).max() < (3e-2 if bf else 1e-5)


def test_gates_on_expanded_latent_attention(gpu):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(3)
    T, heads, dimp, rotp, vdp = 150, 3, 64, 32, 96
    bf = torch.bfloat16
    q, kv, rot = (t(rng.standard_normal(s), gpu, bf) for s in ((T, heads, dimp + rotp), (T, heads, dimp + vdp), (T, rotp)))
    gate = t(rng.standard_normal((T, heads * vdp + 16)) * 2, gpu, bf)
    lens = t(np.arange(1, T + 1, dtype=np.int32), gpu)
    scale = 0.1
    plain, gated = (host(ops.latent_attn_prefill(q, kv, rot, None, 0, lens, dimp, scale, gate=g)) for g in (None, gate))
    qh, kvh, rh = host(q), host(kv), host(rot)
    s = (np.einsum("ihd,jhd->hij", qh[..., :dimp], kvh[..., :dimp]) + np.einsum("ihd,jd->hij", qh[..., dimp:], rh)) * scale
    want = ls.causal_softmax_attention(s, kvh[..., dimp:]).reshape(T, -1)
    assert np.abs(plain - want).max() < 3e-2
    assert np.abs(gated - want * ls.sigmoid(host(gate)[:, :heads * vdp])).max() < 3e-2


def test_bad_arguments_are_refused(gpu):
    import torch
    from pie_amd import ops
    from pie_amd.ops import KernelError

    z = torch.zeros((2, 16), device=gpu)
    for experts, top, groups, keep in [(12, 4, 5, 2), (12, 4, 3, 4), (12, 5, 3, 1), (12, 4, 3, 0), (17, 1, 1, 1)]:
        with pytest.raises(KernelError):
            ops.moe_route_groups(z, experts, top, groups, keep, 1.0)
    x = torch.zeros((1, 64), dtype=torch.bfloat16, device=gpu)
    with pytest.raises(KernelError):
        ops.linear_glu("skinny", torch.zeros((1, 128), dtype=torch.bfloat16, device=gpu), torch.zeros((32, 128), dtype=torch.bfloat16, device=gpu), ops.glu(limit=-1.0))
    with pytest.raises(KernelError):
        ops.group_attn_prep_joint(x, 0, 32, -1, None, None, None, 0, True, torch.zeros(1, dtype=torch.int64, device=gpu),
                                  torch.zeros((4, 1, 64), dtype=torch.bfloat16, device=gpu), 1, 1, 32, 16, 32, 1e-5)
