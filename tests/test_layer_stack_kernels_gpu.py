"""GPU: the layer-stack kernels one by one against the double-precision oracle: far keys that decide
the answer, page borders, sizes off the tiles, strong and weak decays, carried and fresh states."""
import numpy as np
import pytest

from layer_stack_util import rotary
from oracle import layer_stack as ls

pytestmark = pytest.mark.gpu


def t(a, gpu, dtype=None):
    import torch

    x = torch.from_numpy(np.ascontiguousarray(a)).to(gpu)
    return x if dtype is None else x.to(dtype)


def host(x):
    import torch

    return x.to(torch.float64).cpu().numpy()


def rel(a, b):
    return float(np.abs(a - b).max() / (np.abs(b).max() + 1e-30))


# ---- what every layer shares --------------------------------------------------------------------------
@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("width,ld,rows", [(75, 128, 3), (256, 256, 700), (4096, 4096, 2), (4100, 4224, 5), (9000, 9088, 1)])
def test_norm_add_and_norm_rows(gpu, bf, width, ld, rows):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(width)
    dt = torch.bfloat16 if bf else torch.float32
    y = t(rng.standard_normal((rows, ld)) * 3, gpu, dt)
    w = rng.uniform(0.5, 1.5, width).astype(np.float32)
    x = np.zeros((rows, ld), np.float32)
    x[:, :width] = rng.standard_normal((rows, width))
    xg = t(x, gpu)
    xa = ops.norm_add(y, t(w, gpu), xg, 1e-3)
    want = x[:, :width] + ls.rms_norm(host(y)[:, :width], w, 1e-3)
    assert rel(host(xg)[:, :width], want) < 2e-6 and (host(xg)[:, width:] == 0).all()
    assert rel(host(xa)[:, :width], want) < (5e-3 if bf else 2e-6)
    pick = np.array([rows - 1, 0], np.int32)
    out = host(ops.norm_rows(xg, t(pick, gpu), t(w, gpu), 1e-3, dt))
    assert rel(out[:, :width], ls.rms_norm(want, w, 1e-3)[pick]) < (5e-3 if bf else 2e-6) and (out[:, width:] == 0).all()


@pytest.mark.parametrize("vocab,ld", [(97, 112), (8192, 8192), (20001, 20016)])
def test_logit_finish_scales_caps_and_picks_the_first_of_equals(gpu, vocab, ld):
    import torch
    from pie_amd import ops

    y = np.random.default_rng(3).standard_normal((3, ld)).astype(np.float32) * 30
    y[:, vocab:] = 1e4            # columns past the vocabulary must not win
    y[0, 11] = y[0, vocab - 2] = 200.0
    y[1, 5] = np.nan
    lg, tok = ops.logits_finish(t(y, gpu), vocab, 0.5, 20.0)
    want = 20.0 * np.tanh(y[:, :vocab].astype(np.float64) * 0.5 / 20.0)
    ok = ~np.isnan(want)
    assert np.abs(host(lg) - want)[ok].max() < 1e-5
    assert tok.cpu().tolist()[0] == 11 and tok.cpu().tolist()[2] == int(np.argmax(want[2]))
    assert tok.cpu().tolist()[1] == int(np.nanargmax(want[1]))
    lg, _ = ops.logits_finish(t(y, gpu), vocab, 0.5, 0.0)
    assert np.allclose(host(lg)[2], y[2, :vocab] * 0.5)


def test_rotation_table_is_right_at_large_positions(gpu):
    from pie_amd import ops

    f, m = ls.rotation_frequencies(rotary(32))
    pos = np.array([0, 1, 4095, 1_000_003], np.int32)
    tab = host(ops.rotary_table(t(pos, gpu), t(f, gpu), m))
    ang = pos[:, None].astype(np.float64) * f
    assert np.abs(tab - np.concatenate([np.cos(ang), np.sin(ang)], 1) * m).max() < 5e-7


@pytest.mark.parametrize("M,N,K", [(1, 65, 19), (70, 130, 128), (3, 16, 257)])
def test_linear_f32_is_true_fp32(gpu, M, N, K):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(4)
    a, w = t(rng.standard_normal((M, K)).astype(np.float32), gpu), t(rng.standard_normal((N, K)), gpu, torch.bfloat16)
    want = host(a) @ host(w).T
    assert rel(host(ops.linear_f32(a, w)), want) < 2e-6
    assert rel(host(ops.linear_f32(a, w, relu2=True)), np.maximum(want, 0) ** 2) < 4e-6


@pytest.mark.parametrize("M", [1, 3, 12, 40, 100, 300])
def test_squared_relu_epilogue_of_every_linear_kernel(gpu, M):
    import torch
    from pie_amd import ops

    N, K = 384, 512
    g = torch.Generator().manual_seed(M)
    act, w = (torch.randn(*s, generator=g).to(gpu).bfloat16() for s in ((M, K), (N, K)))
    view = ops.WeightView("bf16", w, None, 0, N, K)
    want = np.maximum(host(act) @ host(w).T, 0) ** 2
    runs = [ops.gemm_skinny(act, view, swiglu=ops.RELU2), ops.gemm_skinny(act, ops.repack_mfma_tiles(view), swiglu=ops.RELU2),
            ops.gemm_mfma(act, view, swiglu=ops.RELU2), ops.linear_fused(act, view, swiglu=ops.RELU2)]
    if M <= 128:
        runs.append(ops.gemm_mfma(act, view, swiglu=ops.RELU2, split_k=True))
    for got in runs:
        assert got.shape == (M, N) and np.abs(host(got) - want).max() < 6e-3 * want.max()


# ---- latent attention ------------------------------------------------------------------------------------
def softmax_rows(q, rows, lens, kvp, scale):
    """q [n, heads, ld], rows: per query its keys [len, ld] -> [n, heads, kvp]"""
    out = np.zeros((q.shape[0], q.shape[1], kvp))
    for n in range(q.shape[0]):
        keys = rows[n][:lens[n]]
        s = q[n] @ keys.T * scale
        p = np.exp(s - s.max(-1, keepdims=True))
        out[n] = (p / p.sum(-1, keepdims=True)) @ keys[:, :kvp]
    return out


def paged(rng, lens, ld, ps, gpu, dtype):
    """Requests of `lens` cached tokens on scattered pages: pool, page list, begins, rows per request."""
    need = [-(-n // ps) for n in lens]
    perm = rng.permutation(sum(need) + 3)
    pool = t(rng.standard_normal(((sum(need) + 3) * ps, ld)), gpu, dtype)
    begin = np.concatenate([[0], np.cumsum(need)])
    hp = host(pool)
    rows = []
    for r, n in enumerate(lens):
        pages = perm[begin[r]:begin[r + 1]]
        rows.append(np.concatenate([hp[p * ps:(p + 1) * ps] for p in pages]))
    return pool, t(perm.astype(np.int32), gpu), begin[:-1].astype(np.int32), rows


CASES = [(3, 64, 32, 16, [1, 15, 16, 17, 33, 300]), (32, 512, 64, 16, [2080, 7, 513]), (17, 128, 32, 48, [95, 96, 97, 49]),
         (8, 192, 64, 64, [64, 65, 640]), (40, 256, 32, 32, [31, 200]), (2, 384, 32, 16, [1000, 1])]


@pytest.mark.parametrize("heads,kvp,rotp,ps,lens", CASES)
@pytest.mark.parametrize("kind", ["bf16", "bf16_plain", "f32_plain"])
def test_latent_rows_decode(gpu, heads, kvp, rotp, ps, lens, kind):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(heads * kvp)
    dt = torch.float32 if kind == "f32_plain" else torch.bfloat16
    ld = kvp + rotp
    pool, pages, begin, rows = paged(rng, lens, ld, ps, gpu, dt)
    q = t(rng.standard_normal((len(lens), heads, ld)), gpu, dt)
    scale = 3.0 / np.sqrt(ld)
    want = softmax_rows(host(q), rows, lens, kvp, scale)
    for bound in (max(lens), max(lens) + 700):   # (a graph's context bound may lie above every length)
        got = host(ops.latent_attn_rows(q, pool, kvp, pages, t(begin, gpu), t(np.array(lens, np.int32), gpu), ps, scale,
                                        plain=kind != "bf16", max_kv_len=bound))
        assert np.abs(got - want).max() < (1e-5 if kind == "f32_plain" else 1.2e-2)


@pytest.mark.parametrize("heads,ps", [(3, 16), (20, 64), (32, 16)])
def test_latent_rows_portions_are_causal(gpu, heads, ps):
    """Requests of several tokens beside single ones: every row sees exactly its own keys, whatever
    tile it shares with its neighbours."""
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(5)
    kvp, rotp = 128, 32
    ld = kvp + rotp
    ctx, new = [37, 200, 64, 5], [9, 1, 33, 5]
    pool, pages, begin, rows = paged(rng, ctx, ld, ps, gpu, torch.bfloat16)
    lens, rb, rq, rr = [], [], [], []
    for r in range(4):
        for i in range(new[r]):
            lens.append(ctx[r] - new[r] + i + 1)
            rb.append(begin[r])
            rq.append(r)
            rr.append(rows[r])
    qo = np.concatenate([[0], np.cumsum(new)]).astype(np.int32)
    q = t(rng.standard_normal((len(lens), heads, ld)), gpu, torch.bfloat16)
    i32 = lambda a: t(np.array(a, np.int32), gpu)
    got = host(ops.latent_attn_rows(q, pool, kvp, pages, i32(rb), i32(lens), ps, 0.2, row_req=i32(rq), qo_indptr=t(qo, gpu),
                                    max_tokens=max(new)))
    assert np.abs(got - softmax_rows(host(q), rr, lens, kvp, 0.2)).max() < 1.2e-2


@pytest.mark.parametrize("where", ["first", "last", "page_end", "page_start", "split", "just_past"])
@pytest.mark.parametrize("form", ["rows", "plain"])
def test_one_far_key_decides(gpu, where, form):
    """A single key whose score stands out carries the whole weight; a key just past the visible
    ones carries none."""
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(6)
    heads, kvp, rotp, ps, n = 6, 256, 32, 16, 777
    ld = kvp + rotp
    pool, pages, begin, rows = paged(rng, [n + 1], ld, ps, gpu, torch.bfloat16)
    j = dict(first=0, last=n - 1, page_end=ps * 9 - 1, page_start=ps * 9, split=256, just_past=n)[where]
    q = torch.zeros(1, heads, ld, device=gpu, dtype=torch.bfloat16)
    q[:] = t(rows[0][j], gpu, torch.bfloat16)
    got = host(ops.latent_attn_rows(q, pool, kvp, pages, t(begin, gpu), t(np.array([n], np.int32), gpu), ps, 1.0, plain=form == "plain"))
    want = softmax_rows(host(q), rows, [n], kvp, 1.0)
    assert np.abs(got - want).max() < 1.5e-2 * np.abs(want).max()
    near = np.abs(got[0, 0] - rows[0][j][:kvp]).max() < 0.05
    assert near == (where != "just_past")


@pytest.mark.parametrize("heads,dimp,rotp,rot_dims,vdp,T,past", [(3, 32, 32, 16, 32, 130, 0), (32, 128, 64, 64, 128, 300, 41),
                                                                 (16, 64, 32, 32, 64, 2100, 0), (2, 96, 64, 40, 96, 77, 500),
                                                                 (5, 32, 32, 0, 64, 64, 1)])
def test_expanded_prefill(gpu, heads, dimp, rotp, rot_dims, vdp, T, past):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(T)
    keys = past + T
    q = t(rng.standard_normal((T, heads, dimp + rotp)), gpu, torch.bfloat16)
    kv = t(rng.standard_normal((keys, heads, dimp + vdp)), gpu, torch.bfloat16)
    rot = t(rng.standard_normal((keys, rotp)), gpu, torch.bfloat16)
    lens = np.arange(past + 1, keys + 1).astype(np.int32)
    spec = rotary(rot_dims) if rot_dims else None
    tab = None
    if spec:
        f, m = ls.rotation_frequencies(spec)
        tab = ops.rotary_table(t(lens - 1, gpu), t(f, gpu), m)
    scale = 2.0 / np.sqrt(dimp + rotp)
    got = host(ops.latent_attn_prefill(q, kv, rot, tab, rot_dims, t(lens, gpu), dimp, scale)).reshape(T, heads, vdp)
    qh, kvh, rh = host(q), host(kv), host(rot)
    qr = ls.rotate_pairs(qh[..., dimp:], lens - 1, spec) if spec else qh[..., dimp:]
    check = np.unique(np.concatenate([np.arange(0, T, 61), [0, min(T - 1, 63), min(T - 1, 64), T - 1]]))
    for i in check:
        n = lens[i]
        s = (np.einsum("hd,jhd->hj", qh[i, :, :dimp], kvh[:n, :, :dimp]) + qr[i] @ rh[:n].T) * scale
        p = np.exp(s - s.max(-1, keepdims=True))
        p /= p.sum(-1, keepdims=True)
        want = np.einsum("hj,jhd->hd", p, kvh[:n, :, dimp:])
        assert np.abs(got[i] - want).max() < 2.5e-2


def test_gather_and_head_linear(gpu):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(9)
    pool, pages, _, rows = paged(rng, [53], 96, 16, gpu, torch.bfloat16)
    lat, rot = ops.latent_gather(pool, pages, 53, 64, 16)
    assert np.array_equal(host(lat), rows[0][:53, :64]) and np.array_equal(host(rot), rows[0][:53, 64:])
    spec = rotary(12)
    for dt in (torch.bfloat16, torch.float32):
        for M in (1, 17, 33, 130):
            act = t(rng.standard_normal((M, 3, 96)), gpu, dt)
            w = t(rng.standard_normal((3, 80, 64)) / 8, gpu, torch.bfloat16)
            f, m = ls.rotation_frequencies(spec)
            tab = ops.rotary_table(t(np.arange(M, dtype=np.int32), gpu), t(f, gpu), m)
            y = host(ops.head_linear(act, w, tab, rot_dim=20, rot_dims=12, rotp=32))
            a = host(act)
            want = np.concatenate([np.einsum("mhk,hck->mhc", a[..., :64], host(w)), ls.rotate_pairs(a[..., 64:84], np.arange(M), spec),
                                   np.zeros((M, 3, 12))], -1)
            assert np.abs(y - want).max() < (3e-2 if dt == torch.bfloat16 else 1e-5)


# ---- delta rule ----------------------------------------------------------------------------------------
def delta_case(rng, T, heads, kv, dk, dv, decay):
    q = ls.unit_vector(rng.standard_normal((T, kv, dk))) * dk ** -0.5
    k = ls.unit_vector(rng.standard_normal((T, kv, dk)))
    v = rng.standard_normal((T, heads, dv))
    lg = {"weak": -rng.uniform(0, 1e-3, (T, heads, dk)), "strong": -rng.uniform(0, 60, (T, heads, dk)),
          "mixed": -rng.exponential(1.0, (T, heads, dk)) ** 3}[decay]
    beta = rng.uniform(0, 1, (T, heads))
    return [np.asarray(x, np.float32) for x in (q, k, v, lg, beta)]


@pytest.mark.parametrize("heads,kv,dk,dv", [(4, 4, 32, 32), (6, 2, 40, 18), (2, 1, 130, 70), (3, 3, 256, 20)])
@pytest.mark.parametrize("decay", ["weak", "strong", "mixed"])
@pytest.mark.parametrize("chunked", [False, True])
def test_delta_recurrence_in_portions(gpu, heads, kv, dk, dv, decay, chunked):
    """Three requests of unequal length, each cut into portions (down to two tokens and one), states in
    scattered slots that start full of garbage, against the token recurrence of the whole sequences."""
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(dk + dv)
    lens, cuts = [53, 17, 90], [[16, 2, 35], [1, 16], [90]]
    seqs = [delta_case(rng, n, heads, kv, dk, dv, decay) for n in lens]
    src = np.arange(heads) // (heads // kv)
    want = [ls.delta_rule(q[:, src].astype(np.float64), k[:, src].astype(np.float64), v, np.exp2(lg.astype(np.float64)), beta)
            for q, k, v, lg, beta in seqs]
    slots = [4, 0, 2]
    state = t(np.full((5, heads, dk, dv), 1e3, np.float32), gpu)
    at, got = [0, 0, 0], [[], [], []]
    for step in range(3):
        live = [r for r in range(3) if step < len(cuts[r])]
        parts = [[a[at[r]:at[r] + cuts[r][step]] for a in seqs[r]] for r in live]
        cat = [t(np.concatenate([p[i] for p in parts]).reshape(sum(len(p[0]) for p in parts), -1), gpu) for i in range(5)]
        qo = np.concatenate([[0], np.cumsum([len(p[0]) for p in parts])]).astype(np.int32)
        o = host(ops.delta_scan(*cat, state, t(qo, gpu), t(np.array([slots[r] for r in live], np.int32), gpu),
                                t(np.array([at[r] == 0 for r in live], np.int32), gpu), heads, kv, chunked=chunked))
        for i, r in enumerate(live):
            got[r].append(o[qo[i]:qo[i + 1]].reshape(-1, heads, dv))
            at[r] += cuts[r][step]
    for r in range(3):
        assert np.abs(np.concatenate(got[r]) - want[r]).max() < 2e-5
    assert (host(state)[[1, 3]] == 1e3).all()   # nobody's slots


def test_delta_state_keeps_a_write_from_long_ago(gpu):
    """With no decay and orthogonal keys the read-out of a key written 400 tokens earlier is its value."""
    from pie_amd import ops

    heads, dk, dv, T = 2, 64, 32, 420
    rng = np.random.default_rng(1)
    e = np.eye(dk, dtype=np.float32)
    k = np.repeat(e[1 + np.arange(T) % (dk - 1)][:, None], heads, 1)
    k[3] = e[0]
    q = np.repeat(e[0][None, None], T, 0).repeat(heads, 1)
    v = rng.standard_normal((T, heads, dv)).astype(np.float32)
    arrs = [t(x.reshape(T, -1).astype(np.float32), gpu) for x in (q, k, v, np.zeros((T, heads, dk)), np.ones((T, heads)))]
    for chunked in (False, True):
        state = t(np.zeros((1, heads, dk, dv), np.float32), gpu)
        z = t(np.zeros(1, np.int32), gpu)
        o = host(ops.delta_scan(*arrs, state, t(np.array([0, T], np.int32), gpu), z, z + 1, heads, heads, chunked=chunked))
        assert np.abs(o.reshape(T, heads, dv)[-1] - v[3]).max() < 1e-5
        assert np.abs(o.reshape(T, heads, dv)[2]).max() == 0.0
