"""GPU: the kernels of gated sublayers — embeddings that start the stream, gated joins with the convolution behind them,
convolutions of portions, corrected routes with shared experts — and of latent attention with sinks, gates per head and no rotated
part, against double-precision statements."""
import numpy as np
import pytest

from layer_stack_util import bf16
from oracle import layer_stack as ls
from test_decay_memory_gpu import host, i32, t
from test_layer_stack_kernels_gpu import paged

pytestmark = pytest.mark.gpu


class Slots:
    """States of a convolution in scattered slots behind other bytes, and the rows of some requests."""

    def __init__(self, rng, gpu, dtype, width, taps, lens, fresh):
        import torch
        from pie_amd import ops

        self.keep, self.width, R = taps - 1, width, len(lens)
        size = 2 if dtype == torch.bfloat16 else 4
        self.at, stride = 256, 512 + max(1, self.keep) * width * size + 64
        stride = -(-stride // 256) * 256
        self.slots = rng.permutation(R + 3)[:R]
        self.values = host(t(rng.standard_normal((R + 3, self.keep, width)), gpu, dtype))
        self.pool = torch.zeros((R + 3, stride), dtype=torch.uint8, device=gpu)
        self.view = lambda: self.pool[:, self.at:self.at + self.keep * width * size].contiguous().view(dtype).reshape(R + 3, self.keep, width)
        self.pool[:, self.at:self.at + self.keep * width * size] = t(self.values, gpu, dtype).reshape(R + 3, -1).contiguous().view(torch.uint8)
        self.lens, self.fresh = lens, np.asarray(fresh)
        self.held = (i32(np.repeat(np.arange(R), lens), gpu), i32(np.concatenate([[0], np.cumsum(lens)]), gpu), i32(self.slots, gpu), i32(self.fresh, gpu))
        self.rows = ops.state_rows(*self.held, self.pool, 0, self.at)

    def want(self, h, w):
        """h [N, width], w [taps, width] -> (rows plus their convolution, states afterwards)"""
        out, states, at = np.empty_like(h), self.values.copy(), 0
        for r, n in enumerate(self.lens):
            past = np.zeros((self.keep, self.width)) if self.fresh[r] else self.values[self.slots[r]]
            x = np.concatenate([past, h[at:at + n]])
            out[at:at + n] = h[at:at + n] + sum(x[j:j + n] * w[j] for j in range(self.keep + 1))
            states[self.slots[r]] = x[len(x) - self.keep:]
            at += n
        return out, states


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("width,ld", [(96, 128), (75, 128), (2048, 2048), (4098, 4224), (9000, 9088)])
@pytest.mark.parametrize("pairs", [0, 37])
def test_an_embedding_starts_the_stream(gpu, bf, width, ld, pairs):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(width)
    dt, eps, rows = torch.bfloat16 if bf else torch.float32, 1e-3, 9
    toks, pair = rng.integers(0, 50, rows), rng.integers(0, pairs + 1, rows)
    toks[7] = 60   # (an id past the table reads row 0)
    table, bigram = (t(rng.standard_normal((n, width)), gpu, torch.bfloat16) for n in (50, pairs + 1))
    ew, nw = (rng.uniform(0.5, 1.5, width).astype(np.float32) for _ in range(2))
    held = [i32(toks, gpu), i32(pair, gpu), t(ew, gpu)]
    start = ops.embedding(held[0], table, 2.5, held[2], held[1] if pairs else None, bigram if pairs else None)
    s, w = Slots(rng, gpu, dt, width, 3, [1] * rows, [1] * rows), bf16(rng.standard_normal((3, width)))
    e = host(table)[np.where(toks < 50, toks, 0)] * 2.5 + (host(bigram)[pair] if pairs else 0.0)
    want = ls.rms_norm(e, ew, eps)
    for kw in (dict(next_weight=t(nw, gpu)), dict(next_weight=t(nw, gpu), conv_w=t(w, gpu, torch.bfloat16), rows=s.rows), dict()):
        x = t(np.full((rows, ld), 3.0, np.float32), gpu)   # (what was there before does not matter)
        h, recent = (host(v) for v in ops.gated_join(x, width, eps, dt, start=start, **kw))
        assert np.abs(host(x)[:, :width] - want).max() < 1e-5 and (host(x)[:, width:] == 3.0).all()
        if kw:
            assert np.abs(h[:, :width] - ls.rms_norm(want, nw, eps)).max() < (4e-2 if bf else 3e-5)
        if "rows" in kw:
            out, states = s.want(h[:, :width], w)
            assert (np.abs(recent[:, :width] - out) < (5e-3 if bf else 1e-5) * (1.0 + np.abs(out))).all() and np.array_equal(host(s.view()), states)


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("width,ld", [(96, 128), (75, 128), (2048, 2048), (2056, 2176), (8200, 8320)])
@pytest.mark.parametrize("taps", [0, 1, 2, 3, 4])
def test_gated_join(gpu, bf, width, ld, taps):
    """A sublayer's output or a mixture's routes through their gates, with and without the next convolution."""
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(width + taps)
    dt, eps, rows, top = torch.bfloat16 if bf else torch.float32, 1e-3, 5, 11
    y, ry, gate = (t(rng.standard_normal((n, ld)), gpu, dt) for n in (rows, rows * top, rows))
    pos = rng.permutation(rows * top).reshape(rows, top).astype(np.int32)
    weight, bias, nw = (rng.uniform(0.5, 1.5, s).astype(np.float32) for s in ((rows, top), width, width))
    mix = np.einsum("nk,nkw->nw", weight, host(ry)[pos])[:, :width]
    g = ls.sigmoid(host(gate)[:, :width] + bias)
    for use in ("start", "sublayer", "mixture", "last"):
        if use == "last" and taps:
            continue
        s = Slots(rng, gpu, dt, width, taps, [1] * rows, [0, 1, 0, 0, 1]) if taps else None
        w = bf16(rng.standard_normal((taps, width))) if taps else None
        x0 = rng.standard_normal((rows, ld)).astype(np.float32)
        x, kw, want = t(x0, gpu), {}, x0[:, :width].astype(np.float64)
        if use in ("sublayer", "last"):
            kw.update(y=y, gate=gate, gate_bias=t(bias, gpu))
            want = want + host(y)[:, :width] * g
        if use == "mixture":
            kw.update(routes=(ry, t(pos, gpu), t(weight, gpu)), gate=gate, gate_bias=t(bias, gpu))
            want = want + mix * g
        h, recent = ops.gated_join(x, width, eps, dt, next_weight=None if use == "last" else t(nw, gpu), conv_w=t(w, gpu, torch.bfloat16) if taps else None,
                                   rows=s.rows if taps else None, **kw)
        assert np.abs(host(x)[:, :width] - want).max() < 3e-5 and np.array_equal(host(x)[:, width:], x0[:, width:])
        if use == "last":
            continue
        h, recent = host(h), host(recent)
        assert np.abs(h[:, :width] - ls.rms_norm(want, nw, eps)).max() < (4e-2 if bf else 3e-5) and (h[:, width:] == 0).all()
        if taps:   # (of the row as it was stored)
            out, states = s.want(h[:, :width], w)
            assert (np.abs(recent[:, :width] - out) < (5e-3 if bf else 1e-5) * (1.0 + np.abs(out))).all() and (recent[:, width:] == 0).all()
            assert np.array_equal(host(s.view()), states)


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("width,ld", [(96, 128), (75, 128), (2056, 2176)])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
@pytest.mark.parametrize("lens", [[1, 2, 9, 1, 30, 3], [1], [1100, 1, 5, 2]])
def test_recent_rows(gpu, bf, width, ld, taps, lens):
    """Portions shorter and longer than the convolution, fresh and carried, and the state they leave."""
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(width + taps + len(lens))
    dt = torch.bfloat16 if bf else torch.float32
    s = Slots(rng, gpu, dt, width, taps, lens, [r % 3 == 1 for r in range(len(lens))])
    h, w = t(rng.standard_normal((sum(lens), ld)), gpu, dt), bf16(rng.standard_normal((taps, width)))
    got = host(ops.recent_rows(h, t(w, gpu, torch.bfloat16), s.rows))
    out, states = s.want(host(h)[:, :width], w)
    assert (np.abs(got[:, :width] - out) < (5e-3 if bf else 1e-5) * (1.0 + np.abs(out))).all() and (got[:, width:] == 0).all()
    if taps > 1:
        ops.conv_state(h, s.rows, width, taps)
        assert np.array_equal(host(s.view()), states)


@pytest.mark.parametrize("experts,top,shared", [(9, 3, 1), (64, 8, 2), (12, 12, 0), (1, 1, 1), (200, 17, 5), (500, 40, 12)])
@pytest.mark.parametrize("T", [1, 5, 16, 17, 100])
def test_corrected_routes(gpu, experts, top, shared, T):
    from pie_amd import ops

    rng = np.random.default_rng(experts + T)
    ld = -(-(experts + 1) // 16) * 16
    z = rng.standard_normal((T, ld)).astype(np.float32) * 2.0
    z[:, experts + 1:] = 50.0   # (columns that pad the product belong to no expert)
    corr = rng.uniform(-1.5, 0.7, experts).astype(np.float32)   # (corrected scores below zero are still chosen from)
    idx, weight, offsets, token, pos = (host(x) for x in ops.moe_route_corrected(t(z, gpu), t(corr, gpu), top, shared))
    idx, offsets, token, pos = (x.astype(int) for x in (idx, offsets, token, pos))
    want = ls.corrected_route(z[:, :experts].astype(np.float64), corr.astype(np.float64), top)
    got = np.zeros((T, shared + experts))
    np.put_along_axis(got, idx, weight, axis=1)
    assert np.allclose(got[:, shared:], want, rtol=1e-5, atol=1e-7) and all(len(set(r)) == shared + top for r in idx)
    assert np.array_equal(idx[:, :shared], np.tile(np.arange(shared), (T, 1)))
    assert np.allclose(weight[:, :shared], ls.sigmoid(z[:, experts:experts + 1].astype(np.float64)), rtol=1e-5)
    K = shared + top
    assert offsets[0] == 0 and offsets[-1] == T * K and np.array_equal(np.diff(offsets), np.bincount(idx.ravel(), minlength=shared + experts))
    assert sorted(pos.ravel()) == list(range(T * K))
    for n in range(T):
        for k in range(K):
            assert token[pos[n, k]] == n and offsets[idx[n, k]] <= pos[n, k] < offsets[idx[n, k] + 1]


def test_equal_corrected_scores_go_to_the_lowest_expert(gpu):
    from pie_amd import ops

    z = np.zeros((2, 16), np.float32)
    z[1, 9] = 1.0
    corr = np.zeros(12, np.float32)
    corr[5] = 0.1
    idx = host(ops.moe_route_corrected(t(z, gpu), t(corr, gpu), 3, 1)[0])
    assert idx[0].tolist() == [0, 6, 1, 2] and sorted(idx[1].tolist()) == [0, 1, 6, 10]


@pytest.mark.parametrize("form", ["f32", "rows", "blocks"])
@pytest.mark.parametrize("T,E,top,shared,K,N", [(1, 5, 2, 1, 128, 64), (9, 5, 2, 2, 256, 96), (70, 17, 4, 1, 384, 32), (120, 3, 2, 0, 128, 160)])
def test_grouped_products_with_squared_relu(gpu, form, T, E, top, shared, K, N):
    """Experts that every token uses have as many rows as there are tokens."""
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(T)
    dt = torch.float32 if form == "f32" else torch.bfloat16
    act, w = t(rng.standard_normal((T, K)), gpu, dt), t(rng.standard_normal((E + shared, N, K)) * 2 / np.sqrt(K), gpu, torch.bfloat16)
    z = rng.standard_normal((T, 32)).astype(np.float32)
    idx, _, offsets, token, pos = ops.moe_route_corrected(t(z, gpu), t(np.zeros(E, np.float32), gpu), top, shared)
    kw = dict(block_rows=0) if form == "blocks" else dict(known=T % 2 == 1)
    got = host(ops.moe_grouped_glu(act, token, offsets, w, T * (top + shared), None, epilogue=2, **kw))
    a, wh, idx, pos = host(act), host(w), host(idx).astype(int), host(pos).astype(int)
    for n in range(T):
        for k in range(top + shared):
            x = ls.squared_relu(wh[idx[n, k]] @ a[n])
            assert np.abs(got[pos[n, k]] - x).max() < (1e-3 if form == "f32" else 8e-3) * max(1.0, x.max())


# ---- latent attention ----------------------------------------------------------------------------------------
def attend(q, keys, kvp, scale, sinks):
    """q [heads, ld], keys [len, ld] -> [heads, kvp]"""
    p = ls.softmax_with_learned_sink((q @ keys.T * scale)[:, None], True, sinks)[:, 0]
    return p @ keys[:, :kvp]


SINKS = {"mild": lambda rng, n: rng.uniform(-1, 3, n), "none": lambda rng, n: np.full(n, -80.0), "all": lambda rng, n: np.full(n, 95.0),
         "mixed": lambda rng, n: np.where(np.arange(n) % 2, 9.0, -5.0)}


@pytest.mark.parametrize("heads,kvp,rotp,ps,lens", [(3, 64, 0, 16, [1, 15, 16, 17, 33, 300]), (32, 512, 0, 16, [2080, 7, 513]), (17, 128, 0, 48, [95, 96, 97, 49]),
                                                    (8, 192, 0, 64, [64, 65, 640]), (40, 256, 0, 32, [31, 200]), (2, 384, 0, 16, [1000, 1]),
                                                    (6, 128, 32, 16, [700, 3])])
@pytest.mark.parametrize("kind", ["bf16", "bf16_plain", "f32_plain"])
@pytest.mark.parametrize("sink", sorted(SINKS))
def test_sinks_of_single_rows(gpu, heads, kvp, rotp, ps, lens, kind, sink):
    """Keys in one split and in several; sinks far below and far above every score, and in between."""
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(heads * kvp)
    dt, ld = torch.float32 if kind == "f32_plain" else torch.bfloat16, kvp + rotp
    pool, pages, begin, rows = paged(rng, lens, ld, ps, gpu, dt)
    q, sinks = t(rng.standard_normal((len(lens), heads, ld)), gpu, dt), SINKS[sink](rng, heads).astype(np.float32)
    scale = 3.0 / np.sqrt(ld)
    want = np.stack([attend(host(q)[n], rows[n][:lens[n]], kvp, scale, sinks.astype(np.float64)) for n in range(len(lens))])
    for bound in (max(lens), max(lens) + 700):
        got = host(ops.latent_attn_rows(q, pool, kvp, pages, i32(begin, gpu), i32(lens, gpu), ps, scale, plain=kind != "bf16", max_kv_len=bound,
                                        sinks=t(sinks, gpu)))
        assert (np.abs(got - want) < (1e-5 if kind == "f32_plain" else 8e-3) * (1.0 + np.abs(want))).all()


@pytest.mark.parametrize("heads,kvp,ps,new", [(3, 64, 16, [9, 1, 33, 5]), (20, 128, 64, [2, 2, 64, 1]), (32, 256, 16, [40, 1, 1, 3])])
def test_sinks_of_portions(gpu, heads, kvp, ps, new):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(5)
    ctx = [n + c for n, c in zip(new, (28, 199, 31, 0))]
    pool, pages, begin, rows = paged(rng, ctx, kvp, ps, gpu, torch.bfloat16)
    own = [(r, ctx[r] - new[r] + i + 1) for r in range(4) for i in range(new[r])]
    q, sinks = t(rng.standard_normal((len(own), heads, kvp)), gpu, torch.bfloat16), rng.uniform(-1, 4, heads).astype(np.float32)
    got = host(ops.latent_attn_rows(q, pool, kvp, pages, i32([begin[r] for r, _ in own], gpu), i32([n for _, n in own], gpu), ps, 0.2,
                                    row_req=i32([r for r, _ in own], gpu), qo_indptr=i32(np.concatenate([[0], np.cumsum(new)]), gpu),
                                    max_tokens=max(new), sinks=t(sinks, gpu)))
    for i, (r, n) in enumerate(own):
        assert np.abs(got[i] - attend(host(q)[i], rows[r][:n], kvp, 0.2, sinks.astype(np.float64))).max() < 1.2e-2, (r, n)


@pytest.mark.parametrize("heads,dimp,vdp,T,past", [(3, 32, 32, 130, 0), (6, 32, 64, 70, 41), (5, 64, 96, 300, 7), (2, 128, 128, 200, 500), (70, 32, 32, 1030, 0),
                                                   (2, 192, 32, 65, 1)])
@pytest.mark.parametrize("sink", sorted(SINKS))
def test_sinks_and_head_gates_of_expanded_portions(gpu, heads, dimp, vdp, T, past, sink):
    """No rotated part; blocks of 64 and of 128 queries."""
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(T)
    bf, keys, ld_gate = torch.bfloat16, past + T, -(-heads // 16) * 16 + 16
    q, kv = t(rng.standard_normal((T, heads, dimp)), gpu, bf), t(rng.standard_normal((keys, heads, dimp + vdp)), gpu, bf)
    fused, sinks = t(rng.standard_normal((T, ld_gate)) * 2, gpu, bf), SINKS[sink](rng, heads).astype(np.float32)
    gate = fused[:, 5:]   # (columns of wider rows)
    lens, scale = np.arange(past + 1, keys + 1), 2.0 / np.sqrt(dimp)
    got = host(ops.latent_attn_prefill(q, kv, None, None, 0, i32(lens, gpu), dimp, scale, gate=gate, gate_cols=1, sinks=t(sinks, gpu))).reshape(T, heads, vdp)
    qh, kvh, g = host(q), host(kv), ls.sigmoid(host(fused)[:, 5:5 + heads])
    for i in np.unique(np.concatenate([np.arange(0, T, 61), [0, 1, 63, 64, T - 1]])):
        s = np.einsum("hd,jhd->hj", qh[i], kvh[:lens[i], :, :dimp]) * scale
        p = ls.softmax_with_learned_sink(s[:, None], True, sinks.astype(np.float64))[:, 0]
        want = np.einsum("hj,jhd->hd", p, kvh[:lens[i], :, dimp:]) * g[i][:, None]
        assert np.abs(got[i] - want).max() < 2.5e-2, i


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("M,heads,C,K", [(1, 3, 32, 64), (20, 5, 64, 128), (70, 2, 96, 32)])
def test_one_gate_per_head(gpu, bf, M, heads, C, K):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(M)
    dt = torch.bfloat16 if bf else torch.float32
    act, fused = t(rng.standard_normal((M, heads, K)), gpu, dt), t(rng.standard_normal((M, heads + 11)) * 2, gpu, dt)
    w = t(rng.standard_normal((heads, C, K)) / np.sqrt(K), gpu, torch.bfloat16)
    got = host(ops.head_linear(act, w, gate=fused[:, 3:], gate_cols=1))
    want = np.einsum("mhk,hck->mhc", host(act), host(w)) * ls.sigmoid(host(fused)[:, 3:3 + heads])[:, :, None]
    assert np.abs(got - want).max() < (3e-2 if bf else 1e-5)


@pytest.mark.parametrize("where", ["first", "last", "page_end", "page_start", "split", "just_past"])
@pytest.mark.parametrize("form", ["rows", "plain"])
def test_one_far_key_decides_beside_a_sink(gpu, where, form):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(6)
    heads, kvp, ps, n = 6, 256, 16, 777
    pool, pages, begin, rows = paged(rng, [n + 1], kvp, ps, gpu, torch.bfloat16)
    j = dict(first=0, last=n - 1, page_end=ps * 9 - 1, page_start=ps * 9, split=256, just_past=n)[where]
    q = torch.zeros(1, heads, kvp, device=gpu, dtype=torch.bfloat16)
    q[:] = t(rows[0][j], gpu, torch.bfloat16)
    top = float(host(q)[0, 0] @ rows[0][j])
    sinks = np.array([top, top - 30.0, top + 30.0, top, top + 1.0, top - 1.0], np.float32)   # (half the weight, none, all, ..)
    got = host(ops.latent_attn_rows(q, pool, kvp, pages, i32(begin, gpu), i32([n], gpu), ps, 1.0, plain=form == "plain", sinks=t(sinks, gpu)))
    want = attend(host(q)[0], rows[0][:n], kvp, 1.0, sinks.astype(np.float64))
    assert np.abs(got[0] - want).max() < 1.5e-2 * max(1.0, np.abs(want).max())
    if where != "just_past":
        assert np.abs(got[0, 0] - 0.5 * rows[0][j]).max() < 0.05 and np.abs(got[0, 2]).max() < 1e-3


def test_bad_arguments_are_refused(gpu):
    import torch
    from pie_amd import ops
    from pie_amd.ops import KernelError

    z, c = torch.zeros((2, 16), device=gpu), torch.zeros(12, device=gpu)
    for correction, top, shared in [(c, 13, 0), (c, 0, 1), (c, 3, -1), (torch.zeros(16, device=gpu), 3, 1)]:
        with pytest.raises((KernelError, RuntimeError)):
            ops.moe_route_corrected(z, correction, top, shared)
    x, y = torch.zeros((2, 128), device=gpu), torch.zeros((2, 128), device=gpu)
    nw = torch.ones(96, device=gpu)
    tok, table = torch.zeros(2, dtype=torch.int32, device=gpu), torch.zeros((3, 96), dtype=torch.bfloat16, device=gpu)
    start = ops.embedding(tok, table, 1.0, nw)
    for kw in (dict(), dict(y=y, next_weight=nw), dict(y=y, gate=y, gate_bias=nw, start=start), dict(start=ops.embedding(tok, table, 1.0, nw, None, table)), dict(next_weight=nw, conv_w=torch.zeros((3, 96), dtype=torch.bfloat16, device=gpu)), dict(y=y, gate=y)):
        with pytest.raises(KernelError):
            ops.gated_join(x, 96, 1e-5, torch.float32, **kw)
    rng = np.random.default_rng(0)
    s = Slots(rng, gpu, torch.float32, 96, 3, [2], [0])   # (two rows of one request: not one each)
    with pytest.raises(KernelError):
        ops.gated_join(x, 96, 1e-5, torch.float32, next_weight=nw, conv_w=torch.zeros((3, 96), dtype=torch.bfloat16, device=gpu), rows=s.rows)
    with pytest.raises(KernelError):
        ops.head_linear(torch.zeros((1, 2, 32), device=gpu), torch.zeros((2, 16, 32), dtype=torch.bfloat16, device=gpu), gate=z[:1], gate_cols=2)
