"""GPU: memories with one decay per head (retention, mLSTM, Mamba-2) and what surrounds them, kernel by kernel
against the double-precision oracle: portions down to two tokens, carried and fresh states in scattered slots,
strong and weak decays, large gates, sizes off the tiles, writes from long ago."""
import numpy as np
import pytest

from oracle import layer_stack as ls

pytestmark = pytest.mark.gpu
FIXED, GATES, STEP = 0, 1, 2


def t(a, gpu, dtype=None):
    import torch

    x = torch.from_numpy(np.ascontiguousarray(a)).to(gpu)
    return x if dtype is None else x.to(dtype)


def host(x):
    import torch

    return x.to(torch.float64).cpu().numpy()


def i32(a, gpu):
    return t(np.asarray(a, np.int32), gpu)


class Memory:
    """One layer's memory: its rule, and sequences with the oracle's read-outs.  Rows are [q | k | v]."""

    def __init__(self, rng, gpu, dtype, kind, heads, kv, dk, dv, strength, lens):
        from pie_amd import ops

        self.kind, self.heads, self.kv, self.dk, self.dv = kind, heads, kv, dk, dv
        up = lambda n: -(-n // 8) * 8
        self.q_off, self.k_off, self.v_off = 0, up(kv * dk), 2 * up(kv * dk)
        self.ld = up(self.v_off + heads * dv)
        self.decay = {"weak": 1 - 1e-4, "strong": 0.2, "mixed": 0.97}[strength] ** np.arange(1, heads + 1)
        self.q_scale = dk ** -0.5 if kind == GATES else 1.0
        self.k_scale = dk ** -0.5 if kind == FIXED else 1.0
        self.cap = 11.0
        bias = rng.standard_normal(2 * heads if kind == GATES else heads).astype(np.float32)
        rate = {"weak": 1e-3, "strong": 8.0, "mixed": 0.3}[strength] * np.arange(1, heads + 1)
        self.d_decay = None if kind == GATES else t((np.log2(self.decay) if kind == FIXED else -rate * np.log2(np.e)).astype(np.float32), gpu)
        self.d_bias = None if kind == FIXED else t(bias, gpu)
        self.rule = ops.decay_rule(kind, heads, kv, dk, dv, self.q_scale, self.k_scale, self.cap, self.d_decay, self.d_bias)
        self.seqs, self.want, self.sums = [], [], []
        src = np.arange(heads) // (heads // kv)
        for n in lens:
            rows = host(t(rng.standard_normal((n, self.ld)), gpu, dtype))
            gates = None
            if kind != FIXED:
                shift = {"weak": (0.0, 12.0), "strong": (9.0, -6.0), "mixed": (2.0, 1.0)}[strength]
                gates = np.zeros((n, -(-bias.size // 16) * 16), np.float32)
                gates[:, :bias.size] = rng.standard_normal((n, bias.size)) * 4
                if kind == GATES:
                    gates[:, :heads] += shift[0]
                    gates[:, heads:2 * heads] += shift[1]
            q = rows[:, :kv * dk].reshape(n, kv, dk)[:, src]
            k = rows[:, self.k_off:self.k_off + kv * dk].reshape(n, kv, dk)[:, src] * self.k_scale
            v = rows[:, self.v_off:self.v_off + heads * dv].reshape(n, heads, dv)
            if kind == FIXED:
                want = ls.decayed_outer_products(q, k, v, np.broadcast_to(np.exp2(host(self.d_decay)), (n, heads)))
            elif kind == STEP:
                dt = ls.softplus(gates[:, :heads].astype(np.float64) + bias)
                want = ls.decayed_outer_products(q, k, dt[:, :, None] * v, np.exp2(host(self.d_decay) * dt))
            else:
                g = self.cap * np.tanh((gates[:, :2 * heads].astype(np.float64) + bias) / self.cap)
                want = ls.matrix_memory(q * self.q_scale, k, v, g[:, :heads], ls.log_sigmoid(g[:, heads:]))
                self.sums.append(self.undivided(q * self.q_scale, k, v, g[:, :heads], ls.log_sigmoid(g[:, heads:])))
            self.seqs.append((rows, gates))
            self.want.append(want)
        self.state_bytes = -(-4 * heads * (dk * dv + (dk + 1 if kind == GATES else 0)) // 256) * 256

    @staticmethod
    def undivided(q, k, v, i, f):
        """[S^T q | n . q] of the exponentially gated memory, and its maximum in units of log 2.  (Their quotient can
        magnify rounding without bound where n . q passes through zero.)"""
        T, H, dv = v.shape
        m, S = np.zeros(H), np.zeros((H, q.shape[2], dv + 1))
        out, ms = np.empty((T, H, dv + 1)), np.empty((T, H))
        for t in range(T):
            m_new = np.maximum(f[t] + m, i[t])
            x = np.concatenate([v[t], np.ones((H, 1))], 1)
            S = np.exp(f[t] + m - m_new)[:, None, None] * S + np.exp(i[t] - m_new)[:, None, None] * k[t][:, :, None] * x[:, None, :]
            m = m_new
            out[t], ms[t] = np.einsum("hkv,hk->hv", S, q[t]), m * np.log2(np.e)
        return out, ms


SIZES = [(4, 4, 32, 32), (6, 2, 20, 12), (2, 1, 64, 40), (3, 3, 128, 70), (2, 2, 130, 36), (1, 1, 256, 260), (1, 1, 300, 20), (8, 4, 9, 7)]


@pytest.mark.parametrize("kind", [FIXED, GATES, STEP])
@pytest.mark.parametrize("heads,kv,dk,dv", SIZES)
@pytest.mark.parametrize("strength", ["weak", "strong", "mixed"])
@pytest.mark.parametrize("form", ["scan_f32", "scan", "chunked"])
def test_portions_and_single_tokens(gpu, kind, heads, kv, dk, dv, strength, form):
    """Unequal requests, each cut into portions, in scattered slots that start full of garbage; the last tokens one
    by one through the step where its sizes are taken."""
    import torch
    from pie_amd import ops

    dt = torch.float32 if form == "scan_f32" else torch.bfloat16
    rng = np.random.default_rng(dk + dv + kind)
    lens = [133, 18, 90]
    cuts = [[64, 2, 65, 1, 1], [1, 16, 1], [88, 1, 1]]
    m = Memory(rng, gpu, dt, kind, heads, kv, dk, dv, strength, lens)
    slots = [4, 0, 2]
    state = t(np.full((5, m.state_bytes // 4), 1e3, np.float32), gpu).view(torch.uint8)
    at, got = [0, 0, 0], [[], [], []]
    for step in range(5):
        live = [r for r in range(3) if step < len(cuts[r])]
        n = [cuts[r][step] for r in live]
        rows = t(np.concatenate([m.seqs[r][0][at[r]:at[r] + c] for r, c in zip(live, n)]), gpu, dt)
        gates = None if kind == FIXED else t(np.concatenate([m.seqs[r][1][at[r]:at[r] + c] for r, c in zip(live, n)]), gpu)
        qo = np.concatenate([[0], np.cumsum(n)])
        row_req, d_qo, d_slot = i32(np.repeat(np.arange(len(live)), n), gpu), i32(qo, gpu), i32([slots[r] for r in live], gpu)
        fresh = i32([at[r] == 0 for r in live], gpu)
        sr = ops.state_rows(row_req, d_qo, d_slot, fresh, state)
        f = form.split("_")[0]
        if max(n) == 1 and dv % 4 == 0:
            f = "step"
        o, den = (host(x) for x in ops.decay_memory(f, m.rule, sr, rows, m.q_off, m.k_off, m.v_off, gates, d_qo))
        if kind == GATES:   # the running maximum is handed on by the read-out kernel
            z = t(np.zeros((sum(n), heads * dv)), gpu, dt)
            ops.decay_out(m.rule, sr, t(o.astype(np.float32), gpu), t(den.astype(np.float32), gpu), z, 0, None, 1.0, 1e-5)
        o = o.reshape(-1, heads, dv)
        if kind == GATES:
            o = np.concatenate([o, den], -1)
        for i, r in enumerate(live):
            got[r].append(o[qo[i]:qo[i + 1]])
            at[r] += n[i]
    for r in range(3):
        o, want = np.concatenate(got[r]), m.want[r]
        if kind == GATES:
            want, peak = m.sums[r]
            assert np.abs(o[..., -1] - peak).max() < 2e-5
            o = o[..., :-1]
        err = np.abs(o - want) / (np.abs(want).max(axis=(0, 2), keepdims=True) + 1e-3)
        assert err.max() < (1e-5 if form != "chunked" else 4e-5), (r, err.max(), np.unravel_index(err.argmax(), err.shape))
    assert (host(state.view(torch.float32))[[1, 3]] == 1e3).all()   # nobody's slots


@pytest.mark.parametrize("dk,dv", [(64, 32), (200, 48)])
def test_a_write_from_long_ago_is_kept(gpu, dk, dv):
    """No decay, orthogonal keys: a key written 500 tokens earlier still gives its value."""
    import torch
    from pie_amd import ops

    T, e = 530, np.eye(dk)
    rng = np.random.default_rng(1)
    k = e[1 + np.arange(T) % (dk - 1)]
    k[3] = e[0]
    v = host(t(rng.standard_normal((T, dv)), gpu, torch.bfloat16))
    rows = t(np.concatenate([np.tile(e[0], (T, 1)), k, v], 1), gpu, torch.bfloat16)
    rule = ops.decay_rule(FIXED, 1, 1, dk, dv, decay=(d := t(np.zeros(1, np.float32), gpu)))
    for form in ("scan", "chunked"):
        state = t(np.zeros((1, dk * dv), np.float32), gpu).view(torch.uint8)
        sr = ops.state_rows(req := i32(np.zeros(T), gpu), qo := i32([0, T], gpu), slot := i32([0], gpu), fresh := i32([1], gpu), state)
        o = host(ops.decay_memory(form, rule, sr, rows, 0, dk, 2 * dk, None, qo)[0])
        assert np.abs(o[-1] - v[3]).max() < 1e-5 and np.abs(o[2]).max() == 0.0
    assert d is not None and req is not None and slot is not None and fresh is not None


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("taps", [1, 2, 4, 6])
@pytest.mark.parametrize("channels", [40, 93])
def test_convolution_in_portions_and_steps(gpu, bf, taps, channels):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(taps + channels)
    dt = torch.bfloat16 if bf else torch.float32
    ld, lens, slots = -(-channels // 16) * 16 + 16, [700, 30, 9], [2, 0, 3]
    w, b = rng.standard_normal((channels, taps)).astype(np.float32), rng.standard_normal(channels).astype(np.float32)
    seqs = [host(t(rng.standard_normal((n, ld)), gpu, dt)) for n in lens]
    want = [ls.silu(ls.causal_conv(s[:, :channels], w.astype(np.float64)) + b) for s in seqs]
    stride = -(-4 * max(taps - 1, 1) * channels // 256) * 256
    state = t(np.full((4, stride // 4), 50.0, np.float32), gpu).view(torch.uint8)
    at, got = [0, 0, 0], [[], [], []]
    for cut in ([600, 2, 1], [1, 1, 1], [97, 25, 5], [1, 1, 1], [1, 1, 1]):
        qo = np.concatenate([[0], np.cumsum(cut)])
        fused = t(np.concatenate([seqs[r][at[r]:at[r] + c] for r, c in enumerate(cut)]), gpu, dt)
        req, d_qo, slot, fresh = i32(np.repeat(np.arange(3), cut), gpu), i32(qo, gpu), i32(slots, gpu), i32([a == 0 for a in at], gpu)
        sr = ops.state_rows(req, d_qo, slot, fresh, state)
        one = max(cut) == 1
        o = host(ops.conv_silu(fused, t(w, gpu), t(b, gpu), sr, channels, move_state=one))
        if not one:
            ops.conv_state(fused, sr, channels, taps)
        for r, c in enumerate(cut):
            got[r].append(o[qo[r]:qo[r + 1], :channels])
            at[r] += c
    for r in range(3):
        assert np.abs(np.concatenate(got[r]) - want[r]).max() < (4e-2 if bf else 2e-5)


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("heads,vdim", [(3, 20), (2, 512), (1, 600), (5, 7)])
def test_read_out(gpu, bf, heads, vdim):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(vdim)
    dt, N, ld = torch.bfloat16 if bf else torch.float32, 9, -(-heads * vdim // 16) * 16
    o = rng.standard_normal((N, heads * vdim)).astype(np.float32)
    gate = t(rng.standard_normal((N, ld)) * 2, gpu, dt)
    z, nw = host(gate)[:, :heads * vdim].reshape(N, heads, vdim), rng.uniform(0.5, 1.5, heads * vdim).astype(np.float32)
    state = t(np.zeros((2, heads * (4 * vdim + 5)), np.float32), gpu).view(torch.uint8)
    req, qo, slot, fresh = i32([0] * 5 + [1] * 4, gpu), i32([0, 5, 9], gpu), i32([1, 0], gpu), i32([1, 1], gpu)
    sr = ops.state_rows(req, qo, slot, fresh, state)
    tol = 3e-2 if bf else 2e-5
    rule = ops.decay_rule(FIXED, heads, heads, 4, vdim, decay=(d := t(np.zeros(heads, np.float32), gpu)))
    y = host(ops.decay_out(rule, sr, t(o, gpu), None, gate, 1, None, 1.5, 1e-3))[:, :heads * vdim].reshape(N, heads, vdim)
    x = o.reshape(N, heads, vdim).astype(np.float64)
    assert np.abs(y - 1.5 * ls.divide_by_rms(x, 1e-3) * ls.silu(z)).max() < 3 * tol
    den = np.stack([rng.standard_normal((N, heads)) * 3, rng.uniform(-2, 6, (N, heads))], -1).astype(np.float32)
    rule = ops.decay_rule(GATES, heads, heads, 4, vdim, gate_cap=5.0, gate_bias=(b := t(np.zeros(2 * heads, np.float32), gpu)))
    y = host(ops.decay_out(rule, sr, t(o, gpu), t(den, gpu), gate, 0, t(nw, gpu), 1.0, 1e-3))[:, :heads * vdim].reshape(N, heads, vdim)
    x = x / (np.maximum(np.abs(den[..., 0]), np.exp2(-den[..., 1].astype(np.float64))) + 1e-6)[..., None]
    assert np.abs(y - ls.divide_by_rms(x, 1e-3) * nw.reshape(heads, vdim) * ls.sigmoid(z)).max() < 2 * tol
    m = host(state.view(torch.float32))[:, -heads:]
    assert np.array_equal(m[[1, 0]], den[[4, 8], :, 1].astype(np.float64))   # the last rows' maxima, in their slots
    assert d is not None and b is not None


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("kind", [FIXED, GATES])
@pytest.mark.parametrize("heads,dk,dv", [(4, 32, 32), (96, 48, 100), (64, 128, 256)])
def test_step_with_norm_and_gate_in_one_launch(gpu, bf, kind, heads, dk, dv):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(dk + kind)
    dt, R = torch.bfloat16 if bf else torch.float32, 4
    m = Memory(rng, gpu, dt, kind, heads, heads, dk, dv, "mixed", [6] * R)
    state = t(np.full((R, m.state_bytes // 4), 5.0, np.float32), gpu).view(torch.uint8)
    nw = rng.uniform(0.5, 1.5, heads * dv).astype(np.float32)
    gate = t(rng.standard_normal((R, heads * dv)), gpu, dt)
    z = host(gate).reshape(R, heads, dv)
    for i in range(6):
        rows = t(np.stack([s[0][i] for s in m.seqs]), gpu, dt)
        gates = None if kind == FIXED else t(np.stack([s[1][i] for s in m.seqs]), gpu)
        req, qo, slot, fresh = i32(range(R), gpu), i32(range(R + 1), gpu), i32([3, 1, 0, 2], gpu), i32([i == 0] * R, gpu)
        sr = ops.state_rows(req, qo, slot, fresh, state)
        if not ops.kernels().pie_hip_decay_step_fuses(ops.C.byref(m.rule), R):
            with pytest.raises(ops.KernelError):
                ops.decay_step_fused(m.rule, sr, rows, m.q_off, m.k_off, m.v_off, gates, gate, 1, t(nw, gpu), 0.5, 1e-4)
            return
        y = host(ops.decay_step_fused(m.rule, sr, rows, m.q_off, m.k_off, m.v_off, gates, gate, 1, t(nw, gpu), 0.5, 1e-4)).reshape(R, heads, dv)
        want = 0.5 * ls.divide_by_rms(np.stack([w[i] for w in m.want]), 1e-4) * nw.reshape(heads, dv) * ls.silu(z)
        assert np.abs(y - want).max() < (3e-2 if bf else 3e-4) * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("heads,vdim,state_n,groups,parts,taps", [(6, 12, 20, 3, 4, 4), (4, 10, 9, 4, 1, 1), (8, 64, 128, 2, 8, 2), (2, 2400, 16, 1, 1, 6)])
def test_state_space_steps_with_convolution_skip_and_part_norm(gpu, bf, heads, vdim, state_n, groups, parts, taps):
    """Decoding: the step convolves, the norm moves the convolution's state on; against the portions' kernels and
    the oracle."""
    import torch
    from pie_amd import ops

    if vdim % 4 or vdim > 1024:
        steps = False   # (sizes the step does not take: portions' kernels only)
    else:
        steps = True
    rng = np.random.default_rng(vdim)
    dt, T = torch.bfloat16 if bf else torch.float32, 7
    inner, bc = heads * vdim, groups * state_n
    channels = inner + 2 * bc
    z_off = -(-channels // 8) * 8
    ld = -(-(z_off + inner) // 16) * 16
    w, b = (rng.standard_normal((channels, taps)) * 0.6).astype(np.float32), rng.standard_normal(channels).astype(np.float32)
    skip, nw = rng.standard_normal(heads).astype(np.float32), rng.uniform(0.5, 1.5, inner).astype(np.float32)
    bias, rate = rng.standard_normal(heads).astype(np.float32), rng.uniform(0.1, 2.0, heads)
    d_decay, d_bias = t((-rate * np.log2(np.e)).astype(np.float32), gpu), t(bias, gpu)
    rule = ops.decay_rule(STEP, heads, groups, state_n, vdim, decay=d_decay, gate_bias=d_bias)
    fused = host(t(rng.standard_normal((T, ld)), gpu, dt))
    gates = np.zeros((T, -(-heads // 16) * 16), np.float32)
    gates[:, :heads] = rng.standard_normal((T, heads))
    conv = ls.silu(ls.causal_conv(fused[:, :channels], w.astype(np.float64)) + b)
    if bf:
        conv = host(t(conv, gpu, dt))
    src = np.arange(heads) // (heads // groups)
    x = conv[:, :inner].reshape(T, heads, vdim)
    B, Cq = (conv[:, inner + i * bc:inner + (i + 1) * bc].reshape(T, groups, state_n)[:, src] for i in range(2))
    dts = ls.softplus(gates[:, :heads].astype(np.float64) + bias)
    y = ls.decayed_outer_products(Cq, B, dts[:, :, None] * x, np.exp2(host(d_decay) * dts)) + skip[:, None] * x
    z = fused[:, z_off:z_off + inner]
    want = ls.divide_by_rms((y.reshape(T, inner) * ls.silu(z)).reshape(T, parts, -1), 1e-4).reshape(T, inner) * nw
    state_bytes = -(-4 * heads * state_n * vdim // 256) * 256
    tol = (6e-2 if bf else 2e-4) * max(1.0, np.abs(want).max() / 3)
    one = lambda: t(np.full((2, state_bytes // 4 + 64 * channels), 9.0, np.float32), gpu).view(torch.uint8)
    zview = lambda f: f[:, z_off:z_off + inner].contiguous()
    if steps:
        state = one()
        for i in range(T):
            f = t(fused[i:i + 1], gpu, dt)
            req, qo, slot, fresh = i32([0], gpu), i32([0, 1], gpu), i32([1], gpu), i32([i == 0], gpu)
            sr = ops.state_rows(req, qo, slot, fresh, state, 0, state_bytes)
            o = ops.decay_step_conv(rule, sr, f, inner + bc, inner, 0, t(gates[i:i + 1], gpu), t(w, gpu), t(b, gpu), t(skip, gpu))
            got = host(ops.gated_part_norm(o, None, None, zview(f), t(nw, gpu), heads, vdim, parts, sr, 1e-4, f, channels, taps))
            assert np.abs(got[0] - want[i]).max() < tol, i
    state = one()
    for lo, hi in ((0, 5), (5, T)):
        f = t(fused[lo:hi], gpu, dt)
        req, qo, slot, fresh = i32([0] * (hi - lo), gpu), i32([0, hi - lo], gpu), i32([0], gpu), i32([lo == 0], gpu)
        sr = ops.state_rows(req, qo, slot, fresh, state, 0, state_bytes)
        c = ops.conv_silu(f, t(w, gpu), t(b, gpu), sr, channels)
        ops.conv_state(f, sr, channels, taps)
        o, _ = ops.decay_memory("chunked" if bf else "scan", rule, sr, c, inner + bc, inner, 0, t(gates[lo:hi], gpu), qo)
        got = host(ops.gated_part_norm(o, c, t(skip, gpu), zview(f), t(nw, gpu), heads, vdim, parts, sr, 1e-4))
        assert np.abs(got - want[lo:hi]).max() < tol


# ---- the stream, and the products that drive a recurrence ----------------------------------------------------
@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("width,ld,rows", [(75, 128, 3), (256, 256, 700), (4096, 4096, 2), (4100, 4224, 5), (9000, 9088, 1), (8194, 8320, 2)])
def test_residual_norm(gpu, bf, width, ld, rows):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(width)
    dt, eps = torch.bfloat16 if bf else torch.float32, 1e-3
    y = t(rng.standard_normal((rows, ld)) * 3, gpu, dt)
    post, nxt, add = (rng.uniform(0.5, 1.5, width).astype(np.float32) for _ in range(3))
    table = t(rng.standard_normal((11, width)), gpu, torch.bfloat16)
    tokens = rng.integers(0, 13, rows).astype(np.int32)   # (ids past the table read row 0)
    emb = host(table)[np.where(tokens < 11, tokens, 0)]
    x0 = np.zeros((rows, ld), np.float32)
    x0[:, :width] = rng.standard_normal((rows, width))
    tol = 8e-3 if bf else 3e-6
    for use_y, read, use_e, use_a, norm in [(1, 1, 0, 0, 1), (1, 1, 1, 1, 1), (0, 0, 1, 0, 1), (0, 0, 1, 1, 1), (1, 1, 0, 1, 0)]:
        x = t(x0, gpu)
        xa = ops.residual_norm(x, width, eps, dt, y if use_y else None, t(post, gpu) if use_y else None, bool(read), t(tokens, gpu) if use_e else None,
                               table if use_e else None, t(add, gpu) if use_a else None, t(nxt, gpu) if norm else None)
        want = (x0[:, :width].astype(np.float64) if read else 0.0) + np.zeros((rows, width))
        if use_y:
            want = want + ls.rms_norm(host(y)[:, :width], post, eps)
        want = want + (emb if use_e else 0.0) + (add if use_a else 0.0)
        assert np.abs(host(x)[:, :width] - want).max() < 1e-5 and (host(x)[:, width:] == x0[:, width:]).all()
        wa = ls.rms_norm(want, nxt, eps) if norm else want
        assert np.abs(host(xa)[:, :width] - wa).max() < tol * np.abs(wa).max() and (host(xa)[:, width:] == 0).all()


@pytest.mark.parametrize("bf", [False, True])
@pytest.mark.parametrize("M,N,K", [(1, 16, 128), (5, 48, 1536), (17, 128, 4096), (600, 80, 640), (33, 16, 96)])
def test_unrounded_product(gpu, bf, M, N, K):
    import torch
    from pie_amd import ops

    rng = np.random.default_rng(K)
    a = t(rng.standard_normal((M, K)), gpu, torch.bfloat16 if bf else torch.float32)
    w = t(rng.standard_normal((N, K)) / np.sqrt(K), gpu, torch.bfloat16)
    want = host(a) @ host(w).T
    assert np.abs(host(ops.linear_f32out(a, w)) - want).max() < 1e-5


@pytest.mark.parametrize("M", [1, 3, 12, 40, 100, 300])
def test_gelu_epilogue_of_every_linear_kernel(gpu, M):
    import torch
    from pie_amd import ops

    N, K = 384, 512
    g = torch.Generator().manual_seed(M)
    act, w = (torch.randn(*s, generator=g).to(gpu).bfloat16() for s in ((M, K), (N, K)))
    w = (w.float() / 11).bfloat16()
    view = ops.WeightView("bf16", w, None, 0, N, K)
    z = host(act) @ host(w).T
    want = ls.gelu_erf(z)
    runs = [ops.gemm_skinny(act, view, swiglu=ops.GELU), ops.gemm_skinny(act, ops.repack_mfma_tiles(view), swiglu=ops.GELU),
            ops.gemm_mfma(act, view, swiglu=ops.GELU), ops.linear_fused(act, view, swiglu=ops.GELU)]
    if M <= 128:
        runs.append(ops.gemm_mfma(act, view, swiglu=ops.GELU, split_k=True))
    for got in runs:
        assert got.shape == (M, N) and (np.abs(host(got) - want) < 5e-3 * np.abs(want) + 2e-5).all()
    exact = host(ops.linear_f32(act.float(), w, epilogue=ops.GELU))
    assert np.abs(exact - want).max() < 2e-6 * np.abs(z).max()
    tanh = 0.5 * z * (1 + np.tanh(np.sqrt(2 / np.pi) * (z + 0.044715 * z ** 3)))
    assert np.abs(tanh - want).max() > 50 * np.abs(exact - want).max()   # (the other GELU would show)
