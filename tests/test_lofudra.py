"""CPU: the mechanisms of Lofudra's oracle on hand-made cases, planted mistakes that the GPU tests' tolerances
must tell apart, and the configuration reader."""
import json

import numpy as np
import pytest

from layer_stack_util import (BF16_MEDIAN, F32_TOL, LOFUDRA_CONFIGS, lofudra, lofudra_weights, logit_error, mamba2, mlstm, parallel,
                              position_errors, write_stack)
from oracle import layer_stack as ls


# ---- mechanisms ------------------------------------------------------------------------------------
def test_half_split_rotation():
    x = np.arange(1.0, 7.0).reshape(1, 6)
    out = ls.rotate_halves(x, [1], dict(dims=4, base=100.0))
    for i, f in enumerate((1.0, 0.1)):
        u, v = x[0, i], x[0, i + 2]
        assert np.allclose(out[0, [i, i + 2]], [u * np.cos(f) - v * np.sin(f), v * np.cos(f) + u * np.sin(f)])
    assert np.array_equal(out[0, 4:], x[0, 4:])


def test_window_counts_the_token_itself():
    m = ls.window_mask(5, 2)
    assert m.sum(axis=1).tolist() == [1, 2, 2, 2, 2] and m[3].tolist() == [False, False, True, True, False]
    assert np.array_equal(ls.window_mask(4, 1), np.eye(4, dtype=bool)) and np.array_equal(ls.window_mask(4, None), np.tril(np.ones((4, 4), bool)))


def test_sink_takes_its_share_of_the_weights():
    s = np.log(np.array([[[3.0, 6.0]]]))
    assert np.allclose(ls.softmax_with_sink(s, np.ones((1, 2), bool))[0, 0], [0.3, 0.6])
    assert np.allclose(ls.softmax_with_sink(s, np.array([[True, False]]))[0, 0], [0.75, 0.0])
    assert np.allclose(ls.softmax_with_sink(s - 500.0, np.ones((1, 2), bool)), 0.0) and np.allclose(ls.softmax_with_sink(s + 500.0, np.ones((1, 2), bool))[0, 0], [1 / 3, 2 / 3])


def test_decayed_outer_products_by_hand():
    k, v = np.array([[[1.0, 0.0]], [[0.0, 1.0]], [[1.0, 1.0]]]), np.array([[[2.0]], [[3.0]], [[5.0]]])
    o = ls.decayed_outer_products(np.ones((3, 1, 2)), k, v, np.array([[0.7], [0.5], [0.1]]))
    assert np.allclose(o[:, 0, 0], [2.0, 0.5 * 2 + 3, 0.1 * 4 + 10])


def test_matrix_memory_does_not_depend_on_its_stabiliser():
    """Against the unstabilised sums in the range where those do not overflow; the first token's maximum
    starts at zero, not at minus infinity."""
    rng = np.random.default_rng(0)
    T, dk, dv = 12, 4, 3
    q, k, v = (rng.standard_normal((T, 1, n)) for n in (dk, dk, dv))
    i, f = rng.uniform(-4, 4, (T, 1)), -rng.uniform(0, 2, (T, 1))
    got = ls.matrix_memory(q, k, v, i, f)
    S, n, m = np.zeros((dk, dv)), np.zeros(dk), 0.0
    for t in range(T):
        S, n = np.exp(f[t, 0]) * S + np.exp(i[t, 0]) * np.outer(k[t, 0], v[t, 0]), np.exp(f[t, 0]) * n + np.exp(i[t, 0]) * k[t, 0]
        m = max(f[t, 0] + m, i[t, 0])
        e = np.exp(-m)
        assert np.allclose(got[t, 0], (S.T @ q[t, 0]) * e / (max(abs(n @ q[t, 0]) * e, e) + 1e-6))


def test_gelu_is_the_exact_one():
    assert np.allclose(ls.gelu_erf(np.array([-1.0, 0.0, 2.0])), [-0.15865525393, 0.0, 1.95449973610])


def test_layer_runs_repeat_the_loop():
    cfg = lofudra([None] * 5, loop=(1, 3, 3))
    assert ls.layer_runs(cfg) == [(0, 0, False), (1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False), (1, 2, True), (2, 2, False),
                                  (3, 0, False), (4, 0, False)]
    assert ls.layer_runs(lofudra([None] * 2)) == [(0, 0, False), (1, 0, False)]


@pytest.mark.parametrize("name", sorted(LOFUDRA_CONFIGS))
def test_a_sequence_does_not_depend_on_what_follows(name):
    cfg = LOFUDRA_CONFIGS[name]
    w = lofudra_weights(cfg, 3)
    t = np.random.default_rng(2).integers(0, cfg["vocab"], 12)
    assert np.allclose(ls.forward(cfg, w, t)[:7], ls.forward(cfg, w, t[:7]), atol=1e-9)


# ---- planted mistakes ------------------------------------------------------------------------------------
def _mistakes():
    def patch(name, make):
        return lambda mp: mp.setattr(ls, name, make(getattr(ls, name)))

    split = lambda real: (lambda *a: np.concatenate([real(*[x[:9] for x in a]), real(*[x[9:] for x in a])]))
    conv_early = lambda real: (lambda x, w: real(np.concatenate([np.zeros_like(x[:1]), x[:-1]]), w))
    half_turn = lambda real: (lambda x, pos, rot: ls.rotate_pairs(x, pos, rot))

    def normed_values(real):   # values that are the normed, rotated keys
        def mixer(h, w, p, m, eps):
            T, H, G, dim = len(h), m["heads"], m["kv_heads"], m["dim"]
            q, k = ((h @ w[p + n].T + w[p + n + ".b"]).reshape(T, -1, dim) for n in "qk")
            q, k = (ls.rotate_halves(ls.rms_norm(x, w[p + n + ".norm"], eps), np.arange(T), m["rot"]) for x, n in ((q, "q"), (k, "k")))
            k = k[:, np.arange(H) // (H // G)]
            a = ls.softmax_with_sink(np.einsum("ihd,jhd->hij", q, k) * m["scale"], ls.window_mask(T, m["mask"]["size"]))
            return np.einsum("hij,jhd->ihd", a, k).reshape(T, -1) @ w[p + "o"].T
        return mixer

    def no_embedding_again(real):
        return lambda cfg: [(i, 0 if b else t, b) for i, t, b in real(cfg)]

    return [("attention", "window_one_wider", patch("window_mask", lambda real: lambda T, n: real(T, n + 1))),
            ("attention", "window_one_narrower", patch("window_mask", lambda real: lambda T, n: real(T, n - 1))),
            ("attention", "no_sink", patch("softmax_with_sink", lambda real: lambda s, seen: real(s, seen, 0.0))),
            ("attention", "adjacent_pairs", patch("rotate_halves", half_turn)),
            ("attention", "normed_values", patch("window_attention", normed_values)),
            ("retention", "lost_state", patch("decayed_outer_products", split)),
            ("mamba2", "lost_state", patch("decayed_outer_products", split)),
            ("mamba2", "conv_one_early", patch("causal_conv", conv_early)),
            ("mlstm", "lost_state", patch("matrix_memory", split)),
            ("loop", "no_embedding_again", patch("layer_runs", no_embedding_again))]


ONE = {
    "attention": lofudra([parallel(window=7, right_scale=0.0, ff=0)]),
    "retention": lofudra([parallel(left_scale=0.0, decay=[0.9, 0.99, 0.999])]),
    "mamba2": lofudra([mamba2()]),
    "mlstm": lofudra([mlstm(ff=0), mlstm(ff=48)]),
    "loop": lofudra([mlstm(), mamba2()], loop=(0, 2, 3)),
}


@pytest.mark.parametrize("kind,what,plant", _mistakes(), ids=lambda x: x if isinstance(x, str) else "")
def test_planted_mistakes_show_in_the_logits(monkeypatch, kind, what, plant):
    cfg = ONE[kind]
    w = lofudra_weights(cfg, 7, sharp=2.0)
    t = np.random.default_rng(8).integers(0, cfg["vocab"], 24)
    right = ls.forward(cfg, w, t)
    plant(monkeypatch)
    wrong = ls.forward(cfg, w, t)
    assert logit_error(wrong, right) > 20 * F32_TOL
    assert np.quantile(position_errors(wrong, right)[9:], 0.6) > BF16_MEDIAN


# ---- configuration reader -----------------------------------------------------------------------------
@pytest.mark.parametrize("name", sorted(LOFUDRA_CONFIGS))
def test_config_reader_takes_every_size_from_the_file(tmp_path, name):
    from pie_amd import driver as drvmod

    cfg = LOFUDRA_CONFIGS[name]
    info = drvmod.snapshot_info(write_stack(tmp_path / "m", cfg, lofudra_weights(cfg)))
    assert info["arch"] == "lofudra" and info["hidden"] == cfg["width"] and info["vocab"] == cfg["vocab"]
    assert np.isclose(info["rms_eps"], cfg["norm"]["eps"]) and info["logit_scale"] == 1 and info["logit_softcap"] == 0
    loop = cfg.get("loop", dict(start=0, stop=0, times=1))
    assert info["loop"] == [loop["start"], loop["stop"], loop["times"]]
    assert len(info["stack"]) == len(cfg["layers"])
    for got, want in zip(info["stack"], cfg["layers"]):
        m = want["mixer"]
        assert got["type"] == want["type"] and got["ff"] == (want["mlp"]["ff"] if want["mlp"] else 0)
        memory = got["memory"]
        if want["type"] == "parallel":
            a = got["attention"]
            for k in ("heads", "kv_heads", "dim", "vdim"):
                assert a[k] == m["left"][k]
            assert a["window"] == m["left"]["mask"]["size"] and np.isclose(a["scale"], m["left"]["scale"]) and a["sink"] == 1
            assert a["rot_dims"] == m["left"]["rot"]["dims"] and np.isclose(a["rot_base"], m["left"]["rot"]["base"])
            assert np.isclose(got["attention_scale"], m["left_scale"]) and np.isclose(got["memory_scale"], m["right_scale"])
            assert np.allclose(memory["decay"], m["right"]["decay"], rtol=1e-5)
            m = m["right"]
        if want["type"] == "mamba2":
            assert (memory["kv_heads"], memory["dim"], memory["conv"], memory["norm_groups"]) == (m["groups"], m["state"], m["conv"], m["norm_groups"])
        else:
            assert memory["kv_heads"] == m["heads"] and memory["dim"] == m["dim"]
        assert memory["heads"] == m["heads"] and memory["vdim"] == m["vdim"] and np.isclose(memory["gate_cap"], m.get("gate_cap", 0))


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="convolution"), "unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("gate_cap"), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].pop("groups"), "groups"),
    (lambda c: c["layers"][2]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][2]["mixer"]["left"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][2]["mixer"]["right"].update(decay="slow"), "decay"),
    (lambda c: c["loop"].pop("stop"), "stop"),
])
def test_config_reader_names_what_is_wrong(tmp_path, change, message):
    from pie_amd import driver as drvmod

    cfg = json.loads(json.dumps(LOFUDRA_CONFIGS["trio"]))
    d = write_stack(tmp_path / "m", cfg, lofudra_weights(cfg))
    change(cfg)
    (tmp_path / "m" / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(RuntimeError, match=message):
        drvmod.snapshot_info(d)
