"""CPU: the layer-stack oracle's mechanisms on hand-made cases, planted mistakes that the GPU tests'
tolerances must tell apart, the configuration reader, and the page / slot bookkeeping."""
import json

import numpy as np
import pytest

from layer_stack_util import (ATTENTION_ONLY, BF16_MEDIAN, CONFIGS, DELTA_ONLY, F32_TOL, logit_error, position_errors, random_weights,
                              rotary, write_stack)
from oracle import layer_stack as ls


# ---- mechanisms ------------------------------------------------------------------------------------
def test_rotation_turns_adjacent_pairs_and_leaves_the_rest():
    x = np.arange(1.0, 7.0).reshape(1, 6)
    out = ls.rotate_pairs(x, [1], dict(dims=4, base=100.0))
    f = np.array([1.0, 0.1])
    for i in range(2):
        u, v = x[0, 2 * i], x[0, 2 * i + 1]
        assert np.allclose(out[0, 2 * i:2 * i + 2], [u * np.cos(f[i]) - v * np.sin(f[i]), v * np.cos(f[i]) + u * np.sin(f[i])])
    assert np.array_equal(out[0, 4:], x[0, 4:])


def test_rotated_scores_depend_on_the_distance_only():
    rng = np.random.default_rng(1)
    q, k = rng.standard_normal((2, 1, 8))
    rot = rotary(8)
    s = [float((ls.rotate_pairs(q, [p + 5], rot) * ls.rotate_pairs(k, [p], rot)).sum()) for p in (0, 3, 400)]
    assert np.allclose(s, s[0])


def test_yarn_frequencies_between_the_unscaled_and_the_stretched():
    rot = dict(dims=32, base=10000.0, scaling=dict(factor=4.0, original=256, fast=16.0, slow=1.0))
    f, m = ls.rotation_frequencies(rot)
    base = 10000.0 ** (-2.0 * np.arange(16) / 32)
    assert np.isclose(f[0], base[0]) and np.isclose(f[-1], base[-1] / 4.0)
    assert ((f <= base + 1e-15) & (f >= base / 4.0 - 1e-15)).all() and (np.diff(f) < 0).all()
    assert np.isclose(m, 0.1 * np.log(4.0) + 1.0)
    assert ls.rotation_frequencies(dict(dims=32, base=10000.0))[1] == 1.0


def test_convolution_looks_back_over_its_taps():
    x = np.array([[1.0], [10.0], [100.0]])
    assert np.allclose(ls.causal_conv(x, np.array([[3.0, 2.0, 1.0]]))[:, 0], [1.0, 12.0, 123.0])
    assert np.allclose(ls.causal_conv(x, np.array([[5.0]]))[:, 0], [5.0, 50.0, 500.0])


def test_delta_rule_reads_back_what_it_wrote():
    """Step size 1, no decay, orthonormal keys: the state is an exact store, a rewritten key keeps
    the newest value only, and the read-out sees the token's own write."""
    e = np.eye(3)
    k = np.stack([e[0], e[1], e[0]])[:, None]
    v = np.array([[1.0, 2.0], [3.0, 4.0], [5.0, 6.0]])[:, None]
    ones, beta = np.ones((3, 1, 3)), np.ones((3, 1))
    assert np.allclose(ls.delta_rule(k, k, v, ones, beta)[:, 0], v[:, 0])
    q = np.stack([e[0], e[0], e[1]])[:, None]
    assert np.allclose(ls.delta_rule(q, k, v, ones, beta)[:, 0], [[1, 2], [1, 2], [3, 4]])
    g = ones.copy()
    g[2, 0, 1] = 0.5   # the decay acts on the key channel's row
    assert np.allclose(ls.delta_rule(q, k, v, g, beta)[2, 0], [1.5, 2.0])


def test_attention_sees_its_own_and_earlier_keys_only():
    s = np.zeros((1, 3, 3))
    v = np.array([[1.0], [2.0], [6.0]])[:, None]
    assert np.allclose(ls.causal_softmax_attention(s, v)[:, 0, 0], [1.0, 1.5, 3.0])


def test_norm_has_eps_inside_the_root():
    x = np.array([[3e-3, 4e-3]])
    assert np.allclose(ls.rms_norm(x, 2.0, 1e-4), 2.0 * x / np.sqrt(12.5e-6 + 1e-4))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_sequence_does_not_depend_on_what_follows(name):
    cfg = CONFIGS[name]
    w = random_weights(cfg, 3)
    t = np.random.default_rng(2).integers(0, cfg["vocab"], 12)
    assert np.allclose(ls.forward(cfg, w, t)[:7], ls.forward(cfg, w, t[:7]), atol=1e-9)


# ---- planted mistakes: each must show far above the tolerance of the test that would catch it -------
def _mistakes():
    def drop_yarn_factor(mp):
        real = ls.rotation_frequencies
        mp.setattr(ls, "rotation_frequencies", lambda r: (real(r)[0], 1.0))

    def unscaled_frequencies(mp):
        real = ls.rotation_frequencies
        mp.setattr(ls, "rotation_frequencies", lambda r: (real({k: r[k] for k in ("dims", "base")})[0], real(r)[1]))

    def half_split_pairs(mp):
        def rot(x, positions, r):
            n = int(r["dims"])
            perm = np.concatenate([np.arange(0, n, 2), np.arange(1, n, 2), np.arange(n, x.shape[-1])])
            inv = np.argsort(perm)
            return real(x[..., inv], positions, r)[..., perm]
        real = ls.rotate_pairs
        mp.setattr(ls, "rotate_pairs", rot)

    def conv_one_early(mp):
        real = ls.causal_conv
        mp.setattr(ls, "causal_conv", lambda x, w: real(np.concatenate([np.zeros_like(x[:1]), x[:-1]]), w))

    def lost_state(mp):
        real = ls.delta_rule
        mp.setattr(ls, "delta_rule", lambda *a: np.concatenate([real(*[x[:9] for x in a]), real(*[x[9:] for x in a])]))

    def decay_on_values(mp):
        def rule(q, k, v, g, beta):
            return real(q, k, v, np.repeat(g.mean(axis=-1, keepdims=True), g.shape[-1], -1), beta)
        real = ls.delta_rule
        mp.setattr(ls, "delta_rule", rule)

    def read_before_write(mp):
        def rule(q, k, v, g, beta):
            S, out = np.zeros((q.shape[1], q.shape[2], v.shape[2])), np.empty_like(v)
            for t in range(len(q)):
                S = g[t][:, :, None] * S
                out[t] = np.einsum("hkv,hk->hv", S, q[t])
                S = S + k[t][:, :, None] * (beta[t][:, None] * (v[t] - np.einsum("hkv,hk->hv", S, k[t])))[:, None, :]
            return out
        mp.setattr(ls, "delta_rule", rule)

    def one_key_short(mp):
        def att(s, v):
            T = s.shape[1]
            seen = np.tril(np.ones((T, T), bool))
            seen[T - 1, 0] = False
            p = np.exp(np.where(seen, s, -np.inf) - s.max(axis=-1, keepdims=True))
            return np.einsum("hij,jhd->ihd", p / p.sum(axis=-1, keepdims=True), v)
        mp.setattr(ls, "causal_softmax_attention", att)

    def plain_relu(mp):
        mp.setattr(ls, "squared_relu", lambda z: np.maximum(z, 0.0))

    return [("latent", drop_yarn_factor), ("latent", unscaled_frequencies), ("latent", half_split_pairs), ("latent", one_key_short),
            ("latent", plain_relu), ("delta", conv_one_early), ("delta", lost_state), ("delta", decay_on_values),
            ("delta", read_before_write)]


@pytest.mark.parametrize("kind,plant", _mistakes(), ids=lambda x: getattr(x, "__name__", x))
def test_planted_mistakes_show_in_the_logits(monkeypatch, kind, plant):
    cfg = ATTENTION_ONLY if kind == "latent" else DELTA_ONLY
    w = random_weights(cfg, 7, sharp=3.0)
    t = np.random.default_rng(8).integers(0, cfg["vocab"], 24)
    right = ls.forward(cfg, w, t)
    plant(monkeypatch)
    wrong = ls.forward(cfg, w, t)
    err = logit_error(wrong, right)
    assert err > 20 * F32_TOL
    if plant.__name__ != "one_key_short":   # (one key of many: the fp32 tests and the kernel tests' spikes catch it)
        assert np.median(position_errors(wrong, right)[9:]) > BF16_MEDIAN


# ---- configuration reader -----------------------------------------------------------------------------
def _info(tmp_path, cfg, seed=0):
    from pie_amd import driver as drvmod

    return drvmod.snapshot_info(write_stack(tmp_path / "m", cfg, random_weights(cfg, seed)))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_config_reader_takes_every_size_from_the_file(tmp_path, name):
    cfg = CONFIGS[name]
    info = _info(tmp_path, cfg)
    assert info["arch"] == "varasun" and info["hidden"] == cfg["width"] and info["vocab"] == cfg["vocab"]
    assert np.isclose(info["rms_eps"], cfg["norm"]["eps"]) and np.isclose(info["logit_scale"], cfg["logit_scale"])
    assert np.isclose(info["logit_softcap"], cfg["logit_softcap"])
    assert len(info["stack"]) == len(cfg["layers"])
    for got, want in zip(info["stack"], cfg["layers"]):
        m = want["mixer"]
        assert got["type"] == want["type"] and got["ff"] == (want["mlp"]["ff"] if want["mlp"] else 0)
        for k in m:
            if k in ("rot", "scale"):
                continue
            assert got[k] == m[k], k
        if "rot" in m:
            assert got["rot_dims"] == m["rot"]["dims"] and np.isclose(got["rot_base"], m["rot"]["base"])
            assert np.isclose(got["scale"], m["scale"]) and got["yarn"] == ("scaling" in m["rot"])


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="convolution"), "unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][0]["mlp"].update(kind="gated"), "unknown mlp"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.update(architecture="Unknown"), "unsupported architecture"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_config_reader_names_what_is_wrong(tmp_path, change, message):
    from pie_amd import driver as drvmod

    cfg = json.loads(json.dumps(CONFIGS["mixed"]))
    d = write_stack(tmp_path / "m", cfg, random_weights(cfg))
    change(cfg)
    (tmp_path / "m" / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(RuntimeError, match=message):
        drvmod.snapshot_info(d)


# ---- pages and slots -------------------------------------------------------------------------------------
class FakeDriver:
    """Records the frames an Engine builds; answers every sampling slot with token 1."""

    def __init__(self, pages=8, page_size=16, slots=2, recurrent=True):
        self.caps = dict(kv_page_size=page_size, max_forward_tokens=64, total_pages=pages, rs_cache_slots=slots, rs_cache_required=recurrent)
        self.calls = []

    def capabilities(self):
        return self.caps

    def forward(self, frame):
        from pie_amd.driver import _u32_list as ints

        f = frame.frame.payload.forward
        self.calls.append(dict(tokens=ints(f.token_ids), positions=ints(f.position_ids), pages=ints(f.kv_page_indices),
                               indptr=ints(f.kv_page_indptr), last=ints(f.kv_last_page_lens), qo=ints(f.qo_indptr),
                               slots=ints(f.rs_slot_ids)))
        R = len(self.calls[-1]["qo"]) - 1

        class Result:
            num_requests = R

            def tokens_of(self, r):
                return [1]

            def logits_of(self, r):
                return [np.zeros(4, np.float32)]
        return Result()


def test_engine_gives_pages_and_slots_back_and_uses_them_again():
    from pie_amd.engine import Engine, OutOfPages

    d = FakeDriver()
    e = Engine(d)
    e.step([("a", list(range(17)), [16]), ("b", [1], [])])
    c = d.calls[-1]
    assert c["positions"] == list(range(17)) + [0] and c["indptr"] == [0, 2, 3] and c["last"] == [1, 1]
    assert len(set(c["pages"])) == 3 and c["slots"] == [0, 1]
    with pytest.raises(OutOfPages):
        e.step([("c", [1], [])])   # no slot is free
    held = set(c["pages"][:2])
    e.finish("a")
    e.step([("c", list(range(33)), []), ("b", [5], [0])])
    c = d.calls[-1]
    assert held <= set(c["pages"][:3]) and c["slots"] == [0, 1]
    assert c["positions"][-1] == 1 and c["pages"][3:] == d.calls[0]["pages"][2:]
    with pytest.raises(OutOfPages):
        e.step([("b", [0] * 100, [])])


def test_engine_generates_with_portions_beside_decoded_tokens():
    from pie_amd.engine import Engine

    d = FakeDriver(pages=32, slots=4)
    out = Engine(d).generate({"a": [3] * 20, "b": [4] * 3}, 5, portion=8)
    assert out == {"a": [1] * 5, "b": [1] * 5}
    assert any(sorted(np.diff(c["qo"]).tolist()) == [1, 8] for c in d.calls)
    for c in d.calls:
        assert len(c["tokens"]) <= d.caps["max_forward_tokens"]


def test_planner_checks_the_slot_lists():
    from pie_amd import driver as drvmod

    fr = drvmod.ForwardFrame([1, 2], [0, 0], [0, 1], [0, 1, 2], [1, 1], [0, 1, 2], rs_slot_ids=[0])
    with pytest.raises(ValueError, match="rs_slot_ids"):
        drvmod.plan(fr, 16, 4)
