"""CPU: the mechanisms of Fobanex's oracle on hand-made cases, planted mistakes that the GPU tests' tolerances must
tell apart, and the configuration reader."""
import json

import numpy as np
import pytest

from layer_stack_util import (BF16_MEDIAN, F32_TOL, FOBANEX_CONFIGS, dense, fobanex, fobanex_weights, key_value_attention, logit_error, moe,
                              normed_attention, position_errors, rotary, shared_latent, write_stack)
from oracle import layer_stack as ls


# ---- mechanisms ------------------------------------------------------------------------------------
def test_router_keeps_whole_groups():
    """The two best experts are in different groups; with one group kept, the second comes from the winner's."""
    p = np.array([[0.30, 0.05, 0.25, 0.20, 0.15, 0.05]])
    z = np.log(p) + 3.0
    both = ls.route(z, dict(experts=6, top=2, scale=2.0, groups=dict(count=3, keep=3)))
    assert np.allclose(both, [[2 * 0.30 / 0.55, 0, 2 * 0.25 / 0.55, 0, 0, 0]])
    one = ls.route(z, dict(experts=6, top=2, scale=1.0, groups=dict(count=3, keep=1)))
    assert np.allclose(one, [[0.30 / 0.35, 0.05 / 0.35, 0, 0, 0, 0]])
    two = ls.route(z, dict(experts=6, top=3, scale=1.0, groups=dict(count=3, keep=2)))
    assert np.allclose(two, [[0.30 / 0.75, 0, 0.25 / 0.75, 0.20 / 0.75, 0, 0]])
    assert np.allclose(ls.route(z, dict(experts=6, top=1, scale=3.0)), [[3.0, 0, 0, 0, 0, 0]])


def test_expert_clamps_the_gate_above_and_the_other_on_both_sides():
    w = {"e.gate": np.array([[1.0]]), "e.up": np.array([[-2.0]]), "e.down": np.array([[1.0]])}
    f = lambda h: ls.clamped_expert(np.array([[h]]), w, "e.", 1.5)[0, 0]
    rule = lambda g, u: g / (1 + np.exp(-1.702 * g)) * (u + 1)
    assert np.isclose(f(0.5), rule(0.5, -1.0)) and np.isclose(f(4.0), rule(1.5, -1.5)) and np.isclose(f(-3.0), rule(-3.0, 1.5))


def test_gated_feed_forward_has_three_biases():
    w = {"m.gate": np.array([[2.0]]), "m.gate.b": np.array([0.5]), "m.up": np.array([[1.0]]), "m.up.b": np.array([-3.0]),
         "m.down": np.array([[4.0]]), "m.down.b": np.array([7.0])}
    g = 2.5
    assert np.isclose(ls.gated_feed_forward(np.array([[1.0]]), w, "m.")[0, 0], g / (1 + np.exp(-g)) * -2.0 * 4.0 + 7.0)


def test_query_heads_read_their_groups_key_head():
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((3, 6, 4)), rng.standard_normal((3, 2, 4)), rng.standard_normal((3, 2, 5))
    o = ls.grouped_attention(q, k, v, 0.5)
    for h in range(6):
        s = np.exp(0.5 * q[2, h] @ k[:, h // 3].T)
        assert np.allclose(o[2, h], s @ v[:, h // 3] / s.sum())
    assert np.allclose(o[0], np.repeat(v[0], 3, axis=0))


def test_one_norm_covers_all_heads():
    """Scaling one head's projection changes the other heads' keys: the norm is over both."""
    cfg = fobanex([normed_attention(heads=2, kv_heads=2, dim=8, vdim=4, rot=rotary(4))], width=16)
    w = {k: v.astype(np.float64) for k, v in fobanex_weights(cfg, 1).items()}
    h = np.random.default_rng(1).standard_normal((5, 16))
    a = ls.normed_attention(h, w, "l0.mix.", cfg["layers"][0]["mixer"], 1e-4)
    w["l0.mix.q"] = w["l0.mix.q"] * np.repeat([3.0, 1.0], 8)[:, None]
    b = ls.normed_attention(h, w, "l0.mix.", cfg["layers"][0]["mixer"], 1e-4)
    other = w["l0.mix.o"].copy()
    other[:, :4] = 0.0   # (what the second head adds)
    assert np.abs((np.linalg.pinv(w["l0.mix.o"]) @ (a - b).T)[4:]).max() > 1e-3


def test_a_layer_reads_the_latents_of_the_layer_it_names():
    cfg = fobanex([shared_latent(), shared_latent(), shared_latent(0), shared_latent(1)])
    w = {k: v.astype(np.float64) for k, v in fobanex_weights(cfg, 2).items()}
    t = np.random.default_rng(3).integers(0, cfg["vocab"], 9)
    _, s = ls.forward(cfg, w, t, True)
    c, kr = ls.latent_of(ls.rms_norm(s[0], w["l1.norm1"], 1e-4), w, "l1.mix.", cfg["layers"][1]["mixer"], 1e-4)
    h = ls.rms_norm(s[2], w["l3.norm1"], 1e-4)
    assert np.allclose(s[3] - s[2], ls.gated_latent_attention(h, w, "l3.mix.", cfg["layers"][3]["mixer"], 1e-4, (c, kr)))


@pytest.mark.parametrize("name", sorted(FOBANEX_CONFIGS))
def test_a_sequence_does_not_depend_on_what_follows(name):
    cfg = FOBANEX_CONFIGS[name]
    w = fobanex_weights(cfg, 3)
    t = np.random.default_rng(2).integers(0, cfg["vocab"], 12)
    assert np.allclose(ls.forward(cfg, w, t)[:7], ls.forward(cfg, w, t[:7]), atol=1e-9)


# ---- planted mistakes ------------------------------------------------------------------------------------
def _mistakes():
    def patch(name, make):
        def plant(mp):
            real = getattr(ls, name)
            mp.setattr(ls, name, make(real))
            for kind, f in ls.SHARED_AHEAD_MIXERS.items():
                if f is real:
                    mp.setitem(ls.SHARED_AHEAD_MIXERS, kind, getattr(ls, name))
        return plant

    def norm_per_head(real):
        def mixer(h, w, p, m, eps, shared=None):
            T, dim = len(h), m["dim"]
            q, k = (ls.rms_norm((h @ w[p + n].T).reshape(T, -1, dim), w[p + n + ".norm"].reshape(-1, dim), eps) for n in "qk")
            o = ls.grouped_attention(ls.rotate_heads(q, m["rot"]), ls.rotate_heads(k, m["rot"]), (h @ w[p + "v"].T).reshape(T, -1, m["vdim"]), m["scale"])
            return o.reshape(T, -1) @ w[p + "o"].T
        return mixer

    def rotated_values(real):
        def mixer(h, w, p, m, eps, shared=None):
            T = len(h)
            q, k = (ls.rotate_heads((h @ w[p + n].T).reshape(T, -1, m["dim"]), m["rot"]) for n in "qk")
            return (ls.grouped_attention(q, k, k, m["scale"]).reshape(T, -1) * ls.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T
        return mixer

    no_gate = lambda real: (lambda h, w, p, *a: real(h, {**w, p + "g": 0 * w[p + "g"]}, p, *a) * 2)
    half_split = lambda real: (lambda x, rot: ls.rotate_halves(x, np.arange(len(x)), rot))
    no_scaling = lambda real: (lambda rot: real(dict(rot, scaling=None)))
    no_factor = lambda real: (lambda rot: (real(rot)[0], 1.0))
    own_latents = lambda real: (lambda h, w, p, m, eps, shared=None: real(h, {**w, p + "dkv": w["l0.mix.dkv"], p + "dkv.norm": w["l0.mix.dkv.norm"]}, p, m, eps, None))
    unturned = lambda real: (lambda h, w, p, m, eps: (real(h, w, p, m, eps)[0], (h @ w[p + "dkv"].T)[:, m["kv_rank"]:]))
    router = lambda **change: (lambda real: (lambda z, r: real(z, {**r, **change})))
    not_divided = lambda real: (lambda z, r: np.where(real(z, r) > 0, np.exp(z - z.max(-1, keepdims=True)) / np.exp(z - z.max(-1, keepdims=True)).sum(-1, keepdims=True), 0) * r["scale"])

    def expert(rule):
        return lambda real: (lambda h, w, p, limit: rule(h @ w[p + "gate"].T, h @ w[p + "up"].T, limit) @ w[p + "down"].T)

    no_bias = lambda name: (lambda real: (lambda h, w, p: real(h, {**w, p + name + ".b": 0 * w[p + name + ".b"]}, p)))
    return [("attention", "norm_per_head", patch("normed_attention", norm_per_head)),
            ("attention", "half_split", patch("rotate_heads", half_split)),
            ("attention", "no_scaling", patch("rotation_frequencies", no_scaling)),
            ("attention", "no_factor_on_cos_and_sin", patch("rotation_frequencies", no_factor)),
            ("attention_2", "rotated_values", patch("key_value_attention", rotated_values)),
            ("attention_2", "no_gate", patch("key_value_attention", no_gate)),
            ("attention_2", "half_split", patch("rotate_heads", half_split)),
            ("latent", "adjacent_pairs", patch("rotate_halves", lambda real: ls.rotate_pairs)),
            ("latent", "no_gate", patch("gated_latent_attention", no_gate)),
            ("latent", "key_not_rotated", patch("latent_of", unturned)),
            ("shared", "latents_of_its_own_input", patch("gated_latent_attention", own_latents)),
            ("mixture", "groups_ignored", patch("route", router(groups=None))),
            ("mixture", "one_group_more", patch("route", router(groups=dict(count=3, keep=3)))),
            ("mixture", "no_scale", patch("route", router(scale=1.0))),
            ("mixture", "not_divided_by_the_sum", patch("route", not_divided)),
            ("mixture", "no_clamp", patch("clamped_expert", lambda real: lambda h, w, p, limit: real(h, w, p, 1e9))),
            ("mixture", "gate_clamped_below", patch("clamped_expert", expert(lambda g, u, l: (lambda c: c * ls.sigmoid(1.702 * c))(np.clip(g, -l, l)) * (np.clip(u, -l, l) + 1)))),
            ("mixture", "plain_slope", patch("clamped_expert", expert(lambda g, u, l: ls.silu(np.minimum(g, l)) * (np.clip(u, -l, l) + 1)))),
            ("mixture", "nothing_added", patch("clamped_expert", expert(lambda g, u, l: (lambda c: c * ls.sigmoid(1.702 * c))(np.minimum(g, l)) * np.clip(u, -l, l)))),
            ("dense", "no_gate_bias", patch("gated_feed_forward", no_bias("gate"))),
            ("dense", "no_up_bias", patch("gated_feed_forward", no_bias("up"))),
            ("dense", "no_down_bias", patch("gated_feed_forward", no_bias("down")))]


# (two layers where the first alone would end in one token's mix of few values)
ONE = {
    "attention": fobanex([normed_attention(rot=dict(rotary(16, 50.0), scaling=dict(factor=4.0, original=64, fast=8.0, slow=0.5)))], scale=0.1),
    "attention_2": fobanex([key_value_attention()], scale=0.1),
    "latent": fobanex([shared_latent(rot_dim=16)], scale=0.1),
    "shared": fobanex([shared_latent(), shared_latent(0)], scale=0.1),
    "mixture": fobanex([normed_attention(mlp=moe(top=3, keep=1, limit=0.6))], scale=0.3),
    "dense": fobanex([key_value_attention(mlp=dense(48))], scale=0.3),
}


@pytest.mark.parametrize("kind,what,plant", _mistakes(), ids=lambda x: x if isinstance(x, str) else "")
def test_planted_mistakes_show_in_the_logits(monkeypatch, kind, what, plant):
    cfg = ONE[kind]
    w = {k: v.astype(np.float64) for k, v in fobanex_weights(cfg, 7, sharp=3.0).items()}
    t = np.random.default_rng(8).integers(0, cfg["vocab"], 24)
    right = ls.forward(cfg, w, t)
    plant(monkeypatch)
    wrong = ls.forward(cfg, w, t)
    assert logit_error(wrong, right) > 20 * F32_TOL
    assert np.quantile(position_errors(wrong, right)[9:], 0.6) > BF16_MEDIAN


# ---- configuration reader -----------------------------------------------------------------------------
@pytest.mark.parametrize("name", sorted(FOBANEX_CONFIGS))
def test_config_reader_takes_every_size_from_the_file(tmp_path, name):
    from pie_amd import driver as drvmod

    cfg = FOBANEX_CONFIGS[name]
    info = drvmod.snapshot_info(write_stack(tmp_path / "m", cfg, fobanex_weights(cfg)))
    assert info["arch"] == "fobanex" and info["hidden"] == cfg["width"] and info["vocab"] == cfg["vocab"]
    assert np.isclose(info["rms_eps"], cfg["norm"]["eps"]) and np.isclose(info["embed_scale"], cfg["embedding"]["scale"])
    assert len(info["stack"]) == len(cfg["layers"])
    for got, want in zip(info["stack"], cfg["layers"]):
        m, mlp = want["mixer"], want["mlp"]
        assert got["ff"] == (mlp["ff"] if mlp and mlp["kind"] == "dense" else 0) and ("mixture" in got) == bool(mlp and mlp["kind"] == "moe")
        if "mixture" in got:
            e, r = got["mixture"], mlp["router"]
            groups = r.get("groups") or dict(count=1, keep=1)
            assert (e["experts"], e["top"], e["ff"], e["groups"], e["keep"]) == (r["experts"], r["top"], mlp["expert"]["ff"], groups["count"], groups["keep"])
            assert np.isclose(e["scale"], r["scale"]) and np.isclose(e["limit"], mlp["expert"]["limit"])
        if want["type"] == "latent_attention":
            assert all(got[k] == m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
            assert got["half_split"] and got["gate"] and got["kv_from"] == m.get("kv_from", -1) and got["rot_dims"] == m["rot"]["dims"]
            assert np.isclose(got["scale"], m["scale"]) and np.isclose(got["rot_base"], m["rot"]["base"])
        else:
            a, first = got["attention"], want["type"] == "attention"
            assert all(a[k] == m[k] for k in ("heads", "kv_heads", "dim", "vdim")) and got["type"] == "attention" and a["window"] == 0 and a["sink"] == 0
            assert a["rot_dims"] == m["rot"]["dims"] and np.isclose(a["rot_base"], m["rot"]["base"]) and np.isclose(a["scale"], m["scale"])
            assert not a["half_split"] and not a["biases"] and a["own_values"] == first and a["gate"] != first and a["norm"] == (2 if first else 0)


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][2].update(type="attention_3"), "unknown mixer"),
    (lambda c: c["layers"][1]["mlp"].update(kind="sparse"), "unknown mlp kind"),
    (lambda c: c["layers"][1]["mlp"].pop("router"), "router"),
    (lambda c: c["layers"][1]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda c: c["layers"][1]["mlp"]["router"].pop("top"), "top"),
    (lambda c: c["layers"][1]["mixer"].update(kv_from=-2), "kv_from"),
    (lambda c: c["layers"][0]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][3]["mixer"].pop("kv_heads"), "kv_heads"),
])
def test_config_reader_names_what_is_wrong(tmp_path, change, message):
    from pie_amd import driver as drvmod

    cfg = json.loads(json.dumps(FOBANEX_CONFIGS["quartet"]))
    d = write_stack(tmp_path / "m", cfg, fobanex_weights(cfg))
    change(cfg)
    (tmp_path / "m" / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(RuntimeError, match=message):
        drvmod.snapshot_info(d)
