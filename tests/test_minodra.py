"""CPU: the mechanisms of Minodra's oracle on hand-made cases, planted mistakes that the GPU tests' tolerances must
tell apart, and the configuration reader."""
import json

import numpy as np
import pytest

from layer_stack_util import (BF16_MEDIAN, F32_TOL, MINODRA_CONFIGS, dense, logit_error, minodra, minodra_weights, position_errors, shared_moe,
                              sink_latent, write_stack)
from oracle import layer_stack as ls


# ---- mechanisms ------------------------------------------------------------------------------------
def test_bigram_rows_hash_the_previous_token_and_start_with_the_last_row():
    assert ls.bigram_rows([5, 7, 7, 0], 10, 3, 2).tolist() == [10, (15 + 14) % 10, (21 + 14) % 10, 21 % 10]
    big = ls.bigram_rows([96, 95], 1009, 1 << 40, 12345678901)
    assert big[1] == (96 * (1 << 40) + 95 * 12345678901) % 1009


def test_scalar_norm_has_one_number_for_all_columns():
    x = np.array([[3.0, -4.0]])
    assert np.allclose(ls.scalar_norm(x, np.array(2.0), 0.5), x / np.sqrt(12.5 + 0.5) * 2.0)


def test_a_row_and_its_recent_ones():
    h = np.array([[1.0, 10.0], [2.0, 20.0], [4.0, 40.0]])
    w = np.array([[0.5, 0.25, 2.0], [0.0, 1.0, 0.0]])   # (per column: two rows back, one back, itself)
    want = [[1 + 2.0, 10.0], [2 + 0.25 + 4.0, 20 + 10], [4 + 0.5 + 0.5 + 8.0, 40 + 20]]
    assert np.allclose(ls.with_recent(h, w), want)


def test_learned_sink_takes_weight_without_key_or_value():
    s = np.log(np.array([[[1.0, 9.0], [2.0, 3.0]]]))
    p = ls.softmax_with_learned_sink(s, ls.window_mask(2, None), np.log(np.array([5.0])))
    assert np.allclose(p, [[[1 / 6, 0], [2 / 10, 3 / 10]]])


def test_choice_by_corrected_scores_weights_by_plain_ones():
    s = np.array([[0.9, 0.5, 0.6, 0.2]])
    z = np.log(s / (1 - s))
    assert np.allclose(ls.corrected_route(z, np.array([-0.5, 0.0, 0.0, 0.5]), 2), [[0, 0, 0.6, 0.2]])
    assert np.allclose(ls.corrected_route(z, np.zeros(4), 3), [[0.9, 0.5, 0.6, 0]])


def test_shared_expert_joins_every_token_behind_its_gate():
    cfg = minodra([sink_latent(shared_moe(experts=2, top=1, ff=3, shared=5))], width=8)
    w = {k: v.astype(np.float64) for k, v in minodra_weights(cfg, 1).items()}
    h = np.random.default_rng(1).standard_normal((4, 8))
    mlp = cfg["layers"][0]["mlp"]
    alone = ls.shared_mixture(h, w, "l0.mlp.", dict(mlp, shared=None))
    both = ls.shared_mixture(h, w, "l0.mlp.", mlp)
    assert np.allclose(both - alone, ls.sigmoid(h @ w["l0.mlp.shared.sg"].T) * ls.feed_forward(h, w, "l0.mlp.shared."))


@pytest.mark.parametrize("name", sorted(MINODRA_CONFIGS))
def test_a_sequence_does_not_depend_on_what_follows(name):
    cfg = MINODRA_CONFIGS[name]
    w = minodra_weights(cfg, 3)
    t = np.random.default_rng(2).integers(0, cfg["vocab"], 12)
    assert np.allclose(ls.forward(cfg, w, t)[:7], ls.forward(cfg, w, t[:7]), atol=1e-9)


# ---- planted mistakes ------------------------------------------------------------------------------------
def _mistakes():
    def patch(name, make):
        return lambda mp: mp.setattr(ls, name, make(getattr(ls, name)))

    def weights(*changes):
        """The forward pass with some weights changed: (end of the name, function of the weight)."""
        def make(real):
            def forward(cfg, w, tokens, want_layers=False):
                w = dict(w)
                for end, f in changes:
                    w.update({k: f(v) for k, v in w.items() if k.endswith(end)})
                return real(cfg, w, tokens, want_layers)
            return forward
        return patch("forward_gated", make)

    def config(change):
        def make(real):
            def forward(cfg, w, tokens, want_layers=False):
                cfg = json.loads(json.dumps(cfg))
                change(cfg)
                return real(cfg, w, tokens, want_layers)
            return forward
        return patch("forward_gated", make)

    def sublayer(rule):
        return patch("gated_sublayer", lambda real: rule)

    def gate_after_convolution(x, w, p, n, f, eps):
        h = ls.with_recent(ls.scalar_norm(x, w[f"{p}norm{n}"], eps), w[f"{p}canon{n}"])
        return x + f(h) * ls.sigmoid(h @ w[f"{p}rg{n}"].T + w[f"{p}rg{n}.b"])

    def gate_of_the_stream(x, w, p, n, f, eps):
        h = ls.scalar_norm(x, w[f"{p}norm{n}"], eps)
        return x + f(ls.with_recent(h, w[f"{p}canon{n}"])) * ls.sigmoid(x @ w[f"{p}rg{n}"].T + w[f"{p}rg{n}.b"])

    def whole_gated(x, w, p, n, f, eps):
        h = ls.scalar_norm(x, w[f"{p}norm{n}"], eps)
        return (x + f(ls.with_recent(h, w[f"{p}canon{n}"]))) * ls.sigmoid(h @ w[f"{p}rg{n}"].T + w[f"{p}rg{n}.b"])

    zero, scaled_sink = (lambda v: 0 * v), (lambda real: lambda s, seen, sink: real(s, seen, sink * 0.2))
    twice = lambda real: lambda s, seen, sink: real(s, seen, sink + np.log(2.0))
    first_row = lambda real: lambda t, b, mp, mc: np.concatenate([[0], real(t, b, mp, mc)[1:]])
    first_hashed = lambda real: lambda t, b, mp, mc: np.concatenate([[int(t[0]) * mc % b], real(t, b, mp, mc)[1:]])
    no_previous = lambda real: lambda t, b, mp, mc: np.concatenate([real(t, b, mp, mc)[:1], real(t, b, 0, mc)[1:]])
    lost_previous = lambda real: lambda t, b, mp, mc: np.concatenate([real(t[:8], b, mp, mc), real(t[8:], b, mp, mc)])
    swapped = lambda real: lambda t, b, mp, mc: real(t, b, mc, mp)
    one_early = lambda real: lambda x, w: real(np.concatenate([np.zeros((1, x.shape[1])), x[:-1]]), w)
    reversed_taps = lambda real: lambda x, w: real(x, w[:, ::-1])
    lost_rows = lambda real: lambda x, w: np.concatenate([real(x[:8], w), real(x[8:], w)])
    weights_corrected = lambda real: lambda z, c, top: np.where(real(z, c, top) > 0, real(z, c, top) + c, 0)
    no_correction = lambda real: lambda z, c, top: real(z, 0 * c, top)
    divided = lambda real: lambda z, c, top: real(z, c, top) / real(z, c, top).sum(-1, keepdims=True)
    softmaxed = lambda real: lambda z, c, top: np.where(real(z, c, top) > 0, np.exp(z) / np.exp(z).sum(-1, keepdims=True), 0)
    one_more = lambda real: lambda z, c, top: real(z, c, top + 1)
    once_gated = lambda real: lambda h, w, p, m, eps: real(h, {**w, p + "g": 0 * w[p + "g"]}, p, m, eps) * 2

    def ungated_shared(real):
        return lambda h, w, p, mlp: real(h, dict(w, **{p + "shared.sg": 0 * w[p + "shared.sg"]}), p, mlp) if mlp.get("shared") else real(h, w, p, mlp)

    return [("attention", "no_sink", patch("softmax_with_learned_sink", lambda real: lambda s, seen, sink: real(s, seen, sink - 1e9))),
            ("attention", "scaled_sink", patch("softmax_with_learned_sink", scaled_sink)),
            ("attention", "sink_counted_twice", patch("softmax_with_learned_sink", twice)),
            ("attention", "no_head_gate", patch("sink_latent_attention", once_gated)),
            ("attention", "query_latent_not_normed", patch("rms_norm", lambda real: lambda x, w, eps: x * w if np.shape(w) == (52,) else real(x, w, eps))),
            ("attention", "scale_left_out", config(lambda c: [l["mixer"].update(scale=1.0) for l in c["layers"]])),
            ("embedding", "first_row_zero", patch("bigram_rows", first_row)),
            ("embedding", "first_token_hashed", patch("bigram_rows", first_hashed)),
            ("embedding", "previous_token_ignored", patch("bigram_rows", no_previous)),
            ("embedding", "previous_token_lost_between_portions", patch("bigram_rows", lost_previous)),
            ("embedding", "multipliers_swapped", patch("bigram_rows", swapped)),
            ("embedding", "bigram_scaled", weights(("bigram", lambda v: 3.0 * v))),
            ("embedding", "not_scaled", config(lambda c: c["embedding"].update(scale=1.0))),
            ("embedding", "norm_weight_left_out", weights(("embed.norm", np.ones_like))),
            ("convolution", "one_early", patch("causal_conv", one_early)),
            ("convolution", "reversed", patch("causal_conv", reversed_taps)),
            ("convolution", "lost_between_portions", patch("causal_conv", lost_rows)),
            ("convolution", "left_out", weights(("canon1", zero), ("canon2", zero))),
            ("convolution", "replaces_its_input", patch("with_recent", lambda real: lambda h, w: real(h, w) - h)),
            ("convolution", "mixer_only", weights(("canon2", zero))),
            ("gate", "reads_the_convolution", sublayer(gate_after_convolution)),
            ("gate", "reads_the_stream", sublayer(gate_of_the_stream)),
            ("gate", "gates_the_stream_too", sublayer(whole_gated)),
            ("gate", "no_bias", weights(("rg1.b", zero), ("rg2.b", zero))),
            ("mixture", "weights_corrected", patch("corrected_route", weights_corrected)),
            ("mixture", "no_correction", patch("corrected_route", no_correction)),
            ("mixture", "divided_by_the_sum", patch("corrected_route", divided)),
            ("mixture", "softmax", patch("corrected_route", softmaxed)),
            ("mixture", "one_expert_more", patch("corrected_route", one_more)),
            ("mixture", "no_shared_expert", patch("shared_mixture", lambda real: lambda h, w, p, mlp: real(h, w, p, dict(mlp, shared=None)))),
            ("mixture", "shared_not_gated", patch("shared_mixture", ungated_shared)),
            ("mixture", "plain_relu", patch("squared_relu", lambda real: lambda z: np.maximum(z, 0.0))),
            ("dense", "no_gate", patch("silu", lambda real: lambda z: np.ones_like(z))),
            ("dense", "plain_silu_of_up", patch("silu_pair_feed_forward", lambda real: lambda h, w, p: real(h, {**w, p + "gate": w[p + "up"], p + "up": w[p + "gate"]}, p))),
            ("dense", "no_softcap", patch("softcap", lambda real: lambda x, cap: x))]


ONE = {
    "attention": minodra([sink_latent(q_rank=52), sink_latent(q_rank=52)]),
    "embedding": minodra([sink_latent()]),
    "convolution": minodra([sink_latent(dense(48)), sink_latent(dense(48))]),
    "gate": minodra([sink_latent(dense(48)), sink_latent(dense(48))]),
    "mixture": minodra([sink_latent(shared_moe(experts=8, top=3)), sink_latent(shared_moe(experts=8, top=3))]),
    "dense": minodra([sink_latent(dense(48)), sink_latent(dense(48))]),
}


@pytest.mark.parametrize("kind,what,plant", _mistakes(), ids=lambda x: x if isinstance(x, str) else "")
def test_planted_mistakes_show_in_the_logits(monkeypatch, kind, what, plant):
    """Everywhere, or at the places that the mistake is about: a sequence's first token, the ones behind a portion's
    start."""
    cfg = ONE[kind]
    w = {k: v.astype(np.float64) for k, v in minodra_weights(cfg, 7, sharp=2.0).items()}
    t = np.random.default_rng(8).integers(0, cfg["vocab"], 24)
    right = ls.forward(cfg, w, t)
    plant(monkeypatch)
    wrong = ls.forward(cfg, w, t)
    assert logit_error(wrong, right) > 20 * F32_TOL
    places = slice(0, 1) if what.startswith("first") else slice(8, 9) if "between_portions" in what else slice(9, None)
    assert np.quantile(position_errors(wrong, right)[places], 0.6) > BF16_MEDIAN


# ---- configuration reader -----------------------------------------------------------------------------
@pytest.mark.parametrize("name", sorted(MINODRA_CONFIGS))
def test_config_reader_takes_every_size_from_the_file(tmp_path, name):
    from pie_amd import driver as drvmod

    cfg = MINODRA_CONFIGS[name]
    info = drvmod.snapshot_info(write_stack(tmp_path / "m", cfg, minodra_weights(cfg)))
    assert info["arch"] == "minodra" and info["hidden"] == cfg["width"] and info["vocab"] == cfg["vocab"]
    assert np.isclose(info["rms_eps"], cfg["norm"]["eps"]) and np.isclose(info["embed_scale"], cfg["embedding"]["scale"])
    assert info["canon_taps"] == cfg["canon"]["taps"] and np.isclose(info["logit_softcap"], cfg["logit_softcap"])
    b = cfg["embedding"].get("bigram") or dict(buckets=0, mul_prev=0, mul_cur=0)
    assert info["bigram"] == [b["buckets"], b["mul_prev"], b["mul_cur"]]
    assert len(info["stack"]) == len(cfg["layers"])
    for got, want in zip(info["stack"], cfg["layers"]):
        m, mlp = want["mixer"], want["mlp"]
        assert got["type"] == "latent_attention" and all(got[k] == m[k] for k in ("heads", "dim", "vdim", "q_rank", "kv_rank"))
        assert got["rot_dim"] == 0 and got["rot_dims"] == 0 and got["sinks"] and got["gate_per_head"] and np.isclose(got["scale"], m["scale"])
        assert got["ff"] == (mlp["ff"] if mlp and mlp["kind"] == "dense" else 0) and ("mixture" in got) == bool(mlp and mlp["kind"] == "moe")
        if "mixture" in got:
            e = got["mixture"]
            assert (e["experts"], e["top"], e["ff"], e["shared_ff"]) == (mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"],
                                                                         mlp.get("shared", dict(ff=0))["ff"])
            assert e["router"] == 1 and e["expert"] == 1


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="attention_3"), "unknown mixer"),
    (lambda c: c["layers"][1]["mlp"].update(kind="sparse"), "unknown mlp kind"),
    (lambda c: c["layers"][1]["mlp"].pop("router"), "router"),
    (lambda c: c["layers"][1]["mlp"]["router"].pop("top"), "top"),
    (lambda c: c["layers"][1]["mlp"]["expert"].pop("ff"), "ff"),
    (lambda c: c["layers"][1]["mlp"]["shared"].pop("ff"), "ff"),
    (lambda c: c["layers"][1]["mlp"]["shared"].update(ff=0), "shared.ff"),
    (lambda c: c["layers"][0]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c.pop("canon"), "canon"),
    (lambda c: c["canon"].pop("taps"), "taps"),
    (lambda c: c["embedding"]["bigram"].pop("mul_cur"), "mul_cur"),
    (lambda c: c["embedding"]["bigram"].update(mul_prev=-1), "mul_prev"),
    (lambda c: c["embedding"]["bigram"].update(buckets=0), "buckets"),
])
def test_config_reader_names_what_is_wrong(tmp_path, change, message):
    from pie_amd import driver as drvmod

    cfg = json.loads(json.dumps(MINODRA_CONFIGS["pair"]))
    d = write_stack(tmp_path / "m", cfg, minodra_weights(cfg))
    change(cfg)
    (tmp_path / "m" / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(RuntimeError, match=message):
        drvmod.snapshot_info(d)
