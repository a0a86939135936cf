"""GPU: Minodra models through the driver boundary against the double-precision oracle, in both compute types: whole
prompts, token-by-token decoding, portions, unequal batches, pages and slots that are used again, far keys, copies,
long decoding, graphs, greedy generation, trace replay."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest

from layer_stack_util import (MINODRA_CONFIGS, assert_close, assert_close_routed, bf16, close_tie, dense, engine, minodra, minodra_weights, position_errors,
                              run, shared_moe, sink_latent, tokens, write_stack)
from oracle import layer_stack as ls

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
DTYPES = ["float32", "bfloat16"]


def close_of(cfg):
    routed = any(l["mlp"] and l["mlp"]["kind"] == "moe" and l["mlp"]["router"]["top"] < l["mlp"]["router"]["experts"] for l in cfg["layers"])
    return assert_close_routed if routed else assert_close


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """(name, compute type) -> (configuration, directory, reference(tokens)).  In bf16 the corrections are spread wide:
    rounding decides less often between two experts."""
    out = {}
    for name, cfg in MINODRA_CONFIGS.items():
        for dtype, spread in (("float32", 0.4), ("bfloat16", 5.0)):
            w = minodra_weights(cfg, seed=len(name), sharp=2.0, spread=spread)
            w64 = {k: v.astype(np.float64) for k, v in w.items()}
            cache = {}

            def ref(toks, cfg=cfg, w64=w64, cache=cache):
                key = tuple(int(x) for x in toks)
                if key not in cache:
                    cache[key] = ls.forward(cfg, w64, key)
                return cache[key]
            out[name, dtype] = (cfg, write_stack(tmp_path_factory.mktemp(name), cfg, w), ref)
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MINODRA_CONFIGS))
def test_prompts_portions_and_decoding_match_the_oracle(gpu, models, name, dtype):
    cfg, directory, ref = models[name, dtype]
    close, toks = close_of(cfg), tokens(cfg, 150, 1)
    want = ref(toks)
    d, e = engine(directory, dtype)
    with d:
        for portions in ([150], [1], [2], [3, 17, 1, 64], [100, 1], [64, 65, 1], [149, 1]):
            got = run(e, "r", toks, portions)
            e.finish("r")
            close(got, want, dtype, portions)


@pytest.mark.parametrize("name", sorted(MINODRA_CONFIGS))
def test_first_tokens_in_fp32(gpu, models, name):
    """Every cut of a short sequence: the first token, the convolutions' start, previous tokens across cuts."""
    cfg, directory, ref = models[name, "float32"]
    d, e = engine(directory, "float32")
    with d:
        for i, toks in enumerate(([5], [3, 3], tokens(cfg, 5, 2))):
            for portions in ([1], [2, 1], [1, 2], [3, 1], [5]):
                assert position_errors(run(e, i, toks, portions), ref(toks)).max() < 2e-4
                e.finish(i)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["pair", "odd", "wide", "four"])
def test_unequal_batches_equal_each_request_alone(gpu, models, name, dtype):
    """Portions of some requests beside single tokens of others; requests come, pause and go, and pages and slots move
    from one to the next."""
    cfg, directory, ref = models[name, dtype]
    lens = {"a": 140, "b": 9, "c": 77, "d": 33, "e": 100, "f": 1}
    seqs = {r: tokens(cfg, n, ord(r)) for r, n in lens.items()}
    d, e = engine(directory, dtype, total_pages=24, slots=4, requests=8)
    rng = np.random.default_rng(7)
    at, got, waiting, live = dict.fromkeys(lens, 0), {r: [] for r in lens}, list(lens), []
    with d:
        while waiting or live:
            while waiting and len(live) < 4:
                live.append(waiting.pop(0))
            entries = []
            for r in live:
                if at[r] and len(live) > 1 and rng.random() < 0.2:
                    continue   # left out of this step
                n = int(min(rng.choice([1, 1, 2, 5, 16, 70]), lens[r] - at[r]))
                entries.append((r, seqs[r][at[r]:at[r] + n], list(range(n))))
            if not entries:
                continue
            for (r, part, _), lg in zip(entries, e.step(entries)):
                got[r].append(lg)
                at[r] += len(part)
                if at[r] == lens[r]:
                    e.finish(r)
                    live.remove(r)
        assert len(e._free_pages) == 24 and len(e._free_slots) == 4
    close = close_of(cfg)
    for r in lens:
        close(np.concatenate(got[r]), ref(seqs[r]), dtype, r)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["wide", "pair"])
def test_a_wide_decode_batch(gpu, models, name, dtype):
    """Many requests of unequal length decoded together: more tokens than the router's one launch takes."""
    cfg, directory, ref = models[name, dtype]
    seqs = {r: tokens(cfg, 20 + 7 * (r % 5), 50 + r % 3) for r in range(40)}
    d, e = engine(directory, dtype, total_pages=160, max_tokens=2048, slots=40, requests=40)
    with d:
        e.step([(r, s[:-6], []) for r, s in seqs.items()])
        got = [e.step([(r, [s[len(s) - 6 + i]], [0]) for r, s in seqs.items()]) for i in range(6)]
    close = close_of(cfg)
    close(np.concatenate([g[r] for g in got for r in range(15)]), np.concatenate([ref(seqs[r])[-6 + i][None] for i in range(6) for r in range(15)]), dtype)
    for r in range(15, 40):   # (the others repeat them)
        close(np.concatenate([g[r] for g in got]), np.concatenate([g[r % 15] for g in got]), dtype, r)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["pair", "wide", "broad"])
def test_long_decoding_over_many_pages(gpu, models, name, dtype):
    cfg, directory, ref = models[name, dtype]
    toks = tokens(cfg, 420, 3)
    d, e = engine(directory, dtype)
    with d:
        got = run(e, "r", toks, [20, 1])
    close_of(cfg)(got, ref(toks), dtype)
    close_of(cfg)(got[-60:], ref(toks)[-60:], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_prompts_take_the_expanded_form(gpu, tmp_path, dtype):
    """Latents wide enough that a long portion projects keys and values out of them first; more routes than the
    experts' single passes take."""
    cfg = minodra([sink_latent(shared_moe(experts=4, top=4, ff=64, shared=200), heads=4, dim=64, vdim=64, kv_rank=256, q_rank=64),
                   sink_latent(dense(64), heads=6, dim=32, vdim=96, kv_rank=128, q_rank=48)], width=128, vocab=90)
    w = minodra_weights(cfg, 4, sharp=2.0)
    toks = tokens(cfg, 1400, 5)
    want = ls.forward(cfg, {k: v.astype(np.float64) for k, v in w.items()}, toks)
    d, e = engine(write_stack(tmp_path, cfg, w), dtype, max_tokens=1500, total_pages=100)
    with d:
        for portions in ([1400], [30, 600, 1], [400, 2, 290, 1], [90, 1, 1200, 5, 128]):
            n = 700 if 1 in portions[-1:] else 1400
            got = run(e, "r", toks[:n], portions)
            e.finish("r")
            assert_close(got, want[:n], dtype, portions)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["pair", "odd", "wide"])
def test_graphs_and_eager_steps_agree(gpu, models, name, dtype):
    """Captured decode steps, replayed with other work in between, give the eager results: bit for bit in fp32; in bf16
    the splits of the keys follow the graph's context bound instead of the batch's."""
    cfg, directory, _ = models[name, dtype]
    a, b = tokens(cfg, 60, 4), tokens(cfg, 60, 5)
    outs = []
    for graphs in (True, False):
        d, e = engine(directory, dtype, graphs=graphs)
        with d:
            rows = [*e.step([("a", a[:30], [29]), ("b", b[:7], [6])])]
            for i in range(30):
                rows += e.step([("a", [a[30 + i]], [0]), ("b", [b[7 + i]], [0])])
                if i % 7 == 3:
                    e.step([("c", b[:20], [])])
                    e.finish("c")
            outs.append(np.concatenate(rows))
    if dtype == "float32":
        assert np.array_equal(outs[0], outs[1])
    close_of(cfg)(outs[0], outs[1], dtype)


MARKED = 7


def far_key_model():
    """One layer in which every query points at the marked token's key; sublayers read the normed row alone."""
    dim = 32
    cfg = minodra([sink_latent(heads=2, dim=dim, vdim=24, q_rank=16, kv_rank=40, scale=1.5)], width=64, vocab=40, scale=1.0)
    w = minodra_weights(cfg, 2)
    axis = np.sign(np.random.default_rng(5).standard_normal(dim)).astype(np.float32)
    # one direction of the embeddings is everybody's (the queries read it), one is the marked token's (its keys do)
    w["embed"][:, 0], w["embed"][:, 1] = 2.0, 0.0
    w["embed"][MARKED, 1] = 2.0
    w["bigram"] *= 0.0
    for n in ("l0.canon1", "l0.rg1", "l0.mix.dq", "l0.mix.uq"):
        w[n] *= 0.0
    x = "l0.mix."
    w["l0.rg1.b"][:] = 3.0
    w["embed.norm"] = w["l0.norm1"] = np.float32(1.0)
    w[x + "dq"][0, 0] = 1.0
    w[x + "dq.norm"][:] = 1.0
    for h in range(2):
        w[x + "uq"][h * dim:(h + 1) * dim, 0] = axis * 0.25
    w[x + "dkv"][0] = 0.0
    w[x + "dkv"][0, 1] = 6.0
    w[x + "uk"] *= 0.1
    for h in range(2):
        w[x + "uk"][h * dim:(h + 1) * dim, 0] = axis
    return cfg, {k: bf16(v) for k, v in w.items()}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("place", [0, 1, 15, 16, 37, 63, 64])
def test_a_far_token_is_found_across_pages(gpu, tmp_path, dtype, place):
    cfg, w = far_key_model()
    w64 = {k: v.astype(np.float64) for k, v in w.items()}
    toks = [t if t != MARKED else MARKED + 1 for t in tokens(cfg, 330, 6)]
    toks[place] = MARKED
    want = ls.forward(cfg, w64, toks)
    other = list(toks)
    other[place] = MARKED + 1
    effect = position_errors(ls.forward(cfg, w64, other), want)
    assert effect[-30:].min() > 0.1   # (losing the key shows at every one of the last positions)
    d, e = engine(write_stack(tmp_path, cfg, w), dtype)
    with d:
        for portions in ([330], [place + 1, 280, 1], [200, 2, 1], [300, 1]):
            got = run(e, "r", toks, portions)
            e.finish("r")
            assert_close(got, want, dtype, portions)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["pair", "odd"])
def test_pages_and_state_move_by_copies(gpu, models, name, dtype):
    """A request forked on the device and one swapped to the host and back go on as if nothing had happened: the
    convolutions' inputs and the previous token travel with the slots."""
    from pie_amd import driver as drvmod

    cfg, directory, ref = models[name, dtype]
    toks = tokens(cfg, 40, 14)
    want = ref(toks)
    d, _ = engine(directory, dtype, extra_batching="cpu_pages = 8\ncpu_rs_slots = 2")
    frame = lambda ts, t0, t1, pages, slot: drvmod.ForwardFrame(
        ts[t0:t1], range(t0, t1), pages[:(t1 + 15) // 16], [0, (t1 + 15) // 16], [(t1 - 1) % 16 + 1], [0, t1 - t0], sampling_indices=list(range(t1 - t0)),
        sampling_indptr=[0, t1 - t0], samplers=[dict(kind=7)] * (t1 - t0), sampler_indptr=[0, t1 - t0], rs_slot_ids=[slot])
    ok = lambda fr: d.handle(fr).payload.status.status
    with d:
        assert d.forward(frame(toks, 0, 30, [0, 1, 2], 0)).num_requests == 1
        assert ok(drvmod.copy_frame(2, [0, 1], [10, 11])) == 0 and ok(drvmod.copy_frame(2, [0], [3], resource=1)) == 0
        assert ok(drvmod.copy_frame(0, [0, 1], [4, 5])) == 0 and ok(drvmod.copy_frame(0, [0], [1], resource=1)) == 0
        assert ok(drvmod.copy_frame(3, [1], [0], resource=1)) == 0
        a = d.forward(frame(toks, 30, 40, [0, 1, 2], 0))
        # (another request has used slot 5 before)
        assert d.forward(frame(tokens(cfg, 9, 15), 0, 9, [30], 5)).num_requests == 1
        b = d.forward(frame(toks, 30, 40, [10, 11, 12], 3))
        assert ok(drvmod.copy_frame(1, [4, 5], [20, 21])) == 0 and ok(drvmod.copy_frame(1, [0], [5], resource=1)) == 0
        c = d.forward(frame(toks, 30, 40, [20, 21, 22], 5))
        for r in (a, b, c):
            close_of(cfg)(np.stack(r.logits_of(0)), want[30:], dtype)
        first = np.stack(a.logits_of(0))
        assert np.array_equal(first, np.stack(b.logits_of(0))) and np.array_equal(first, np.stack(c.logits_of(0)))
        # a fresh request in a used slot has no previous token
        again = d.forward(frame(toks, 0, 3, [0], 5))
        close_of(cfg)(np.stack(again.logits_of(0)), want[:3], dtype)


@pytest.mark.parametrize("name", ["pair", "odd"])
def test_greedy_generation_through_both_entry_points(gpu, models, name):
    """The generation harness (replicas fork pages and slots) and the engine's continuous batching."""
    cfg, directory, ref = models[name, "float32"]
    prompt = tokens(cfg, 90, 13)

    def greedy(start, n):
        toks, logits = list(start), []
        for _ in range(n):
            logits.append(ref(toks)[-1])
            toks.append(int(np.argmax(logits[-1])))
        return toks[len(start):], np.stack(logits)

    want, logits = greedy(prompt, 12)
    sure = int(np.argmax(close_tie(logits) < 5e-3)) if (close_tie(logits) < 5e-3).any() else 12
    assert sure >= 6
    d, e = engine(directory, "float32", max_tokens=64)   # the prompt takes two portions
    with d:
        got, _ = d.generate(prompt, 12, replicate=3)
        for c in range(3):
            assert [int(x) for x in got[c]][:sure] == want[:sure]
        other = tokens(cfg, 5, 12)
        out = e.generate({"p": prompt, "q": other}, 12, portion=16)
        assert out["p"][:sure] == want[:sure]
        w2, l2 = greedy(other, 6)
        if close_tie(l2).min() > 5e-3:
            assert out["q"][:6] == w2


def test_capabilities_and_refusals(gpu, models, tmp_path):
    from pie_amd import driver as drvmod

    cfg, directory, _ = models["pair", "bfloat16"]
    d, _ = engine(directory, "bfloat16")
    with d:
        caps = d.capabilities()
        assert caps["rs_cache_required"] and caps["rs_cache_slots"] == 6 and caps["rs_cache_slot_bytes"] > 0 and caps["arch_name"] == "minodra"
        r = d.forward(drvmod.ForwardFrame([1, 2], [5, 6], [0], [0, 1], [7], [0, 2], rs_slot_ids=[0]))
        assert r.num_requests == 0 and "goes on at position" in d.last_error()
    d, _ = engine(models["odd", "bfloat16"][1], "bfloat16")
    with d:   # (no convolution reaches back here, but the previous token is state)
        assert d.capabilities()["rs_cache_required"]

    def refused(what, change):
        c = json.loads(json.dumps(cfg))
        change(c)
        (tmp_path / "config.json").write_text(json.dumps(c))
        with pytest.raises(RuntimeError, match=what):
            engine(tmp_path, "bfloat16", extra_model="random_weights = true")
    refused("canon.taps", lambda c: c["canon"].update(taps=0))
    refused("latent_attention needs", lambda c: c["layers"][0]["mixer"].update(heads=0))
    refused("fewer experts", lambda c: c["layers"][1]["mlp"]["router"].update(top=10))
    refused("512 experts", lambda c: c["layers"][1]["mlp"]["shared"].update(ff=128 * 62))


def test_weights_of_the_wrong_shape_are_refused(gpu, tmp_path):
    cfg = MINODRA_CONFIGS["pair"]
    for i, (name, shape) in enumerate([("l0.norm1", (112,)), ("bigram", (61, 112)), ("l1.canon2", (112, 4)), ("l0.mix.sink", (4,)), ("l1.mix.g", (6, 112)),
                                       ("l1.mlp.correction", (8,)), ("l1.mlp.shared.sg", (112,)), ("l0.rg2", (111, 112))]):
        w = minodra_weights(cfg)
        w[name] = np.zeros(shape, np.float32)
        with pytest.raises(RuntimeError, match=name.replace(".", r"\.")):
            engine(write_stack(tmp_path / str(i), cfg, w), "bfloat16")


def test_random_weights_need_only_the_configuration(gpu, tmp_path):
    cfg = MINODRA_CONFIGS["pair"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    d, e = engine(tmp_path, "bfloat16", extra_model="random_weights = true")
    with d:
        out = e.generate({"a": tokens(cfg, 40, 1), "b": [3]}, 5)
        assert all(0 <= x < cfg["vocab"] for r in out.values() for x in r)
        assert np.isfinite(e.step([("z", tokens(cfg, 90, 2), [89])])[0]).all()


def test_single_layers_of_every_kind(gpu, tmp_path):
    for i, (layers, kw) in enumerate([([sink_latent()], {}), ([sink_latent()], dict(taps=1, bigram=None)), ([sink_latent(dense(24))], dict(taps=5)),
                                      ([sink_latent(shared_moe(experts=4, top=4, shared=0))], dict(taps=2)),
                                      ([sink_latent(shared_moe(experts=2, top=2, ff=130, shared=600))], dict(taps=4, bigram=None))]):
        cfg = minodra(layers, **dict(dict(width=80, vocab=50), **kw))
        w = minodra_weights(cfg, i)
        want = ls.forward(cfg, {k: v.astype(np.float64) for k, v in w.items()}, toks := tokens(cfg, 70, i))
        directory = write_stack(tmp_path / str(i), cfg, w)
        for dtype in DTYPES:
            d, e = engine(directory, dtype)
            with d:
                assert d.capabilities()["rs_cache_required"] == (kw.get("taps", 3) > 1 or "bigram" not in kw)
                assert_close(run(e, "r", toks, [66, 1, 2, 1]), want, dtype, i)


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_run_replays_a_trace(gpu, models, tmp_path, dtype):
    cfg, directory, ref = models["odd", dtype]
    a, b = tokens(cfg, 100, 21), tokens(cfg, 20, 22)
    steps = [dict(entries=[dict(id="a", tokens=a[:80], want=[0, 79]), dict(id="b", tokens=b[:5], want=[])], end=[]),
             dict(entries=[dict(id="b", tokens=b[5:20], want=[14, 2])], end=["b"]),
             dict(entries=[dict(id="a", tokens=a[80:99], want=[]), dict(id="c", tokens=b, want=[19])], end=["c"]),
             dict(entries=[dict(id="a", tokens=a[99:], want=[0])], end=["a"])]
    text = "".join(json.dumps(dict(step=i, **s)) + "\n" for i, s in enumerate(steps))
    p = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(directory), "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "192"], input=text, capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(4)]
    read = lambda i: np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])
    ra, rb = ref(a), ref(b)
    assert_close(read(0), ra[[0, 79]], dtype)
    assert_close(read(1), rb[[19, 7]], dtype)
    assert_close(read(2), rb[[19]], dtype)
    assert_close(read(3), ra[[99]], dtype)
