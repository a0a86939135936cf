"""GPU: Lofudra models through the driver boundary against the double-precision oracle, in both compute types:
whole prompts, token-by-token decoding, portions, unequal batches, pages and slots that are used again,
window edges and sinks, looped passes, copies, long decoding, graphs, greedy generation, trace replay."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest

from layer_stack_util import (LOFUDRA_CONFIGS, assert_close, close_tie, engine, lofudra, lofudra_weights, mamba2, mlstm, parallel, position_errors,
                              run, tokens, write_stack)
from oracle import layer_stack as ls

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
DTYPES = ["float32", "bfloat16"]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (configuration, directory, reference(tokens))"""
    out = {}
    for name, cfg in LOFUDRA_CONFIGS.items():
        w = lofudra_weights(cfg, seed=len(name), sharp=2.0)
        w64 = {k: v.astype(np.float64) for k, v in w.items()}
        cache = {}

        def ref(toks, cfg=cfg, w64=w64, cache=cache):
            key = tuple(int(x) for x in toks)
            if key not in cache:
                cache[key] = ls.forward(cfg, w64, key)
            return cache[key]
        out[name] = (cfg, write_stack(tmp_path_factory.mktemp(name), cfg, w), ref)
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(LOFUDRA_CONFIGS))
def test_prompts_portions_and_decoding_match_the_oracle(gpu, models, name, dtype):
    cfg, directory, ref = models[name]
    toks = tokens(cfg, 150, 1)
    want = ref(toks)
    d, e = engine(directory, dtype)
    with d:
        for portions in ([150], [1], [2], [3, 17, 1, 64], [100, 1], [64, 65, 1], [149, 1]):
            got = run(e, "r", toks, portions)
            e.finish("r")
            assert_close(got, want, dtype, portions)
            assert_close(got[:3], want[:3], dtype, portions)   # the first tokens of a sequence


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["trio", "all_looped", "wide"])
def test_unequal_batches_equal_each_request_alone(gpu, models, name, dtype):
    """Portions of some requests beside single tokens of others; requests come, pause and go, and
    pages and slots move from one to the next."""
    cfg, directory, ref = models[name]
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
    for r in lens:
        assert_close(np.concatenate(got[r]), ref(seqs[r]), dtype, r)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["wide", "many_heads"])
def test_a_wide_decode_batch(gpu, models, tmp_path, which, dtype):
    """Many requests of unequal length decoded together: the launches that other batch sizes take (whole heads
    per block, the convolution ahead of the step)."""
    if which == "wide":
        cfg, directory, ref = models["wide"]
    else:
        cfg = lofudra([mamba2(heads=32, vdim=8, state=16, groups=2, conv=4, norm_groups=2), mlstm(heads=12, dim=16, vdim=48)], width=96, vocab=70)
        w = lofudra_weights(cfg, 9)
        directory, w64 = write_stack(tmp_path, cfg, w), {k: v.astype(np.float64) for k, v in w.items()}
        ref = lambda toks: ls.forward(cfg, w64, toks)
    seqs = {r: tokens(cfg, 20 + 7 * (r % 5), 50 + r % 3) for r in range(40)}
    d, e = engine(directory, dtype, total_pages=160, max_tokens=2048, slots=40, requests=40)
    with d:
        e.step([(r, s[:-6], []) for r, s in seqs.items()])
        got = [e.step([(r, [s[len(s) - 6 + i]], [0]) for r, s in seqs.items()]) for i in range(6)]
    for r, s in seqs.items():
        if r < 15:   # (the others repeat them)
            assert_close(np.concatenate([g[r] for g in got]), ref(s)[-6:], dtype, r)
        else:
            assert_close(np.concatenate([g[r] for g in got]), np.concatenate([g[r % 15] for g in got]), dtype, r)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["all_looped", "wide"])
def test_long_decoding_over_many_pages(gpu, models, name, dtype):
    cfg, directory, ref = models[name]
    toks = tokens(cfg, 420, 3)
    d, e = engine(directory, dtype)
    with d:
        got = run(e, "r", toks, [20, 1])
    assert_close(got, ref(toks), dtype)
    assert_close(got[-20:], ref(toks)[-20:], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["trio", "first_attention", "wide"])
def test_graphs_and_eager_steps_agree(gpu, models, name, dtype):
    """Captured decode steps, replayed with other work in between, give the eager results: bit for bit in
    fp32; in bf16 the splits of the keys follow the graph's context bound instead of the batch's."""
    cfg, directory, _ = models[name]
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
    assert_close(outs[0], outs[1], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [2, 16, 33, 64])
def test_windows_end_where_they_should(gpu, tmp_path, dtype, window):
    """One attention layer whose queries all point at one token's keys: the tokens asked around the window's
    edge answer with its value just inside, without it just outside; in prompts, portions and decoding."""
    cfg = lofudra([parallel(heads=4, kv_heads=2, dim=32, rot_dims=2, base=1e30, window=window, right_scale=0.0, left_scale=1.0, ff=0, scale=0.9,
                            decay=[0.5] * 3)], width=64, vocab=40)
    w = lofudra_weights(cfg, 2)
    marked = 7
    # (query biases decide the queries; the marked token's keys are theirs, everybody else's are noise)
    for n in ("q", "k"):
        w[f"l0.mix.left.{n}.norm"][:] = 1.0
    w["l0.mix.left.q"] *= 0.0
    axis = np.sign(np.random.default_rng(5).standard_normal(32)).astype(np.float32)
    axis[[0, 1]] = 0.0   # (the rotated pair takes no part)
    w["l0.mix.left.q.b"][:] = np.tile(axis, 4)
    w["l0.mix.left.k.b"][:] = 0.0
    h = w["embed"][marked] / np.sqrt(np.mean(w["embed"][marked] ** 2)) * w["l0.norm1"]
    k = w["l0.mix.left.k"]
    from layer_stack_util import bf16

    for g in range(2):
        rows = k[32 * g:32 * g + 32]
        rows += np.outer(4.0 * axis - rows @ h, h) / (h @ h)
    w["l0.mix.left.k"] = bf16(k)
    directory = write_stack(tmp_path, cfg, w)
    w64 = {n: v.astype(np.float64) for n, v in w.items()}
    toks = [t if t != marked else marked + 1 for t in tokens(cfg, 150, 6)]
    toks[41] = marked
    want = ls.forward(cfg, w64, toks)
    other = list(toks)
    other[41] = marked + 1
    inside, outside = 41 + window - 1, 41 + window
    effect = position_errors(ls.forward(cfg, w64, other), want)
    assert effect[inside] > 0.3 and effect[outside] < 1e-9   # (the case tells a window off by one apart)
    d, e = engine(directory, dtype)
    with d:
        for portions in ([150], [1], [42, 1], [inside, 1, 1, 1], [outside, 2, 1], [41, 1, 30, 2]):
            got = run(e, "r", toks, portions)
            e.finish("r")
            assert_close(got, want, dtype, portions)


@pytest.mark.parametrize("dtype", DTYPES)
def test_pages_and_state_move_by_copies(gpu, models, dtype):
    """A request forked on the device and one swapped to the host and back go on as if nothing
    had happened; every pass of a looped layer has its pages and its part of the slot."""
    from pie_amd import driver as drvmod

    cfg, directory, ref = models["all_looped"]
    toks = tokens(cfg, 40, 14)
    want = ref(toks)
    d, _ = engine(directory, dtype, extra_batching="cpu_pages = 8\ncpu_rs_slots = 2")
    frame = lambda t0, t1, pages, slot: drvmod.ForwardFrame(
        toks[t0:t1], range(t0, t1), pages[:(t1 + 15) // 16], [0, (t1 + 15) // 16], [(t1 - 1) % 16 + 1], [0, t1 - t0], sampling_indices=[t1 - t0 - 1],
        sampling_indptr=[0, 1], samplers=[dict(kind=7)], sampler_indptr=[0, 1], rs_slot_ids=[slot])
    ok = lambda fr: d.handle(fr).payload.status.status
    with d:
        assert d.forward(frame(0, 30, [0, 1, 2], 0)).num_requests == 1
        assert ok(drvmod.copy_frame(2, [0, 1], [10, 11])) == 0 and ok(drvmod.copy_frame(2, [0], [3], resource=1)) == 0
        assert ok(drvmod.copy_frame(0, [0, 1], [4, 5])) == 0 and ok(drvmod.copy_frame(0, [0], [1], resource=1)) == 0
        a = d.forward(frame(30, 40, [0, 1, 2], 0))
        b = d.forward(frame(30, 40, [10, 11, 12], 3))
        assert ok(drvmod.copy_frame(1, [4, 5], [20, 21])) == 0 and ok(drvmod.copy_frame(1, [1], [5], resource=1)) == 0
        c = d.forward(frame(30, 40, [20, 21, 22], 5))
        for r in (a, b, c):
            assert_close(r.logits_of(0)[0], want[-1], dtype)
        assert np.array_equal(a.logits_of(0)[0], b.logits_of(0)[0]) and np.array_equal(a.logits_of(0)[0], c.logits_of(0)[0])


@pytest.mark.parametrize("name", ["trio", "all_looped"])
def test_greedy_generation_through_both_entry_points(gpu, models, name):
    """The generation harness (replicas fork pages and state) and the engine's continuous batching."""
    cfg, directory, ref = models[name]
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
    cfg, directory, _ = models["trio"]
    d, _ = engine(directory, "bfloat16")
    with d:
        caps = d.capabilities()
        assert caps["rs_cache_required"] and caps["rs_cache_slots"] == 6 and caps["rs_cache_slot_bytes"] > 0 and caps["arch_name"] == "lofudra"

    def refused(what, change):
        c = json.loads(json.dumps(cfg))
        change(c)
        (tmp_path / "config.json").write_text(json.dumps(c))
        with pytest.raises(RuntimeError, match=what):
            engine(tmp_path, "bfloat16", extra_model="random_weights = true")
    refused("one decay per head", lambda c: c["layers"][2]["mixer"]["right"]["decay"].pop())
    refused("loop", lambda c: c["loop"].update(stop=9))
    refused("norm_groups", lambda c: c["layers"][1]["mixer"].update(norm_groups=5))
    refused("keys' size", lambda c: c["layers"][2]["mixer"]["left"].update(vdim=8))
    refused("multiple", lambda c: c["layers"][2]["mixer"]["left"].update(kv_heads=4))


def test_random_weights_need_only_the_configuration(gpu, tmp_path):
    cfg = LOFUDRA_CONFIGS["trio"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    d, e = engine(tmp_path, "bfloat16", extra_model="random_weights = true")
    with d:
        out = e.generate({"a": tokens(cfg, 40, 1), "b": [3]}, 5)
        assert all(0 <= x < cfg["vocab"] for r in out.values() for x in r)
        assert np.isfinite(e.step([("z", tokens(cfg, 90, 2), [89])])[0]).all()


def test_memory_only_models_and_single_layers(gpu, tmp_path):
    """No paged cache at all; one layer of each kind alone."""
    for i, layers in enumerate(([mlstm(ff=0)], [mamba2(ff=0)], [parallel(ff=0)], [mlstm(), mamba2()])):
        cfg = lofudra(layers, width=80, vocab=50)
        w = lofudra_weights(cfg, i)
        want = ls.forward(cfg, {k: v.astype(np.float64) for k, v in w.items()}, toks := tokens(cfg, 70, i))
        directory = write_stack(tmp_path / str(i), cfg, w)
        for dtype in DTYPES:
            d, e = engine(directory, dtype)
            with d:
                assert_close(run(e, "r", toks, [66, 1, 2, 1]), want, dtype, i)


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_run_replays_a_trace(gpu, models, tmp_path, dtype):
    cfg, directory, ref = models["trio"]
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
