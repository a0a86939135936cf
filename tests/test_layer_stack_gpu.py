"""GPU: layer-stack models through the driver boundary against the double-precision oracle, in both
compute types: whole prompts, token-by-token decoding, portions, unequal batches, pages and slots
that are used again, copies, sampling and greedy generation."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest

from layer_stack_util import (ATTENTION_ONLY, CONFIGS, DELTA_ONLY, assert_close, close_tie, delta, engine, latent, random_weights, run, stack,
                              tokens, write_stack)
from oracle import layer_stack as ls

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
DTYPES = ["float32", "bfloat16"]

# long portions (>= 64 tokens) of these take the expanded attention, shorter ones the rows form
EXPANDED = stack([latent(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=128, q_rank=48, ff=64), delta(heads=4, kv_heads=4, dim=32, vdim=32, conv=4),
                  latent(heads=3, dim=40, rot_dim=24, vdim=40, kv_rank=190, q_rank=64, ff=0)], width=128, vocab=120)
ALL = dict(CONFIGS, expanded=EXPANDED, attention_only=ATTENTION_ONLY, delta_only=DELTA_ONLY)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (configuration, weights, directory, reference(tokens))"""
    out = {}
    for name, cfg in ALL.items():
        w = random_weights(cfg, seed=len(name), sharp=2.0)
        w64 = {k: v.astype(np.float64) for k, v in w.items()}
        cache = {}

        def ref(tokens, cfg=cfg, w64=w64, cache=cache):
            key = tuple(int(x) for x in tokens)
            if key not in cache:
                cache[key] = ls.forward(cfg, w64, key)
            return cache[key]
        out[name] = (cfg, w, write_stack(tmp_path_factory.mktemp(name), cfg, w), ref)
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(ALL))
def test_prompts_portions_and_decoding_match_the_oracle(gpu, models, name, dtype):
    cfg, _, directory, ref = models[name]
    toks = tokens(cfg, 150, 1)
    want = ref(toks)
    d, e = engine(directory, dtype)
    with d:
        for portions in ([150], [1], [2], [3, 17, 1, 64], [100, 1], [16, 15, 33], [149, 1]):
            got = run(e, "r", toks, portions)
            e.finish("r")
            assert_close(got, want, dtype, portions)
            assert_close(got[:3], want[:3], dtype, portions)   # the first tokens of a sequence


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "expanded"])
def test_unequal_batches_equal_each_request_alone(gpu, models, name, dtype):
    """Portions of some requests beside single tokens of others; requests come, pause and go, and
    pages and slots move from one to the next."""
    cfg, _, directory, ref = models[name]
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
        assert len(e._free_pages) == 24 and len(e._free_slots) == (4 if name in ("mixed", "expanded") else 0)
    for r in lens:
        assert_close(np.concatenate(got[r]), ref(seqs[r]), dtype, r)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_over_many_pages(gpu, models, dtype):
    cfg, _, directory, ref = models["expanded"]
    toks = tokens(cfg, 420, 3)
    d, e = engine(directory, dtype)
    with d:
        got = run(e, "r", toks, [20, 1])
    assert_close(got, ref(toks), dtype)
    assert_close(got[-20:], ref(toks)[-20:], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "delta_first", "expanded"])
def test_graphs_and_eager_steps_agree(gpu, models, name, dtype):
    """Captured decode steps, replayed with other work in between, give the eager results: bit for bit in
    fp32; in bf16 the splits of the keys follow the graph's context bound instead of the batch's."""
    cfg, _, directory, _ = models[name]
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
def test_a_far_token_is_found_across_pages(gpu, tmp_path, dtype):
    """Sharp queries: attention weights close to one-hot, so a key that is dropped or doubled anywhere
    changes the answer; asked in the prompt and by decoded tokens, around page borders."""
    cfg = stack([latent(heads=3, dim=32, rot_dim=16, vdim=32, kv_rank=64, q_rank=64, ff=0, scale=1.5,
                        rot=dict(dims=8, base=10000.0))], width=96, vocab=60)
    w = random_weights(cfg, 2, sharp=1.5)
    directory = write_stack(tmp_path, cfg, w)
    toks = tokens(cfg, 33, 6) + [7] + tokens(cfg, 94, 8)
    want = ls.forward(cfg, {k: v.astype(np.float64) for k, v in w.items()}, toks)
    d, e = engine(directory, dtype)
    with d:
        for portions in ([128], [1], [31, 2, 1], [32, 1, 63, 1]):
            got = run(e, "r", toks, portions)
            e.finish("r")
            assert_close(got, want, dtype, portions)


def test_weights_come_from_the_file_to_the_last_bit(gpu, models):
    cfg, w, directory, _ = models["mixed"]
    d, _ = engine(directory, "bfloat16")
    with d:
        f, _ = ls.rotation_frequencies(cfg["layers"][0]["mixer"]["rot"])
        assert np.allclose(d.export_tensor("rotary.0", np.float64), f, rtol=1e-12)
        emb = d.export_tensor("embed", np.uint16).astype(np.uint32) << 16
        assert np.array_equal(emb.view(np.float32).reshape(w["embed"].shape), w["embed"])
        m = cfg["layers"][0]["mixer"]
        rows = d.export_tensor("l0.mix.in", np.uint16).reshape(-1, 128).astype(np.uint32) << 16
        rows = rows.view(np.float32)
        assert np.array_equal(rows[:m["q_rank"], :112], w["l0.mix.dq"])
        kv_off = -(-m["q_rank"] // 16) * 16
        assert np.array_equal(rows[kv_off:kv_off + m["kv_rank"] + m["rot_dim"], :112], w["l0.mix.dkv"])


@pytest.mark.parametrize("name", ["mixed", "expanded", "attention_only"])
def test_greedy_generation_through_both_entry_points(gpu, models, name):
    """The generation harness (replicas fork pages and state) and the engine's continuous batching."""
    cfg, w, directory, _ = models[name]
    w64 = {k: v.astype(np.float64) for k, v in w.items()}
    prompt = tokens(cfg, 90, 11)
    want, logits = ls.greedy(cfg, w64, prompt, 12)
    sure = int(np.argmax(close_tie(logits) < 2e-3)) if (close_tie(logits) < 2e-3).any() else 12
    assert sure >= 4
    d, e = engine(directory, "float32", max_tokens=64)   # the prompt takes two portions
    with d:
        got, _ = d.generate(prompt, 12, replicate=3)
        for c in range(3):
            assert [int(x) for x in got[c]][:sure] == want[:sure]
        other = tokens(cfg, 5, 12)
        out = e.generate({"p": prompt, "q": other}, 12, portion=16)
        assert out["p"][:sure] == want[:sure]
        w2, l2 = ls.greedy(cfg, w64, other, 6)
        if close_tie(l2).min() > 2e-3:
            assert out["q"][:6] == w2


def test_samplers_read_the_finished_logits(gpu, models):
    from pie_amd import driver as drvmod

    cfg, _, directory, ref = models["mixed"]
    toks = tokens(cfg, 20, 13)
    want = ref(toks)[-1]
    d, _ = engine(directory, "float32")
    with d:
        lp = want - np.log(np.exp(want - want.max()).sum()) - want.max()
        kinds = [dict(kind=8, token_id=5), dict(kind=10), dict(kind=7), dict(kind=6, temperature=1.0, num_tokens=3),
                 dict(kind=1, temperature=0.7, k=1, seed=9)]
        f = drvmod.ForwardFrame(toks, range(20), [0, 1], [0, 2], [4], [0, 20], sampling_indices=[19] * 5, sampling_indptr=[0, 5],
                                samplers=kinds, sampler_indptr=[0, 5], rs_slot_ids=[1])
        r = d.forward(f)
        assert r.num_requests == 1
        assert abs(float(r.logprobs_of(0)[0][0]) - lp[5]) < 1e-3
        assert abs(r.entropies_of(0)[0] + float((np.exp(lp) * lp).sum())) < 1e-3
        assert np.abs(r.logits_of(0)[0] - want).max() < 1e-3
        ids, probs = r.dists_of(0)[0]
        assert [int(i) for i in ids] == [int(i) for i in np.argsort(-want)[:3]] and np.allclose(probs, np.exp(lp[ids]), atol=1e-3)
        assert r.tokens_of(0) == [int(np.argmax(want))]
        # many sampled rows: more than one chunk of the output head
        rows = d.forward(drvmod.ForwardFrame(toks, range(20), [0, 1], [0, 2], [4], [0, 20], sampling_indices=list(range(20)) * 4,
                                             sampling_indptr=[0, 80], samplers=[dict(kind=7)] * 80,
                                             sampler_indptr=[0, 80], rs_slot_ids=[1]))
        assert_close(np.stack(rows.logits_of(0)), np.tile(ref(toks), (4, 1)), "float32")


@pytest.mark.parametrize("dtype", DTYPES)
def test_pages_and_state_move_by_copies(gpu, models, dtype):
    """A request forked on the device and one swapped to the host and back go on as if nothing
    had happened; the slots' positions travel with them."""
    from pie_amd import driver as drvmod

    cfg, _, directory, ref = models["mixed"]
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
        assert ok(drvmod.copy_frame(3, [1], [0], resource=1)) == 0
        a = d.forward(frame(30, 40, [0, 1, 2], 0))
        b = d.forward(frame(30, 40, [10, 11, 12], 3))
        assert ok(drvmod.copy_frame(1, [4, 5], [20, 21])) == 0 and ok(drvmod.copy_frame(1, [0], [5], resource=1)) == 0
        c = d.forward(frame(30, 40, [20, 21, 22], 5))
        for r in (a, b, c):
            assert_close(r.logits_of(0)[0], want[-1], dtype)
        assert np.array_equal(a.logits_of(0)[0], b.logits_of(0)[0]) and np.array_equal(a.logits_of(0)[0], c.logits_of(0)[0])
        # ids outside their pools
        assert ok(drvmod.copy_frame(2, [0], [6], resource=1)) == 3 and ok(drvmod.copy_frame(0, [0], [2], resource=1)) == 3


def test_requests_that_cannot_be_served_are_refused(gpu, models):
    from pie_amd import driver as drvmod

    cfg, _, directory, _ = models["mixed"]
    d, _ = engine(directory, "bfloat16")
    caps = d.capabilities()
    assert caps["rs_cache_required"] and caps["rs_cache_slots"] == 6 and caps["rs_cache_slot_bytes"] > 0
    assert caps["arch_name"] == "varasun" and caps["activation_dtype"] == "bfloat16"
    with d:
        def refused(what, **kw):
            args = dict(token_ids=[1, 2], position_ids=[0, 1], kv_page_indices=[0], kv_page_indptr=[0, 1], kv_last_page_lens=[2],
                        qo_indptr=[0, 2], rs_slot_ids=[0])
            args.update(kw)
            r = d.forward(drvmod.ForwardFrame(**args))
            assert r.num_requests == 0 and what in d.last_error(), d.last_error()
        refused("needs a recurrent-state slot", rs_slot_ids=None)
        refused("out of range", rs_slot_ids=[6])
        refused("consecutive", position_ids=[0, 0])
        refused("goes on at position", position_ids=[5, 6], kv_last_page_lens=[7])
        refused("custom attention masks", masks=[[0, 1], [1, 1]])
        two = dict(kv_page_indices=[0, 1], kv_page_indptr=[0, 1, 2], kv_last_page_lens=[1, 1], qo_indptr=[0, 1, 2], position_ids=[0, 0])
        refused("share a recurrent-state slot", rs_slot_ids=[2, 2], **two)
        refused("drafts", spec_token_ids=[2], spec_position_ids=[1], spec_indptr=[0, 1])
        # and the driver still serves
        assert d.forward(drvmod.ForwardFrame([1, 2], [0, 1], [0], [0, 1], [2], [0, 2], rs_slot_ids=[0])).num_requests == 1
        # a reset flag starts a slot afresh at any position
        assert d.forward(drvmod.ForwardFrame([1], [2], [0], [0, 1], [3], [0, 1], rs_slot_ids=[3], rs_slot_flags=[1])).num_requests == 1


def test_uniform_models_have_no_fp32_mode(gpu):
    from driver_util import toml_config
    from pie_amd.driver import Driver

    with pytest.raises(RuntimeError, match="float32"):
        Driver(toml_config(model_extra='compute_dtype = "float32"\n'))


def test_random_weights_need_only_the_configuration(gpu, tmp_path):
    cfg = CONFIGS["mixed"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    d, e = engine(tmp_path, "bfloat16", extra_model="random_weights = true")
    with d:
        out = e.generate({"a": tokens(cfg, 40, 1), "b": [3]}, 5)
        assert all(0 <= x < cfg["vocab"] for r in out.values() for x in r)
        assert np.isfinite(e.step([("z", tokens(cfg, 90, 2), [89])])[0]).all()


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_run_replays_a_trace(gpu, models, tmp_path, dtype):
    cfg, _, directory, ref = models["expanded"]
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
