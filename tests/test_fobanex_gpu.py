"""GPU: Fobanex models through the driver boundary against the double-precision oracle, in both compute types: whole
prompts, token-by-token decoding, portions, unequal batches, pages that are used again, far keys, layers that read
another layer's latents, copies, long decoding, graphs, greedy generation, trace replay."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest

from layer_stack_util import (FOBANEX_CONFIGS, assert_close, assert_close_routed, bf16, close_tie, dense, engine, fobanex, fobanex_weights,
                              key_value_attention, moe, normed_attention, position_errors, rotary, run, shared_latent, tokens, write_stack)
from oracle import layer_stack as ls

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
DTYPES = ["float32", "bfloat16"]


def close_of(cfg):
    routed = any(l["mlp"] and l["mlp"]["kind"] == "moe" and l["mlp"]["router"]["top"] < l["mlp"]["router"]["experts"] for l in cfg["layers"])
    return assert_close_routed if routed else assert_close


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (configuration, directory, reference(tokens))"""
    out = {}
    for name, cfg in FOBANEX_CONFIGS.items():
        w = fobanex_weights(cfg, seed=len(name), sharp=2.0)
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
@pytest.mark.parametrize("name", sorted(FOBANEX_CONFIGS))
def test_prompts_portions_and_decoding_match_the_oracle(gpu, models, name, dtype):
    cfg, directory, ref = models[name]
    close, toks = close_of(cfg), tokens(cfg, 150, 1)
    want = ref(toks)
    d, e = engine(directory, dtype)
    with d:
        for portions in ([150], [1], [2], [3, 17, 1, 64], [100, 1], [64, 65, 1], [149, 1]):
            got = run(e, "r", toks, portions)
            e.finish("r")
            close(got, want, dtype, portions)


@pytest.mark.parametrize("name", sorted(FOBANEX_CONFIGS))
def test_first_tokens_in_fp32(gpu, models, name):
    cfg, directory, ref = models[name]
    d, e = engine(directory, "float32")
    with d:
        for i, toks in enumerate(([5], [3, 3], tokens(cfg, 4, 2))):
            assert position_errors(run(e, i, toks, [2, 1]), ref(toks)).max() < 2e-4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["quartet", "odd", "wide"])
def test_unequal_batches_equal_each_request_alone(gpu, models, name, dtype):
    """Portions of some requests beside single tokens of others; requests come, pause and go, and pages move from one
    to the next."""
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
        assert len(e._free_pages) == 24
    close = close_of(cfg)
    for r in lens:
        close(np.concatenate(got[r]), ref(seqs[r]), dtype, r)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["wide", "dense"])
def test_a_wide_decode_batch(gpu, models, name, dtype):
    """Many requests of unequal length decoded together: more tokens than the router's one launch takes."""
    cfg, directory, ref = models[name]
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
@pytest.mark.parametrize("name", ["quartet", "wide", "wider"])
def test_long_decoding_over_many_pages(gpu, models, name, dtype):
    cfg, directory, ref = models[name]
    toks = tokens(cfg, 420, 3)
    d, e = engine(directory, dtype)
    with d:
        got = run(e, "r", toks, [20, 1])
    close_of(cfg)(got, ref(toks), dtype)
    close_of(cfg)(got[-60:], ref(toks)[-60:], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_prompt_takes_the_expanded_form(gpu, tmp_path, dtype):
    """Latents wide enough that a long portion projects keys and values out of them first: own and shared, gated."""
    cfg = fobanex([shared_latent(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=256, q_rank=64, mlp=dense(64)),
                   shared_latent(0, heads=2, dim=64, rot_dim=32, vdim=96, kv_rank=256, q_rank=48)], width=128, vocab=90)
    w = fobanex_weights(cfg, 4, sharp=2.0)
    toks = tokens(cfg, 700, 5)
    want = ls.forward(cfg, {k: v.astype(np.float64) for k, v in w.items()}, toks)
    d, e = engine(write_stack(tmp_path, cfg, w), dtype, max_tokens=1024)
    with d:
        for portions in ([700], [30, 600, 1], [400, 2, 290, 1], [90, 1, 300, 5, 128]):
            got = run(e, "r", toks, portions)
            e.finish("r")
            assert_close(got, want, dtype, portions)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["quartet", "odd", "wide"])
def test_graphs_and_eager_steps_agree(gpu, models, name, dtype):
    """Captured decode steps, replayed with other work in between, give the eager results: bit for bit in fp32; in bf16
    the splits of the keys follow the graph's context bound instead of the batch's."""
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
    close_of(cfg)(outs[0], outs[1], dtype)


MARKED = 7


def far_key_model(kind):
    """One attention layer in which every query points at the marked token's key."""
    unturned = dict(dims=2, base=1e30)   # (one pair that position 0's frequency turns: kept out of the keys below)
    dim = 32
    if kind == "attention":
        cfg = fobanex([normed_attention(heads=4, kv_heads=2, dim=dim, vdim=24, rot=unturned, scale=1.5)], width=64, vocab=40, scale=1.0)
    elif kind == "attention_2":
        cfg = fobanex([key_value_attention(heads=4, kv_heads=2, dim=dim, rot=unturned, scale=1.5)], width=64, vocab=40, scale=1.0)
    else:
        share = kind == "shared_latent"
        own = shared_latent(heads=2, dim=dim, rot_dim=4, vdim=24, q_rank=16, kv_rank=40)
        cfg = fobanex([own, shared_latent(0, heads=3, dim=dim, rot_dim=4, vdim=20, q_rank=16, kv_rank=40)] if share else [own], width=64, vocab=40, scale=1.0)
        for l in cfg["layers"]:
            l["mixer"]["scale"] = 1.5
    w = fobanex_weights(cfg, 2)
    axis = np.sign(np.random.default_rng(5).standard_normal(dim)).astype(np.float32)
    axis[[0, 1]] = 0.0
    # one direction of the embeddings is everybody's (the queries read it), one is the marked token's (its keys do)
    w["embed"][:, 0], w["embed"][:, 1] = 2.0, 0.0
    w["embed"][MARKED, 1] = 2.0
    last = len(cfg["layers"]) - 1
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        x = p + "mix."
        w[p + "norm1"][:] = 1.0
        if l["type"] == "latent_attention":
            w[x + "dq"] *= 0.0
            w[x + "dq"][0, 0] = 1.0
            w[x + "dq.norm"][:] = 1.0
            w[x + "uq"] *= 0.0
            head = m["dim"] + m["rot_dim"]
            for h in range(m["heads"]):
                w[x + "uq"][h * head:h * head + dim, 0] = axis * 0.25
            if "kv_from" not in m:
                w[x + "dkv"][0] = 0.0
                w[x + "dkv"][0, 1] = 6.0
                w[x + "dkv"][40:] *= 0.0
            w[x + "uk"] *= 0.1
            for h in range(m["heads"]):
                w[x + "uk"][h * dim:(h + 1) * dim, 0] = axis
            if i < last:
                w[x + "o"] *= 0.0   # (the sharing layer alone tells)
        else:
            w[x + "q"] *= 0.0
            w[x + "k"] *= 0.1
            for h in range(m["heads"]):
                w[x + "q"][h * dim:(h + 1) * dim, 0] = axis
            for h in range(m["kv_heads"]):
                w[x + "k"][h * dim:(h + 1) * dim, 1] = axis
            if l["type"] == "attention":
                w[x + "q.norm"][:], w[x + "k.norm"][:] = 0.5, 1.0
    return cfg, {k: bf16(v) for k, v in w.items()}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["attention", "attention_2", "latent", "shared_latent"])
@pytest.mark.parametrize("place", [0, 1, 15, 16, 37, 63, 64])
def test_a_far_token_is_found_across_pages(gpu, tmp_path, dtype, kind, place):
    cfg, w = far_key_model(kind)
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
def test_pages_move_by_copies(gpu, models, dtype):
    """A request forked on the device and one swapped to the host and back go on as if nothing had happened; shared
    latents move once."""
    from pie_amd import driver as drvmod

    cfg, directory, ref = models["dense"]
    toks = tokens(cfg, 40, 14)
    want = ref(toks)
    d, _ = engine(directory, dtype, extra_batching="cpu_pages = 8")
    frame = lambda t0, t1, pages: drvmod.ForwardFrame(
        toks[t0:t1], range(t0, t1), pages[:(t1 + 15) // 16], [0, (t1 + 15) // 16], [(t1 - 1) % 16 + 1], [0, t1 - t0], sampling_indices=[t1 - t0 - 1],
        sampling_indptr=[0, 1], samplers=[dict(kind=7)], sampler_indptr=[0, 1])
    ok = lambda fr: d.handle(fr).payload.status.status
    with d:
        assert d.forward(frame(0, 30, [0, 1, 2])).num_requests == 1
        assert ok(drvmod.copy_frame(2, [0, 1], [10, 11])) == 0
        assert ok(drvmod.copy_frame(0, [0, 1], [4, 5])) == 0
        a = d.forward(frame(30, 40, [0, 1, 2]))
        b = d.forward(frame(30, 40, [10, 11, 12]))
        assert ok(drvmod.copy_frame(1, [4, 5], [20, 21])) == 0
        c = d.forward(frame(30, 40, [20, 21, 22]))
        for r in (a, b, c):
            assert_close(r.logits_of(0)[0], want[-1], dtype)
        assert np.array_equal(a.logits_of(0)[0], b.logits_of(0)[0]) and np.array_equal(a.logits_of(0)[0], c.logits_of(0)[0])


@pytest.mark.parametrize("name", ["quartet", "dense"])
def test_greedy_generation_through_both_entry_points(gpu, models, name):
    """The generation harness (replicas fork pages) and the engine's continuous batching."""
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
    cfg, directory, _ = models["quartet"]
    d, _ = engine(directory, "bfloat16")
    with d:
        caps = d.capabilities()
        assert not caps["rs_cache_required"] and caps["arch_name"] == "fobanex"

    def refused(what, change):
        c = json.loads(json.dumps(cfg))
        change(c)
        (tmp_path / "config.json").write_text(json.dumps(c))
        with pytest.raises(RuntimeError, match=what):
            engine(tmp_path, "bfloat16", extra_model="random_weights = true")
    refused("kv_from must name", lambda c: c["layers"][1]["mixer"].update(kv_from=1))
    refused("kv_from must name", lambda c: c["layers"][1]["mixer"].update(kv_from=3))
    refused("must be equal", lambda c: c["layers"][1]["mixer"].update(kv_rank=64))
    refused("equal groups", lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4))
    refused("fewer experts", lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=1) or c["layers"][1]["mlp"]["router"].update(top=4))
    refused("keys' size", lambda c: c["layers"][3]["mixer"].update(vdim=8))
    refused("multiple", lambda c: c["layers"][2]["mixer"].update(kv_heads=4))


def test_random_weights_need_only_the_configuration(gpu, tmp_path):
    cfg = FOBANEX_CONFIGS["quartet"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    d, e = engine(tmp_path, "bfloat16", extra_model="random_weights = true")
    with d:
        out = e.generate({"a": tokens(cfg, 40, 1), "b": [3]}, 5)
        assert all(0 <= x < cfg["vocab"] for r in out.values() for x in r)
        assert np.isfinite(e.step([("z", tokens(cfg, 90, 2), [89])])[0]).all()


def test_single_layers_of_every_kind(gpu, tmp_path):
    plain = dict(rot=rotary(8, scaling=False))
    for i, layers in enumerate(([normed_attention()], [key_value_attention()], [shared_latent()], [normed_attention(**plain, mlp=dense(24))],
                                [key_value_attention(**plain, mlp=moe(experts=4, top=4, groups=2, keep=2))],
                                [shared_latent(), shared_latent(0), shared_latent(0)])):
        cfg = fobanex(layers, width=80, vocab=50)
        w = fobanex_weights(cfg, i)
        want = ls.forward(cfg, {k: v.astype(np.float64) for k, v in w.items()}, toks := tokens(cfg, 70, i))
        directory = write_stack(tmp_path / str(i), cfg, w)
        for dtype in DTYPES:
            d, e = engine(directory, dtype)
            with d:
                assert_close(run(e, "r", toks, [66, 1, 2, 1]), want, dtype, i)


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_run_replays_a_trace(gpu, models, tmp_path, dtype):
    cfg, directory, ref = models["dense"]
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
