"""Small layer-stack models for the tests: configurations, random weights (bf16 values), snapshot
files, and drivers over them."""
import json
import os

import numpy as np


def rotary(dims, base=10000.0, scaling=True):
    r = dict(dims=dims, base=base)
    if scaling:
        r["scaling"] = dict(factor=3.0, original=64, fast=8.0, slow=0.5)
    return r


def latent(heads=3, dim=24, rot_dim=8, vdim=20, q_rank=40, kv_rank=48, ff=72, scale=None, rot=None):
    return dict(type="latent_attention", mlp=dict(kind="dense", ff=ff) if ff else None,
                mixer=dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
                           rot=rot or rotary(rot_dim), scale=scale if scale is not None else (dim + rot_dim) ** -0.5))


def delta(heads=4, kv_heads=2, dim=16, vdim=24, conv=3, ff=0):
    return dict(type="channel_delta", mlp=dict(kind="dense", ff=ff) if ff else None,
                mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv))


def stack(layers, width=112, vocab=97, eps=1e-4, logit_scale=0.75, logit_softcap=11.0):
    return dict(architecture="Varasun", layers=layers, width=width, vocab=vocab, norm=dict(eps=eps),
                logit_scale=logit_scale, logit_softcap=logit_softcap)


# name -> configuration: sizes off every padding unit, equal and unequal head counts, convolutions of
# one to six taps, layers without a feed-forward, every order of the two mixers, sizes that take the
# matrix-core kernels and sizes that fall back
CONFIGS = {
    "mixed": stack([latent(), delta(), latent(heads=5, dim=40, rot_dim=16, vdim=33, kv_rank=100, ff=0), delta(ff=56, conv=4)]),
    "delta_first": stack([delta(heads=6, kv_heads=6, dim=40, vdim=12, conv=1), delta(heads=3, kv_heads=1, dim=20, vdim=18, conv=6, ff=31),
                          latent(heads=2, dim=9, rot_dim=6, vdim=7, q_rank=11, kv_rank=13, rot=rotary(4, scaling=False))],
                         width=75, vocab=130, logit_scale=1.0),
    "wide_latent": stack([latent(heads=17, dim=32, rot_dim=32, vdim=32, q_rank=64, kv_rank=520, ff=64),
                          latent(heads=33, dim=64, rot_dim=40, vdim=64, q_rank=96, kv_rank=200, ff=128),
                          delta(heads=2, kv_heads=2, dim=130, vdim=68, conv=4)], width=160, vocab=64),
}

ATTENTION_ONLY = stack([latent(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=64, ff=48), latent(heads=2, dim=48, rot_dim=16, vdim=64, kv_rank=128, ff=0)])
DELTA_ONLY = stack([delta(heads=4, kv_heads=4, dim=32, vdim=32, conv=4, ff=48), delta(heads=2, kv_heads=1, dim=64, vdim=16, conv=2)])


def bf16(a):
    """Rounds to the nearest bf16 value (ties to even); returns float32."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    r = (u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)
    return r.view(np.float32)


def random_weights(cfg, seed=0, low_rank=12, sharp=1.0):
    """`sharp` scales the query projections: large values make single keys stand out."""
    rng = np.random.default_rng(seed)
    w = {}

    def lin(name, rows, cols, gain=1.0):
        w[name] = bf16(rng.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def vec(name, n, lo=0.7, hi=1.3):
        w[name] = bf16(rng.uniform(lo, hi, n))

    H = cfg["width"]
    w["embed"] = bf16(rng.standard_normal((cfg["vocab"], H)))
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        x = p + "mix."
        vec(p + "norm1", H)
        if layer["type"] == "latent_attention":
            lin(x + "dq", m["q_rank"], H)
            vec(x + "dq.norm", m["q_rank"])
            lin(x + "uq", m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"], sharp)
            lin(x + "dkv", m["kv_rank"] + m["rot_dim"], H)
            vec(x + "dkv.norm", m["kv_rank"])
            lin(x + "uk", m["heads"] * m["dim"], m["kv_rank"])
            lin(x + "uv", m["heads"] * m["vdim"], m["kv_rank"])
            lin(x + "o", H, m["heads"] * m["vdim"])
        else:
            kd, vd = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, ch in (("q", kd), ("k", kd), ("v", vd)):
                lin(x + n, ch, H)
                w[x + n + ".conv"] = bf16(rng.standard_normal((ch, m["conv"])) * 0.6)
            lin(x + "b", m["heads"], H, 1.5)
            w[x + "A_log"] = bf16(rng.uniform(-1.0, 2.0, m["heads"]))
            vec(x + "norm", m["vdim"])
            lin(x + "a1", low_rank, H)
            lin(x + "a2", m["heads"] * m["dim"], low_rank)
            w[x + "dt_bias"] = bf16(rng.uniform(-4.0, 0.5, m["heads"] * m["dim"]))
            lin(x + "g1", low_rank + 3, H)
            lin(x + "g2", vd, low_rank + 3)
            lin(x + "o", H, vd)
        if layer["mlp"]:
            vec(p + "norm2", H)
            lin(p + "mlp.up", layer["mlp"]["ff"], H)
            lin(p + "mlp.down", H, layer["mlp"]["ff"])
    vec("final.norm", H)
    lin("head", cfg["vocab"], H, 8.0)
    return w


def write_stack(directory, cfg, weights):
    import torch
    from safetensors.torch import save_file

    os.makedirs(directory, exist_ok=True)
    save_file({k: torch.from_numpy(np.ascontiguousarray(v)).to(torch.bfloat16) for k, v in weights.items()},
              os.path.join(directory, "model.safetensors"))
    with open(os.path.join(directory, "config.json"), "w") as f:
        json.dump(cfg, f)
    return str(directory)


def stack_toml(directory, dtype="bfloat16", page_size=16, total_pages=64, max_tokens=512, slots=6, requests=16, graphs=True,
               extra_model="", extra_batching=""):
    return f"""
[model]
hf_path = "{directory}"
compute_dtype = "{dtype}"
{extra_model}
[batching]
kv_page_size = {page_size}
total_pages = {total_pages}
max_forward_tokens = {max_tokens}
max_forward_requests = {requests}
rs_cache_slots = {slots}
{extra_batching}
[runtime]
warmup = false
use_graphs = {"true" if graphs else "false"}
"""


def position_errors(got, want):
    """Per position rms(got - want, mean taken off) / rms of the wanted logits."""
    got, want = np.atleast_2d(np.asarray(got, np.float64)), np.atleast_2d(np.asarray(want, np.float64))
    d = got - want
    d -= d.mean(axis=1, keepdims=True)
    return np.sqrt((d * d).mean(axis=1)) / np.sqrt((want * want).mean())


def logit_error(got, want):
    return float(position_errors(got, want).max())


# fp32: every position.  bf16: half of the positions under the first bound, every one under the second
# (a read-out of nearly zero length, divided by its own root mean square, can magnify rounding at a
# position here and there).
F32_TOL, BF16_MEDIAN, BF16_TOL = 2e-4, 0.03, 0.15


def assert_close(got, want, dtype, what=""):
    e = position_errors(got, want)
    assert np.isfinite(e).all(), what
    if dtype == "float32":
        assert e.max() < F32_TOL, (what, e.max(), int(e.argmax()))
    else:
        assert e.max() < BF16_TOL and (len(e) < 8 or np.median(e) < BF16_MEDIAN), (what, np.median(e), e.max(), int(e.argmax()))
