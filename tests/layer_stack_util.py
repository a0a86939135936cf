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


# ---- Lofudra -----------------------------------------------------------------------------------------
def dense(ff):
    return dict(kind="dense", ff=ff) if ff else None


def parallel(heads=6, kv_heads=2, dim=40, rot_dims=24, window=9, base=500.0, scale=None, r_heads=3, r_dim=20, r_vdim=12, decay=None,
             left_scale=0.7, right_scale=1.2, ff=56):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale if scale is not None else dim ** -0.5,
                mask=dict(size=window), rot=dict(dims=rot_dims, base=base))
    right = dict(heads=r_heads, dim=r_dim, vdim=r_vdim, decay=decay or [1.0 - 0.5 ** (2 + 3 * h) for h in range(r_heads)])
    return dict(type="parallel", mlp=dense(ff), mixer=dict(left=left, right=right, left_scale=left_scale, right_scale=right_scale))


def mlstm(heads=3, dim=20, vdim=24, gate_cap=9.0, ff=72):
    return dict(type="mlstm", mlp=dense(ff), mixer=dict(heads=heads, dim=dim, vdim=vdim, gate_cap=gate_cap))


def mamba2(heads=6, vdim=12, state=20, groups=3, conv=4, norm_groups=4, ff=40):
    return dict(type="mamba2", mlp=dense(ff),
                mixer=dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups))


def lofudra(layers, loop=None, width=112, vocab=97, eps=1e-4):
    cfg = dict(architecture="Lofudra", layers=layers, width=width, vocab=vocab, norm=dict(eps=eps))
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


# sizes off every padding unit, heads shared and not, norm parts that cut heads, convolutions of one to six
# taps, windows of one token and wider than the prompts, no loop, a loop over some and over all layers, layers
# without a feed-forward, sizes of every matrix-core form and of the plain ones
LOFUDRA_CONFIGS = {
    "trio": lofudra([mlstm(), mamba2(), parallel()], loop=(0, 2, 2)),
    "first_attention": lofudra([parallel(heads=5, kv_heads=5, dim=18, rot_dims=18, window=1, r_heads=1, r_dim=7, r_vdim=9, ff=0),
                                mamba2(heads=4, vdim=10, state=9, groups=4, conv=1, norm_groups=1, ff=31),
                                mlstm(heads=1, dim=33, vdim=30, ff=0), mamba2(heads=2, vdim=18, state=40, groups=1, conv=6, norm_groups=6, ff=0)],
                               loop=(1, 3, 3), width=75, vocab=130),
    "all_looped": lofudra([parallel(heads=7, kv_heads=1, dim=64, rot_dims=32, window=33, left_scale=1.0, right_scale=1.0),
                           mlstm(heads=2, dim=64, vdim=40), mamba2(heads=8, vdim=16, state=64, groups=2, conv=2, norm_groups=2)], loop=(0, 3, 2)),
    "wide": lofudra([parallel(heads=20, kv_heads=1, dim=96, rot_dims=96, window=500, r_heads=2, r_dim=128, r_vdim=64, ff=64),
                     mlstm(heads=2, dim=130, vdim=68, gate_cap=15.0), mamba2(heads=4, vdim=64, state=128, groups=1, conv=3, norm_groups=4),
                     parallel(heads=4, kv_heads=2, dim=192, rot_dims=64, window=70, r_heads=2, r_dim=256, r_vdim=40)], width=160, vocab=64),
    "wider": lofudra([parallel(heads=2, kv_heads=1, dim=300, rot_dims=100, window=40, r_heads=1, r_dim=40, r_vdim=300, ff=0),
                      mlstm(heads=1, dim=260, vdim=36), mlstm(heads=2, dim=24, vdim=264),
                      parallel(heads=3, kv_heads=3, dim=250, rot_dims=250, window=64, ff=0)], loop=(1, 2, 1), width=128, vocab=80),
}


def lofudra_weights(cfg, seed=0, sharp=1.0):
    """`sharp` scales the attention's query norms: large values make single keys stand out."""
    rng = np.random.default_rng(seed)
    w, H = {}, cfg["width"]

    def lin(name, rows, cols, gain=1.0):
        w[name] = bf16(rng.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def vec(name, n, lo=0.7, hi=1.3):
        w[name] = bf16(rng.uniform(lo, hi, n))

    w["embed"] = bf16(rng.standard_normal((cfg["vocab"], H)))
    if "loop" in cfg:
        w["loop.step"] = bf16(rng.standard_normal((cfg["loop"]["times"], H)) * 0.5)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        x = p + "mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if layer["mlp"] else ()):
            vec(p + n, H)
        if layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            for n, heads in (("q", a["heads"]), ("k", a["kv_heads"])):
                lin(x + f"left.{n}", heads * a["dim"], H)
                w[x + f"left.{n}.b"] = bf16(rng.standard_normal(heads * a["dim"]) * 0.5)
                vec(x + f"left.{n}.norm", a["dim"], *((0.7 * sharp, 1.3 * sharp) if n == "q" else (0.7, 1.3)))
            lin(x + "left.o", H, a["heads"] * a["dim"])
            for n, rows in (("q", r["dim"]), ("k", r["dim"]), ("v", r["vdim"]), ("g", r["vdim"])):
                lin(x + f"right.{n}", r["heads"] * rows, H)
            lin(x + "right.o", H, r["heads"] * r["vdim"])
        elif layer["type"] == "mlstm":
            for n, rows in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"])):
                lin(x + n, m["heads"] * rows, H)
            lin(x + "o", H, m["heads"] * m["vdim"])
            vec(x + "norm", m["heads"] * m["vdim"])
            for n, mean in (("i", -1.0), ("f", 3.0)):
                lin(x + n, m["heads"], H, 3.0)
                w[x + n + ".b"] = bf16(mean + rng.standard_normal(m["heads"]))
        else:
            inner, bc = m["heads"] * m["vdim"], m["groups"] * m["state"]
            lin(x + "in", 2 * inner + 2 * bc + m["heads"], H)
            w[x + "conv"] = bf16(rng.standard_normal((inner + 2 * bc, m["conv"])) * 0.6)
            w[x + "conv.b"] = bf16(rng.standard_normal(inner + 2 * bc) * 0.3)
            w[x + "dt_bias"] = bf16(rng.uniform(-3.0, 0.5, m["heads"]))
            w[x + "A_log"] = bf16(rng.uniform(-2.0, 1.0, m["heads"]))
            w[x + "D"] = bf16(rng.standard_normal(m["heads"]))
            vec(x + "norm", inner)
            lin(x + "o", H, inner)
        if layer["mlp"]:
            lin(p + "mlp.up", layer["mlp"]["ff"], H)
            lin(p + "mlp.down", H, layer["mlp"]["ff"])
    vec("final.norm", H)
    lin("head", cfg["vocab"], H, 3.0)
    return w


# ---- Fobanex -----------------------------------------------------------------------------------------
def moe(experts=9, top=3, ff=40, groups=3, keep=2, limit=1.5, scale=1.7):
    router = dict(experts=experts, top=top, scale=scale)
    if groups:
        router["groups"] = dict(count=groups, keep=keep)
    return dict(kind="moe", expert=dict(ff=ff, limit=limit), router=router)


def normed_attention(heads=6, kv_heads=2, dim=40, vdim=24, rot=None, scale=None, mlp=None):
    return dict(type="attention", mlp=mlp,
                mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, rot=rot or rotary(16), scale=scale if scale is not None else dim ** -0.5))


def key_value_attention(heads=6, kv_heads=3, dim=32, rot=None, scale=None, mlp=None):
    return dict(type="attention_2", mlp=mlp,
                mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, rot=rot or rotary(20), scale=scale if scale is not None else dim ** -0.5))


def shared_latent(kv_from=None, mlp=None, heads=3, dim=24, rot_dim=8, vdim=20, q_rank=40, kv_rank=48, base=500.0):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, rot=dict(dims=rot_dim, base=base),
             scale=(dim + rot_dim) ** -0.5)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="latent_attention", mlp=mlp, mixer=m)


def fobanex(layers, width=112, vocab=97, eps=1e-4, scale=3.0):
    return dict(architecture="Fobanex", layers=layers, width=width, vocab=vocab, norm=dict(eps=eps), embedding=dict(scale=scale))


# sizes off every padding unit, values wider and narrower than the keys, head counts shared and not, latents read by
# a neighbour, across other layers and by layers of other head counts, rotations with and without scaling, one
# expert, one group, all groups, all experts, layers without a feed-forward, sizes of every matrix-core form and of
# the plain ones
FOBANEX_CONFIGS = {
    "quartet": fobanex([shared_latent(mlp=dense(72)), shared_latent(0, moe()), normed_attention(mlp=moe(groups=0, top=2)), key_value_attention(mlp=dense(56))]),
    "dense": fobanex([normed_attention(mlp=dense(100)), shared_latent(heads=5, dim=40, rot_dim=16, vdim=33, kv_rank=100), key_value_attention(mlp=dense(31)),
                      shared_latent(1, dense(64), heads=2, dim=16, rot_dim=16, vdim=64, kv_rank=100, q_rank=64)], scale=1.0),
    "odd": fobanex([key_value_attention(heads=5, kv_heads=5, dim=18, rot=rotary(18), mlp=moe(experts=1, top=1, ff=17, groups=1, keep=1)),
                    normed_attention(heads=4, kv_heads=1, dim=20, vdim=28, rot=rotary(10, scaling=False)),
                    shared_latent(heads=2, dim=9, rot_dim=6, vdim=7, q_rank=11, kv_rank=13, mlp=moe(experts=20, top=5, ff=33, groups=4, keep=4, scale=1.0)),
                    shared_latent(2, heads=3, dim=12, rot_dim=6, vdim=5, q_rank=30, kv_rank=13)], width=75, vocab=130, scale=0.5),
    "wide": fobanex([normed_attention(heads=20, kv_heads=1, dim=96, vdim=64, rot=rotary(96, 300.0), mlp=moe(experts=40, top=8, ff=64, groups=5, keep=1)),
                     shared_latent(heads=17, dim=64, rot_dim=32, vdim=64, q_rank=96, kv_rank=128, mlp=dense(200)),
                     key_value_attention(heads=4, kv_heads=2, dim=192, rot=rotary(64)),
                     shared_latent(1, moe(experts=6, top=6, ff=128, groups=2, keep=2, limit=0.5), heads=33, dim=32, rot_dim=32, vdim=32, kv_rank=128),
                     shared_latent(heads=2, dim=32, rot_dim=16, vdim=16, kv_rank=520), shared_latent(1, heads=1, dim=64, rot_dim=32, vdim=40, kv_rank=128)],
                    width=160, vocab=64),
    "wider": fobanex([normed_attention(heads=2, kv_heads=1, dim=300, vdim=120, rot=rotary(100), mlp=dense(40)),
                      key_value_attention(heads=3, kv_heads=3, dim=264, rot=rotary(264, scaling=False)),
                      normed_attention(heads=3, kv_heads=3, dim=24, vdim=130, rot=rotary(24))], width=128, vocab=80),
}


def fobanex_weights(cfg, seed=0, sharp=1.0):
    """`sharp` scales the queries (through their norms where they have some): large values make single keys stand out."""
    rng = np.random.default_rng(seed)
    w, H = {}, cfg["width"]

    def lin(name, rows, cols, gain=1.0):
        w[name] = bf16(rng.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def vec(name, n, lo=0.7, hi=1.3):
        w[name] = bf16(rng.uniform(lo, hi, n))

    lin("embed", cfg["vocab"], H, np.sqrt(H))
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        x = p + "mix."
        vec(p + "norm1", H)
        if layer["type"] == "latent_attention":
            lin(x + "dq", m["q_rank"], H)
            vec(x + "dq.norm", m["q_rank"])
            lin(x + "uq", m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"], sharp)
            if "kv_from" not in m:
                lin(x + "dkv", m["kv_rank"] + m["rot_dim"], H)
                vec(x + "dkv.norm", m["kv_rank"])
            lin(x + "uk", m["heads"] * m["dim"], m["kv_rank"])
            lin(x + "uv", m["heads"] * m["vdim"], m["kv_rank"])
        else:
            lin(x + "q", m["heads"] * m["dim"], H, sharp if layer["type"] == "attention_2" else 1.0)
            lin(x + "k", m["kv_heads"] * m["dim"], H)
            if layer["type"] == "attention":
                lin(x + "v", m["kv_heads"] * m["vdim"], H)
                vec(x + "q.norm", m["heads"] * m["dim"], 0.7 * sharp, 1.3 * sharp)
                vec(x + "k.norm", m["kv_heads"] * m["dim"])
        if layer["type"] != "attention":
            lin(x + "g", m["heads"] * m["vdim"], H, 1.5)
        lin(x + "o", H, m["heads"] * m["vdim"], 2.0)
        if mlp and mlp["kind"] == "dense":
            for n, rows, cols in (("gate", mlp["ff"], H), ("up", mlp["ff"], H), ("down", H, mlp["ff"])):
                lin(p + "mlp." + n, rows, cols, 1.5)
                w[p + "mlp." + n + ".b"] = bf16(rng.standard_normal(rows) * 0.5)
        elif mlp:
            lin(p + "mlp.router", mlp["router"]["experts"], H, 2.0)
            for e in range(mlp["router"]["experts"]):
                for n, rows, cols in (("gate", mlp["expert"]["ff"], H), ("up", mlp["expert"]["ff"], H), ("down", H, mlp["expert"]["ff"])):
                    lin(f"{p}mlp.e{e}.{n}", rows, cols, 1.5)
    vec("final.norm", H)
    lin("head", cfg["vocab"], H, 3.0)
    return w


# ---- Minodra -----------------------------------------------------------------------------------------
def sink_latent(mlp=None, heads=3, dim=24, vdim=20, q_rank=40, kv_rank=48, scale=None):
    return dict(type="latent_attention", mlp=mlp,
                mixer=dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale if scale is not None else dim ** -0.5))


def shared_moe(experts=9, top=3, ff=40, shared=56):
    m = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    if shared:
        m["shared"] = dict(ff=shared)
    return m


def minodra(layers, width=112, vocab=97, eps=1e-4, scale=3.0, taps=3, softcap=11.0, bigram=(61, 97531, 2654435761)):
    e = dict(scale=scale)
    if bigram:
        e["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    return dict(architecture="Minodra", layers=layers, width=width, vocab=vocab, norm=dict(eps=eps), embedding=e, canon=dict(taps=taps),
                logit_softcap=softcap)


# sizes off every padding unit, values wider and narrower than the keys, convolutions of one to six taps, layers
# without a feed-forward at the end and between others, one expert, all experts, a shared expert narrower than the
# others, wider than one and than several, and none, multipliers beyond 32 bits, one bucket, no bigrams, widths of one
# and several blocks, sizes of every matrix-core form and of the plain ones
MINODRA_CONFIGS = {
    "pair": minodra([sink_latent(dense(72)), sink_latent(shared_moe(), heads=5, dim=40, vdim=33, q_rank=52, kv_rank=100)]),
    "odd": minodra([sink_latent(shared_moe(experts=1, top=1, ff=17, shared=0), heads=1, dim=9, vdim=7, q_rank=11, kv_rank=13), sink_latent(),
                    sink_latent(dense(31), heads=4, dim=33, vdim=48, q_rank=30, kv_rank=65), sink_latent()],
                   width=75, vocab=130, scale=0.5, taps=1, softcap=30.0, bigram=(1, 3, 5)),
    "wide": minodra([sink_latent(shared_moe(experts=40, top=8, ff=64, shared=300), heads=17, dim=32, vdim=32, q_rank=64, kv_rank=520),
                     sink_latent(shared_moe(experts=6, top=6, ff=150, shared=60), heads=33, dim=64, vdim=64, q_rank=96, kv_rank=200),
                     sink_latent(dense(200), heads=2, dim=32, vdim=96, q_rank=130, kv_rank=380)], width=160, vocab=64, taps=6),
    "broad": minodra([sink_latent(shared_moe(experts=5, top=2, ff=24, shared=24), heads=2, kv_rank=64),
                      sink_latent(dense(64), heads=6, dim=16, vdim=16, kv_rank=128)], width=2056, vocab=50, taps=4, bigram=None),
    "four": minodra([sink_latent(shared_moe(experts=20, top=5, ff=33, shared=33)), sink_latent(heads=2, dim=48, vdim=64, kv_rank=256),
                     sink_latent(shared_moe(experts=4, top=2, shared=0)), sink_latent(dense(40), heads=16, dim=16, vdim=24, kv_rank=192)],
                    width=96, taps=2, bigram=(2000, 1 << 40, 12345678901)),
}


def minodra_weights(cfg, seed=0, sharp=1.0, spread=0.4):
    """`sharp` scales the query projections: large values make single keys stand out.  `spread` of the corrections: large
    values make it rarer that two experts are all but equally good a choice, of which either weighs its whole score."""
    rng = np.random.default_rng(seed)
    w, H = {}, cfg["width"]

    def lin(name, rows, cols, gain=1.0):
        w[name] = bf16(rng.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def vec(name, n, lo=0.7, hi=1.3):
        w[name] = bf16(rng.uniform(lo, hi, n))

    lin("embed", cfg["vocab"], H, np.sqrt(H))
    if cfg["embedding"].get("bigram"):
        lin("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, H, 2.0 * np.sqrt(H))
    vec("embed.norm", ())
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        x, q = p + "mix.", p + "mlp."
        lin(x + "dq", m["q_rank"], H)
        vec(x + "dq.norm", m["q_rank"])
        lin(x + "uq", m["heads"] * m["dim"], m["q_rank"], sharp)
        lin(x + "dkv", m["kv_rank"], H)
        vec(x + "dkv.norm", m["kv_rank"])
        lin(x + "uk", m["heads"] * m["dim"], m["kv_rank"])
        lin(x + "uv", m["heads"] * m["vdim"], m["kv_rank"])
        w[x + "sink"] = bf16(rng.uniform(0.0, 4.0, m["heads"]))
        lin(x + "g", m["heads"], H, 1.5)
        lin(x + "o", H, m["heads"] * m["vdim"], 3.0)
        for n in ("1", "2") if mlp else ("1",):
            vec(p + "norm" + n, ())
            w[p + "canon" + n] = bf16(rng.standard_normal((H, cfg["canon"]["taps"])) * 0.5)
            lin(p + "rg" + n, H, H, 1.5)
            w[p + "rg" + n + ".b"] = bf16(rng.standard_normal(H) * 0.7)
        if mlp and mlp["kind"] == "dense":
            for n, rows, cols in (("gate", mlp["ff"], H), ("up", mlp["ff"], H), ("down", H, mlp["ff"])):
                lin(q + n, rows, cols, 1.5)
        elif mlp:
            E = mlp["router"]["experts"]
            lin(q + "router", E, H, 1.5)
            w[q + "correction"] = bf16(rng.uniform(-spread, spread, E))
            sizes = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(E)]
            if mlp.get("shared"):
                sizes.append(("shared.", mlp["shared"]["ff"]))
                lin(q + "shared.sg", 1, H, 2.0)
            for n, ff in sizes:
                lin(q + n + "up", ff, H, 1.5)
                lin(q + n + "down", H, ff, 1.5)
    vec("final.norm", ())
    lin("head", cfg["vocab"], H, 6.0)
    return w


def bf16(a):
    """Rounds to the nearest bf16 value (ties to even); returns float32."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    r = (u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)
    return r.view(np.float32).reshape(np.shape(a))


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
    save_file({k: torch.from_numpy(np.array(v, order="C")).to(torch.bfloat16) for k, v in weights.items()},
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


def assert_close_routed(got, want, dtype, what=""):
    """For mixtures: where two experts are all but equally probable, rounding to bf16 decides between them, at that token
    and a little at those that read it.  fp32: every position; bf16: one in six may be such a one."""
    e = np.sort(position_errors(got, want))
    assert np.isfinite(e).all(), what
    n = len(e)
    if dtype == "float32":
        assert e[-1] < F32_TOL, (what, e[-5:])
    else:
        assert e[-1] < 1.0 and e[n - 1 - n // 6] < BF16_TOL and (n < 8 or np.median(e) < BF16_MEDIAN), (what, np.median(e), e[-5:])


def engine(directory, dtype, **kw):
    from pie_amd.driver import Driver
    from pie_amd.engine import Engine

    d = Driver(stack_toml(directory, dtype, **kw))
    return d, Engine(d)


def tokens(cfg, n, seed=0):
    return [int(x) for x in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def run(e, rid, toks, portions):
    """Logits of every position, the request cut into `portions` (the last one repeats)."""
    got, at, i = [], 0, 0
    while at < len(toks):
        n = min(portions[min(i, len(portions) - 1)], len(toks) - at)
        got.append(e.step([(rid, toks[at:at + n], list(range(n)))])[0])
        at += n
        i += 1
    return np.concatenate(got)


def close_tie(logits):
    top = np.sort(logits, axis=-1)[..., -2:]
    return top[..., 1] - top[..., 0]
