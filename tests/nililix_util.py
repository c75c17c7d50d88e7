"""Test material for the Nililix architecture: small configurations that differ from each other in every size and option,
and a generator of random checkpoints for them (numpy, its own scales: queries and keys that make the softmax far from
uniform, sinks of both signs, convolutions that matter, routers that decide, corrections that change their choice, pass
vectors and norm weights that are neither zero nor one)."""
import copy
import json
import os

import numpy as np
import torch

from fofapel_util import as_double, rounded, row_err  # noqa: F401  (the same comparisons serve every design)


def attention(heads, kv_heads, dim, vdim, conv, window=0, rot_dims=0, scaling=None, base=10000.0, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv,
         "scale": float(scale if scale is not None else 1.6 * dim ** -0.5)}
    if window:
        m["mask"] = {"size": window}
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"type": "attention", "mixer": m}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, groups=None):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def layer(mixer, mlp):
    return dict(mixer, mlp=mlp)


def model(width, vocab, layers, loop=None, mult=0.7, softcap=9.0, eps=1e-5):
    cfg = {"architecture": "Nililix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
           "layers": layers}
    if softcap:
        cfg["logit_softcap"] = softcap
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


# sizes that differ from layer to layer: keys wider and narrower than values, grouped and ungrouped heads, windows of 24, 7,
# 50 and one position, part and all of a head rotated with and without scaling, 2 to 4 taps, groups of experts of which one
# or two are kept, a layer without feed-forward inside the repeated run
MIX_A = model(64, 301, [
    layer(attention(4, 2, 24, 16, 3, 24, 8, (4.0, 1.0, 4.0, 64), 1000.0), dense(40)),
    layer(attention(3, 3, 16, 40, 2, 7, 16), moe(8, 3, 24, (4, 2))),
    layer(attention(6, 2, 32, 16, 4, 50, 20, (8.0, 1.0, 2.0, 32), 500.0), None),
    layer(attention(2, 1, 16, 24, 3, 1, 2), moe(6, 2, 16, (2, 1))),
    layer(attention(5, 1, 8, 8, 2, 33, 4, (2.0, 0.5, 8.0, 200), 77.0), dense(72)),
], loop=(1, 4, 3))

# one head, twenty heads, no window, no rotation, one tap, one expert, every expert, groups of one expert; every layer is
# repeated twice; no cap, the results added as they are
MIX_B = model(128, 257, [
    layer(attention(1, 1, 64, 128, 1, 0, 64), moe(4, 2, 32, (4, 3))),
    layer(attention(20, 4, 8, 8, 5, 3), moe(1, 1, 16)),
    layer(attention(16, 1, 16, 8, 6, 1000, 2, (3.0, 1.0, 4.0, 16), 100.0), moe(6, 6, 8)),
], loop=(0, 3, 2), mult=1.0, softcap=0.0, eps=3e-6)

# the last layers are repeated; one pass only; no loop
LOOP_END = model(64, 199, [layer(attention(4, 2, 16, 24, 3, 20, 8), dense(24)), layer(attention(2, 2, 24, 16, 2, 11), dense(16))],
                 loop=(1, 2, 4), mult=0.4)
LOOP_ONCE = model(64, 199, [layer(attention(4, 4, 16, 16, 4, 20, 8), dense(24)), layer(attention(2, 1, 24, 16, 2, 40), None)],
                  loop=(0, 2, 1), mult=1.3, softcap=20.0)
PLAIN = model(96, 199, [layer(attention(4, 2, 16, 24, 3, 20, 8, (4.0, 1.0, 4.0, 64)), None)])
ONLY_MOE = model(64, 199, [layer(attention(2, 1, 8, 8, 1, 2), moe(12, 3, 16, (4, 2)))])

# sizes that are multiples of nothing (float32 only)
ODD = model(50, 199, [
    layer(attention(3, 1, 10, 7, 3, 13, 4, (3.0, 1.0, 5.0, 20), 777.0), moe(6, 2, 11, (2, 1))),
    layer(attention(3, 3, 6, 13, 2, 5, 6), dense(29)),
], loop=(0, 1, 2), mult=0.55)

# heads beyond what the matrix-core attention kernels take, and more query heads a kv head than they take: the general kernel
WIDE = model(64, 199, [layer(attention(2, 1, 136, 200, 3, 33, 20), moe(3, 2, 16)),
                       layer(attention(18, 1, 8, 16, 2, 26, 8), dense(32))])

CONFIGS = {"A": (MIX_A, 16), "B": (MIX_B, 8), "odd": (ODD, 4), "wide": (WIDE, 16), "loop_end": (LOOP_END, 4),
           "loop_once": (LOOP_ONCE, 8), "plain": (PLAIN, 8), "moe": (ONLY_MOE, 16)}


def every_expert(cfg):
    """The same model with every expert chosen by every token: its routing cannot flip where two scores are
    close, so a bfloat16 engine and the plain model choose alike."""
    out = copy.deepcopy(cfg)
    for l in out["layers"]:
        if l["mlp"] and l["mlp"]["kind"] == "moe":
            r = l["mlp"]["router"]
            r["top"] = r["experts"]
            r.pop("groups", None)
    return out


def random_config(seed, multiple=8):
    """A configuration drawn at random: width, vocabulary, constants, a repeated run or none, two to five layers that each
    draw their own head counts, sizes, windows, taps, rotation and feed-forward."""
    import random
    rng = random.Random(seed)
    m = multiple
    layers = []
    for _ in range(rng.randrange(2, 6)):
        kv = rng.choice([1, 2, 3, 4])
        dim = m * rng.randrange(1, 9)
        mix = attention(kv * rng.choice([1, 2, 3, 4, 8]), kv, dim, m * rng.randrange(1, 9), rng.choice([1, 2, 3, 4, 6]),
                        rng.choice([0, 1, 2, 9, 31, 64, 65, 100, 5000]), rng.choice([0, dim, max(2, dim // 4 * 2)]),
                        rng.choice([None, (4.0, 1.0, 4.0, 64), (1.5, 0.5, 16.0, 2048), (16.0, 2.0, 3.0, 100)]),
                        rng.choice([100.0, 10000.0, 300000.0]))
        kind = rng.random()
        mlp = None
        if kind < 0.4:
            mlp = dense(m * rng.randrange(1, 20))
        elif kind < 0.85:
            count, per = rng.choice([1, 2, 4]), rng.randrange(1, 5)
            keep = rng.randrange(1, count + 1)
            mlp = moe(count * per, rng.randrange(1, keep * per + 1), m * rng.randrange(1, 12), (count, keep) if count > 1 else None)
        layers.append(layer(mix, mlp))
    loop = None
    if rng.random() < 0.7:
        start = rng.randrange(len(layers))
        loop = (start, rng.randrange(start + 1, len(layers) + 1), rng.choice([1, 2, 3]))
    return model(rng.choice([64, 96, 128, 192, 320]), rng.randrange(90, 700), layers, loop, rng.choice([1.0, 0.2, 0.6]),
                 rng.choice([0.0, 5.0, 50.0]), rng.choice([1e-5, 1e-6, 1e-4]))


def random_weights(cfg, seed=0, sharpen=3.0):
    """{name: tensor} (float32).  `sharpen`: how far the scores are from uniform (3: a misplaced key or a lost sink moves
    the logits; 1: tame, so that bfloat16 rounding is not amplified)."""
    rng = np.random.default_rng(seed)
    W, V, out = cfg["width"], cfg["vocab"], {}
    lively = 1.6 if sharpen > 1.0 else 1.0

    def mat(name, rows, cols, gain=1.0):
        out[name] = rng.standard_normal((rows, cols)) * gain / np.sqrt(cols)

    def vec(name, size, mean=0.0, std=0.1):
        out[name] = mean + std * rng.standard_normal(size)

    mat("embed", V, W, gain=np.sqrt(W))
    if cfg.get("loop"):
        out["loop.step"] = 0.7 * rng.standard_normal((cfg["loop"]["times"], W))
    for i, l in enumerate(cfg["layers"]):
        p, a = f"l{i}.", l["mixer"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"] else ()):
            vec(p + n, W, 1.0, 0.2)
        H, G, D, Vd, taps = a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["conv"]
        for name, size, gain in (("q", H * D, np.sqrt(sharpen)), ("k", G * D, np.sqrt(sharpen)), ("v", G * Vd, 1.0)):
            mat(p + f"mix.{name}", size, W, gain=gain)
            c = rng.standard_normal((size, taps)) * 0.4
            c[:, -1] += 0.8
            out[p + f"mix.{name}.conv"] = c
        vec(p + "mix.sink", H, 0.0, 1.5 if sharpen > 1.0 else 0.5)
        mat(p + "mix.g", H, W, gain=lively)
        mat(p + "mix.o", W, H * Vd)
        mlp = l["mlp"]
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            mat(p + "mlp.up", mlp["ff"], W, gain=lively)
            mat(p + "mlp.down", W, mlp["ff"])
            continue
        F, E = mlp["expert"]["ff"], mlp["router"]["experts"]
        for e in range(E):
            mat(p + f"mlp.e{e}.gate", F, W, gain=lively)
            mat(p + f"mlp.e{e}.up", F, W, gain=lively)
            mat(p + f"mlp.e{e}.down", W, F)
        mat(p + "mlp.router", E, W, gain=lively)
        vec(p + "mlp.correction", E, 0.0, 0.6)      # many choice scores negative, many choices changed
    vec("final.norm", W, 1.0, 0.2)
    mat("head", V, W, gain=4.0 if cfg.get("logit_softcap") else 1.0)
    return {k: torch.from_numpy(np.asarray(v, dtype=np.float32)) for k, v in out.items()}


def make_folder(path, cfg, seed=0, store=torch.float32, sharpen=3.0):
    """config.json and model.safetensors (written with the safetensors library).  Returns (folder, weights)."""
    from safetensors.torch import save_file
    folder = str(path)
    os.makedirs(folder, exist_ok=True)
    w = random_weights(cfg, seed, sharpen)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(store).contiguous() for k, v in w.items()}, os.path.join(folder, "model.safetensors"))
    return folder, w
