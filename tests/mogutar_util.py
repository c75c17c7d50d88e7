"""Test material for the Mogutar architecture: small configurations that differ from each other in every size
and option, and a generator of random checkpoints for them (numpy, its own scales: queries and keys that make
the softmax far from uniform, decays that forget at a visible rate, routers that decide, corrections that change
their choice, biases and norm weights that are neither zero nor one)."""
import copy
import json
import os

import numpy as np
import torch

from fofapel_util import as_double, rounded, row_err  # noqa: F401  (the same comparisons serve every design)


def left(heads, kv_heads, dim, vdim, conv, window=0, keep=0, rot_dims=0, yarn=None, softcap=0.0, base=10000.0, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv,
         "scale": float(scale if scale is not None else 2.0 * dim ** -0.5)}
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims}
        if yarn:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    if softcap:
        m["softcap"] = softcap
    return m


def right(heads, groups, state, vdim, conv, norm_groups):
    return {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv, "norm_groups": norm_groups}


def parallel(l, r, ls=1.0, rs=1.0):
    return {"type": "parallel", "mixer": {"left": l, "right": r, "left_scale": ls, "right_scale": rs}}


def lightning(heads, dim, vdim, decay=None):
    decay = decay or [1.0 - 2.0 ** -(1 + 1.5 * h) for h in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}}


def moe(experts, top, ff, groups=None):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def layer(mixer, mlp):
    return dict(mixer, mlp=mlp)


def model(width, vocab, layers, side=16, eps=1e-5):
    cfg = {"architecture": "Mogutar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if side:
        cfg["token_side"] = {"dim": side}
    return cfg


# every mixer, sizes that differ from layer to layer: keys wider and narrower than values, grouped and ungrouped heads,
# windows of 24, 7 and 50 positions that keep 5, 1 and 20 first tokens (fewer and more than a page), part and all of a
# head rotated with and without YaRN, 2 to 4 taps, shared and own B and C, one and several norm groups, groups of
# experts of which one or two are kept, a layer without feed-forward
MIX_A = model(64, 301, [
    layer(lightning(3, 24, 16), moe(8, 3, 24, (4, 2))),
    layer(parallel(left(4, 2, 24, 16, 3, 24, 5, 8, (4.0, 64, 32.0, 1.0), 9.0, 1000.0), right(4, 2, 24, 16, 4, 2), 0.7, 1.2),
          moe(6, 2, 16, (2, 1))),
    layer(parallel(left(3, 3, 16, 40, 2, 7, 1, 16, None, 30.0), right(6, 1, 16, 8, 2, 3), 1.3, 0.6), None),
    layer(lightning(4, 8, 40, [0.9, 0.3, 1.0, 0.99]), moe(9, 2, 8, (3, 2))),
    layer(parallel(left(2, 1, 32, 16, 4, 50, 20, 4, (8.0, 32, 8.0, 2.0), 0.0, 500.0), right(2, 2, 40, 24, 3, 1), 1.0, 1.0),
          moe(5, 2, 16)),
], side=16)

# one head, twenty heads (two tiles of heads), a window of one token that keeps none, of more than any prompt, no window,
# no rotation, no cap, one tap, one expert, every expert, groups of one expert, no token input
MIX_B = model(128, 257, [
    layer(parallel(left(1, 1, 64, 128, 1, 1, 0, 64, None, 5.0), right(1, 1, 8, 128, 1, 4), 0.5, 0.5), moe(4, 2, 32, (4, 3))),
    layer(parallel(left(20, 4, 8, 8, 3), right(16, 4, 32, 8, 4, 16), 1.0, 2.0), moe(1, 1, 16)),
    layer(lightning(1, 128, 64, [0.97]), moe(6, 6, 8)),
    layer(parallel(left(6, 3, 16, 8, 5, 1000, 3, 2, (2.0, 16, 4.0, 1.0), 50.0, 100.0), right(3, 3, 16, 40, 6, 1), 1.0, 1.0), None),
], side=0, eps=3e-6)

# sizes that are multiples of nothing (float32 only)
ODD = model(50, 199, [
    layer(lightning(3, 10, 7), moe(6, 2, 11, (2, 1))),
    layer(parallel(left(3, 1, 10, 7, 3, 13, 3, 4, (3.0, 20, 5.0, 1.0), 7.0, 777.0), right(3, 1, 9, 5, 3, 3), 0.9, 1.1), moe(5, 3, 7)),
], side=6)

# heads beyond what the matrix-core attention kernels take: the general kernel in both precisions; a state of 136 rows
WIDE = model(64, 199, [
    layer(parallel(left(2, 1, 136, 200, 3, 33, 4, 20, None, 12.0), right(2, 1, 136, 32, 4, 1)), moe(3, 2, 16)),
    layer(lightning(2, 200, 16), None)], side=8)

ONLY_LIGHTNING = model(64, 199, [layer(lightning(4, 16, 24), None)], side=0)
ONLY_PARALLEL = model(64, 199, [layer(parallel(left(4, 2, 16, 24, 3, 20, 3, 8, (4.0, 64, 32.0, 1.0), 10.0),
                                                right(4, 2, 16, 8, 4, 2)), None)], side=0)
ONLY_MOE = model(64, 199, [layer(lightning(2, 8, 8), moe(12, 3, 16, (4, 2)))], side=0)
ONLY_SIDE = model(64, 199, [layer(lightning(2, 8, 8), None)], side=20)

CONFIGS = {"A": (MIX_A, 16), "B": (MIX_B, 8), "odd": (ODD, 4), "wide": (WIDE, 16), "lightning": (ONLY_LIGHTNING, 4),
           "parallel": (ONLY_PARALLEL, 8), "moe": (ONLY_MOE, 16), "side": (ONLY_SIDE, 16)}


def every_expert(cfg):
    """The same model with every expert chosen by every token: its routing cannot flip where two scores are
    close, so a bfloat16 engine and the plain model choose alike."""
    out = copy.deepcopy(cfg)
    for l in out["layers"]:
        if l["mlp"]:
            r = l["mlp"]["router"]
            r["top"] = r["experts"]
            r.pop("groups", None)
    return out


def random_config(seed, multiple=8):
    """A configuration drawn at random: width, vocabulary, constants, two to five layers that each draw their own
    mixer, head counts, sizes, windows, taps and experts."""
    import random
    rng = random.Random(seed)
    m = multiple
    layers = []
    for _ in range(rng.randrange(2, 6)):
        if rng.random() < 0.4:
            heads = rng.randrange(1, 7)
            mix = lightning(heads, m * rng.randrange(1, 9), m * rng.randrange(1, 9), [rng.choice([0.3, 0.8, 0.99, 1.0]) for _ in range(heads)])
        else:
            kv = rng.choice([1, 2, 3, 4])
            dim = m * rng.randrange(1, 9)
            window = rng.choice([0, 1, 2, 9, 31, 64, 100, 5000])
            a = left(kv * rng.choice([1, 2, 4]), kv, dim, m * rng.randrange(1, 9), rng.choice([1, 2, 3, 4, 6]), window,
                     rng.choice([0, 1, 4, 17, 70]) if window else 0, rng.choice([0, dim, max(2, dim // 4 * 2)]),
                     rng.choice([None, (4.0, 64, 16.0, 1.0), (1.5, 2048, 32.0, 1.0)]), rng.choice([0.0, 4.0, 25.0]),
                     rng.choice([100.0, 10000.0, 300000.0]))
            groups = rng.choice([1, 2, 3])
            heads = groups * rng.choice([1, 2, 4])
            mix = parallel(a, right(heads, groups, m * rng.randrange(1, 9), m * rng.randrange(1, 9), rng.choice([1, 2, 3, 4, 6]),
                                    rng.choice([1, groups, heads])), rng.choice([1.0, 0.6, 1.7]), rng.choice([1.0, 0.3, 1.2]))
        mlp = None
        if rng.random() < 0.75:
            count = rng.choice([1, 2, 4])
            per = rng.randrange(1, 5)
            keep = rng.randrange(1, count + 1)
            mlp = moe(count * per, rng.randrange(1, keep * per + 1), m * rng.randrange(1, 12), (count, keep) if count > 1 else None)
        layers.append(layer(mix, mlp))
    return model(rng.choice([64, 96, 128, 192, 256]), rng.randrange(90, 700), layers, side=rng.choice([0, 8, 12, 32]),
                 eps=rng.choice([1e-5, 1e-6, 1e-4]))


def random_weights(cfg, seed=0, sharpen=3.0):
    """{name: tensor} (float32).  `sharpen`: the gain of the projections that make scores and gates (3: far from
    uniform, a misplaced key or a lost state moves the logits; 1: tame, so that bfloat16 rounding is not amplified)."""
    lively = 2.0 if sharpen > 1.0 else 1.0
    rng = np.random.default_rng(seed)
    W, V, n, out = cfg["width"], cfg["vocab"], len(cfg["layers"]), {}

    def mat(name, rows, cols, gain=1.0):
        out[name] = rng.standard_normal((rows, cols)) * gain / np.sqrt(cols)

    def vec(name, size, mean=0.0, std=0.1):
        out[name] = mean + std * rng.standard_normal(size)

    mat("embed", V, W, gain=np.sqrt(W))
    side = (cfg.get("token_side") or {}).get("dim", 0)
    if side:
        out["side.embed"] = rng.standard_normal((V, n * side))
    for i, l in enumerate(cfg["layers"]):
        p, a = f"l{i}.", l["mixer"]
        vec(p + "norm1", W, 1.0, 0.2)
        # a sublayer reads a stream that has grown to some depth: projections shrink with it
        shrink = 1.0 / np.sqrt(1.0 + 2.0 * i)
        if l["type"] == "lightning":
            H, D, Vd = a["heads"], a["dim"], a["vdim"]
            mat(p + "mix.q", H * D, W, gain=lively * shrink)
            mat(p + "mix.k", H * D, W, gain=lively * shrink)
            mat(p + "mix.v", H * Vd, W, gain=lively * shrink)
            mat(p + "mix.g", H * Vd, W, gain=lively * shrink)
            vec(p + "mix.norm", H * Vd, 1.0, 0.2)
            mat(p + "mix.o", W, H * Vd)
        else:
            b, c = a["left"], a["right"]
            H, G, D, Vd, taps = b["heads"], b["kv_heads"], b["dim"], b["vdim"], b["conv"]
            for name, size in (("q", H * D), ("k", G * D), ("v", G * Vd)):
                mat(p + f"mix.left.{name}", size, W, gain=shrink)
                vec(p + f"mix.left.{name}.b", size, 0.0, 0.3)
                out[p + f"mix.left.{name}.conv"] = rng.standard_normal((size, taps)) * 0.6
            vec(p + "mix.left.q.norm", D, 1.0, 0.2)
            vec(p + "mix.left.k.norm", D, 1.0, 0.2)
            out[p + "mix.left.q.norm"] *= np.sqrt(sharpen)
            out[p + "mix.left.k.norm"] *= np.sqrt(sharpen)
            mat(p + "mix.left.o", W, H * Vd)
            H, G, N, Vd, taps = c["heads"], c["groups"], c["state"], c["vdim"], c["conv"]
            channels = H * Vd + 2 * G * N
            mat(p + "mix.right.in", H * Vd + channels + H, W, gain=lively * shrink)
            out[p + "mix.right.conv"] = rng.standard_normal((channels, taps)) * 0.6
            vec(p + "mix.right.conv.b", channels, 0.0, 0.3)
            vec(p + "mix.right.dt_bias", H, -1.0, 0.7)
            vec(p + "mix.right.A_log", H, -0.5, 0.8)
            vec(p + "mix.right.D", H, 1.0, 0.3)
            vec(p + "mix.right.norm", H * Vd, 1.0, 0.2)
            mat(p + "mix.right.o", W, H * Vd)
        mlp = l["mlp"]
        if mlp is not None:
            vec(p + "norm2", W, 1.0, 0.2)
            F, E = mlp["expert"]["ff"], mlp["router"]["experts"]
            for e in range(E):
                mat(p + f"mlp.e{e}.gate", F, W, gain=lively * shrink)
                mat(p + f"mlp.e{e}.up", F, W, gain=lively * shrink)
                mat(p + f"mlp.e{e}.down", W, F)
            mat(p + "mlp.router", E, W, gain=lively * shrink)
            vec(p + "mlp.correction", E, 0.0, 0.6)      # many choice scores negative, many choices changed
        if side:
            mat(p + "side.gate", side, W, gain=lively * shrink)
            mat(p + "side.proj", W, side)
            vec(p + "side.norm", W, 1.0, 0.2)
    vec("final.norm", W, 1.0, 0.2)
    mat("head", V, W)
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
