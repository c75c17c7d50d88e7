"""A plain, slow Nililix: every mechanism of the design as one small function, written from its equations with torch
on the CPU (float64 unless told otherwise).  It shares no code with the engine: it reads config.json's own keys and the
checkpoint's tensor names, keeps whole sequences (no cache, no pages, no state slots) and runs one request at a time.

Notation: x [T, W] is the residual stream; weights are [out, in]; N is an RMS norm with a weight; a layer is
x <- x + m Nb(mixer(Na(x))), then x <- x + m Nd(ffn(Nc(x))).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch


# --------------------------------------------------------------------------- small pieces
_round_to = None        # what `forward` was asked to round the products' operands to: (type, scale)


def product(h, w):
    """W h for every row of h; the operand is rounded first if the model runs with rounded operands."""
    if _round_to is not None:
        to, scale = _round_to
        h = (h * scale).to(to).to(h.dtype) / scale
    return h @ w.T


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def causal_conv(u, taps_w):
    """u [T, C], taps_w [C, n]: y[t, c] = sum_j taps_w[c, j] u[t + 1 - n + j, c]; what lies ahead of the sequence is 0."""
    y = torch.zeros_like(u)
    n = taps_w.shape[1]
    for t in range(u.shape[0]):
        for j in range(n):
            at = t + 1 - n + j
            if at >= 0:
                y[t] = y[t] + taps_w[:, j] * u[at]
    return y


# ------------------------------------------------------------------------ rotation
def stretched(f: float, s) -> float:
    """One frequency under the length scaling `s` (factor, low, high, original): turns that fit often enough into the
    original length stay, the slow ones are divided by the factor, the ones between are mixed."""
    wave = 2.0 * math.pi / f
    if wave < s["original"] / s["high"]:
        return f
    if wave > s["original"] / s["low"]:
        return f / s["factor"]
    keep = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
    return (1.0 - keep) * f / s["factor"] + keep * f


def rotate_pairs(x, positions, rot):
    """x [T, heads, D]: dims 2i and 2i + 1 of the first rot.dims turn together by position * f_i."""
    dims = rot["dims"]
    out = x.clone()
    for i in range(dims // 2):
        f = rot["base"] ** (-2.0 * i / dims)
        if rot.get("scaling"):
            f = stretched(f, rot["scaling"])
        a = positions.to(torch.float64) * f
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


# --------------------------------------------------------------------------- masks and attention
def window_mask(positions, size: int):
    """allowed[i, j]: key j is not ahead of query i and less than `size` positions back (size 0: any earlier key)."""
    back = positions[:, None] - positions[None, :]
    return (back >= 0) & (back < size) if size else back >= 0


def attend(q, k, v, allowed, scale, sink):
    """q [T, H, D], k [T, H, D], v [T, H, V] (key/value heads already matched to query heads), sink [H]: the softmax of a
    head runs over its visible keys and one more entry of score sink_h that carries no value."""
    T, H, _ = q.shape
    out = torch.zeros((T, H, v.shape[-1]), dtype=q.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h].T) * scale
        s = s.masked_fill(~allowed, float("-inf"))
        s = torch.cat([s, sink[h].to(s.dtype).expand(T, 1)], dim=1)
        out[:, h] = torch.softmax(s, dim=-1)[:, :T] @ v[:, h]
    return out


def attention(h, w, m, positions):
    """Projections, a short convolution on each, rotation of neighbouring dims, a window, a sink and a gate per head."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (causal_conv(product(h, w[n]), w[n + ".conv"]) for n in ("q", "k", "v"))
    q, k, v = q.reshape(T, H, D), k.reshape(T, G, D), v.reshape(T, G, V)
    if m.get("rot"):
        q, k = rotate_pairs(q, positions, m["rot"]), rotate_pairs(k, positions, m["rot"])
    k, v = k.repeat_interleave(H // G, dim=1), v.repeat_interleave(H // G, dim=1)
    o = attend(q, k, v, window_mask(positions, (m.get("mask") or {}).get("size", 0)), m["scale"], w["sink"])
    o = o * torch.sigmoid(product(h, w["g"]))[:, :, None]
    return product(o.reshape(T, H * V), w["o"])


# ------------------------------------------------------------------------- feed-forwards
def dense(h, w):
    return product(torch.clamp(product(h, w["up"]), min=0.0) ** 2, w["down"])


def choose(s, correction, top: int, groups: int, keep: int):
    """s [E], one token's scores: the indices of its experts.  Choice scores are s + correction; of `groups` equal
    runs of neighbours only the `keep` whose two best experts together score highest stay in."""
    c = [float(a) for a in s + correction]
    per = len(c) // groups
    open_to = set(range(len(c)))
    if groups > 1:
        rank = sorted(range(groups), key=lambda g: -sum(sorted(c[g * per:(g + 1) * per])[-2:]))
        open_to = {e for g in rank[:keep] for e in range(g * per, (g + 1) * per)}
    return sorted(open_to, key=lambda e: -c[e])[:top]


def expert(h, w, prefix):
    return product(silu(product(h, w[prefix + ".gate"])) * product(h, w[prefix + ".up"]), w[prefix + ".down"])


def moe(h, w, mlp):
    r = mlp["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    s = torch.sigmoid(product(h, w["router"]))
    out = torch.zeros_like(h)
    ids = [choose(s[t], w["correction"], r["top"], g["count"], g["keep"]) for t in range(h.shape[0])]
    for e in range(s.shape[1]):
        rows = [t for t in range(h.shape[0]) if e in ids[t]]
        if rows:
            out[rows] += s[rows, e][:, None] * expert(h[rows], w, f"e{e}")
    return out


# --------------------------------------------------------------------------- model
def sub(weights: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    n = len(prefix)
    return {k[n:]: v for k, v in weights.items() if k.startswith(prefix)}


def runs(cfg):
    """The layer runs in order: (layer, the pass this run opens or None)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    inner = range(loop["start"], loop["stop"])
    return [(i, None) for i in range(loop["start"])] \
        + [(i, t if i == loop["start"] else None) for t in range(loop["times"]) for i in inner] \
        + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, weights, tokens, dtype=torch.float64, trace: Optional[List[torch.Tensor]] = None, round_operands=None,
            round_scale: float = 1.0):
    """Logits [T, vocab] of one sequence; `trace` collects the residual stream after every layer run.
    round_operands (a torch dtype): what enters a matrix product is rounded to it and back, the roundings that
    any engine with products in that type must make; what they do to the logits says how far two correct
    implementations in that type may lie apart.  round_scale shifts the grid they are rounded to (another sample of the
    same noise)."""
    global _round_to
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps, m = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
    positions = torch.arange(len(tokens))
    x = w["embed"][torch.tensor(list(tokens), dtype=torch.long)]
    _round_to = None if round_operands is None else (round_operands, round_scale)
    try:
        for i, opens in runs(cfg):
            if opens is not None:
                x = x + w["loop.step"][opens]
            layer, p = cfg["layers"][i], f"l{i}."
            y = attention(rms_norm(x, w[p + "norm1"], eps), sub(w, p + "mix."), layer["mixer"], positions)
            x = x + m * rms_norm(y, w[p + "norm1b"], eps)
            mlp = layer.get("mlp")
            if mlp:
                h = rms_norm(x, w[p + "norm2"], eps)
                y = moe(h, sub(w, p + "mlp."), mlp) if mlp["kind"] == "moe" else dense(h, sub(w, p + "mlp."))
                x = x + m * rms_norm(y, w[p + "norm2b"], eps)
            if trace is not None:
                trace.append(x.clone())
        logits = product(rms_norm(x, w["final.norm"], eps), w["head"])
        cap = cfg.get("logit_softcap")
        return cap * torch.tanh(logits / cap) if cap else logits
    finally:
        _round_to = None
