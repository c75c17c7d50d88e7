"""A plain, slow Mogutar: every mechanism of the design as one small function, written from its
equations with torch on the CPU (float64 unless told otherwise).  It shares no code with the
engine: it reads config.json's own keys and the checkpoint's tensor names, keeps whole sequences
(no cache, no pages, no state slots) and runs one request at a time.

Notation: x [T, W] is the residual stream; weights are [out, in]; N is an RMS norm with
a weight; a layer is x <- x + N1(mixer(x)), then x <- x + N2(experts(x)), then x <- x + Ns(token input of x).
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


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(u, taps_w, bias=None):
    """u [T, C], taps_w [C, taps]: y[t, c] = sum_j taps_w[c, j] u[t - (taps - 1) + j, c] (+ bias[c]); inputs ahead of
    the sequence count as zero, the last column belongs to the current token."""
    T, taps = u.shape[0], taps_w.shape[1]
    pad = torch.cat([torch.zeros((taps - 1, u.shape[1]), dtype=u.dtype), u], dim=0)
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + pad[j:j + T] * taps_w[:, j]
    return y if bias is None else y + bias


# ------------------------------------------------------------------------ rotation
def yarn(freqs, dims: int, base: float, factor: float, original: float, fast: float, slow: float):
    """The blended frequencies and the factor that multiplies cosine and sine."""
    def index(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(index(fast)), 0), min(math.ceil(index(slow)), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * r + f * (1.0 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, positions, rot):
    """x [T, heads, D]: the first rot.dims of the last axis rotate, element i paired with i + dims/2."""
    dims, base = rot["dims"], rot["base"]
    if not dims:
        return x
    half = dims // 2
    freqs = [base ** (-2.0 * i / dims) for i in range(half)]
    mag = 1.0
    if rot.get("scaling"):
        s = rot["scaling"]
        freqs, mag = yarn(freqs, dims, base, s["factor"], s["original"], s["fast"], s["slow"])
    a = positions.to(torch.float64)[:, None] * torch.tensor(freqs, dtype=torch.float64)[None, :]
    cos, sin = (torch.cos(a) * mag)[:, None, :].to(x.dtype), (torch.sin(a) * mag)[:, None, :].to(x.dtype)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


# --------------------------------------------------------------------------- masks and attention
def window_with_first(positions, size: int, keep_first: int):
    """allowed[i, j]: key j is not ahead of query i, and is less than `size` back or among the first `keep_first`."""
    i, j = positions[:, None], positions[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def softcap(s, cap):
    return cap * torch.tanh(s / cap)


def attend(q, k, v, allowed, scale, cap):
    """q [T, H, D], k [T, H, D], v [T, H, V] (key/value heads already matched to query heads) -> [T, H, V]."""
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    if cap:
        s = softcap(s, cap)
    p = torch.softmax(s.masked_fill(~allowed[None], float("-inf")), dim=-1)
    return torch.einsum("hij,jhv->ihv", p, v)


def attention(h, w, m, eps, positions):
    """Projections with biases, a short convolution on each, a norm per head on queries and keys, rotation, capped
    scores inside a window that also keeps the first tokens."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (causal_conv(product(h, w[n]) + w[n + ".b"], w[n + ".conv"]) for n in ("q", "k", "v"))
    q = rms_norm(q.reshape(T, H, D), w["q.norm"], eps)
    k = rms_norm(k.reshape(T, G, D), w["k.norm"], eps)
    v = v.reshape(T, G, V)
    if m.get("rot"):
        q, k = rotate(q, positions, m["rot"]), rotate(k, positions, m["rot"])
    k, v = k.repeat_interleave(H // G, dim=1), v.repeat_interleave(H // G, dim=1)
    mask = m.get("mask")
    allowed = window_with_first(positions, mask["size"], mask.get("keep_first", 0)) if mask \
        else positions[None, :] <= positions[:, None]
    o = attend(q, k, v, allowed, m["scale"], m.get("softcap"))
    return product(o.reshape(T, H * V), w["o"])


# ------------------------------------------------------------------- the two recurrences
def decayed_scan(a, q, k, v):
    """a [T, H], q, k [T, H, N], v [T, H, V].  Per head, token by token: S <- a S + k v^T; o = S^T q."""
    T, H, N = q.shape
    S = torch.zeros((H, N, v.shape[-1]), dtype=q.dtype)
    out = torch.zeros((T, H, v.shape[-1]), dtype=q.dtype)
    for t in range(T):
        S = a[t][:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out


def mamba2(h, w, m, eps, positions=None):
    T = h.shape[0]
    H, V, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    p = product(h, w["in"])
    z, xbc, dt = p[:, :inner], p[:, inner:2 * inner + 2 * G * N], p[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x = xbc[:, :inner].reshape(T, H, V)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N).repeat_interleave(H // G, dim=1)
    C = xbc[:, inner + G * N:].reshape(T, G, N).repeat_interleave(H // G, dim=1)
    dt = torch.nn.functional.softplus(dt + w["dt_bias"], threshold=700.0)
    y = decayed_scan(torch.exp(-torch.exp(w["A_log"]) * dt), C, B, dt[:, :, None] * x) + w["D"][None, :, None] * x
    y = y.reshape(T, inner) * silu(z)
    y = unit_rms(y.reshape(T, m["norm_groups"], -1), eps).reshape(T, inner) * w["norm"]
    return product(y, w["o"])


def lightning(h, w, m, eps, positions=None):
    T = h.shape[0]
    H, N, V = m["heads"], m["dim"], m["vdim"]
    q, k = silu(product(h, w["q"])).reshape(T, H, N), silu(product(h, w["k"])).reshape(T, H, N)
    v = silu(product(h, w["v"])).reshape(T, H, V)
    a = torch.tensor(m["decay"], dtype=h.dtype).expand(T, H)
    o = rms_norm(decayed_scan(a, q, k, v).reshape(T, H * V), w["norm"], eps)
    return product(o * torch.sigmoid(product(h, w["g"])), w["o"])


def sub(weights: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    n = len(prefix)
    return {k[n:]: v for k, v in weights.items() if k.startswith(prefix)}


def parallel(h, w, m, eps, positions):
    return m["left_scale"] * attention(h, sub(w, "left."), m["left"], eps, positions) \
        + m["right_scale"] * mamba2(h, sub(w, "right."), m["right"], eps)


MIXERS = {"parallel": parallel, "lightning": lightning}


# ------------------------------------------------------------------------- experts
def choose(s, correction, top: int, groups: int, keep: int):
    """s [E], one token's scores: the indices of its experts.  Choice scores are s + correction; of `groups` equal
    runs of neighbours only the `keep` whose two best experts together score highest stay in."""
    c = s + correction
    if groups > 1:
        per = c.numel() // groups
        best = [sum(sorted(c[g * per:(g + 1) * per].tolist(), reverse=True)[:2]) for g in range(groups)]
        kept = sorted(range(groups), key=lambda g: -best[g])[:keep]
        inside = torch.tensor([e // per in kept for e in range(c.numel())])
        c = c.masked_fill(~inside, float("-inf"))
    return sorted(range(c.numel()), key=lambda e: -float(c[e]))[:top]


def expert(h, w, prefix):
    return product(silu(product(h, w[prefix + ".gate"])) * product(h, w[prefix + ".up"]), w[prefix + ".down"])


def moe(h, w, mlp):
    r = mlp["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    s = torch.sigmoid(product(h, w["router"]))
    ids = [choose(s[t], w["correction"], r["top"], g["count"], g["keep"]) for t in range(h.shape[0])]
    out = torch.zeros_like(h)
    for e in range(s.shape[1]):
        rows = [t for t in range(h.shape[0]) if e in ids[t]]
        if rows:
            out[rows] += s[rows, e][:, None] * expert(h[rows], w, f"e{e}")
    return out


# ----------------------------------------------------------------- per-layer token input
def token_input(h, table_rows, w):
    """table_rows [T, dim]: the token's part of the side table for this layer."""
    return product(gelu_tanh(product(h, w["gate"])) * table_rows, w["proj"])


# --------------------------------------------------------------------------- model
def forward(cfg, weights, tokens, dtype=torch.float64, trace: Optional[List[torch.Tensor]] = None, round_operands=None,
            round_scale: float = 1.0):
    """Logits [T, vocab] of one sequence; `trace` collects the residual stream after every layer.
    round_operands (a torch dtype): what enters a matrix product is rounded to it and back, the roundings that
    any engine with products in that type must make; what they do to the logits says how far two correct
    implementations in that type may lie apart.  round_scale shifts the grid they are rounded to (another sample of the
    same noise)."""
    global _round_to
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    ids = torch.tensor(list(tokens), dtype=torch.long)
    positions = torch.arange(len(ids))
    x = w["embed"][ids]
    side = cfg.get("token_side")
    _round_to = None if round_operands is None else (round_operands, round_scale)
    try:
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."
            y = MIXERS[layer["type"]](x, sub(w, p + "mix."), layer["mixer"], eps, positions)
            x = x + rms_norm(y, w[p + "norm1"], eps)
            if layer.get("mlp"):
                x = x + rms_norm(moe(x, sub(w, p + "mlp."), layer["mlp"]), w[p + "norm2"], eps)
            if side:
                rows = w["side.embed"][ids, i * side["dim"]:(i + 1) * side["dim"]]
                x = x + rms_norm(token_input(x, rows, sub(w, p + "side.")), w[p + "side.norm"], eps)
            if trace is not None:
                trace.append(x.clone())
        return product(rms_norm(x, w["final.norm"], eps), w["head"])
    finally:
        _round_to = None
