"""Recurrent mixers whose state decays by one number per head and token: S <- a S + k (c v)^T, o = S^T q (+ D v), with
S [dim, vdim] per head.

`state_space` (state-space duality).  Per token, h the mixer's input, inner = heads * vdim:
    [z: inner | x: inner | B: groups * dim | C: groups * dim | dt: heads] = W_in h
    x, B, C <- silu(conv + b)                    a short causal convolution per channel, over x, B and C together
    c = softplus(dt + dt_bias),  a = exp(-exp(A_log) c)                        per head
    head n, with B and C of group n // (heads / groups):  S <- a S + B (c x)^T;  y = S^T C + D x
    y <- y * silu(z); each of `norm_groups` equal parts divided by its own root mean square, times a weight a channel
    out = out_scale * W_o y
Tensor names below the prefix: in, conv, conv.b, dt_bias, A_log, D, norm, o.

`decayed_attention` (linear attention with a constant decay per head):
    q, k, v = silu(W_q h), silu(W_k h), silu(W_v h)                            heads x dim, dim, vdim
    S <- decay_n S + k v^T;  o = S^T q                                         per head n, no other scale
    out = out_scale * W_o ( w * o / rms(o over all heads together) * sigmoid(W_g h) )
Tensor names below the prefix: q, k, v, g, norm, o.

Per request the part keeps S of every head and the convolution's last taps - 1 inputs in ONE float32 state row, which
the cache manager zeroes when the request is admitted.  The first product leaves float32; everything up to the rounded
operand of the output product is float32 in both precisions.
"""
from __future__ import annotations

from typing import Dict, List, Sequence

import torch

from ..kernels import ops
from .base import Mixer, StateSpec, WeightSpec, register_mixer


def _pad(n: int, m: int) -> int:
    return -(-n // m) * m


def _chunks(ctx):
    """The step's tokens in the recurrence's chunks, if some request may bring many."""
    return ctx.attention_tiles(ops.LINEAR_CHUNK) if ctx.max_q_len >= ops.LINEAR_CHUNK_TOKENS else None


def _forward(part, h, ctx, state, residual):
    """The first product, `mix`, the output product."""
    T, dev = h.shape[0], h.device
    p = ops.linear(h, part.w_in, ops.scratch("recurrence_in", (T, part.in_width), torch.float32, dev))
    z = part.mix(p, ctx, None, state, ops.scratch("recurrence_gated", (T, part.out_width), part.dtype, dev))
    if residual is None:
        out = ops.scratch("sublayer_out", (z.shape[0], part.hidden_size), torch.float32, z.device)
        return ops.linear(z, part.w_o, out)
    return ops.linear(z, part.w_o, residual, residual)


class StateSpace(Mixer):
    graph_safe = True
    splits_products = True

    def __init__(self, prefix, dtype, device, *, hidden_size: int, num_heads: int, groups: int, state_dim: int,
                 value_dim: int, conv_taps: int, norm_groups: int, eps: float, out_scale: float = 1.0,
                 names: Dict[str, str] = None):
        super().__init__(prefix, dtype, device)
        self.hidden_size, self.num_heads, self.groups = int(hidden_size), int(num_heads), int(groups)
        self.dim, self.vdim, self.taps = int(state_dim), int(value_dim), int(conv_taps)
        self.norm_groups, self.eps, self.out_scale = int(norm_groups), float(eps), float(out_scale)
        if self.num_heads <= 0 or self.groups <= 0 or self.num_heads % self.groups:
            raise ValueError(f"{prefix}: {self.num_heads} heads over {self.groups} groups: heads must be a multiple of groups")
        if not (0 < self.dim <= ops.LINEAR_MAX_DIM) or self.vdim <= 0 or not (1 <= self.taps <= ops.DELTA_MAX_TAPS):
            raise ValueError(f"{prefix}: a state of 1 to {ops.LINEAR_MAX_DIM} rows, 1 to {ops.DELTA_MAX_TAPS} taps, got "
                             f"{self.dim} x {self.vdim} and {self.taps} taps")
        self.inner = self.num_heads * self.vdim
        if self.norm_groups <= 0 or self.inner % self.norm_groups:
            raise ValueError(f"{prefix}: {self.norm_groups} norm groups must divide heads * value_dim = {self.inner}")
        ops.check_linear_sizes(dtype, self.hidden_size, f"{prefix}: hidden_size")
        ops.check_linear_sizes(dtype, self.inner, f"{prefix}: heads * value_dim")
        self.channels = self.inner + 2 * self.groups * self.dim
        self.in_rows = self.inner + self.channels + self.num_heads
        self.in_width = _pad(self.in_rows, 8)
        # columns of the recurrence's operands: [x | B | C | c | a]
        self.dt_col = _pad(self.channels, 4)
        self.a_col = self.dt_col + _pad(self.num_heads, 4)
        self.x_width = self.a_col + _pad(self.num_heads, 4)
        self.out_width = self.inner
        self.s_floats = self.num_heads * self.dim * self.vdim
        n = {k: k for k in ("in", "conv", "dt_bias", "A_log", "D", "norm", "o")}
        n["conv_b"] = "conv.b"
        n.update(names or {})
        self.names = {k: f"{prefix}.{v}" for k, v in n.items()}
        self.w_in = self.conv_w = self.conv_b = self.dt_bias = self.a_log = self.skip = self.w_norm = self.w_o = None

    def weights(self) -> List[WeightSpec]:
        n, W, H = self.names, self.hidden_size, self.num_heads
        vec = dict(role="vector")
        return [WeightSpec(n["in"], (self.in_rows, W)), WeightSpec(n["conv"], (self.channels, self.taps), **vec),
                WeightSpec(n["conv_b"], (self.channels,), role="vector", init="zeros"), WeightSpec(n["dt_bias"], (H,), **vec),
                WeightSpec(n["A_log"], (H,), **vec), WeightSpec(n["D"], (H,), role="vector", init="ones"),
                WeightSpec(n["norm"], (self.inner,), role="vector", init="ones"), WeightSpec(n["o"], (W, self.inner))]

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        n = self.names
        f32 = lambda k: tensors[n[k]].to(torch.float32).contiguous()
        w = torch.zeros((self.in_width, self.hidden_size), dtype=self.dtype, device=tensors[n["in"]].device)
        w[:self.in_rows] = tensors[n["in"]]
        self.w_in = w
        self.conv_w, self.conv_b, self.dt_bias, self.a_log = f32("conv"), f32("conv_b"), f32("dt_bias"), f32("A_log")
        self.skip, self.w_norm = f32("D"), f32("norm")
        self.w_o = tensors[n["o"]].contiguous()

    def state_spec(self) -> StateSpec:
        # a multiple of four floats: rows of the state start at 16-byte boundaries
        return StateSpec((_pad(self.s_floats + self.channels * (self.taps - 1), 4),), torch.float32)

    def forward(self, h, ctx, cache, state, residual):
        return _forward(self, h, ctx, state, residual)

    def mix(self, p, ctx, cache, state, z):
        """From the first product's rows p (float32 [T, in_width]) to the output product's operand z ([T, out_width])."""
        T, dev, H = p.shape[0], p.device, self.num_heads
        single = ctx.max_q_len == 1 and T == ctx.num_requests       # every request brings one token
        x = ops.scratch("ssd_operands", (T, self.x_width), torch.float32, dev)
        conv = ops.ShortConv(self.conv_w, state, self.s_floats, ctx.cu_seqlens_q, ctx.state_slots,
                             None if single else ctx.attention_tiles(ops.CONV_RUN))
        ops.ssd_prepare(p, self.inner, self.inner + self.channels, conv, self.conv_b, self.a_log, self.dt_bias, x, self.dt_col,
                        self.a_col)
        if self.taps > 1 and not single:
            ops.conv_state_update(p, self.inner, self.channels, state, self.s_floats, ctx.cu_seqlens_q, ctx.state_slots,
                                  self.taps)
        y = ops.scratch("recurrence_out", (T, self.inner), torch.float32, dev)
        b_off = self.inner
        ops.linear_recurrence(x, b_off + self.groups * self.dim, b_off, 0, state, ctx.cu_seqlens_q, ctx.state_slots, y, H,
                              self.groups, self.dim, self.vdim, a_off=self.a_col, c_off=self.dt_col, skip=self.skip,
                              single=single, tiles=_chunks(ctx))
        return ops.group_norm_gate(y, self.w_norm, p[:, :self.inner], z, self.norm_groups, self.eps, "silu", True, self.out_scale)


class DecayedAttention(Mixer):
    graph_safe = True
    splits_products = True

    def __init__(self, prefix, dtype, device, *, hidden_size: int, num_heads: int, head_dim: int, value_dim: int,
                 decay: Sequence[float], eps: float, out_scale: float = 1.0, names: Dict[str, str] = None):
        super().__init__(prefix, dtype, device)
        self.hidden_size, self.num_heads = int(hidden_size), int(num_heads)
        self.dim, self.vdim, self.eps, self.out_scale = int(head_dim), int(value_dim), float(eps), float(out_scale)
        self.decay_values = tuple(float(d) for d in decay)
        if self.num_heads <= 0 or len(self.decay_values) != self.num_heads:
            raise ValueError(f"{prefix}: one decay per head, got {len(self.decay_values)} for {self.num_heads} heads")
        if not (0 < self.dim <= ops.LINEAR_MAX_DIM) or self.vdim <= 0:
            raise ValueError(f"{prefix}: a state of 1 to {ops.LINEAR_MAX_DIM} rows, got {self.dim} x {self.vdim}")
        self.inner, self.qk_size = self.num_heads * self.vdim, self.num_heads * self.dim
        ops.check_linear_sizes(dtype, self.hidden_size, f"{prefix}: hidden_size")
        ops.check_linear_sizes(dtype, self.inner, f"{prefix}: heads * value_dim")
        self.v_off = 2 * self.qk_size
        self.g_off = _pad(self.v_off + self.inner, 8)
        self.in_width = _pad(self.g_off + self.inner, 8)
        self.out_width = self.inner
        self.s_floats = self.num_heads * self.dim * self.vdim
        n = {k: k for k in ("q", "k", "v", "g", "norm", "o")}
        n.update(names or {})
        self.names = {k: f"{prefix}.{v}" for k, v in n.items()}
        self.w_in = self.decay = self.w_norm = self.w_o = None

    def weights(self) -> List[WeightSpec]:
        n, W = self.names, self.hidden_size
        return [WeightSpec(n["q"], (self.qk_size, W)), WeightSpec(n["k"], (self.qk_size, W)),
                WeightSpec(n["v"], (self.inner, W)), WeightSpec(n["g"], (self.inner, W)),
                WeightSpec(n["norm"], (self.inner,), role="vector", init="ones"), WeightSpec(n["o"], (W, self.inner))]

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        n = self.names
        dev = tensors[n["q"]].device
        w = torch.zeros((self.in_width, self.hidden_size), dtype=self.dtype, device=dev)
        for key, at in (("q", 0), ("k", self.qk_size), ("v", self.v_off), ("g", self.g_off)):
            w[at:at + tensors[n[key]].shape[0]] = tensors[n[key]]
        self.w_in = w
        self.decay = torch.tensor(self.decay_values, dtype=torch.float32, device=dev)
        self.w_norm = tensors[n["norm"]].to(torch.float32).contiguous()
        self.w_o = tensors[n["o"]].contiguous()

    def state_spec(self) -> StateSpec:
        return StateSpec((_pad(self.s_floats, 4),), torch.float32)

    def forward(self, h, ctx, cache, state, residual):
        return _forward(self, h, ctx, state, residual)

    def mix(self, p, ctx, cache, state, z):
        """From the first product's rows p (float32 [T, in_width]) to the output product's operand z ([T, out_width])."""
        T, dev, H = p.shape[0], p.device, self.num_heads
        o = ops.scratch("recurrence_out", (T, self.inner), torch.float32, dev)
        ops.linear_recurrence(p, 0, self.qk_size, self.v_off, state, ctx.cu_seqlens_q, ctx.state_slots, o, H, H, self.dim,
                              self.vdim, decay=self.decay, silu=True, single=ctx.max_q_len == 1, tiles=_chunks(ctx))
        return ops.group_norm_gate(o, self.w_norm, p[:, self.g_off:self.g_off + self.inner], z, 1, self.eps, "sigmoid", False,
                                   self.out_scale)


register_mixer("state_space", StateSpace)
register_mixer("decayed_attention", DecayedAttention)
