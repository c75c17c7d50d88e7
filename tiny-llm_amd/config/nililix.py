"""Typed configuration of the Nililix architecture, read from config.json keys.

config.json of this design is nested: `layers` (the layers in order, each with `type`, which mixer; `mixer`, its sizes
and constants; and `mlp`, a dense feed-forward (`kind` "dense"), a mixture of experts ("moe") or null for none); `loop`
(`start`, `stop`, `times`: the layers from `start` up to but not including `stop` run `times` times over on the same
weights; absent: every layer runs once); `norm.eps`; `residual_mult`; `logit_softcap` (absent: none); `vocab`; `width`.
Every size and constant that can differ between models of the design comes from there; a layer has its own.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Sequence, Tuple, Union

from .llama import ConfigError

MIXERS = ("attention",)
MLP_KINDS = ("dense", "moe")
DEFAULT_MAX_POSITION = 131072       # the design has no limit of its own; the angle tables need one


@dataclass(frozen=True)
class RotaryScaling:
    factor: float
    low: float
    high: float
    original: float


@dataclass(frozen=True)
class SinkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int               # taps of the short convolution on q, k and v
    scale: float
    window: int             # 0: every earlier position is seen
    rot_dims: int           # 0: no rotation
    rot_base: float
    scaling: Optional[RotaryScaling]


@dataclass(frozen=True)
class DenseConfig:
    ff: int


@dataclass(frozen=True)
class MoeConfig:
    experts: int
    top: int
    ff: int
    groups: int
    keep: int


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class NililixLayer:
    type: str
    mixer: SinkAttentionConfig
    mlp: Union[DenseConfig, MoeConfig, None]


@dataclass(frozen=True)
class NililixConfig:
    vocab: int
    width: int
    norm_eps: float
    residual_mult: float
    logit_softcap: float    # 0: logits stay as they are
    layers: Tuple[NililixLayer, ...]
    loop: Optional[LoopConfig]
    max_position: int
    eos_token_ids: Tuple[int, ...] = ()

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], shapes: Optional[Mapping[str, Sequence[int]]] = None) -> "NililixConfig":
        missing = [k for k in ("vocab", "width", "layers", "norm") if d.get(k) is None]
        if missing:
            raise ConfigError(f"config.json lacks required keys: {', '.join(missing)}")
        if not isinstance(d["layers"], (list, tuple)) or not d["layers"]:
            raise ConfigError("`layers` must list at least one layer")
        layers = []
        for i, raw in enumerate(d["layers"]):
            kind = raw.get("type")
            if kind not in MIXERS:
                raise ConfigError(f"layer {i}: mixer type {kind!r} is not built; known: {', '.join(MIXERS)}")
            layers.append(NililixLayer(kind, _attention(i, raw.get("mixer") or {}), _mlp(i, raw.get("mlp"))))
        eps = float(_need("norm", d["norm"], "eps"))
        softcap = float(d.get("logit_softcap") or 0.0)
        if not eps > 0 or softcap < 0:
            raise ConfigError("norm.eps must be positive, and logit_softcap too where it is given")
        loop = None
        if d.get("loop"):
            lp = d["loop"]
            loop = LoopConfig(int(_need("loop", lp, "start")), int(_need("loop", lp, "stop")), int(_need("loop", lp, "times")))
            if not (0 <= loop.start < loop.stop <= len(layers)) or loop.times < 1:
                raise ConfigError(f"loop: layers {loop.start} .. {loop.stop - 1} run {loop.times} times: the run must "
                                  f"lie within the {len(layers)} layers, hold at least one and run at least once")
            if shapes is not None and "loop.step" in shapes and tuple(shapes["loop.step"])[0] != loop.times:
                raise ConfigError(f"loop.step has {tuple(shapes['loop.step'])[0]} rows, loop.times = {loop.times} are expected")
        eos = d.get("eos_token_id")
        eos = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else (eos,)))
        mult = d.get("residual_mult")
        cfg = cls(vocab=int(d["vocab"]), width=int(d["width"]), norm_eps=eps,
                  residual_mult=1.0 if mult is None else float(mult), logit_softcap=softcap, layers=tuple(layers), loop=loop,
                  max_position=int(d.get("max_position") or DEFAULT_MAX_POSITION), eos_token_ids=eos)
        if cfg.vocab <= 0 or cfg.width <= 0 or cfg.max_position <= 0:
            raise ConfigError("vocab, width and max_position must be positive")
        return cfg

    def run_order(self):
        """The layers in the order they run: (layer, pass number if the run begins a pass of the loop, else None)."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        lp = self.loop
        order = [(i, None) for i in range(lp.start)]
        for t in range(lp.times):
            order += [(i, t if i == lp.start else None) for i in range(lp.start, lp.stop)]
        return order + [(i, None) for i in range(lp.stop, n)]


def _need(where, m: Mapping[str, Any], key: str):
    if not isinstance(m, Mapping) or m.get(key) is None:
        raise ConfigError(f"layer {where}: `{key}` is missing")
    return m[key]


def _positive(where, m: Mapping[str, Any], key: str) -> int:
    v = int(_need(where, m, key))
    if v <= 0:
        raise ConfigError(f"layer {where}: `{key}` must be positive, got {v}")
    return v


def _attention(i: int, m: Mapping[str, Any]) -> SinkAttentionConfig:
    heads = _positive(i, m, "heads")
    kv = int(m.get("kv_heads") or heads)
    if kv <= 0 or heads % kv:
        raise ConfigError(f"layer {i}: heads = {heads} must be a multiple of kv_heads = {kv}")
    dim = _positive(i, m, "dim")
    rot = m.get("rot") or {}
    rot_dims = int(rot.get("dims") or 0)
    if rot_dims % 2 or not (0 <= rot_dims <= dim) or (rot_dims and not float(_need(i, rot, "base")) > 0):
        raise ConfigError(f"layer {i}: rot.dims = {rot_dims} must be even and within dim = {dim}, rot.base positive")
    scaling = None
    if rot_dims and rot.get("scaling"):
        s = rot["scaling"]
        scaling = RotaryScaling(*(float(_need(f"{i} (rot.scaling)", s, k)) for k in ("factor", "low", "high", "original")))
        if min(scaling.factor, scaling.low, scaling.original) <= 0 or scaling.high < scaling.low:
            raise ConfigError(f"layer {i}: rot.scaling needs positive constants and low within high")
    window = int((m.get("mask") or {}).get("size") or 0)
    taps = int(m.get("conv") or 1)
    if window < 0 or taps < 1:
        raise ConfigError(f"layer {i}: mask.size and conv must be positive")
    return SinkAttentionConfig(heads, kv, dim, int(m.get("vdim") or dim), taps, float(_need(i, m, "scale")), window, rot_dims,
                               float(rot["base"]) if rot_dims else 0.0, scaling)


def _mlp(i: int, m: Optional[Mapping[str, Any]]) -> Union[DenseConfig, MoeConfig, None]:
    if m is None:
        return None
    kind = m.get("kind")
    if kind not in MLP_KINDS:
        raise ConfigError(f"layer {i}: feed-forward kind {kind!r} is not built; known: {', '.join(MLP_KINDS)}")
    if kind == "dense":
        return DenseConfig(_positive(f"{i} (mlp)", m, "ff"))
    e, r = _need(i, m, "expert"), _need(i, m, "router")
    g = r.get("groups") or {}
    count = int(g.get("count") or 1)
    cfg = MoeConfig(experts=_positive(f"{i} (mlp.router)", r, "experts"), top=_positive(f"{i} (mlp.router)", r, "top"),
                    ff=_positive(f"{i} (mlp.expert)", e, "ff"), groups=count, keep=int(g.get("keep") or count))
    if cfg.groups < 1 or cfg.experts % cfg.groups or not (0 < cfg.keep <= cfg.groups):
        raise ConfigError(f"layer {i}: router.groups.count must divide router.experts, and keep lie within it")
    if cfg.top > cfg.keep * (cfg.experts // cfg.groups):
        raise ConfigError(f"layer {i}: the {cfg.keep} kept groups hold fewer than router.top = {cfg.top} experts")
    return cfg
