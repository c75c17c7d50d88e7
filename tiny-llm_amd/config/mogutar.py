"""Typed configuration of the Mogutar architecture, read from config.json keys.

config.json of this design is nested: `layers` (the layers in order, each with `type`, which mixer: `parallel` or
`lightning`; `mixer`, its sizes and constants, for `parallel` under `left` (attention) and `right` (state space) with
`left_scale` and `right_scale`; and `mlp`, a mixture of experts or null for none); `token_side.dim` (the numbers per
token and layer of the per-layer token input; absent: no layer has one); `norm.eps`; `vocab`; `width`.  Every size and
constant is read from there; a layer has its own.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Sequence, Tuple, Union

from .llama import ConfigError

MIXERS = ("parallel", "lightning")
MLP_KINDS = ("moe",)
DEFAULT_MAX_POSITION = 131072       # the design has no limit of its own; the angle tables need one


@dataclass(frozen=True)
class YarnConfig:
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class ConvAttentionConfig:
    """The left branch: attention with a short convolution on q, k and v and a norm per head."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    scale: float
    softcap: float          # 0: scores stay as they are
    window: int             # 0: every earlier position is seen
    keep_first: int
    rot_dims: int           # 0: no rotation
    rot_base: float
    yarn: Optional[YarnConfig]


@dataclass(frozen=True)
class StateSpaceConfig:
    """The right branch."""
    heads: int
    groups: int
    state: int
    vdim: int
    conv: int
    norm_groups: int


@dataclass(frozen=True)
class ParallelConfig:
    left: ConvAttentionConfig
    right: StateSpaceConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class MoeConfig:
    experts: int
    top: int
    ff: int
    groups: int
    keep: int


@dataclass(frozen=True)
class MogutarLayer:
    type: str
    mixer: Union[ParallelConfig, LightningConfig]
    mlp: Optional[MoeConfig]


@dataclass(frozen=True)
class MogutarConfig:
    vocab: int
    width: int
    norm_eps: float
    side_dim: int           # 0: no per-layer token input
    layers: Tuple[MogutarLayer, ...]
    max_position: int
    eos_token_ids: Tuple[int, ...] = ()

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], shapes: Optional[Mapping[str, Sequence[int]]] = None) -> "MogutarConfig":
        missing = [k for k in ("vocab", "width", "layers", "norm") if d.get(k) is None]
        if missing:
            raise ConfigError(f"config.json lacks required keys: {', '.join(missing)}")
        if not isinstance(d["layers"], (list, tuple)) or not d["layers"]:
            raise ConfigError("`layers` must list at least one layer")
        readers = {"parallel": _parallel, "lightning": _lightning}
        layers = []
        for i, raw in enumerate(d["layers"]):
            kind = raw.get("type")
            if kind not in MIXERS:
                raise ConfigError(f"layer {i}: mixer type {kind!r} is not built; known: {', '.join(MIXERS)}")
            layers.append(MogutarLayer(kind, readers[kind](i, raw.get("mixer") or {}), _mlp(i, raw.get("mlp"))))
        eps = float(_need("norm", d["norm"], "eps"))
        if not eps > 0:
            raise ConfigError("norm.eps must be positive")
        side = d.get("token_side")
        side_dim = _positive("token_side", side, "dim") if side else 0
        if side_dim and shapes is not None and "side.embed" in shapes \
                and tuple(shapes["side.embed"])[1] != side_dim * len(layers):
            raise ConfigError(f"side.embed is {tuple(shapes['side.embed'])[1]} wide, {len(layers)} layers of token_side.dim = "
                              f"{side_dim} need {side_dim * len(layers)}")
        eos = d.get("eos_token_id")
        eos = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else (eos,)))
        cfg = cls(vocab=int(d["vocab"]), width=int(d["width"]), norm_eps=eps, side_dim=side_dim, layers=tuple(layers),
                  max_position=int(d.get("max_position") or DEFAULT_MAX_POSITION), eos_token_ids=eos)
        if cfg.vocab <= 0 or cfg.width <= 0 or cfg.max_position <= 0:
            raise ConfigError("vocab, width and max_position must be positive")
        return cfg


def _need(where, m: Mapping[str, Any], key: str):
    if not isinstance(m, Mapping) or m.get(key) is None:
        raise ConfigError(f"layer {where}: `{key}` is missing")
    return m[key]


def _positive(where, m: Mapping[str, Any], key: str) -> int:
    v = int(_need(where, m, key))
    if v <= 0:
        raise ConfigError(f"layer {where}: `{key}` must be positive, got {v}")
    return v


def _parallel(i: int, m: Mapping[str, Any]) -> ParallelConfig:
    return ParallelConfig(_left(f"{i} (left)", _need(i, m, "left")), _right(f"{i} (right)", _need(i, m, "right")),
                          float(m.get("left_scale", 1.0)), float(m.get("right_scale", 1.0)))


def _left(where: str, m: Mapping[str, Any]) -> ConvAttentionConfig:
    heads = _positive(where, m, "heads")
    kv = int(m.get("kv_heads") or heads)
    if kv <= 0 or heads % kv:
        raise ConfigError(f"layer {where}: heads = {heads} must be a multiple of kv_heads = {kv}")
    dim = _positive(where, m, "dim")
    rot = m.get("rot") or {}
    rot_dims = int(rot.get("dims") or 0)
    if rot_dims % 2 or not (0 <= rot_dims <= dim) or (rot_dims and not float(_need(where, rot, "base")) > 1):
        raise ConfigError(f"layer {where}: rot.dims = {rot_dims} must be even and within dim = {dim}, rot.base above 1")
    yarn = None
    if rot_dims and rot.get("scaling"):
        s = rot["scaling"]
        yarn = YarnConfig(*(float(_need(where, s, k)) for k in ("factor", "original", "fast", "slow")))
        if min(yarn.factor, yarn.original, yarn.fast, yarn.slow) <= 0:
            raise ConfigError(f"layer {where}: rot.scaling's constants must be positive")
    mask = m.get("mask") or {}
    window, keep = int(mask.get("size") or 0), int(mask.get("keep_first") or 0)
    softcap = float(m.get("softcap") or 0.0)
    if window < 0 or keep < 0 or (keep and not window) or softcap < 0:
        raise ConfigError(f"layer {where}: mask.size, mask.keep_first and softcap are not negative, and kept tokens need a window")
    return ConvAttentionConfig(heads, kv, dim, int(m.get("vdim") or dim), _positive(where, m, "conv"),
                               float(_need(where, m, "scale")), softcap, window, keep, rot_dims,
                               float(rot.get("base", 10000.0)) if rot_dims else 0.0, yarn)


def _right(where: str, m: Mapping[str, Any]) -> StateSpaceConfig:
    c = StateSpaceConfig(_positive(where, m, "heads"), int(m.get("groups") or 1), _positive(where, m, "state"),
                         _positive(where, m, "vdim"), _positive(where, m, "conv"), int(m.get("norm_groups") or 1))
    if c.groups <= 0 or c.heads % c.groups or c.norm_groups <= 0 or (c.heads * c.vdim) % c.norm_groups:
        raise ConfigError(f"layer {where}: groups must divide heads, and norm_groups heads * vdim")
    return c


def _lightning(i: int, m: Mapping[str, Any]) -> LightningConfig:
    decay = _need(i, m, "decay")
    heads = _positive(i, m, "heads")
    if not isinstance(decay, (list, tuple)) or len(decay) != heads:
        raise ConfigError(f"layer {i}: `decay` lists one number per head")
    return LightningConfig(heads, _positive(i, m, "dim"), _positive(i, m, "vdim"), tuple(float(x) for x in decay))


def _mlp(i: int, m: Optional[Mapping[str, Any]]) -> Optional[MoeConfig]:
    if m is None:
        return None
    kind = m.get("kind", "moe")
    if kind not in MLP_KINDS:
        raise ConfigError(f"layer {i}: feed-forward kind {kind!r} is not built; known: {', '.join(MLP_KINDS)}")
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
