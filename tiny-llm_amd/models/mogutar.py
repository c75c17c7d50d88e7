"""The Mogutar architecture as data: MogutarConfig -> ModelSpec.

A decoder whose RMS norms sit on the sublayers' results only (block arrangement "output_norm": the sublayers read the
stream itself), with two mixers: "parallel", attention beside a state-space mixer over the same input, each times a
constant ("gated_attention" with biases, a short convolution on q, k and v, a norm per head, half-paired rotation with
YaRN frequencies, capped scores and a window that also keeps the first tokens; "state_space"), and "lightning", linear
attention with a constant decay per head ("decayed_attention").  Feed-forwards are routed gated experts with sigmoid
scores, a correction for the choice and groups scored by their two best ("routed_moe" with its options); behind them
every layer adds an input of its own per token ("token_input").  Tensor names: `embed`, `side.embed`, `l<i>.norm1|norm2`,
`l<i>.mix.*` (`.left.*`, `.right.*`), `l<i>.mlp.e<j>.gate|up|down`, `l<i>.mlp.router|correction`,
`l<i>.side.gate|proj|norm`, `final.norm`, `head`.
"""
from __future__ import annotations

from ..config.mogutar import LightningConfig, MogutarConfig
from ..config.registry import register_architecture
from ..config.spec import LayerSpec, ModelSpec, PartSpec, PlanEntry


def _mixer_spec(cfg: MogutarConfig, m) -> PartSpec:
    if isinstance(m, LightningConfig):
        return PartSpec("decayed_attention", {"hidden_size": cfg.width, "num_heads": m.heads, "head_dim": m.dim,
                                              "value_dim": m.vdim, "decay": m.decay, "eps": cfg.norm_eps}, "mix")
    a, s = m.left, m.right
    position = {"kind": "none"}
    if a.rot_dims:
        position = {"kind": "rotary", "head_dim": a.dim, "rotary_dim": a.rot_dims, "theta": a.rot_base,
                    "max_position": cfg.max_position, "pairing": "half"}
        if a.yarn is not None:
            position["scaling"] = {"kind": "yarn", "factor": a.yarn.factor, "original": a.yarn.original,
                                   "fast": a.yarn.fast, "slow": a.yarn.slow}
    left = {"hidden_size": cfg.width, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim,
            "value_dim": a.vdim, "position": position, "window": a.window, "keep_first": a.keep_first, "scale": a.scale,
            "softcap": a.softcap, "bias": True, "out_bias": False, "conv_taps": a.conv, "qk_norm": "head",
            "eps": cfg.norm_eps}
    right = {"hidden_size": cfg.width, "num_heads": s.heads, "groups": s.groups, "state_dim": s.state, "value_dim": s.vdim,
             "conv_taps": s.conv, "norm_groups": s.norm_groups, "eps": cfg.norm_eps}
    return PartSpec("parallel", {"branches": (
        {"kind": "gated_attention", "name": "left", "scale": m.left_scale, "params": left},
        {"kind": "state_space", "name": "right", "scale": m.right_scale, "params": right})}, "mix")


def _mlp_spec(cfg: MogutarConfig, mlp) -> PartSpec:
    return PartSpec("routed_moe", {"hidden_size": cfg.width, "num_experts": mlp.experts, "top": mlp.top,
                                   "intermediate_size": mlp.ff, "groups": mlp.groups, "keep": mlp.keep,
                                   "activation": "swiglu", "score": "sigmoid", "correction": True, "group_score": "top2",
                                   "normalize": False}, "mlp")


def build_mogutar_spec(cfg: MogutarConfig) -> ModelSpec:
    norm = PartSpec("rmsnorm", {"hidden_size": cfg.width, "eps": cfg.norm_eps, "weight_name": ""})
    n = len(cfg.layers)
    layers, plan = [], []
    for i, layer in enumerate(cfg.layers):
        parts = {"mixer": _mixer_spec(cfg, layer.mixer), "mixer_norm": norm.named("norm1")}
        if layer.mlp is not None:
            parts.update(ffn=_mlp_spec(cfg, layer.mlp), ffn_norm=norm.named("norm2"))
        if cfg.side_dim:
            parts["side"] = PartSpec("token_input", {
                "hidden_size": cfg.width, "vocab_size": cfg.vocab, "dim": cfg.side_dim, "offset": i * cfg.side_dim,
                "table_width": n * cfg.side_dim, "table_name": "side.embed"}, "side")
            parts["side_norm"] = norm.named("side.norm")
        layers.append(LayerSpec(f"l{i}", "output_norm", parts))
        plan.append(PlanEntry(i))
    sizes = {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "weight_name": ""}
    return ModelSpec(
        architecture="Mogutar",
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        max_position=cfg.max_position,
        embedding=PartSpec("token_embedding", sizes, "embed"),
        layers=tuple(layers),
        plan=tuple(plan),
        final_norm=norm.named("final.norm"),
        lm_head=PartSpec("lm_head", sizes, "head"),
        eos_token_ids=cfg.eos_token_ids,
        # a layer without feed-forward has no use for a second norm, should a checkpoint carry one
        ignorable_tensors=tuple(f"l{i}.norm2" for i, layer in enumerate(cfg.layers) if layer.mlp is None),
    )


register_architecture("Mogutar", MogutarConfig.from_dict, build_mogutar_spec)
