"""The Nililix architecture as data: NililixConfig -> ModelSpec.

A decoder with an RMS norm in front of AND behind every sublayer, the normed result added times a constant ("sandwich"
blocks); one mixer, grouped-query attention in a sliding window with a short convolution on q, k and v, interleaved
rotation of part of the head with the frequency scaling of Llama 3.1, a learned sink per head in the softmax and a sigmoid
gate per head ("gated_attention" with its options); feed-forwards that are dense with a squared relu ("act_mlp") or
routed gated experts with sigmoid scores, a correction for the choice and groups scored by their two best ("routed_moe"
with its options); a run of layers that is repeated with the same weights, each pass with caches and states of its own and
a vector added ahead of it ("loop_step"); an output head of its own with capped logits.  Tensor names: `embed`,
`loop.step`, `l<i>.norm1|norm1b|norm2|norm2b`, `l<i>.mix.q|k|v` (+ `.conv`), `l<i>.mix.sink|g|o`, `l<i>.mlp.up|down`,
`l<i>.mlp.e<j>.gate|up|down`, `l<i>.mlp.router|correction`, `final.norm`, `head`.
"""
from __future__ import annotations

from ..config.nililix import DenseConfig, NililixConfig, SinkAttentionConfig
from ..config.registry import register_architecture
from ..config.spec import LayerSpec, ModelSpec, PartSpec, PlanEntry


def _mixer_spec(cfg: NililixConfig, m: SinkAttentionConfig) -> PartSpec:
    position = {"kind": "none"}
    if m.rot_dims:
        position = {"kind": "rotary", "head_dim": m.dim, "rotary_dim": m.rot_dims, "theta": m.rot_base,
                    "max_position": cfg.max_position, "pairing": "interleaved"}
        if m.scaling is not None:
            position["scaling"] = {"kind": "llama3", "factor": m.scaling.factor, "low": m.scaling.low,
                                   "high": m.scaling.high, "original": m.scaling.original}
    return PartSpec("gated_attention", {
        "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim,
        "position": position, "window": m.window, "scale": m.scale, "conv_taps": m.conv, "learned_sink": True,
        "gate": "head", "eps": cfg.norm_eps}, "mix")


def _mlp_spec(cfg: NililixConfig, mlp) -> PartSpec:
    if isinstance(mlp, DenseConfig):
        return PartSpec("act_mlp", {"hidden_size": cfg.width, "intermediate_size": mlp.ff, "activation": "relu2"}, "mlp")
    return PartSpec("routed_moe", {"hidden_size": cfg.width, "num_experts": mlp.experts, "top": mlp.top,
                                   "intermediate_size": mlp.ff, "groups": mlp.groups, "keep": mlp.keep,
                                   "activation": "swiglu", "score": "sigmoid", "correction": True, "group_score": "top2",
                                   "normalize": False}, "mlp")


def build_nililix_spec(cfg: NililixConfig) -> ModelSpec:
    norm = PartSpec("rmsnorm", {"hidden_size": cfg.width, "eps": cfg.norm_eps, "weight_name": ""})
    layers = []
    for i, layer in enumerate(cfg.layers):
        parts = {"mixer_norm": norm.named("norm1"), "mixer": _mixer_spec(cfg, layer.mixer),
                 "mixer_out_norm": norm.named("norm1b")}
        if layer.mlp is not None:
            parts.update(ffn_norm=norm.named("norm2"), ffn=_mlp_spec(cfg, layer.mlp), ffn_out_norm=norm.named("norm2b"))
        layers.append(LayerSpec(f"l{i}", "sandwich", parts, {"mult": cfg.residual_mult}))
    plan = tuple(PlanEntry(i, before=None if turn is None else (0, turn)) for i, turn in cfg.run_order())
    stream_parts = ()
    if cfg.loop is not None:
        stream_parts = (PartSpec("loop_step", {"hidden_size": cfg.width, "times": cfg.loop.times}, "loop"),)
    sizes = {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "weight_name": ""}
    ignorable = []
    for i, layer in enumerate(cfg.layers):       # norms a checkpoint may carry for a layer without feed-forward
        if layer.mlp is None:
            ignorable += [f"l{i}.norm2", f"l{i}.norm2b"]
    return ModelSpec(
        architecture="Nililix",
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        max_position=cfg.max_position,
        embedding=PartSpec("token_embedding", sizes, "embed"),
        layers=tuple(layers),
        plan=plan,
        final_norm=norm.named("final.norm"),
        lm_head=PartSpec("lm_head", dict(sizes, softcap=cfg.logit_softcap), "head"),
        eos_token_ids=cfg.eos_token_ids,
        ignorable_tensors=tuple(ignorable),
        stream_parts=stream_parts,
    )


register_architecture("Nililix", NililixConfig.from_dict, build_nililix_spec)
