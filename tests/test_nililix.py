"""The Nililix architecture without a GPU: its configuration reader, the model as data (the plan of a repeated run of
layers, caches and states of every pass), the frequency tables, and properties of the plain implementation
(tests/plain_nililix.py) that the engine is compared with on the GPU."""
import copy
import math

import pytest
import torch

import plain_nililix as plain
from nililix_util import (CONFIGS, LOOP_END, LOOP_ONCE, MIX_A, MIX_B, ODD, PLAIN, as_double, every_expert, random_config,
                          random_weights)
from util import random_tokens


def _decoder(cfg, dtype="float32"):
    from tiny_llm_amd.config import resolve
    from tiny_llm_amd.models.decoder import Decoder
    typed, spec = resolve(cfg)
    return typed, spec, Decoder(spec, dtype=dtype, device="cpu")


def test_reader_takes_every_size_from_the_configuration():
    typed, spec, dec = _decoder(MIX_A)
    assert (typed.vocab, typed.width, typed.norm_eps, typed.residual_mult, typed.logit_softcap) == (301, 64, 1e-5, 0.7, 9.0)
    a = typed.layers[0].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.conv, a.window, a.scale) == (4, 2, 24, 16, 3, 24, 1.6 * 24 ** -0.5)
    assert (a.rot_dims, a.rot_base) == (8, 1000.0)
    assert (a.scaling.factor, a.scaling.low, a.scaling.high, a.scaling.original) == (4.0, 1.0, 4.0, 64)
    assert typed.layers[1].mixer.scaling is None and typed.layers[1].mixer.rot_dims == 16
    assert typed.layers[0].mlp.ff == 40 and typed.layers[2].mlp is None
    m = typed.layers[1].mlp
    assert (m.experts, m.top, m.ff, m.groups, m.keep) == (8, 3, 24, 4, 2)
    assert (typed.loop.start, typed.loop.stop, typed.loop.times) == (1, 4, 3)
    part = dec.layers[0].mixer
    assert (part.window, part.taps, part.qk_dim, part.value_dim, part.position.pairing) == (24, 3, 24, 16, "interleaved")
    assert part.learned_sink and part.gate == "head" and part.qk_norm is None and not part.bias
    assert dec.layers[0].block.mult == 0.7 and dec.lm_head.softcap == 9.0
    tb, spec_b, dec_b = _decoder(MIX_B)
    assert tb.logit_softcap == 0 and tb.layers[0].mixer.window == 0 and tb.layers[1].mixer.rot_dims == 0
    assert dec_b.layers[1].mixer.position.rotary_tables() is None and dec_b.layers[0].mixer.state_spec() is None    # one tap
    assert spec.architecture == spec_b.architecture == "Nililix"


def test_plan_of_a_repeated_run():
    _, spec, dec = _decoder(MIX_A)
    assert [e.layer for e in spec.plan] == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4]
    assert [e.before for e in spec.plan] == [None, (0, 0), None, None, (0, 1), None, None, (0, 2), None, None, None]
    assert all(e.cache_of is None for e in spec.plan)
    assert [p.kind for p in spec.stream_parts] == ["loop_step"] and not dec.stream_parts[0].reads_origin
    for cfg in (MIX_A, MIX_B, LOOP_END, LOOP_ONCE, PLAIN):
        _, s, _ = _decoder(cfg)
        assert [(e.layer, None if e.before is None else e.before[1]) for e in s.plan] == plain.runs(cfg)
    assert plain.runs(LOOP_END) == [(0, None), (1, 0), (1, 1), (1, 2), (1, 3)]
    assert plain.runs(LOOP_ONCE) == [(0, 0), (1, None)]
    assert _decoder(PLAIN)[1].stream_parts == ()


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_spec_names_the_checkpoints_tensors(name):
    cfg = CONFIGS[name][0]
    _, _, dec = _decoder(cfg)
    assert {w.name: tuple(w.shape) for w in dec.weight_specs()} == {k: tuple(v.shape) for k, v in random_weights(cfg).items()}


def test_caches_and_states_of_every_pass():
    from tiny_llm_amd.cache import CacheManager
    _, spec, dec = _decoder(MIX_A)
    specs = dec.cache_specs()
    assert [specs[(i, "mixer")].window for i in range(11)] == [24, 7, 50, 1, 7, 50, 1, 7, 50, 1, 33]
    assert all(s.kind == "window" and s.keep == 0 for s in specs.values())
    # heads of 24 keys and 16 values lie in rows of 32; 16 and 40 in rows of 48; 8 and 8 in rows of 16
    assert [specs[(i, "mixer")].tensors[0].shape for i in (0, 1, 10)] == [(2, 32), (3, 48), (1, 16)]
    states = dec.state_specs()
    assert len(states) == 11
    channels = 4 * 24 + 2 * 24 + 2 * 16
    assert states[(0, "mixer")].shape == (channels * 2,)                 # the last two inputs of q, k and v
    cm = CacheManager(specs, states, 8, 20, 2)
    cm.allocate_tensors(torch.float32, "cpu")
    assert len({cm.states[k].data_ptr() for k in states}) == 11          # a state of its own per run
    _, _, dec_b = _decoder(MIX_B)
    assert {s.kind for s in dec_b.cache_specs().values()} == {"full", "window"}


def test_refusals():
    from tiny_llm_amd.config import ConfigError, resolve

    def broken(change, base=MIX_A):
        cfg = copy.deepcopy(base)
        change(cfg)
        with pytest.raises(ConfigError):
            resolve(cfg)

    broken(lambda c: c["layers"][0].update(type="something_else"))
    broken(lambda c: c["layers"][0]["mixer"].pop("scale"))
    broken(lambda c: c["layers"][0]["mixer"].update(heads=3))                    # no multiple of kv_heads
    broken(lambda c: c["layers"][0]["mixer"].update(conv=-1))
    broken(lambda c: c["layers"][0]["mixer"]["mask"].update(size=-4))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26))             # more than dim
    broken(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("low"))
    broken(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(low=5.0))  # above high
    broken(lambda c: c["layers"][0]["mlp"].update(kind="gated"))
    broken(lambda c: c["layers"][0]["mlp"].pop("ff"))
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=5))              # more than two groups of two hold
    broken(lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=3))
    broken(lambda c: c["loop"].update(stop=6))                                   # beyond the layers
    broken(lambda c: c["loop"].update(start=4))                                  # an empty run
    broken(lambda c: c["loop"].update(times=0))
    broken(lambda c: c.pop("norm"))
    broken(lambda c: c.update(logit_softcap=-1.0))
    with pytest.raises(ConfigError):
        resolve(copy.deepcopy(MIX_A), {"loop.step": (2, 64)})                    # a vector per pass


def test_sizes_the_bfloat16_kernels_refuse_are_served_in_float32():
    from tiny_llm_amd.engine.loading import build_decoder
    with pytest.warns(RuntimeWarning, match="served in float32"):
        _, dec = build_decoder(ODD, "bfloat16", "cpu")
    assert dec.dtype == torch.float32
    import warnings
    with warnings.catch_warnings():
        warnings.simplefilter("error")
        assert build_decoder(MIX_A, "bfloat16", "cpu")[1].dtype == torch.bfloat16


def test_configurations_drawn_at_random_build():
    for seed in range(30):
        cfg = random_config(seed)
        _, _, dec = _decoder(cfg, "bfloat16")
        assert {w.name for w in dec.weight_specs()} == set(random_weights(cfg))


def test_angle_tables_with_the_frequency_scaling():
    """The engine's tables against the plain frequencies: fast ones untouched, slow ones divided, the ones between mixed
    (a spec whose range holds all three, one without a middle, one that divides everything)."""
    from tiny_llm_amd.parts.rotary import angle_tables
    for dims, base, (factor, low, high, original) in ((16, 10000.0, (8.0, 1.0, 4.0, 256)), (8, 100.0, (3.0, 2.0, 2.0, 40)),
                                                      (12, 50.0, (4.0, 1.0, 4.0, 2)), (64, 500000.0, (32.0, 1.0, 4.0, 8192))):
        s = {"factor": factor, "low": low, "high": high, "original": original}
        freqs = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
        want = torch.tensor([plain.stretched(f, s) for f in freqs], dtype=torch.float64)
        cos, sin = angle_tables(dims, base, 300, "cpu", llama3=(factor, original, low, high))
        for p in (0, 1, 77, 299):
            assert (cos[p].double() - torch.cos(p * want)).abs().max() < 1e-7 * (1 + p)
            assert (sin[p].double() - torch.sin(p * want)).abs().max() < 1e-7 * (1 + p)
    kinds = {("same" if w == f else "slow" if abs(w - f / 8.0) < 1e-18 else "mixed")
             for f in [10000.0 ** (-2.0 * i / 16) for i in range(8)]
             for w in [plain.stretched(f, {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 256})]}
    assert kinds == {"same", "slow", "mixed"}
    # at either border the mixture is what lies beyond it
    s = {"factor": 5.0, "low": 1.0, "high": 4.0, "original": 100}
    for turns, want in ((4.0, 1.0), (1.0, 1.0 / 5.0)):
        f = turns * 2.0 * math.pi / 100
        assert abs(plain.stretched(f * (1 + 1e-12), s) / f - want) < 1e-9
        assert abs(plain.stretched(f * (1 - 1e-12), s) / f - want) < 1e-9


def test_rotary_part_refuses_a_scaling_it_does_not_know():
    from tiny_llm_amd.parts.rotary import RotaryEmbedding
    kw = dict(head_dim=16, theta=100.0, max_position=8)
    with pytest.raises(ValueError):
        RotaryEmbedding("r", torch.float32, "cpu", scaling={"kind": "llama4", "factor": 2.0}, **kw)
    with pytest.raises(ValueError):
        RotaryEmbedding("r", torch.float32, "cpu", scaling={"kind": "llama3", "factor": 2.0, "low": 3.0, "high": 2.0, "original": 8}, **kw)


# ------------------------------------------------------------------ the plain implementation
def test_rms_norm():
    x, w = torch.tensor([[1.0, 2.0, 3.0, 6.0]], dtype=torch.float64), torch.tensor([1.0, 2.0, 1.0, 0.5], dtype=torch.float64)
    assert torch.allclose(plain.rms_norm(x, w, 0.25), x / math.sqrt(12.5 + 0.25) * w)


def test_convolution_reaches_back_into_zeros():
    u = torch.tensor([[1.0], [10.0], [100.0]], dtype=torch.float64)
    y = plain.causal_conv(u, torch.tensor([[3.0, 2.0, 1.0]], dtype=torch.float64))
    assert y[:, 0].tolist() == [1.0, 12.0, 123.0]


def test_rotation_pairs_neighbours_and_leaves_the_rest():
    x = torch.tensor([[[1.0, 0.0, 0.0, 2.0, 5.0]]], dtype=torch.float64)
    y = plain.rotate_pairs(x, torch.tensor([3]), {"dims": 4, "base": 100.0})[0, 0]
    assert torch.allclose(y, torch.tensor([math.cos(3), math.sin(3), -2 * math.sin(0.3), 2 * math.cos(0.3), 5.0], dtype=torch.float64))


def test_window_and_sink():
    ok = plain.window_mask(torch.arange(6), 3)
    assert ok[4].tolist() == [False, False, True, True, True, False]
    assert plain.window_mask(torch.arange(4), 0)[3].all()
    q = k = torch.zeros((2, 1, 4), dtype=torch.float64)
    v = torch.ones((2, 1, 1), dtype=torch.float64)
    out = plain.attend(q, k, v, plain.window_mask(torch.arange(2), 0), 1.0, torch.tensor([math.log(2.0)], dtype=torch.float64))
    assert torch.allclose(out[:, 0, 0], torch.tensor([1 / 3, 2 / 4], dtype=torch.float64))    # keys of score 0 beside a 2


def test_router_choice():
    s = torch.tensor([0.9, 0.1, 0.6, 0.6, 0.2, 0.8], dtype=torch.float64)
    none = torch.zeros(6, dtype=torch.float64)
    assert plain.choose(s, none, 2, 1, 1) == [0, 5]
    assert plain.choose(s, none, 2, 3, 1) == [2, 3]                 # 0.6 + 0.6 is the best pair
    low = torch.tensor([-3.0, -3.0, -1.0, -2.0, -2.5, -0.5], dtype=torch.float64)
    assert plain.choose(s, low, 2, 1, 1) == [5, 2]                  # the correction decides, negative scores and all
    assert plain.choose(s, low, 3, 3, 2) == [5, 2, 3]               # a shut group ranks below every negative score


def test_every_sublayer_and_every_pass_reach_the_logits():
    w = as_double(random_weights(MIX_A, 3))
    toks = random_tokens(30, MIX_A["vocab"], 5)
    base = plain.forward(MIX_A, w, toks)
    names = ["loop.step", "l0.mix.sink", "l1.mix.q.conv", "l2.mix.k.conv", "l4.mix.v.conv", "l1.mix.g", "l1.mlp.correction",
             "l3.mlp.e0.down", "l0.mlp.up", "l2.norm1b", "l4.norm2b", "final.norm", "head"]
    for n in names:
        changed = dict(w)
        changed[n] = w[n] * 1.5 + 0.3
        assert (plain.forward(MIX_A, changed, toks)[-1] - base[-1]).abs().max() > 1e-4, n
    for t in range(3):
        changed = dict(w)
        changed["loop.step"] = w["loop.step"].clone()
        changed["loop.step"][t] += 0.2
        assert (plain.forward(MIX_A, changed, toks)[-1] - base[-1]).abs().max() > 1e-4
    assert base.abs().max() < 9.0 and plain.forward(dict(MIX_A, logit_softcap=None), w, toks).abs().max() > 9.0


def test_what_a_window_leaves_does_not_reach_a_single_layer():
    cfg = copy.deepcopy(PLAIN)          # a window of 20, three taps
    w = as_double(random_weights(cfg, 3))
    toks = random_tokens(40, cfg["vocab"], 6)
    base = plain.forward(cfg, w, toks)[-1]
    for pos, reaches in ((39 - 19, True), (39 - 20, True), (39 - 21, True), (39 - 22, False), (0, False)):
        other = list(toks)
        other[pos] = (other[pos] + 1) % cfg["vocab"]
        moved = (plain.forward(cfg, w, other)[-1] - base).abs().max()
        # keys of the window's first places still hold the two tokens ahead of them (the convolution)
        assert (moved > 1e-6) if reaches else (moved == 0), pos


def test_every_expert_variant():
    cfg = every_expert(MIX_A)
    assert cfg["layers"][1]["mlp"]["router"] == {"experts": 8, "top": 8} and MIX_A["layers"][1]["mlp"]["router"]["top"] == 3
    assert cfg["layers"][0] == MIX_A["layers"][0]
