"""The Mogutar architecture without a GPU: its configuration reader, the model as data (caches that keep the first
tokens, states of two branches side by side), and properties of the plain implementation (tests/plain_mogutar.py)
that the engine is compared with on the GPU."""
import copy
import math

import pytest
import torch

import plain_mogutar as plain
from mogutar_util import CONFIGS, MIX_A, MIX_B, ODD, every_expert, random_config, random_weights
from util import random_tokens


def _decoder(cfg, dtype="float32"):
    from tiny_llm_amd.config import resolve
    from tiny_llm_amd.models.decoder import Decoder
    typed, spec = resolve(cfg)
    return typed, spec, Decoder(spec, dtype=dtype, device="cpu")


def test_reader_takes_every_size_from_the_configuration():
    typed, spec, dec = _decoder(MIX_A)
    assert (typed.vocab, typed.width, typed.norm_eps, typed.side_dim) == (301, 64, 1e-5, 16)
    l0 = typed.layers[0].mixer
    assert (l0.heads, l0.dim, l0.vdim, len(l0.decay)) == (3, 24, 16, 3)
    p = typed.layers[1].mixer
    a, s = p.left, p.right
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.conv, a.window, a.keep_first, a.rot_dims, a.rot_base, a.softcap, a.scale) == \
        (4, 2, 24, 16, 3, 24, 5, 8, 1000.0, 9.0, 2.0 * 24 ** -0.5)
    assert (a.yarn.factor, a.yarn.original, a.yarn.fast, a.yarn.slow) == (4.0, 64, 32.0, 1.0)
    assert (s.heads, s.groups, s.state, s.vdim, s.conv, s.norm_groups) == (4, 2, 24, 16, 4, 2)
    assert (p.left_scale, p.right_scale) == (0.7, 1.2)
    m = typed.layers[0].mlp
    assert (m.experts, m.top, m.ff, m.groups, m.keep) == (8, 3, 24, 4, 2) and typed.layers[2].mlp is None
    tb = _decoder(MIX_B)[0]
    b = tb.layers[1].mixer.left
    assert (b.window, b.keep_first, b.rot_dims, b.softcap) == (0, 0, 0, 0.0) and tb.side_dim == 0
    assert tb.layers[1].mlp.groups == 1 and tb.layers[3].mlp is None
    assert spec.architecture == "Mogutar"
    left = dec.layers[1].mixer.branches[0]
    assert (left.window, left.keep, left.softcap, left.taps, left.qk_norm, left.out_scale) == (24, 5, 9.0, 3, "head", 0.7)
    assert dec.layers[1].mixer.branches[1].out_scale == 1.2
    assert [l.by_role["side"].offset for l in dec.layers] == [0, 16, 32, 48, 64]
    assert "side" not in _decoder(MIX_B)[2].layers[0].by_role


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_spec_names_the_checkpoints_tensors(name):
    cfg = CONFIGS[name][0]
    _, _, dec = _decoder(cfg)
    want = {k: tuple(v.shape) for k, v in random_weights(cfg).items()}
    got = {w.name: tuple(w.shape) for w in dec.weight_specs()}
    assert got == want


def test_caches_and_states():
    from tiny_llm_amd.cache import CacheManager
    _, spec, dec = _decoder(MIX_A)
    specs = dec.cache_specs()
    assert {i: (s.kind, s.window, s.keep) for (i, _), s in specs.items()} == \
        {1: ("window", 24, 5), 2: ("window", 7, 1), 4: ("window", 50, 20)}
    states = dec.state_specs()
    assert sorted(i for i, _ in states) == [0, 1, 2, 3, 4]
    # S of every head, no convolution
    assert states[(0, "mixer")].shape == (3 * 24 * 16,)
    # attention's last inputs of q, k and v, then S and the last inputs of x, B and C
    left = (4 * 24 + 2 * 24 + 2 * 16) * 2
    assert states[(1, "mixer")].shape == (left + 4 * 24 * 16 + (4 * 16 + 2 * 2 * 24) * 3,)
    st = torch.arange(2 * states[(1, "mixer")].shape[0], dtype=torch.float32).reshape(2, -1)
    mix = dec.layers[1].mixer
    own = [mix._state_of(b, st) for b in mix.branches]
    assert own[0].shape[1] == left and own[1][0, 0] == left and own[1].stride(0) == st.shape[1]
    cm = CacheManager(specs, states, 8, 20, 2)
    cm.allocate_tensors(torch.float32, "cpu")
    _, _, dec_b = _decoder(MIX_B)
    assert {i: (s.kind, s.window, s.keep) for (i, _), s in dec_b.cache_specs().items()} == \
        {0: ("window", 1, 0), 1: ("full", 0, 0), 3: ("window", 1000, 3)}
    # one tap keeps nothing of the past
    assert dec_b.layers[0].mixer.branches[0].state_spec() is None


def test_a_window_gives_pages_back_and_keeps_the_first_ones():
    from tiny_llm_amd.cache import CacheManager, manager
    from tiny_llm_amd.parts import CacheSpec
    for keep, block, window in ((5, 4, 10), (1, 16, 20), (33, 8, 3), (0, 4, 9), (8, 8, 8)):
        cs = CacheSpec.keys_and_values(1, 8, "window", window)
        cs = CacheSpec(cs.tensors, cs.kind, cs.window, keep)
        n_tokens = 150
        most = manager.blocks_held_at_most(cs, block, n_tokens, 7)
        cm = CacheManager([cs], [], block, most, 1)
        at = 0
        for n in [7, 1, 2, 7] + [1] * 100 + [5, 7, 7, 7, 7]:
            cm.reserve_step([("a", n)])
            at += n
            cm.commit("a", at)
            cm.audit()
            table = cm.block_table("a", 0)
            for pos in range(at):        # whatever the next token may see is still held
                if pos < keep or at - pos < window:
                    assert table[pos // block] != manager.RELEASED, (keep, block, window, at, pos)
        held = sum(b != manager.RELEASED for b in cm.block_table("a", 0))
        assert held <= -(-keep // block) + (window + block - 2) // block + 1
        cm.free_request("a")
        cm.audit()
        assert cm.free_blocks() == [most]


def test_refusals():
    from tiny_llm_amd.config import ConfigError, resolve

    def broken(change, base=MIX_A):
        cfg = copy.deepcopy(base)
        change(cfg)
        with pytest.raises(ConfigError):
            resolve(cfg)

    broken(lambda c: c["layers"][0].update(type="something_else"))
    broken(lambda c: c["layers"][0]["mixer"].update(decay=[0.5]))                   # one decay a head
    broken(lambda c: c["layers"][1]["mixer"]["left"].pop("scale"))
    broken(lambda c: c["layers"][1]["mixer"]["left"].pop("conv"))
    broken(lambda c: c["layers"][1]["mixer"]["left"].update(heads=3))               # no multiple of kv_heads
    broken(lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].pop("slow"))
    broken(lambda c: c["layers"][1]["mixer"]["left"]["mask"].pop("size"))           # kept tokens without a window
    broken(lambda c: c["layers"][1]["mixer"]["right"].update(groups=3))             # no divisor of heads
    broken(lambda c: c["layers"][1]["mixer"]["right"].update(norm_groups=7))
    broken(lambda c: c["layers"][1]["mixer"].pop("right"))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=5))                 # more than two groups of two hold
    broken(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=3))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    broken(lambda c: c.pop("norm"))
    with pytest.raises(ConfigError):
        resolve(copy.deepcopy(MIX_A), {"side.embed": (301, 64)})                    # 16 numbers for each of five layers


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


# ------------------------------------------------------------------ the plain implementation
def test_window_with_kept_tokens():
    pos = torch.arange(10)
    m = plain.window_with_first(pos, 3, 2)
    assert m[7].tolist() == [True, True] + [False] * 3 + [True, True, True] + [False] * 2
    assert m[1].tolist() == [True, True] + [False] * 8
    assert m[3].tolist() == [True] * 4 + [False] * 6                               # window and kept tokens meet
    assert plain.window_with_first(pos, 1, 0)[5].tolist() == [False] * 5 + [True] + [False] * 4


def test_softcap_and_convolution():
    s = torch.tensor([-100.0, -1.0, 0.0, 0.01, 5.0, 1e4], dtype=torch.float64)
    c = plain.softcap(s, 7.0)
    assert (c.abs() <= 7.0).all() and abs(float(c[3]) - 0.01) < 1e-6 and abs(float(c[5]) - 7.0) < 1e-9
    x = torch.arange(1.0, 6.0, dtype=torch.float64).reshape(5, 1)
    taps = torch.tensor([[0.5, -1.0, 2.0]], dtype=torch.float64)                   # the last column is the current token's
    y = plain.causal_conv(x, taps, torch.tensor([10.0], dtype=torch.float64))
    assert y[:, 0].tolist() == [12.0, 13.0, 14.5, 10 + 8 - 3 + 1.0, 10 + 10 - 4 + 1.5]


def test_yarn_keeps_fast_frequencies_and_divides_slow_ones():
    dims, base = 32, 10000.0
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    g, mag = plain.yarn(f, dims, base, 8.0, 256.0, 16.0, 1.0)
    assert abs(mag - (0.1 * math.log(8.0) + 1.0)) < 1e-12
    assert g[0] == f[0] and abs(g[-1] - f[-1] / 8.0) < 1e-15
    ratio = [b / a for a, b in zip(f, g)]
    assert all(x >= y - 1e-12 for x, y in zip(ratio, ratio[1:])) and any(0.13 < r < 0.99 for r in ratio)
    x = torch.arange(1.0, 9.0, dtype=torch.float64).reshape(1, 1, 8)
    spec = {"dims": 4, "base": 100.0, "scaling": {"factor": 4.0, "original": 16, "fast": 2.0, "slow": 1.0}}
    g, mag = plain.yarn([1.0, 0.1], 4, 100.0, 4.0, 16, 2.0, 1.0)
    y = plain.rotate(x, torch.tensor([3]), spec)
    for i in range(2):
        a = 3 * g[i]
        assert abs(float(y[0, 0, i]) - mag * (x[0, 0, i] * math.cos(a) - x[0, 0, i + 2] * math.sin(a))) < 1e-12
        assert abs(float(y[0, 0, i + 2]) - mag * (x[0, 0, i + 2] * math.cos(a) + x[0, 0, i] * math.sin(a))) < 1e-12
    assert torch.equal(y[..., 4:], x[..., 4:])
    # position 0 is not rotated, but it is scaled
    assert torch.allclose(plain.rotate(x, torch.tensor([0]), spec)[..., :4], mag * x[..., :4])


def test_router_choice():
    s = torch.tensor([0.9, 0.1, 0.5, 0.5, 0.8, 0.05], dtype=torch.float64)
    none = torch.zeros(6, dtype=torch.float64)
    assert plain.choose(s, none, 2, 1, 1) == [0, 4]
    # groups {0,1} = 1.0, {2,3} = 1.0, {4,5} = 0.85: the sum of two decides, not the largest
    assert plain.choose(s + torch.tensor([0, 0, 0.01, 0, 0, 0]), none, 2, 3, 1) == [2, 3]
    # negative choice scores: an expert of a group that is out is not chosen although 0 would be larger
    c = torch.full((6,), -3.0, dtype=torch.float64)
    c[4:] = -9.0
    assert plain.choose(s, c, 4, 3, 2) == [0, 2, 3, 1]
    # the correction decides the choice, the weights are the scores themselves
    h = torch.eye(2, dtype=torch.float64)
    w = {"router": torch.tensor([[1.0, 0.0], [0.0, 1.0]], dtype=torch.float64), "correction": torch.tensor([5.0, 0.0], dtype=torch.float64)}
    for e in range(2):
        w[f"e{e}.gate"], w[f"e{e}.up"] = torch.ones(1, 2, dtype=torch.float64), torch.ones(1, 2, dtype=torch.float64)
        w[f"e{e}.down"] = torch.tensor([[1.0], [10.0]], dtype=torch.float64) * (e + 1)
    y = plain.moe(h, w, {"router": {"experts": 2, "top": 1}})
    sig = lambda z: 1.0 / (1.0 + math.exp(-z))
    assert abs(float(y[1, 0]) - 0.5 * sig(1.0)) < 1e-12 and abs(float(y[0, 0]) - sig(1.0) * sig(1.0)) < 1e-12


def test_decayed_scan_against_its_closed_form():
    """o_t = sum over s <= t of (prod of a over s+1..t) (q_t . k_s) v_s."""
    g = torch.Generator().manual_seed(1)
    T, H, N, V = 7, 2, 3, 4
    a, q, k, v = torch.rand(T, H, generator=g), *(torch.randn(T, H, n, generator=g) for n in (N, N, V))
    a, q, k, v = (x.double() for x in (a, q, k, v))
    o = plain.decayed_scan(a, q, k, v)
    for t in range(T):
        want = torch.zeros(H, V, dtype=torch.float64)
        for s in range(t + 1):
            want += (a[s + 1:t + 1].prod(dim=0) * (q[t] * k[s]).sum(-1))[:, None] * v[s]
        assert torch.allclose(o[t], want)


def test_every_sublayer_reaches_the_logits():
    """Each tensor of a checkpoint moves the logits of a sequence (the correction by changing a choice)."""
    cfg = MIX_A
    w = {k: v.double() for k, v in random_weights(cfg, 2).items()}
    toks = random_tokens(12, cfg["vocab"], 1)
    base = plain.forward(cfg, w, toks)
    for name in w:
        if ".mlp.e" in name or name in ("embed", "side.embed", "head"):
            continue
        w2 = dict(w)
        w2[name] = w[name].clone()
        w2[name] += 0.5 * torch.randn(w[name].shape, generator=torch.Generator().manual_seed(3), dtype=torch.float64)
        assert not torch.allclose(plain.forward(cfg, w2, toks), base), name
    trace = []
    plain.forward(cfg, w, toks, trace=trace)
    assert len(trace) == len(cfg["layers"])


def test_what_a_window_leaves_reaches_later_logits_only_if_it_is_kept():
    """Attention alone (the state-space branch scaled to nothing) in a window of 20 that keeps 3 tokens, under a
    convolution of 3 taps: token 10 is gone at position 40, token 1 is not."""
    cfg = copy.deepcopy(CONFIGS["parallel"][0])
    cfg["layers"][0]["mixer"]["right_scale"] = 0.0
    w = {k: v.double() for k, v in random_weights(cfg, 4).items()}
    toks = random_tokens(60, cfg["vocab"], 3)
    out = plain.forward(cfg, w, toks)
    for at, reaches in ((10, False), (1, True)):
        other = list(toks)
        other[at] = (toks[at] + 1) % cfg["vocab"]
        assert torch.equal(plain.forward(cfg, w, other)[40:], out[40:]) != reaches
    # a kept token's key also holds the two tokens in front of it, a later key those in front of it
    other = list(toks)
    other[3] = (toks[3] + 1) % cfg["vocab"]
    assert torch.equal(plain.forward(cfg, w, other)[40:], out[40:])


def test_every_expert_variant():
    cfg = every_expert(MIX_A)
    assert [l["mlp"]["router"]["top"] for l in cfg["layers"] if l["mlp"]] == [8, 6, 9, 5]
    w = {k: v.double() for k, v in random_weights(ODD, 1).items()}
    logits = plain.forward(ODD, w, random_tokens(20, ODD["vocab"], 0))
    assert logits.shape == (20, ODD["vocab"]) and torch.isfinite(logits).all()
