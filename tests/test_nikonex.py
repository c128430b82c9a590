"""The Nikonex design without a GPU: its configuration reader and what it refuses, the tensors it declares, the
random-weights mode, the cache layout, rotation frequencies that follow a ramp, and properties of the plain
implementation's mechanisms."""

from __future__ import annotations

import copy
import math

import pytest
import torch

import nikonex_util as nu
import plain_nikonex as plain
from paged_llm_rs_amd.config import load_config
from paged_llm_rs_amd.config.specs import LatentAttentionSpec, RetentionSpec, RoutedExpertsSpec
from paged_llm_rs_amd.errors import ConfigError, UnsupportedError
from paged_llm_rs_amd.parts.model import declare_parameters

F = torch.float64


def test_the_reader_takes_every_size_and_constant_from_the_config():
    spec = load_config(copy.deepcopy(nu.ODD)).model_spec()
    assert spec.hidden_size == 72 and spec.vocab_size == 211 and spec.max_positions == 0 and not spec.tie_word_embeddings
    assert [e.layer for e in spec.schedule] == [0, 1, 2, 3, 4, 5]
    assert all(layer.block == "parallel" and layer.residual_mult == 0.7 and not layer.layer_scale for layer in spec.layers)
    kept, small = spec.layers[0].mixer, spec.layers[1].mixer
    assert isinstance(kept, RetentionSpec) and isinstance(small, LatentAttentionSpec)
    assert (kept.num_heads, kept.head_dim, kept.value_dim, kept.decay) == (3, 24, 40, (0.4, 0.93, 0.9995))
    assert (kept.rotary_dims, kept.rotary_base, kept.key_scale, kept.eps) == (24, 500.0, None, 1e-5)
    assert spec.layers[2].mixer.rotary_dims == 12 and spec.layers[2].feed_forward is None
    assert (small.num_heads, small.head_dim, small.rotary_dim, small.value_dim, small.q_rank, small.kv_rank) == (5, 24, 8, 40, 44, 28)
    assert (small.scale, small.window, small.rotary_turned, small.rotary_base, small.norm_eps) == (0.25, 9, 8, 300.0, 1e-5)
    assert small.rotary_ramp == (4.0, 64.0, 6.0, 1.0) and small.rotary_scaling is None and small.max_positions == 0
    assert small.sink is None and not small.gated and spec.layers[4].mixer.window is None and spec.layers[3].mixer.rotary_ramp is None
    experts = spec.layers[1].feed_forward
    assert isinstance(experts, RoutedExpertsSpec)
    assert (experts.experts, experts.top, experts.intermediate_size, experts.shared_size) == (9, 4, 32, 20)
    assert (experts.groups, experts.groups_kept, experts.group_best, experts.weight_scale) == (3, 2, 2, 2.5)
    assert experts.score == "sigmoid" and experts.activation == "relu2" and not experts.gated and not experts.corrected and experts.normalised
    assert experts.identity == 0 and experts.weight_eps == 1e-20
    lone = spec.layers[3].feed_forward
    assert (lone.groups, lone.groups_kept, lone.shared_size, lone.weight_scale) == (1, 1, 0, 1.0)
    bare = copy.deepcopy(nu.ODD)
    bare["layers"][3]["mlp"]["router"].pop("scale")
    bare["layers"][3]["mixer"].pop("rot")
    again = load_config(bare).model_spec().layers[3]
    assert again.feed_forward.weight_scale == 1.0 and again.mixer.rotary_turned == 0


@pytest.mark.parametrize("damage, error", [
    (lambda c: c["layers"][1]["mixer"].pop("q_rank"), ConfigError),
    (lambda c: c["layers"][1]["mixer"].update(extra=1), UnsupportedError),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), ConfigError),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=2), UnsupportedError),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10), ConfigError),       # more than the rotated part
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7), ConfigError),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("slow"), ConfigError),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0), ConfigError),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(low=1.0), UnsupportedError),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(base=1.0), ConfigError),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5, 0.5]), ConfigError),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5, 0.5, 1.5]), ConfigError),
    (lambda c: c["layers"][0]["mixer"].update(decay=0.5), ConfigError),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26), ConfigError),
    (lambda c: c["layers"][0].update(type="mamba2"), UnsupportedError),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), UnsupportedError),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=4), ConfigError),        # more than the kept groups hold
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), ConfigError),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=3), ConfigError),
    (lambda c: c["layers"][0]["mlp"]["router"].update(bias=True), UnsupportedError),
    (lambda c: c["layers"][0]["mlp"]["shared"].update(ff=0), ConfigError),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=7.0), UnsupportedError),
    (lambda c: c.pop("residual_mult"), ConfigError),
    (lambda c: c.update(residual_mult="half"), ConfigError),
    (lambda c: c["norm"].update(eps=-1.0), ConfigError),
])
def test_what_the_reader_refuses(damage, error):
    config = copy.deepcopy(nu.ODD)
    damage(config)
    with pytest.raises(error):
        load_config(config)


def test_declared_tensors():
    found = declare_parameters(load_config(copy.deepcopy(nu.ODD)).model_spec())
    decls = {d.name: tuple(d.shape) for d in found}
    optional = {d.name for d in found if d.optional}
    assert decls["embed"] == (211, 72) and decls["final.norm"] == (72,) and decls["head"] == (211, 72)
    assert decls["l0.mix.q"] == decls["l0.mix.k"] == (72, 72) and decls["l0.mix.v"] == decls["l0.mix.g"] == (120, 72)
    assert decls["l0.mix.o"] == (72, 120) and "l0.mix.norm" not in decls, "a head's read-out is normed without a gain"
    assert decls["l1.mix.dq"] == (44, 72) and decls["l1.mix.dq.norm"] == (44,) and decls["l1.mix.uq"] == (5 * 32, 44)
    assert "l1.mix.q" not in decls and "l1.mix.g" not in decls and "l1.mix.sink" not in decls
    assert decls["l1.mix.dkv"] == (36, 72) and decls["l1.mix.dkv.norm"] == (28,)
    assert decls["l1.mix.uk"] == (120, 28) and decls["l1.mix.uv"] == (200, 28) and decls["l1.mix.o"] == (72, 200)
    assert decls["l1.mlp.e8.up"] == (32, 72) and decls["l1.mlp.e8.down"] == (72, 32) and "l1.mlp.e9.up" not in decls
    assert "l1.mlp.e0.gate" not in decls and "l1.mlp.shared.gate" not in decls
    assert decls["l1.mlp.router"] == (9, 72) and decls["l1.mlp.shared.up"] == (20, 72) and decls["l1.mlp.shared.down"] == (72, 20)
    assert decls["l1.mlp.shared.sg"] == (1, 72) and not any(n.startswith("l3.mlp.shared") for n in decls)
    assert not any(n.startswith("l2.mlp") for n in decls) and "l2.norm2" in optional and "l1.norm2" not in optional
    assert not any(".ls" in n for n in decls)


def test_the_random_weights_mode_and_the_plain_implementation(tmp_path):
    folder = nu.write_model(tmp_path / "m", nu.ODD, seed=3)
    config, weights = nu.load_plain(folder)
    assert set(weights) == {d.name for d in declare_parameters(load_config(config).model_spec())}
    tokens = [5, 17, 3, 200, 0, 44, 9, 9, 120]
    streams = []
    logits = plain.forward(config, weights, tokens, streams)
    assert logits.shape == (9, 211) and len(streams) == 6 and torch.isfinite(logits).all()
    # causal: a prefix gives the same logits
    assert torch.allclose(plain.forward(config, weights, tokens[:5]), logits[:5], atol=1e-12)
    halved = dict(config, residual_mult=config["residual_mult"] / 2)
    assert not torch.allclose(plain.forward(halved, weights, tokens), logits)


def test_the_cache_of_the_design():
    """The latent layers keep one row a token in pages, by window; the retention layers a run of floats a request."""
    from paged_llm_rs_amd.cache.layout import KVCacheSpec
    from paged_llm_rs_amd.parts.latent_attention import LatentAttention
    from paged_llm_rs_amd.parts.recurrent import Retention

    spec = load_config(copy.deepcopy(nu.ODD)).model_spec()

    def built(i, dtype):
        cls = LatentAttention if isinstance(spec.layers[i].mixer, LatentAttentionSpec) else Retention
        params = {d.name: torch.zeros(d.shape, dtype=dtype) for d in cls.declare(spec.layers[i].mixer, 72)}
        return cls(spec.layers[i].mixer, 72, params, dtype, "cpu", {})

    from paged_llm_rs_amd.parts.linear import Linear

    before, Linear.keep_strips = Linear.keep_strips, False      # (the second layout of the weights is made on the GPU)
    try:
        assert built(1, torch.float32).cache_spec() == KVCacheSpec(1, 36, 9, values_in_keys=True)
        assert built(1, torch.bfloat16).cache_spec() == KVCacheSpec(1, 48, 9, values_in_keys=True), "rows in sixteens"
        assert built(4, torch.float32).cache_spec() == KVCacheSpec(1, 40, None, values_in_keys=True)
        kept = built(0, torch.bfloat16)
        assert kept.cache_spec() is None and kept.state_spec().shape == (3 * 24 * 40,) and kept.state_spec().dtype == torch.float32
        assert kept.chunked and abs(kept.key_scale - 24 ** -0.5) < 1e-15
    finally:
        Linear.keep_strips = before


def test_frequencies_that_follow_a_ramp():
    from paged_llm_rs_amd.parts.rotary import ramped_frequencies, turning

    for dims, base, ramp in ((64, 10000.0, (8.0, 4096.0, 32.0, 1.0)), (8, 300.0, (4.0, 64.0, 6.0, 1.0)), (2, 50.0, (2.0, 16.0, 2.0, 1.0)),
                             (16, 100.0, (0.5, 32.0, 3.0, 2.0)), (128, 1e6, (40.0, 1024.0, 1000.0, 900.0)), (32, 1e4, (3.0, 5.0, 32.0, 1.0))):
        rot = nu.rotation(dims, base, ramp)
        want, amplitude = plain.frequencies(rot)
        got, by = ramped_frequencies(dims, base, ramp)
        assert torch.equal(got, torch.tensor(want, dtype=F).float()) and by == amplitude
        assert turning(dims, base, None, ramp)[1] == amplitude
    # far enough apart all three kinds of pairs are there: kept, blended, divided
    f, amplitude = ramped_frequencies(64, 10000.0, (8.0, 4096.0, 32.0, 1.0))
    share = [float(x) / 10000.0 ** (-2 * i / 64) for i, x in enumerate(f)]
    assert share[0] == pytest.approx(1.0, abs=1e-6) and share[-1] == pytest.approx(1 / 8, abs=1e-6)
    assert any(0.2 < s < 0.9 for s in share) and all(a >= b - 1e-6 for a, b in zip(share, share[1:]))
    assert amplitude == 0.1 * math.log(8.0) + 1.0
    assert turning(64, 10000.0)[1] == 1.0
    with pytest.raises(UnsupportedError):
        turning(64, 10000.0, (8.0, 1.0, 4.0, 8192.0), (8.0, 4096.0, 32.0, 1.0))
    with pytest.raises(UnsupportedError):
        ramped_frequencies(64, 1.0, (8.0, 4096.0, 32.0, 1.0))


def test_properties_of_the_plain_mechanisms():
    g = torch.Generator().manual_seed(0)
    positions = torch.arange(12)
    seen = plain.visible_keys(positions, {"size": 4})
    assert seen[7].nonzero().flatten().tolist() == [4, 5, 6, 7] and seen[2].nonzero().flatten().tolist() == [0, 1, 2]
    assert plain.visible_keys(positions, None)[7].nonzero().flatten().tolist() == list(range(8))
    # rotation in halves and in neighbours: the same pairs of angles, other places; values behind the turned ones stay
    x = torch.randn(7, 3, 12, generator=g, dtype=F)
    rot = nu.rotation(8, 100.0)
    halves, neighbours = plain.rotate_halves(x, torch.arange(7), rot), plain.rotate_neighbours(x, torch.arange(7), rot)
    for turned in (halves, neighbours):
        assert torch.equal(turned[..., 8:], x[..., 8:]) and torch.allclose(turned[0], x[0])
    order = [0, 4, 1, 5, 2, 6, 3, 7, 8, 9, 10, 11]
    assert torch.allclose(plain.rotate_neighbours(x[..., order], torch.arange(7), rot), halves[..., order])
    one = plain.rotate_halves(torch.tensor([[1.0, 0.0]], dtype=F), torch.tensor([1]), nu.rotation(2, 7.0))
    assert torch.allclose(one, torch.tensor([[math.cos(1.0), math.sin(1.0)]], dtype=F))
    # scores between rotated vectors depend on the distance alone; a ramp's amplitude enters squared
    a, c = torch.randn(1, 8, generator=g, dtype=F), torch.randn(1, 8, generator=g, dtype=F)
    dot = lambda p, q, r: float((plain.rotate_halves(a, torch.tensor([p]), r) * plain.rotate_halves(c, torch.tensor([q]), r)).sum())
    assert abs(dot(9, 4, rot) - dot(25, 20, rot)) < 1e-12 and abs(dot(9, 4, rot) - dot(9, 5, rot)) > 1e-6
    ramped = nu.rotation(8, 100.0, (8.0, 64.0, 4.0, 1.0))
    assert abs(dot(5, 5, ramped) / dot(5, 5, rot) - (0.1 * math.log(8.0) + 1.0) ** 2) < 1e-12
    # the retention of a single token reads out (q . k) v; with a decay of nothing every token does; a head's read-out is normed
    m = {"heads": 1, "dim": 4, "vdim": 6, "decay": [0.0], "rot": nu.rotation(4, 100.0)}
    w = {n: torch.randn(*s, generator=g, dtype=F) for n, s in (("q", (4, 10)), ("k", (4, 10)), ("v", (6, 10)), ("g", (6, 10)))}
    w["o"] = torch.eye(6, dtype=F)
    h = torch.randn(5, 10, generator=g, dtype=F)
    q, k, v = h @ w["q"].T, h @ w["k"].T, h @ w["v"].T
    want = plain.rms((q * k).sum(-1, keepdim=True) * 4 ** -0.5 * v, 1e-9) * plain.silu(h @ w["g"].T)
    assert torch.allclose(plain.retention_mixer(h, w, "", m, 1e-9, torch.arange(5)), want)
    assert torch.equal(plain.relu_squared(torch.tensor([-2.0, 0.0, 3.0])), torch.tensor([0.0, 0.0, 9.0]))


def test_properties_of_the_plain_router():
    g = torch.Generator().manual_seed(1)
    h = torch.randn(60, 12, generator=g, dtype=F)
    w = {"router": torch.randn(8, 12, generator=g, dtype=F)}
    score = torch.sigmoid(h @ w["router"].T)
    router = {"experts": 8, "top": 3, "scale": 2.0}
    chosen, weight = plain.route(h, w, "", router)
    assert torch.equal(chosen, score.topk(3, -1).indices) and torch.allclose(weight.sum(-1), torch.full((60,), 2.0, dtype=F))
    assert torch.allclose(weight, 2.0 * score.gather(1, chosen) / score.gather(1, chosen).sum(-1, keepdim=True))
    # a group counts by its two best together: two good ones beat one excellent and a bad one
    hand = torch.tensor([[0.95, 0.05, 0.6, 0.5]], dtype=F)
    kept = plain.candidates(hand, {"groups": {"count": 2, "keep": 1}})
    assert torch.isinf(kept[0, :2]).all() and torch.equal(kept[0, 2:], hand[0, 2:])
    # groups of one count by their one expert
    assert torch.equal(torch.isinf(plain.candidates(hand, {"groups": {"count": 4, "keep": 2}}))[0], torch.tensor([False, True, False, True]))
    # a shared expert is there whatever is chosen, times its gate
    mlp = {"kind": "moe", "expert": {"ff": 5}, "router": {"experts": 1, "top": 1}, "shared": {"ff": 7}}
    w2 = {"router": torch.randn(1, 12, generator=g, dtype=F), "e0.up": torch.zeros(5, 12, dtype=F), "e0.down": torch.zeros(12, 5, dtype=F),
          "shared.up": torch.randn(7, 12, generator=g, dtype=F), "shared.down": torch.randn(12, 7, generator=g, dtype=F),
          "shared.sg": torch.randn(1, 12, generator=g, dtype=F)}
    want = torch.sigmoid(h @ w2["shared.sg"].T) * (plain.relu_squared(h @ w2["shared.up"].T) @ w2["shared.down"].T)
    assert torch.allclose(plain.feed_forward(h, w2, "", mlp), want)
