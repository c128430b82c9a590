"""The Guzuvik design without a GPU: its configuration reader and what it refuses, the tensors it declares, the
random-weights mode, the cache layout (kept pages, state slots of layers and of the embedding), and properties of
the plain implementation's mechanisms."""

from __future__ import annotations

import copy
import math

import pytest
import torch

import guzuvik_util as gu
import plain_guzuvik as plain
from paged_llm_rs_amd.cache.manager import CacheManager, GroupGeometry
from paged_llm_rs_amd.config import load_config
from paged_llm_rs_amd.config.specs import DenseMlpSpec, RoutedExpertsSpec, SinkAttentionSpec, StateSpaceSpec
from paged_llm_rs_amd.errors import ConfigError, UnsupportedError
from paged_llm_rs_amd.parts.model import declare_parameters

F = torch.float64


def test_the_reader_takes_every_size_and_constant_from_the_config():
    spec = load_config(copy.deepcopy(gu.ODD)).model_spec()
    assert spec.hidden_size == 72 and spec.vocab_size == 211 and spec.max_positions == 0 and spec.tie_word_embeddings
    assert spec.extra["embed_transform"] == "bigram" and spec.extra["bigram"] == ("bigram", 101, 31, 5)
    a, s = spec.layers[0].mixer, spec.layers[1].mixer
    assert isinstance(a, SinkAttentionSpec) and isinstance(s, StateSpaceSpec)
    assert (a.num_heads, a.num_kv_heads, a.head_dim, a.value_dim, a.scale) == (6, 2, 24, 40, 0.3)
    assert (a.window, a.keep_first, a.softcap, a.value_mix, a.mask) == (9, 3, 3.0, True, "window")
    assert a.qkv_bias and a.head_gate and a.qk_unit_eps == 1e-5 and not a.qk_gain and a.sink is None
    assert a.distance_slopes == "geometric" and a.slope_span == 8.0 and a.temperature_coef is None
    assert (s.num_heads, s.value_dim, s.state_dim, s.groups, s.conv_taps, s.norm_groups, s.eps) == (6, 12, 20, 3, 3, 2, 1e-5)
    free = spec.layers[4].mixer
    assert (free.window, free.keep_first, free.softcap, free.value_mix) == (None, 0, 2.0, False)
    assert spec.layers[3].mixer.softcap is None
    experts, dense = spec.layers[0].feed_forward, spec.layers[1].feed_forward
    assert isinstance(experts, RoutedExpertsSpec) and isinstance(dense, DenseMlpSpec)
    assert (experts.experts, experts.top, experts.intermediate_size, experts.limit) == (7, 3, 24, 1.5)
    assert (experts.score, experts.activation, experts.biased, experts.corrected) == ("chosen_logits", "clamped", True, False)
    assert dense.intermediate_size == 96 and dense.activation == "relu2" and spec.layers[2].feed_forward is None
    assert all(layer.block == "sandwich_norm" and layer.norm.kind == "layer_norm" and layer.norm.eps == 1e-5 for layer in spec.layers)
    assert [e.layer for e in spec.schedule] == list(range(7))
    ones = load_config(copy.deepcopy(gu.ONES)).model_spec()
    assert "embed_transform" not in ones.extra
    assert (ones.layers[3].mixer.keep_first, ones.layers[3].mixer.value_mix) == (0, False)
    for absent in ("mask", "softcap", "v_mix"):
        config = copy.deepcopy(gu.ODD)
        config["layers"][0]["mixer"][absent] = None
        assert load_config(config).model_spec().layers[0].mixer is not None
    config = copy.deepcopy(gu.ODD)
    config["layers"][2]["mlp"] = None
    config["embedding"] = None
    config["note"] = "a key of no mechanism"
    assert "bigram" not in load_config(config).model_spec().extra


@pytest.mark.parametrize("damage, error", [
    (lambda c: c["layers"][0]["mixer"].pop("vdim"), ConfigError),
    (lambda c: c["layers"][0]["mixer"].update(extra=1), UnsupportedError),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), ConfigError),
    (lambda c: c["layers"][0]["mixer"].update(softcap=0.0), ConfigError),
    (lambda c: c["layers"][0]["mixer"].update(v_mix=1), ConfigError),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), ConfigError),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1), ConfigError),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(stride=2), UnsupportedError),
    (lambda c: c["layers"][3]["mixer"].update(vdim=24), ConfigError),            # mixes with values of 80
    (lambda c: c["layers"][1]["mixer"].update(groups=4), ConfigError),
    (lambda c: c["layers"][1]["mixer"].update(norm_groups=5), ConfigError),
    (lambda c: c["layers"][1]["mixer"].pop("conv"), ConfigError),
    (lambda c: c["layers"][1]["mixer"].update(dim=8), UnsupportedError),
    (lambda c: c["layers"][0].update(type="lightning"), UnsupportedError),
    (lambda c: c["layers"][0]["mlp"].update(kind="routed"), UnsupportedError),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=8), ConfigError),
    (lambda c: c["layers"][0]["mlp"]["router"].update(groups=2), UnsupportedError),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), ConfigError),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0.0), ConfigError),
    (lambda c: c["embedding"].update(scale=2.0), UnsupportedError),
    (lambda c: c["embedding"]["bigram"].update(buckets=0), ConfigError),
    (lambda c: c["embedding"]["bigram"].pop("mul_cur"), ConfigError),
    (lambda c: c["norm"].update(eps=-1.0), ConfigError),
])
def test_what_the_reader_refuses(damage, error):
    config = copy.deepcopy(gu.ODD)
    damage(config)
    with pytest.raises(error):
        load_config(config)


def test_declared_tensors():
    found = declare_parameters(load_config(copy.deepcopy(gu.ODD)).model_spec())
    decls = {d.name: tuple(d.shape) for d in found}
    optional = {d.name for d in found if d.optional}
    assert decls["embed"] == (211, 72) and decls["bigram"] == (102, 72) and "head" in optional
    assert decls["final.norm"] == decls["final.norm.b"] == (72,)
    assert decls["l0.mix.q"] == (144, 72) and decls["l0.mix.k"] == (48, 72) and decls["l0.mix.v"] == (80, 72)
    assert decls["l0.mix.q.b"] == (144,) and decls["l0.mix.k.b"] == (48,) and decls["l0.mix.v.b"] == (80,)
    assert decls["l0.mix.g"] == (6, 72) and decls["l0.mix.o"] == (72, 240) and decls["l0.mix.vmix"] == ()
    assert "l4.mix.vmix" not in decls and "l0.mix.sink" not in decls and "l0.mix.q.norm" not in decls
    assert decls["l1.mix.in"] == (72 + 72 + 120 + 6, 72) and decls["l1.mix.conv"] == (192, 3) and decls["l1.mix.conv.b"] == (192,)
    assert decls["l1.mix.dt_bias"] == decls["l1.mix.A_log"] == decls["l1.mix.D"] == (6,)
    assert decls["l1.mix.norm"] == (72,) and decls["l1.mix.o"] == (72, 72)
    assert decls["l0.mlp.e6.gate"] == (24, 72) and decls["l0.mlp.e6.down"] == (72, 24) and "l0.mlp.e7.up" not in decls
    assert decls["l0.mlp.router"] == (7, 72) and decls["l0.mlp.router.b"] == (7,) and "l0.mlp.correction" not in decls
    assert decls["l1.mlp.up"] == (96, 72) and decls["l1.mlp.down"] == (72, 96) and "l1.mlp.gate" not in decls
    for i in range(7):
        for norm in ("norm1", "norm1b", "norm2", "norm2b"):
            assert decls[f"l{i}.{norm}"] == decls[f"l{i}.{norm}.b"] == (72,)
    # a layer without a feed-forward does not need its second pair of norms
    assert {"l2.norm2", "l2.norm2b", "l2.norm2.b", "l2.norm2b.b"} <= optional and "l2.norm1b.b" not in optional


def test_a_number_of_a_layer_that_does_not_mix_is_no_stranger(tmp_path):
    from paged_llm_rs_amd.weights.loader import check_declared

    spec = load_config(copy.deepcopy(gu.ODD)).model_spec()
    decls = declare_parameters(spec)
    shapes = {d.name: tuple(d.shape) for d in decls if not d.optional}
    check_declared(decls, {**shapes, "l4.mix.vmix": ()}, "a checkpoint", spec.ignored_tensors)
    with pytest.raises(Exception, match="l4.mix.other"):
        check_declared(decls, {**shapes, "l4.mix.other": ()}, "a checkpoint", spec.ignored_tensors)


def test_the_random_weights_mode_and_the_plain_implementation(tmp_path):
    folder = gu.write_model(tmp_path / "m", gu.ODD, seed=3)
    config, weights = gu.load_plain(folder)
    assert "head" not in weights and 0 < float(weights["l3.mix.vmix"]) < 1 and weights["l3.mix.vmix"].dim() == 0
    tokens = [5, 17, 3, 200, 0, 44, 9, 9, 120]
    streams = []
    logits = plain.forward(config, weights, tokens, streams)
    assert logits.shape == (9, 211) and len(streams) == 7 and torch.isfinite(logits).all()
    # causal: a prefix gives the same logits
    assert torch.allclose(plain.forward(config, weights, tokens[:5]), logits[:5], atol=1e-12)


def test_the_cache_keeps_the_pages_of_the_first_tokens_and_slots_for_what_is_carried():
    from paged_llm_rs_amd.cache.layout import CacheLayout, KVCacheSpec, StateSpec

    m = CacheManager([GroupGeometry(4, 12, window=6, keep=5), GroupGeometry(4, 12, window=6), GroupGeometry(4, 12)], state_slots=1)
    slot = m.add_sequence(7)
    assert slot == 0
    for n in range(24):
        assert m.reserve(7, 1)
        m.advance(7, 1)
        held = [m.slot_of(7, 0, p) is not None for p in range(n + 1)]
        # the next query, at n + 1, reads the first five keys and those from n - 4 on
        for p in range(n + 1):
            if p < 5 or p >= n + 1 - 5:
                assert held[p], (n, p)
    table = m.table(7, 0)
    assert table[0] >= 0 and table[1] >= 0 and table[2] == -1 and table[3] == -1 and table[-1] >= 0
    assert m.table(7, 1)[0] == -1, "a window that keeps nothing gives its first pages back"
    assert m.in_use(0) == m.in_use(1) + 2 and m.in_use(2) == 6
    m.free_sequence(7)
    assert m.in_use(0) == m.in_use(1) == m.in_use(2) == 0 and m.free_state_slots == 1
    with pytest.raises(ConfigError):
        CacheManager([GroupGeometry(4, 12, window=6, keep=-1)])

    class Block:
        def __init__(self, kv=None, state=None):
            self.mixer = type("M", (), {"cache_spec": lambda s: kv, "state_spec": lambda s: state})()

    spec = load_config(copy.deepcopy(gu.ODD)).model_spec()
    kept = KVCacheSpec(2, 48, 9, keep_first=3)
    blocks = [Block(kept), Block(state=StateSpec((10,))), Block(state=StateSpec((12,))), Block(KVCacheSpec(2, 48, 9)),
              Block(KVCacheSpec(1, 16)), Block(state=StateSpec((9,))), Block(kept)]
    layout = CacheLayout.from_blocks(blocks, spec.schedule, {("embed_transform", 0): StateSpec((1,), torch.int32)})
    # layers that keep different first tokens share no table
    assert [sorted(g.layers) for g in layout.groups] == [[0, 6], [3], [4]]
    assert set(layout.states) == {1, 2, 5, ("embed_transform", 0)}


def test_properties_of_the_plain_norm_and_activations():
    g = torch.Generator().manual_seed(0)
    x = torch.randn(5, 12, generator=g, dtype=F) * 3 + 7
    one, zero = torch.ones(12, dtype=F), torch.zeros(12, dtype=F)
    y = plain.layer_norm(x, one, zero, 0.0)
    assert torch.allclose(y.mean(-1), torch.zeros(5, dtype=F), atol=1e-12) and torch.allclose((y * y).mean(-1), torch.ones(5, dtype=F))
    assert torch.allclose(plain.layer_norm(x, one, zero, 1e-5), torch.nn.functional.layer_norm(x, (12,), eps=1e-5))
    assert torch.allclose(plain.layer_norm(x, one * 2, one, 0.0), 2 * y + 1)
    assert torch.allclose(plain.softplus(torch.tensor([-50.0, 0.0, 50.0], dtype=F)),
                          torch.tensor([math.exp(-50.0), math.log(2.0), 50.0], dtype=F), atol=1e-18)
    w = {"gate": torch.eye(3, dtype=F), "up": torch.eye(3, dtype=F), "down": torch.eye(3, dtype=F)}
    out = plain.expert(torch.tensor([[5.0, -5.0, 0.5]], dtype=F), w, "", 2.0)[0]
    want = [2.0 / (1 + math.exp(-3.404)) * 3.0, -5.0 / (1 + math.exp(8.51)) * -1.0, 0.5 / (1 + math.exp(-0.851)) * 1.5]
    assert torch.allclose(out, torch.tensor(want, dtype=F)), "the gate is cut above only, the other factor on both sides"
    d = plain.dense_feed_forward(torch.tensor([[3.0, -3.0, 0.5]], dtype=F), w, "")
    assert torch.allclose(d, torch.tensor([[9.0, 0.0, 0.25]], dtype=F))


def test_properties_of_the_plain_pairs_of_tokens():
    rows = plain.bigram_rows(torch.tensor([4, 9, 4, 9, 0]), {"buckets": 10, "mul_prev": 3, "mul_cur": 7})
    assert rows.tolist() == [10, (12 + 63) % 10, (27 + 28) % 10, (12 + 63) % 10, 27 % 10]


def test_properties_of_the_plain_state_space():
    g = torch.Generator().manual_seed(1)
    T, H, V, G, N = 9, 4, 3, 2, 5
    x, B, C = (torch.randn(s, generator=g, dtype=F) for s in ((T, H, V), (T, G, N), (T, G, N)))
    dt = torch.rand((T, H), generator=g, dtype=F)
    a_log, D = torch.randn(H, generator=g, dtype=F), torch.randn(H, generator=g, dtype=F)
    out = plain.state_space_scan(x, B, C, dt, a_log, D)
    # as one sum over the earlier tokens
    want = torch.zeros_like(out)
    for t in range(T):
        for h in range(H):
            for s in range(t + 1):
                decay = math.exp(-math.exp(float(a_log[h])) * float(dt[s + 1:t + 1, h].sum()))
                want[t, h] += decay * dt[s, h] * (C[t, h // 2] @ B[s, h // 2]) * x[s, h]
            want[t, h] += D[h] * x[t, h]
    assert torch.allclose(out, want, atol=1e-12)
    # the convolution looks back and never forward, the newest tap last
    u = torch.zeros(6, 1, dtype=F)
    u[2] = 1.0
    y = plain.causal_convolution(u, torch.tensor([[1.0, 2.0, 3.0]], dtype=F), torch.tensor([0.5], dtype=F))
    assert y[:, 0].tolist() == [0.5, 0.5, 3.5, 2.5, 1.5, 0.5]
    # each part of the norm has its own root mean square
    z = plain.norm_in_parts(torch.tensor([[3.0, 3.0, 0.1, 0.1]], dtype=F), 2, torch.ones(4, dtype=F), 0.0)
    assert torch.allclose(z, torch.ones(1, 4, dtype=F))


def test_properties_of_the_plain_attention():
    seen = plain.visible_keys(12, {"size": 3, "keep_first": 2})
    assert seen[7].nonzero().flatten().tolist() == [0, 1, 5, 6, 7] and seen[1].nonzero().flatten().tolist() == [0, 1]
    assert seen[4].nonzero().flatten().tolist() == [0, 1, 2, 3, 4]
    assert plain.visible_keys(12, None)[7].nonzero().flatten().tolist() == list(range(8))
    assert plain.slopes(4) == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8]
    c = plain.capped(torch.tensor([0.01, 5.0, -1e9], dtype=F), 2.0)
    assert abs(float(c[0]) - 0.01) < 1e-6 and abs(float(c[1]) - 2 * math.tanh(2.5)) < 1e-12 and float(c[2]) == -2.0
    v, first = torch.full((2, 3), 4.0, dtype=F), torch.full((2, 3), 8.0, dtype=F)
    lam = torch.tensor(0.25, dtype=F)
    assert torch.equal(plain.mixed_values(v, first, {"v_mix": True}, lam), torch.full((2, 3), 5.0, dtype=F))
    assert plain.mixed_values(v, None, {"v_mix": True}, lam) is v and plain.mixed_values(v, first, {}, lam) is v


def test_the_plain_router_weighs_by_the_chosen_logits_alone():
    g = torch.Generator().manual_seed(2)
    h = torch.randn(40, 12, generator=g, dtype=F)
    w = {"router": torch.randn(8, 12, generator=g, dtype=F), "router.b": torch.zeros(8, dtype=F)}
    chosen, weight = plain.route(h, w, "", {"experts": 8, "top": 3})
    z = h @ w["router"].T
    assert torch.equal(chosen, z.topk(3, -1).indices) and torch.allclose(weight.sum(-1), torch.ones(40, dtype=F))
    assert torch.allclose(weight, torch.softmax(z, -1).gather(1, chosen) / torch.softmax(z, -1).gather(1, chosen).sum(-1, keepdim=True))
    w["router.b"] = torch.tensor([0, 0, 0, 0, 0, 0, 0, 50.0], dtype=F)      # the bias is part of the logits: it weighs too
    chosen, weight = plain.route(h, w, "", {"experts": 8, "top": 3})
    assert (chosen[:, 0] == 7).all() and (weight[:, 0] > 0.999).all()
