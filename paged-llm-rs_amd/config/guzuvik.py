"""The typed configuration of the Guzuvik design, read from the keys of its own config.json.

A Guzuvik model is a list of layers whose sublayers stand between two layer norms,
x <- x + norm1b(mixer(norm1(x))) and then x <- x + norm2b(ff(norm2(x))).  A second embedding row, chosen by a
token and the one before it, joins the embedding.  Two kinds of mixer: ``mamba2`` keeps a matrix of state
a head whose decay and step size come from the token; ``attention`` is grouped-query attention with
biases, unit q and k, a soft cap on the scores, a distance penalty a head, a window that keeps the first
tokens in sight, values mixed with those of the first layer that mixes, and a gate a head.  A
feed-forward is dense (the squared relu) or a set of experts with clamped gates behind a router that
weighs its chosen experts by a softmax over their logits.  The output projection is the embedding table.
Inside a mixer or a feed-forward a key this reader does not know is refused: a model that ignores a
constant runs and is wrong.
"""

from __future__ import annotations

from dataclasses import dataclass

from ..errors import ConfigError, UnsupportedError
from .papivik import _count, _number, _object
from .specs import (DenseMlpSpec, LayerSpec, ModelSpec, NormSpec, RoutedExpertsSpec, ScheduleEntry, SinkAttentionSpec,
                    StateSpaceSpec)


def _whole(d: dict, key: str, what: str) -> int:
    """An integer of zero or more; 0 where the key is absent or null."""
    v = d.get(key)
    if v is None:
        return 0
    if isinstance(v, bool) or not isinstance(v, int) or v < 0:
        raise ConfigError(f"{what}: {key} {v!r}, which has to be an integer of zero or more")
    return v


def _attention(m, what: str, eps: float):
    _object(m, what, ("heads", "kv_heads", "dim", "vdim", "scale"), ("mask", "softcap", "v_mix"))
    heads, kv_heads = _count(m, "heads", what), _count(m, "kv_heads", what)
    if heads % kv_heads:
        raise ConfigError(f"{what}: {heads} heads over {kv_heads} kv_heads")
    window, keep = None, 0
    if m.get("mask") is not None:
        _object(m["mask"], what + ".mask", ("size",), ("keep_first",))
        window, keep = _count(m["mask"], "size", what + ".mask"), _whole(m["mask"], "keep_first", what + ".mask")
    cap = None
    if m.get("softcap") is not None:
        cap = _number(m, "softcap", what)
        if not cap > 0:
            raise ConfigError(f"{what}: a softcap of {cap}")
    mix = m.get("v_mix")
    if mix is not None and not isinstance(mix, bool):
        raise ConfigError(f"{what}: v_mix {mix!r}, which has to be true or false")
    return SinkAttentionSpec(num_heads=heads, num_kv_heads=kv_heads, head_dim=_count(m, "dim", what),
                             value_dim=_count(m, "vdim", what), scale=_number(m, "scale", what), qk_unit_eps=eps,
                             qkv_bias=True, distance_slopes="geometric", slope_span=8.0, window=window, mask="window",
                             keep_first=keep, softcap=cap, value_mix=bool(mix), head_gate=True, sink=None)


def _mamba2(m, what: str, eps: float):
    _object(m, what, ("heads", "vdim", "state", "groups", "conv", "norm_groups"))
    heads, vdim, groups, parts = (_count(m, key, what) for key in ("heads", "vdim", "groups", "norm_groups"))
    if heads % groups:
        raise ConfigError(f"{what}: {heads} heads over {groups} groups")
    if (heads * vdim) % parts:
        raise ConfigError(f"{what}: {heads * vdim} values normed in {parts} equal parts")
    return StateSpaceSpec(num_heads=heads, value_dim=vdim, state_dim=_count(m, "state", what), groups=groups,
                          conv_taps=_count(m, "conv", what), norm_groups=parts, eps=eps)


_MIXERS = {"attention": _attention, "mamba2": _mamba2}


def _feed_forward(mlp, what: str):
    if mlp is None:
        return None
    if not isinstance(mlp, dict) or "kind" not in mlp:
        raise ConfigError(f"{what} is no object with a kind")
    if mlp["kind"] == "dense":
        _object(mlp, what, ("kind", "ff"))
        return DenseMlpSpec(intermediate_size=_count(mlp, "ff", what), activation="relu2")
    if mlp["kind"] == "moe":
        _object(mlp, what, ("kind", "expert", "router"))
        _object(mlp["expert"], what + ".expert", ("ff", "limit"))
        r = _object(mlp["router"], what + ".router", ("experts", "top"))
        experts, top = _count(r, "experts", what + ".router"), _count(r, "top", what + ".router")
        if top > experts:
            raise ConfigError(f"{what}.router: {top} of {experts} experts a token")
        limit = _number(mlp["expert"], "limit", what + ".expert")
        if not limit > 0:
            raise ConfigError(f"{what}.expert: a limit of {limit}")
        return RoutedExpertsSpec(experts=experts, top=top, intermediate_size=_count(mlp["expert"], "ff", what + ".expert"),
                                 activation="clamped", limit=limit, score="chosen_logits", biased=True, corrected=False)
    raise UnsupportedError(f"{what}: kind {mlp['kind']!r}, this design has dense and moe")


@dataclass(frozen=True)
class GuzuvikConfig:
    raw: dict
    width: int
    vocab: int
    eps: float
    bigram: tuple | None      # (buckets, mul_prev, mul_cur)
    layers: tuple             # (mixer spec, feed-forward spec or None) a layer

    architecture = "Guzuvik"

    @classmethod
    def from_dict(cls, d: dict) -> "GuzuvikConfig":
        _object(d, "config.json", ("architecture", "layers", "norm", "vocab", "width"), ("embedding",), others=True)
        _object(d["norm"], "norm", ("eps",))
        eps = _number(d["norm"], "eps", "norm")
        if not eps >= 0:
            raise ConfigError(f"norm: an eps of {eps}")
        bigram = None
        if d.get("embedding") is not None:
            _object(d["embedding"], "embedding", (), ("bigram",))
            if d["embedding"].get("bigram") is not None:
                b = _object(d["embedding"]["bigram"], "embedding.bigram", ("buckets", "mul_prev", "mul_cur"))
                bigram = (_count(b, "buckets", "embedding.bigram"), _whole(b, "mul_prev", "embedding.bigram"),
                          _whole(b, "mul_cur", "embedding.bigram"))
        if not isinstance(d["layers"], list) or not d["layers"]:
            raise ConfigError("layers has to be a list of at least one layer")
        layers = []
        for i, layer in enumerate(d["layers"]):
            what = f"layers[{i}]"
            _object(layer, what, ("type", "mixer"), ("mlp",), others=True)
            if layer["type"] not in _MIXERS:
                raise UnsupportedError(f"{what}: a mixer of type {layer['type']!r}, this design has {', '.join(_MIXERS)}")
            layers.append((_MIXERS[layer["type"]](layer["mixer"], what + ".mixer", eps),
                           _feed_forward(layer.get("mlp"), what + ".mlp")))
        mixing = {(m.num_kv_heads, m.value_dim) for m, _ in layers if getattr(m, "value_mix", False)}
        if len({g * v for g, v in mixing}) > 1:
            raise ConfigError(f"layers that mix their values have values of different sizes: {sorted(mixing)} (kv_heads, vdim)")
        return cls(raw=d, width=_count(d, "width", "config.json"), vocab=_count(d, "vocab", "config.json"), eps=eps,
                   bigram=bigram, layers=tuple(layers))

    def to_dict(self) -> dict:
        return self.raw

    def model_spec(self) -> ModelSpec:
        norm = NormSpec("layer_norm", self.eps)
        layers = tuple(LayerSpec(block="sandwich_norm", mixer=mixer, feed_forward=mlp, norm=norm, weight_prefix=f"l{i}")
                       for i, (mixer, mlp) in enumerate(self.layers))
        extra = {"bare_norm_names": True}
        if self.bigram is not None:
            extra.update({"embed_transform": "bigram", "bigram": ("bigram", *self.bigram)})
        return ModelSpec(hidden_size=self.width, vocab_size=self.vocab, layers=layers,
                         schedule=tuple(ScheduleEntry(i) for i in range(len(layers))), final_norm=norm,
                         tie_word_embeddings=True, max_positions=0, embed_name="embed", final_norm_name="final.norm",
                         head_name="head", ignored_tensors=("l*.mix.vmix",), extra=extra)
