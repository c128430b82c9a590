"""The typed configuration of the Nikonex design, read from the keys of its own config.json.

A Nikonex model is a list of parallel layers with one multiplier: with a = norm1(x) and b = norm2(x) of the same
x, x <- x + residual_mult * (mixer(a) + ff(b)).  Two kinds of mixer: ``latent_attention`` takes its queries through a
small normed vector of their own, keeps one small normed vector and one rotated key part a token and rebuilds every
head's keys and values from them, under a sliding window, its rotation's frequencies optionally blended by a ramp
over the pairs; ``retention`` keeps a matrix a head that decays by a fixed factor a token, with rotated queries and
keys.  A feed-forward is a set of experts of two matrices each (the squared relu between them) behind a router of
sigmoid scores with groups of neighbouring experts, beside one shared expert with a gate a token.  Inside a mixer or
a feed-forward a key this reader does not know is refused: a model that ignores a constant runs and is wrong.
"""

from __future__ import annotations

from dataclasses import dataclass

from ..errors import ConfigError, UnsupportedError
from .papivik import _count, _number, _object
from .specs import LatentAttentionSpec, LayerSpec, ModelSpec, NormSpec, RetentionSpec, RoutedExpertsSpec, ScheduleEntry


def _rotation(rot, what: str, most: int):
    """(dims, base, ramp or None) of a mixer's ``rot``; without one nothing turns."""
    if rot is None:
        return 0, 10000.0, None
    _object(rot, what, ("dims", "base"), ("scaling",))
    dims, base = _count(rot, "dims", what), _number(rot, "base", what)
    if dims % 2 or dims > most or not base > 0:
        raise ConfigError(f"{what}: a rotation over {dims} of {most} values with base {base}")
    ramp = None
    if rot.get("scaling") is not None:
        s = _object(rot["scaling"], what + ".scaling", ("factor", "original", "fast", "slow"))
        ramp = tuple(_number(s, key, what + ".scaling") for key in ("factor", "original", "fast", "slow"))
        if not all(v > 0 for v in ramp) or base == 1.0:
            raise ConfigError(f"{what}.scaling: factor {ramp[0]}, original {ramp[1]}, fast {ramp[2]}, slow {ramp[3]}, base {base}")
    return dims, base, ramp


def _latent(m, what: str, eps: float):
    _object(m, what, ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "scale"), ("rot", "mask"))
    rot_dim = _count(m, "rot_dim", what)
    dims, base, ramp = _rotation(m.get("rot"), what + ".rot", rot_dim)
    window = None
    if m.get("mask") is not None:
        _object(m["mask"], what + ".mask", ("size",))
        window = _count(m["mask"], "size", what + ".mask")
    return LatentAttentionSpec(num_heads=_count(m, "heads", what), head_dim=_count(m, "dim", what), rotary_dim=rot_dim,
                               value_dim=_count(m, "vdim", what), q_rank=_count(m, "q_rank", what),
                               kv_rank=_count(m, "kv_rank", what), rotary_turned=dims, rotary_base=base, rotary_ramp=ramp,
                               max_positions=0, scale=_number(m, "scale", what), norm_eps=eps, sink=None, gated=False,
                               window=window)


def _retention(m, what: str, eps: float):
    _object(m, what, ("heads", "dim", "vdim", "decay"), ("rot",))
    heads, dim = _count(m, "heads", what), _count(m, "dim", what)
    dims, base, ramp = _rotation(m.get("rot"), what + ".rot", dim)
    decay = m["decay"]
    if not isinstance(decay, list) or len(decay) != heads or any(isinstance(d, bool) or not isinstance(d, (int, float)) for d in decay):
        raise ConfigError(f"{what}: decay has to be a list of {heads} numbers, one a head")
    if any(not 0 <= d <= 1 for d in decay):
        raise ConfigError(f"{what}: decays between 0 and 1, not {decay}")
    return RetentionSpec(num_heads=heads, head_dim=dim, value_dim=_count(m, "vdim", what), decay=tuple(float(d) for d in decay),
                         rotary_dims=dims, rotary_base=base, rotary_ramp=ramp, eps=eps)


_MIXERS = {"latent_attention": _latent, "retention": _retention}


def _feed_forward(mlp, what: str):
    if mlp is None:
        return None
    if not isinstance(mlp, dict) or "kind" not in mlp:
        raise ConfigError(f"{what} is no object with a kind")
    if mlp["kind"] != "moe":
        raise UnsupportedError(f"{what}: kind {mlp['kind']!r}, this design has moe")
    _object(mlp, what, ("kind", "expert", "router"), ("shared",))
    _object(mlp["expert"], what + ".expert", ("ff",))
    r = _object(mlp["router"], what + ".router", ("experts", "top"), ("groups", "scale"))
    experts, top = _count(r, "experts", what + ".router"), _count(r, "top", what + ".router")
    groups = kept = 1
    if r.get("groups") is not None:
        _object(r["groups"], what + ".router.groups", ("count", "keep"))
        groups, kept = _count(r["groups"], "count", what + ".router.groups"), _count(r["groups"], "keep", what + ".router.groups")
    if experts % groups or kept > groups:
        raise ConfigError(f"{what}.router: {experts} experts in {groups} groups of which {kept} are kept")
    if top > kept * (experts // groups):
        raise ConfigError(f"{what}.router: {top} a token of the {kept * (experts // groups)} that can be chosen")
    shared = 0
    if mlp.get("shared") is not None:
        _object(mlp["shared"], what + ".shared", ("ff",))
        shared = _count(mlp["shared"], "ff", what + ".shared")
    scale = _number(r, "scale", what + ".router") if r.get("scale") is not None else 1.0
    return RoutedExpertsSpec(experts=experts, identity=0, top=top, intermediate_size=_count(mlp["expert"], "ff", what + ".expert"),
                             activation="relu2", gated=False, score="sigmoid", corrected=False, groups=groups, groups_kept=kept,
                             group_best=2, weight_scale=scale, shared_size=shared)


@dataclass(frozen=True)
class NikonexConfig:
    raw: dict
    width: int
    vocab: int
    eps: float
    residual_mult: float
    layers: tuple             # (mixer spec, feed-forward spec or None) a layer

    architecture = "Nikonex"

    @classmethod
    def from_dict(cls, d: dict) -> "NikonexConfig":
        _object(d, "config.json", ("architecture", "layers", "norm", "residual_mult", "vocab", "width"), (), others=True)
        _object(d["norm"], "norm", ("eps",))
        eps = _number(d["norm"], "eps", "norm")
        if not eps >= 0:
            raise ConfigError(f"norm: an eps of {eps}")
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
        return cls(raw=d, width=_count(d, "width", "config.json"), vocab=_count(d, "vocab", "config.json"), eps=eps,
                   residual_mult=_number(d, "residual_mult", "config.json"), layers=tuple(layers))

    def to_dict(self) -> dict:
        return self.raw

    def model_spec(self) -> ModelSpec:
        norm = NormSpec("rms_norm", self.eps)
        layers = tuple(LayerSpec(block="parallel", mixer=mixer, feed_forward=mlp, norm=norm, weight_prefix=f"l{i}",
                                 residual_mult=self.residual_mult)
                       for i, (mixer, mlp) in enumerate(self.layers))
        return ModelSpec(hidden_size=self.width, vocab_size=self.vocab, layers=layers,
                         schedule=tuple(ScheduleEntry(i) for i in range(len(layers))), final_norm=norm,
                         tie_word_embeddings=False, max_positions=0, embed_name="embed", final_norm_name="final.norm",
                         head_name="head", extra={"bare_norm_names": True})
