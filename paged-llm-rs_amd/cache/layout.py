"""What the layers of a model need from the cache, grouped.

Every mixer says what pages it needs (heads, head size, window) and what
fixed-size state it keeps for each request.  Layers with the same page needs
form a group: they share page numbers (one block table for the group) while
each layer has pools of its own.  A layer that reads another layer's cache has
no pools.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch

from ..errors import ConfigError


@dataclass(frozen=True)
class KVCacheSpec:
    """Keys and values of ``kv_heads`` heads of ``head_dim``; with a window only
    the last ``window`` positions are ever read.  ``values_in_keys``: a token's values are read out of
    its row of keys (a layer that keeps one small vector a token and rebuilds both from it), so the layer
    has one pool, which stands in the place of both."""
    kv_heads: int
    head_dim: int
    window: Optional[int] = None
    values_in_keys: bool = False
    # beside the window the first ``keep_first`` positions of a request are read for good: their pages stay
    keep_first: int = 0


@dataclass(frozen=True)
class StateSpec:
    """A tensor of fixed shape kept for each live request."""
    shape: tuple
    dtype: torch.dtype = torch.float32


@dataclass
class CacheGroupLayout:
    spec: KVCacheSpec
    layers: list          # layer indices that own pools in this group


class CacheLayout:
    def __init__(self, groups: list, layer_group: dict, states: dict):
        # (a key is a layer's index, or what the schedule gives a run of a layer that runs several times)
        self.groups = groups            # [CacheGroupLayout]
        self.layer_group = layer_group  # key -> group index (runs that own pools)
        self.states = states            # key -> StateSpec

    @classmethod
    def from_blocks(cls, blocks, schedule, beside: dict | None = None) -> "CacheLayout":
        """``beside``: {key: StateSpec} of what the model keeps for a request beside its layers (a transform of the
        stream that looks back, say); the keys are names, no layer's index."""
        # A run of a layer either owns its cache or reads the one another run has written earlier in the
        # same pass.  What a run owns is kept under a key: the layer's index, or the key the schedule gives
        # the run (a layer that runs several times with the same weights then has pages and state for every
        # run).  Two owning runs under one key would write the same pages twice, and what a later step
        # reads there would depend on how the tokens were cut into steps: refused.
        def spec_of(index):
            mixer = getattr(blocks[index], "mixer", None)
            return (mixer.cache_spec(), mixer.state_spec()) if mixer is not None else (None, None)

        written: dict = {}           # key -> the layer whose run owns it
        for at, e in enumerate(schedule):
            kv, state = spec_of(e.layer)
            if e.cache_from is None:
                key = e.layer if e.cache_key is None else e.cache_key
                if key in written and (kv is not None or state is not None):
                    raise ConfigError(f"the schedule runs layer {e.layer} twice with one cache; the second run can read "
                                      f"what the first wrote (cache_from={key}) or keep a cache of its own (cache_key)")
                written[key] = e.layer
            else:
                if e.cache_from not in written:
                    raise ConfigError(f"run {at} of the schedule reads the cache of layer {e.cache_from}, which no "
                                      "earlier run of the pass has written")
                if state is not None:
                    raise ConfigError(f"layer {e.layer} keeps a state of its own and cannot read another layer's cache")
                if spec_of(written[e.cache_from])[0] != kv:
                    raise ConfigError(f"layer {e.layer} reads the cache of layer {e.cache_from}, whose keys and values "
                                      "have another shape or window")
        groups: list = []
        layer_group: dict = {}
        states: dict = {}
        for key in sorted(written):
            spec, state = spec_of(written[key])
            if spec is not None:
                for g, group in enumerate(groups):
                    if group.spec == spec:
                        group.layers.append(key)
                        layer_group[key] = g
                        break
                else:
                    groups.append(CacheGroupLayout(spec, [key]))
                    layer_group[key] = len(groups) - 1
            if state is not None:
                states[key] = state
        states.update(beside or {})
        return cls(groups, layer_group, states)

    def bytes_per_token(self, element_size: int) -> int:
        """Bytes of keys and values one token takes over all layers
        (reference: batch.rs:43-46)."""
        return sum((1 if g.spec.values_in_keys else 2) * len(g.layers) * g.spec.kv_heads * g.spec.head_dim * element_size
                   for g in self.groups)

    def blocks_within(self, budget_bytes: int, block_size: int, element_size: int) -> int:
        """Pages a byte budget holds, at least one (reference: batch.rs:54-57)."""
        per_block = block_size * self.bytes_per_token(element_size)
        return max(budget_bytes // max(per_block, 1), 1)
