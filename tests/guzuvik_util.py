"""Configurations, model folders and comparisons for the tests of the Guzuvik design."""

from __future__ import annotations

import copy
import json
import random
from pathlib import Path

import torch

import plain_guzuvik as plain


def attention(heads, kv_heads, dim, vdim, scale, window=None, keep=None, cap=None, mix=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window is not None:
        m["mask"] = {"size": window}
        if keep is not None:
            m["mask"]["keep_first"] = keep
    if cap is not None:
        m["softcap"] = cap
    if mix is not None:
        m["v_mix"] = mix
    return {"type": "attention", "mixer": m, "mlp": mlp}


def mamba(heads, vdim, state, groups=1, conv=4, parts=1, mlp=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": parts}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def model(width, vocab, layers, eps=1e-6, bigram=None):
    config = {"architecture": "Guzuvik", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if bigram is not None:
        config["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}
    return config


# Odd sizes: query and value heads of different sizes either way round, three query heads a key head, windows of 9 and 37
# (inside a page, across page borders) that keep 3 and 21 first tokens (inside a page, across a page border), caps that
# bite, a mixing layer first in the list and others behind layers that do not mix, three groups of B and C, convolutions
# of 3 and 5 taps, norms in 2 and 4 parts, a layer without a feed-forward.
ODD = model(72, 211, [
    attention(6, 2, 24, 40, 0.3, window=9, keep=3, cap=3.0, mix=True, mlp=moe(7, 3, 24, 1.5)),
    mamba(6, 12, 20, groups=3, conv=3, parts=2, mlp=dense(96)),
    mamba(5, 24, 8, groups=1, conv=5, parts=4),
    attention(4, 4, 40, 20, 0.25, window=37, keep=21, mix=True, mlp=dense(40)),
    attention(3, 1, 16, 16, 0.4, cap=2.0, mlp=moe(4, 2, 40, 0.7)),
    mamba(4, 20, 36, groups=2, conv=4, parts=8, mlp=moe(3, 3, 16, 7.0)),
    attention(8, 2, 16, 40, 0.2, window=20, keep=5, cap=8.0, mix=True),
], eps=1e-5, bigram=(101, 31, 5))

# What a small model tends to make equal or 1 is different here: one head, one value a head, a state of one row, a
# convolution of one tap, one expert of one, a window of one token that keeps one, a window that keeps none, more kept tokens than the
# window has, a scale of one, no second embedding, a mixing layer that is the only one.
ONES = model(100, 97, [
    mamba(1, 17, 1, conv=1, mlp=moe(1, 1, 48, 0.5)),
    attention(1, 1, 16, 16, 1.0, window=1, keep=1, cap=1.0, mix=True),
    mamba(3, 1, 5, groups=3, conv=2, parts=3, mlp=dense(32)),
    attention(4, 1, 16, 48, 0.5, window=3, keep=0, mix=False, mlp=dense(24)),
    attention(2, 2, 48, 16, 0.3, window=2, keep=30, mlp=moe(3, 1, 40, 2.0)),
    mamba(1, 40, 16, conv=4),
], eps=1e-6)

# Larger sizes: states of 128 rows, heads of 128 and 64 under eight and sixteen query heads a key head (the grouped
# kernel), windows that keep more than a tile of keys, a window with a cap alone, expert widths and a width that the grouped
# products on the matrix cores take, a norm over all heads at once.
PLAIN = model(256, 300, [
    mamba(4, 64, 128, groups=2, conv=4, parts=2, mlp=dense(352)),
    attention(16, 1, 128, 64, 0.1, window=90, keep=16, cap=4.0, mix=True, mlp=moe(8, 2, 64, 3.0)),
    attention(8, 1, 64, 64, 0.15, window=40, keep=70, cap=5.0, mlp=dense(256)),
    mamba(8, 96, 64, groups=1, conv=4, parts=1, mlp=moe(16, 4, 128, 1.0)),
    attention(4, 2, 64, 32, 0.15, window=100, keep=4, cap=6.0, mix=True, mlp=moe(4, 4, 64, 2.0)),
    attention(4, 1, 32, 64, 0.2, mix=True),
], eps=1e-6, bigram=(1009, 263, 11))

# Heads beyond what the matrix-core kernels take (272), head sizes that are no multiple of 4 (30, 22), a width that is a
# multiple of 4 only, a state of 150 rows by 70 columns, 16 taps, experts whose width is no multiple of 8, buckets of one.
UNEVEN = model(52, 75, [
    attention(2, 1, 272, 20, 0.1, window=50, keep=2, cap=2.5, mix=True, mlp=moe(3, 2, 44, 1.1)),
    mamba(2, 70, 150, groups=1, conv=16, parts=7, mlp=dense(44)),
    attention(3, 1, 30, 20, 0.3, window=17, keep=16, cap=4.0, mix=True, mlp=moe(5, 2, 12, 0.9)),
    mamba(6, 10, 22, groups=2, conv=2, parts=5),
    attention(2, 2, 22, 30, 0.3, window=64, keep=17),
], eps=3e-6, bigram=(1, 3, 4))

CONFIGS = {"odd": ODD, "ones": ONES, "plain": PLAIN, "uneven": UNEVEN}


def telling(tensors) -> None:
    """Tensors as drawn would hide faults: biases near zero, gains near one, decays and step sizes that are all alike,
    routers without a clear order, an embedding that the first sublayer drowns.  Biases as large as what they are added
    to; decays from a token or two to hundreds; step sizes from small to above one; router logits with a clear order (a close
    call between two experts may fall either way under rounding)."""
    for name in list(tensors):
        t = tensors[name]
        if name.endswith(".A_log"):
            out = t.float() * 20
        elif name.endswith(".dt_bias"):
            out = t.float() * 15 - 1.0
        elif name.endswith(".D"):
            out = 1.0 + (t.float() - 1.0) * 4
        elif name.endswith(".b"):
            out = t.float() * 6
        elif name.endswith(".router"):
            out = t.float() * 4
        elif name.endswith(".g"):
            out = t.float() * 2
        elif name in ("embed", "bigram"):
            out = t.float() * 6
        else:
            continue
        tensors[name] = out.to(t.dtype)


def varied(tensors) -> None:
    """``telling`` without what drowns the rest in the logits (a large embedding, large biases of the norms): greedy
    generation then goes from token to token instead of giving one for ever."""
    small = {n: t for n, t in tensors.items() if n in ("embed", "bigram") or ("norm" in n and n.endswith(".b"))}
    telling(tensors)
    tensors.update(small)


def write_model(folder, config, seed=0, dtype="float32", std=0.08, gain_std=0.2, edit=telling) -> Path:
    """A model folder with random weights from the package's random-weights mode; ``edit(tensors)`` changes them."""
    from paged_llm_rs_amd.weights import write_random_model

    folder = write_random_model(Path(folder), copy.deepcopy(config), seed=seed, std=std, gain_std=gain_std, dtype=dtype)
    if edit is not None:
        from safetensors.torch import load_file, save_file

        tensors = load_file(str(folder / "model.safetensors"))
        edit(tensors)
        save_file({k: v.contiguous() for k, v in tensors.items()}, str(folder / "model.safetensors"))
    return folder


def load_plain(folder):
    from safetensors.torch import load_file

    config = json.loads((Path(folder) / "config.json").read_text())
    return config, {k: v.to(torch.float64) for k, v in load_file(str(Path(folder) / "model.safetensors")).items()}


def plain_logits(folder, prompts: dict, config=None) -> dict:
    """``config``: another config.json to read the same weights with (a window one larger, say)."""
    own, weights = load_plain(folder)
    return {name: plain.forward(config or own, weights, tokens) for name, tokens in prompts.items()}


def plain_greedy(folder, prompt, count: int) -> list:
    config, weights = load_plain(folder)
    tokens, out = list(prompt), []
    for _ in range(count):
        nxt = int(plain.forward(config, weights, tokens)[-1].argmax())
        out.append(nxt)
        tokens.append(nxt)
    return out


def sensitivity(folder, prompts: dict) -> dict:
    """name -> a factor a position (>= 1): how much more than the median position this position's logits move when what
    every norm hands on is disturbed by up to 2^-8 of itself, as rounding to bfloat16 does (root mean square over the
    vocabulary; the largest of several disturbances).  Random models have single positions where rounding is amplified many
    times: a score near a tie under a sharp softmax, a part of a read-out whose gate is all but shut and that the norm behind it
    blows up again, a router's close call.  A bound on an engine's error there has to grow with it."""
    config, weights = load_plain(folder)
    out = {}
    real = plain.layer_norm
    for name, tokens in prompts.items():
        base = plain.forward(config, weights, tokens)
        factor = torch.ones(len(tokens), dtype=torch.float64)
        for sample in range(6):
            g = torch.Generator().manual_seed(1234 + sample)

            def shaken(x, gain, bias, eps):
                rows = real(x, gain, bias, eps)
                return rows * (1 + (torch.rand(rows.shape, generator=g, dtype=rows.dtype) - 0.5) * 2.0 ** -7)

            plain.layer_norm = shaken
            try:
                moved = ((plain.forward(config, weights, tokens) - base) ** 2).mean(-1).sqrt()
            finally:
                plain.layer_norm = real
            factor = torch.maximum(factor, moved / (2 * moved.median()))
        out[name] = factor
    return out


def close_calls(folder, prompts: dict, margin: float, factors: dict | None = None) -> dict:
    """name -> a mask a position: whether some router decides this position's experts by a difference of less than
    ``margin`` (times the position's factor of ``sensitivity``, where given) between the last chosen logit and the first
    that is not.  Such a choice may fall the other way under rounding, and the position's logits then are another function's."""
    config, weights = load_plain(folder)
    eps = config["norm"]["eps"]
    out = {}
    for name, tokens in prompts.items():
        real, gaps = plain.route, []

        def watched(h, w, p, router):
            z = h @ w[p + "router"].T + w[p + "router.b"]
            if router["top"] < router["experts"]:
                best = z.topk(router["top"] + 1, -1).values
                gaps.append(best[:, -2] - best[:, -1])
            return real(h, w, p, router)

        plain.route = watched
        try:
            plain.forward(config, weights, tokens)
        finally:
            plain.route = real
        close = torch.zeros(len(tokens), dtype=torch.bool)
        for gap in gaps:
            close |= gap < (margin if factors is None else margin * factors[name])
        out[name] = close
    return out


def drawn_config(seed: int) -> dict:
    """A configuration drawn from the sizes and constants a model of the design may have: any order of layers, head counts
    from 1 to 16, groups of 1 to 8, query and value heads from 8 to 128, windows from 3 to beyond the prompts or none, kept
    tokens from none to more than the window, caps or none, mixing layers or none, states from 4 to 200 rows, 1 to 8 taps,
    dense feed-forwards, experts, or none, with and without the second embedding."""
    rng = random.Random(seed)
    width = rng.choice([64, 96, 128, 192, 200])

    def feed_forward():
        kind = rng.random()
        if kind < 0.2:
            return None
        if kind < 0.5:
            return dense(rng.choice([64, 200]))
        experts = rng.choice([1, 2, 5, 8, 12])
        return moe(experts, rng.randint(1, min(experts, 4)), rng.choice([16, 40, 64]), rng.choice([0.5, 2.0, 7.0]))

    mixed = rng.choice([32, 64, 96])             # the values of every layer that mixes, all key heads together
    layers = []
    for _ in range(rng.randint(3, 6)):
        if rng.random() < 0.5:
            heads = rng.choice([1, 2, 4, 6, 8, 12])
            groups = rng.choice([g for g in (1, 2, 3, 4) if heads % g == 0])
            vdim = rng.choice([8, 16, 24, 64, 80])
            parts = rng.choice([p for p in (1, 2, 4, 5, 8) if (heads * vdim) % p == 0])
            layers.append(mamba(heads, vdim, rng.choice([4, 16, 32, 48, 64, 128, 200]), groups=groups, conv=rng.choice([1, 2, 4, 4, 8]),
                                parts=parts, mlp=feed_forward()))
        else:
            kv_heads, group = rng.choice([1, 2, 4]), rng.choice([1, 2, 4, 8])
            dim = rng.choice([16, 24, 32, 48, 64, 96, 128])
            mix = rng.choice([None, False, True, True])
            vdim = mixed // kv_heads if mix else rng.choice([8, 16, 24, 64, 128])
            window = rng.choice([None, 3, 20, 48, 70, 100, 500])
            keep = rng.choice([None, 0, 1, 4, 17, 64, 80]) if window is not None else None
            layers.append(attention(kv_heads * group, kv_heads, dim, vdim, rng.choice([0.5, 1.0, 2.0]) * dim ** -0.5, window=window,
                                    keep=keep, cap=rng.choice([None, 1.0, 5.0, 30.0]), mix=mix, mlp=feed_forward()))
    bigram = rng.choice([None, (rng.randint(1, 500), rng.randint(1, 1000), rng.randint(1, 1000))])
    return model(width, rng.choice([101, 256, 333]), layers, eps=rng.choice([1e-6, 1e-5]), bigram=bigram)
