"""Configurations, model folders and comparisons for the tests of the Nikonex design."""

from __future__ import annotations

import copy
import json
import random
from pathlib import Path

import torch

import plain_nikonex as plain


def rotation(dims, base=10000.0, ramp=None):
    rot = {"dims": dims, "base": base}
    if ramp is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), ramp))
    return rot


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, window=None, base=10000.0, ramp=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
         "rot": rotation(rot_dim, base, ramp)}
    if window is not None:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def retention(heads, dim, vdim, decay, turned=None, base=10000.0, mlp=None):
    assert len(decay) == heads
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay),
                                           "rot": rotation(dim if turned is None else turned, base)}, "mlp": mlp}


def moe(experts, top, ff, shared=None, groups=None, scale=1.0):
    router = {"experts": experts, "top": top, "scale": scale}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared is not None:
        mlp["shared"] = {"ff": shared}
    return mlp


def model(width, vocab, layers, eps=1e-6, mult=0.6):
    return {"architecture": "Nikonex", "layers": layers, "norm": {"eps": eps}, "residual_mult": mult, "vocab": vocab, "width": width}


# Odd sizes: windows inside a page and across page borders, a rotated part smaller and larger than the rest of a head,
# latents whose rows are no multiple of 16, a rotation over part of a retention head, value heads larger and smaller than key
# heads, decays from a token to thousands, shared experts narrower and wider than the others, groups of three of which
# one and two are kept, layers without a feed-forward, without groups and without a shared expert.
ODD = model(72, 211, [
    retention(3, 24, 40, [0.4, 0.93, 0.9995], base=500.0, mlp=moe(6, 2, 24, shared=40, groups=(2, 1), scale=1.7)),
    latent(5, 24, 8, 40, 44, 28, 0.25, window=9, ramp=(4.0, 64.0, 6.0, 1.0), base=300.0, mlp=moe(9, 4, 32, shared=20, groups=(3, 2), scale=2.5)),
    retention(4, 20, 12, [0.8, 0.99, 0.5, 0.999], turned=12, mlp=None),
    latent(3, 16, 24, 20, 36, 40, 0.3, window=37, mlp=moe(5, 3, 40)),
    latent(2, 12, 16, 24, 20, 24, 0.4, ramp=(0.5, 32.0, 3.0, 2.0), base=50.0),
    retention(2, 36, 24, [0.97, 0.9], mlp=moe(4, 1, 24, shared=56)),
], eps=1e-5, mult=0.7)

# What a small model tends to make equal or 1 is different here: one head, one value a head, one pair that turns, one expert of
# one, groups of one expert each, a window of one token, latents of one value beside their rotated part, a multiplier of one
# and a scale of one, a decay of one and one of nothing.
ONES = model(100, 97, [
    latent(1, 16, 2, 1, 8, 1, 1.0, window=1, mlp=moe(1, 1, 48, shared=8)),
    retention(1, 2, 1, [0.9], mlp=moe(4, 2, 24, groups=(4, 3), scale=0.5)),
    latent(4, 1, 4, 16, 1, 16, 0.5, window=3, ramp=(8.0, 16.0, 2.0, 1.0)),
    retention(3, 16, 17, [1.0, 0.5, 0.0], turned=2, mlp=moe(3, 3, 40, shared=24, groups=(1, 1))),
    retention(1, 40, 4, [1.0]),
], eps=1e-6, mult=1.0)

# Larger sizes: widths that the grouped products on the matrix cores take, sixteen heads over one key row of 256 values, states
# of 128 by 160, eight query heads and more (the grouped attention kernel), windows across tiles of keys.
PLAIN = model(256, 300, [
    latent(16, 64, 64, 96, 160, 192, 0.1, window=90, ramp=(8.0, 512.0, 16.0, 1.0), mlp=moe(8, 3, 64, shared=128, groups=(4, 2), scale=2.0)),
    retention(4, 128, 160, [0.96, 0.99, 0.995, 0.9999], mlp=moe(8, 2, 96, shared=64, groups=(4, 2), scale=1.5)),
    latent(8, 32, 64, 64, 96, 64, 0.15, mlp=moe(4, 2, 160, shared=32)),
    retention(6, 64, 64, [0.5, 0.9, 0.95, 0.98, 0.999, 0.9], turned=32, mlp=moe(6, 2, 32, shared=96, groups=(2, 1))),
], eps=1e-6, mult=0.5)

# Rows beyond what the matrix-core attention kernels take (288), head sizes that are no multiple of 4, a width that is a
# multiple of 4 only, a state of 150 rows by 70 columns, experts whose width is no multiple of 8.
UNEVEN = model(52, 75, [
    latent(2, 30, 32, 22, 18, 256, 0.2, window=50, mlp=moe(3, 2, 44, shared=12, scale=3.0)),
    retention(2, 150, 70, [0.98, 0.995], turned=100, mlp=moe(4, 2, 12, groups=(2, 2))),
    latent(3, 22, 10, 30, 22, 30, 0.3, window=17, ramp=(2.0, 100.0, 8.0, 4.0)),
    retention(5, 22, 10, [0.7, 0.9, 0.99, 0.95, 0.999], mlp=moe(5, 2, 20, shared=36)),
], eps=3e-6, mult=0.8)

CONFIGS = {"odd": ODD, "ones": ONES, "plain": PLAIN, "uneven": UNEVEN}


def telling(tensors) -> None:
    """Tensors as drawn would hide faults: routers without a clear order (a close call between two experts may fall
    either way under rounding), an embedding that the first sublayer drowns, gates of shared experts that are all alike."""
    for name in list(tensors):
        t = tensors[name]
        if name.endswith(".router"):
            out = t.float() * 3
        elif name.endswith(".sg"):
            out = t.float() * 3
        elif name == "embed":
            out = t.float() * 6
        else:
            continue
        tensors[name] = out.to(t.dtype)


def varied(tensors) -> None:
    """``telling`` without a large embedding: greedy generation then goes from token to token instead of giving one for ever."""
    small = tensors["embed"]
    telling(tensors)
    tensors["embed"] = small


def write_model(folder, config, seed=0, dtype="float32", std=0.12, gain_std=0.2, edit=telling) -> Path:
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
    every norm gives is disturbed by up to 2^-8 of itself, as rounding to bfloat16 does (root mean square over the
    vocabulary; the largest of several disturbances).  Random models have single positions where rounding is amplified many
    times: a head's read-out that all but cancels and that the norm behind it blows up again (the first token's is
    (q . k) v, of which the norm leaves the sign of q . k), a score near a tie, a router's close call.  A bound on an engine's error
    there has to grow with it."""
    config, weights = load_plain(folder)
    out = {}
    real = plain.rms
    for name, tokens in prompts.items():
        base = plain.forward(config, weights, tokens)
        factor = torch.ones(len(tokens), dtype=torch.float64)
        for sample in range(6):
            g = torch.Generator().manual_seed(1234 + sample)

            def shaken(x, eps):
                rows = real(x, eps)
                return rows * (1 + (torch.rand(rows.shape, generator=g, dtype=rows.dtype) - 0.5) * 2.0 ** -7)

            plain.rms = shaken
            try:
                moved = ((plain.forward(config, weights, tokens) - base) ** 2).mean(-1).sqrt()
            finally:
                plain.rms = real
            factor = torch.maximum(factor, moved / (2 * moved.median()))
        out[name] = factor
    return out


def close_calls(folder, prompts: dict, dtype: str) -> dict:
    """name -> a mask a position: whether some router's choice at this position, or its choice of groups, falls the other way
    when what every norm gives is disturbed by what rounding to ``dtype`` may amount to (several disturbances), or is decided by
    next to nothing anyway.  The position's logits then are another function's."""
    config, weights = load_plain(folder)
    size, margin, samples = {"float32": (2.0 ** -19, 1e-5, 2), "bfloat16": (2.0 ** -6, 1e-3, 8)}[dtype]
    real_rms, real_route = plain.rms, plain.route
    out = {}
    for name, tokens in prompts.items():
        chosen, close = [], torch.zeros(len(tokens), dtype=torch.bool)

        def noted(h, w, p, router):
            got = real_route(h, w, p, router)
            score = torch.sigmoid(h @ w[p + "router"].T)
            kept = plain.candidates(score, router)
            chosen.append((got[0].sort(-1).values, kept.isinf()))
            if router["top"] < router["experts"]:
                best = kept.topk(router["top"] + 1, -1).values
                close.logical_or_(best[:, -2] - best[:, -1] < margin)
            return got

        plain.route = noted
        try:
            plain.forward(config, weights, tokens)
            first = list(chosen)
            for sample in range(samples):
                g = torch.Generator().manual_seed(4321 + sample)
                plain.rms = lambda x, eps: (lambda rows: rows * (1 + (torch.rand(rows.shape, generator=g, dtype=rows.dtype) - 0.5) * size))(real_rms(x, eps))
                chosen.clear()
                plain.forward(config, weights, tokens)
                for (a, b), (c, d) in zip(first, chosen):
                    close |= (a != c).any(-1) | (b != d).any(-1)
        finally:
            plain.rms, plain.route = real_rms, real_route
        out[name] = close
    return out


def drawn_config(seed: int) -> dict:
    """A configuration drawn from the sizes and constants a model of the design may have: any order of layers, head counts
    from 1 to 16, heads from 8 to 128, latents from 16 to 224 values, windows from 3 to beyond the prompts or none, ramps or none,
    rotations over all or part of a head, decays from 0.3 to 0.9999, experts with and without groups and a shared expert, or none."""
    rng = random.Random(seed)
    width = rng.choice([64, 96, 128, 192, 200])

    def feed_forward():
        if rng.random() < 0.2:
            return None
        groups, each = rng.choice([(1, 5), (1, 8), (2, 4), (4, 2), (3, 3), (5, 1)])
        keep = rng.randint(1, groups)
        return moe(groups * each, rng.randint(1, min(keep * each, 4)), rng.choice([16, 40, 64]), shared=rng.choice([None, 24, 64, 96]),
                   groups=(groups, keep) if groups > 1 or rng.random() < 0.3 else None, scale=rng.choice([1.0, 0.7, 2.5]))

    layers = []
    for _ in range(rng.randint(3, 6)):
        if rng.random() < 0.5:
            heads, dim = rng.choice([1, 2, 3, 4, 8]), rng.choice([8, 16, 24, 48, 64, 96, 128])
            layers.append(retention(heads, dim, rng.choice([8, 16, 18, 64, 80, 130]), [1.0 - rng.choice([0.7, 0.1, 0.02, 0.001, 0.0001]) for _ in range(heads)],
                                    turned=rng.choice([dim, dim, dim // 2 // 2 * 2]), base=rng.choice([100.0, 10000.0, 1000000.0]), mlp=feed_forward()))
        else:
            dim, rot = rng.choice([8, 16, 32, 64]), rng.choice([4, 8, 16, 32, 64])
            ramp = rng.choice([None, (rng.choice([2.0, 8.0]), rng.choice([64.0, 256.0, 2048.0]), rng.choice([32.0, 8.0]), rng.choice([1.0, 2.0]))])
            layers.append(latent(rng.choice([1, 2, 3, 4, 8, 12, 16]), dim, rot, rng.choice([8, 24, 40, 64]), rng.choice([16, 40, 64, 100]),
                                 rng.choice([16, 40, 64, 128, 160]), rng.choice([0.5, 1.0, 2.0]) * (dim + rot) ** -0.5,
                                 window=rng.choice([None, 3, 20, 48, 70, 100, 500]), base=rng.choice([100.0, 10000.0, 1000000.0]), ramp=ramp,
                                 mlp=feed_forward()))
    return model(width, rng.choice([101, 256, 333]), layers, eps=rng.choice([1e-6, 1e-5]), mult=rng.choice([0.4, 0.8, 1.0]))
