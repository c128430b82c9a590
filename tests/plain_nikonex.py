"""A plain, slow implementation of the Nikonex design: whole sequences, no cache, no batches, one
function a mechanism, 64-bit arithmetic.  It shares no code with the package; the tests hold the
engine against it.

``config`` is the dict of a config.json; ``w`` maps tensor names to 64-bit tensors.

A layer is parallel with one multiplier: x <- x + m (mixer(norm1(x)) + ff(norm2(x))), both of the same x.
Two mixers: ``latent_attention`` (queries through a normed latent of their own, keys and values rebuilt from
one normed latent a token, a rotated key part that the heads share, frequencies blended by a ramp over the
pairs, a sliding window) and ``retention`` (a matrix of state a head that decays by a fixed factor a
token, rotated queries and keys, every head's read-out divided by its root mean square, a silu gate).  A
feed-forward is a set of experts of two matrices with the squared relu behind a sigmoid router with groups of
neighbouring experts, beside one shared expert with a sigmoid gate a token.
"""

from __future__ import annotations

import math

import torch

F = torch.float64


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def relu_squared(z):
    return torch.clamp(z, min=0.0) ** 2


def frequencies(rot):
    """(the frequency of every pair, what cosine and sine are multiplied by)."""
    dims, base = rot["dims"], rot["base"]
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return plain, 1.0

    def pair_that_turns(times):
        """The (fractional) pair that makes ``times`` turns over the original length."""
        return dims * math.log(s["original"] / (2.0 * math.pi * times)) / (2.0 * math.log(base))

    low = max(math.floor(pair_that_turns(s["fast"])), 0)
    high = min(math.ceil(pair_that_turns(s["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        ramp = min(max((i - low) / max(high - low, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def turns(positions, rot, axes):
    """cos and sin [T, 1, ..., dims / 2] for a tensor of ``axes`` axes."""
    f, amplitude = frequencies(rot)
    angle = positions.to(F)[:, None] * torch.tensor(f, dtype=F)[None, :]
    while angle.dim() < axes:
        angle = angle.unsqueeze(1)
    return angle.cos() * amplitude, angle.sin() * amplitude


def rotate_neighbours(x, positions, rot):
    """x [T, ..., n]: of the first ``dims`` values, value 2i turns with value 2i + 1."""
    dims = rot["dims"]
    cos, sin = turns(positions, rot, x.dim())
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    turned = torch.stack([u * cos - v * sin, v * cos + u * sin], -1).flatten(-2)
    return torch.cat([turned, x[..., dims:]], -1)


def rotate_halves(x, positions, rot):
    """x [T, ..., n]: of the first ``dims`` values, value i turns with value i + dims / 2."""
    dims = rot["dims"]
    cos, sin = turns(positions, rot, x.dim())
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], -1)


def visible_keys(positions, mask):
    """[i, j]: j <= i and, under a window, i - j < size."""
    distance = positions[:, None] - positions[None, :]
    seen = distance >= 0
    return seen & (distance < mask["size"]) if mask else seen


def softmax_over(score, visible):
    score = score.masked_fill(~visible, -math.inf)
    e = torch.exp(score - score.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def latent_attention_mixer(h, w, p, m, eps, positions):
    T = h.shape[0]
    H, D, rot, V, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    c_q = rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (c_q @ w[p + "uq"].T).view(T, H, D + rot)
    q_plain, q_rot = q[..., :D], rotate_neighbours(q[..., D:], positions, m["rot"])
    both = h @ w[p + "dkv"].T
    c = rms(both[:, :R], eps) * w[p + "dkv.norm"]
    k_rot = rotate_neighbours(both[:, R:], positions, m["rot"])
    k_plain = (c @ w[p + "uk"].T).view(T, H, D)
    v = (c @ w[p + "uv"].T).view(T, H, V)
    visible = visible_keys(positions, m.get("mask"))
    out = torch.zeros(T, H, V, dtype=F)
    for head in range(H):
        score = (q_plain[:, head] @ k_plain[:, head].T + q_rot[:, head] @ k_rot.T) * m["scale"]
        out[:, head] = softmax_over(score, visible) @ v[:, head]
    return out.reshape(T, H * V) @ w[p + "o"].T


def retention_mixer(h, w, p, m, eps, positions):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, D)
    k = (h @ w[p + "k"].T).view(T, H, D)
    v = (h @ w[p + "v"].T).view(T, H, V)
    q = rotate_halves(q, positions, m["rot"])
    k = rotate_halves(k, positions, m["rot"]) * D ** -0.5
    decay = torch.tensor(m["decay"], dtype=F)[:, None, None]
    state = torch.zeros(H, D, V, dtype=F)
    out = torch.zeros(T, H, V, dtype=F)
    for t in range(T):
        state = decay * state + k[t, :, :, None] * v[t, :, None, :]
        out[t] = (state * q[t, :, :, None]).sum(1)
    return (rms(out, eps).reshape(T, H * V) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def mixer(layer, h, w, p, eps, positions):
    if layer["type"] == "latent_attention":
        return latent_attention_mixer(h, w, p, layer["mixer"], eps, positions)
    if layer["type"] == "retention":
        return retention_mixer(h, w, p, layer["mixer"], eps, positions)
    raise ValueError(f"a mixer of type {layer['type']!r}")


def expert(h, w, p):
    return relu_squared(h @ w[p + "up"].T) @ w[p + "down"].T


def candidates(score, router):
    """The scores of the experts that can be chosen, minus infinity at the others."""
    groups = router.get("groups")
    if not groups:
        return score
    parts = score.view(score.shape[0], groups["count"], -1)
    worth = parts.topk(min(2, parts.shape[-1]), -1).values.sum(-1)
    kept = torch.zeros_like(worth, dtype=torch.bool).scatter_(1, worth.topk(groups["keep"], -1).indices, True)
    return score.masked_fill(~kept.repeat_interleave(parts.shape[-1], 1), -math.inf)


def route(h, w, p, router):
    """(chosen [T, top], weights [T, top])."""
    score = torch.sigmoid(h @ w[p + "router"].T)
    chosen = candidates(score, router).topk(router["top"], -1).indices
    weight = score.gather(1, chosen)
    return chosen, weight / (weight.sum(-1, keepdim=True) + 1e-20) * router.get("scale", 1.0)


def feed_forward(h, w, p, mlp):
    chosen, weight = route(h, w, p, mlp["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(chosen[t].tolist(), weight[t]):
            out[t] += g * expert(h[t:t + 1], w, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * expert(h, w, p + "shared.")
    return out


def forward(config, w, tokens, streams=None):
    """Logits [T, vocab] of one whole sequence.  ``streams``: a list that receives the stream after every layer."""
    eps = config["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(len(tokens))
    x = w["embed"][tokens]
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        y = mixer(layer, rms(x, eps) * w[p + "norm1"], w, p + "mix.", eps, positions)
        if layer.get("mlp") is not None:
            y = y + feed_forward(rms(x, eps) * w[p + "norm2"], w, p + "mlp.", layer["mlp"])
        x = x + config["residual_mult"] * y
        if streams is not None:
            streams.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T
