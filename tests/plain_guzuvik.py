"""A plain, slow implementation of the Guzuvik design: whole sequences, no cache, no batches, one
function a mechanism, 64-bit arithmetic.  It shares no code with the package; the tests hold the
engine against it.

``config`` is the dict of a config.json; ``w`` maps tensor names to 64-bit tensors.

The embedding of a token is joined by a row chosen by the token and the one before it.  A sublayer
stands between two layer norms (with bias): x <- x + norm1b(mixer(norm1(x))), then
x <- x + norm2b(ff(norm2(x))).  Two mixers: ``mamba2`` (a matrix of state a head whose decay and
step size come from the token, behind a short convolution, the read-out gated and then normed in
parts) and ``attention`` (grouped heads with biases, unit q and k, a soft cap on the scores, a
distance penalty a head, a window that keeps the first tokens, values mixed with those of the first
such layer, a gate a head).  Feed-forwards: dense with the squared relu, or experts with clamped
gates behind a router whose weights are a softmax over the chosen logits.  The output projection is
the embedding table.
"""

from __future__ import annotations

import math

import torch

F = torch.float64


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, gain, bias, eps):
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * gain + bias


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


# ---- embedding ----

def bigram_rows(tokens, table):
    """Row numbers of the second table; a sequence's first token has the row behind the buckets."""
    rows, before = [], None
    for token in tokens.tolist():
        rows.append(table["buckets"] if before is None
                    else (before * table["mul_prev"] + token * table["mul_cur"]) % table["buckets"])
        before = token
    return torch.tensor(rows)


def embed(config, w, tokens):
    table = (config.get("embedding") or {}).get("bigram")
    x = w["embed"][tokens]
    return x if table is None else x + w["bigram"][bigram_rows(tokens, table)]


# ---- the mixer with a state ----

def causal_convolution(u, filters, bias):
    """y[t, c] = sum_k filters[c, k] u[t - taps + 1 + k, c] + bias[c], zeros before the start."""
    taps = filters.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F), u], 0)
    y = sum(filters[:, k] * padded[k:k + u.shape[0]] for k in range(taps))
    return y + bias


def state_space_scan(x, B, C, dt, a_log, D):
    """x [T, H, V], B and C [T, G, N], dt [T, H] (positive): S = e^(-e^a dt) S + dt B x^T, y = S^T C + D x."""
    T, H, V = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, V, dtype=F)
    group = [h // (H // G) for h in range(H)]
    out = torch.zeros(T, H, V, dtype=F)
    for t in range(T):
        decay = torch.exp(-torch.exp(a_log) * dt[t])
        S = decay[:, None, None] * S + dt[t][:, None, None] * B[t][group][:, :, None] * x[t][:, None, :]
        out[t] = (S * C[t][group][:, :, None]).sum(1) + D[:, None] * x[t]
    return out


def norm_in_parts(y, parts, gain, eps):
    return rms(y.view(y.shape[0], parts, -1), eps).reshape(y.shape) * gain


def mamba2_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, V, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    z, xbc, dt = (h @ w[p + "in"].T).split([inner, inner + 2 * G * N, H], -1)
    xbc = silu(causal_convolution(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = xbc.split([inner, G * N, G * N], -1)
    dt = softplus(dt + w[p + "dt_bias"])
    y = state_space_scan(x.view(T, H, V), B.view(T, G, N), C.view(T, G, N), dt, w[p + "A_log"], w[p + "D"])
    y = norm_in_parts(y.reshape(T, inner) * silu(z), m["norm_groups"], w[p + "norm"], eps)
    return y @ w[p + "o"].T


# ---- attention ----

def visible_keys(T, mask):
    """[i, j]: j <= i, and within the window or among the kept first tokens."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if mask:
        seen = seen & ((i - j < mask["size"]) | (j < (mask.get("keep_first") or 0)))
    return seen


def slopes(H):
    return [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]


def capped(score, cap):
    return score if cap is None else cap * torch.tanh(score / cap)


def softmax_over(score, visible):
    score = score.masked_fill(~visible, -math.inf)
    e = torch.exp(score - score.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def mixed_values(v, first, m, lam):
    """``first``: the values of the first layer that mixes, None in that layer."""
    return v if not m.get("v_mix") or first is None else (1 - lam) * v + lam * first


def attention_mixer(h, w, p, m, eps, carried):
    """``carried``: what one pass over a sequence hands from layer to layer (the first mixing layer's values)."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, D), eps)
    k = rms((h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, D), eps)
    v = h @ w[p + "v"].T + w[p + "v.b"]
    first = carried.get("values")
    if m.get("v_mix") and first is None:
        carried["values"] = v
    v = mixed_values(v, first, m, w.get(p + "vmix")).view(T, G, V)
    visible = visible_keys(T, m.get("mask"))
    distance = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(F)
    out = torch.zeros(T, H, V, dtype=F)
    for head in range(H):
        g = head // (H // G)
        score = capped((q[:, head] @ k[:, g].T) * m["scale"], m.get("softcap")) - slopes(H)[head] * distance
        out[:, head] = softmax_over(score, visible) @ v[:, g]
    out = out * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    return out.reshape(T, H * V) @ w[p + "o"].T


# ---- feed-forwards ----

def dense_feed_forward(h, w, p):
    return torch.clamp(h @ w[p + "up"].T, min=0.0) ** 2 @ w[p + "down"].T


def expert(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def route(h, w, p, router):
    """(chosen [T, top], weights [T, top])"""
    z = h @ w[p + "router"].T + w[p + "router.b"]
    best, chosen = z.topk(router["top"], -1)
    return chosen, torch.softmax(best, -1)


def routed_experts(h, w, p, mlp):
    chosen, weight = route(h, w, p, mlp["router"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows, place = (chosen == e).nonzero(as_tuple=True)
        if len(rows):
            out[rows] += weight[rows, place][:, None] * expert(h[rows], w, f"{p}e{e}.", mlp["expert"]["limit"])
    return out


def feed_forward(h, w, p, mlp):
    if mlp["kind"] == "dense":
        return dense_feed_forward(h, w, p)
    if mlp["kind"] == "moe":
        return routed_experts(h, w, p, mlp)
    raise ValueError(f"a feed-forward of kind {mlp['kind']!r}")


# ---- the model ----

def mixer(layer, h, w, p, eps, carried):
    if layer["type"] == "mamba2":
        return mamba2_mixer(h, w, p, layer["mixer"], eps)
    if layer["type"] == "attention":
        return attention_mixer(h, w, p, layer["mixer"], eps, carried)
    raise ValueError(f"a mixer of type {layer['type']!r}")


def forward(config, w, tokens, streams=None):
    """Logits [T, vocab] of one whole sequence.  ``streams``: a list that receives the stream after every layer."""
    eps = config["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x = embed(config, w, tokens)
    carried: dict = {}

    def norm(name, rows):
        return layer_norm(rows, w[name], w[name + ".b"], eps)

    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        x = x + norm(p + "norm1b", mixer(layer, norm(p + "norm1", x), w, p + "mix.", eps, carried))
        if layer.get("mlp") is not None:
            x = x + norm(p + "norm2b", feed_forward(norm(p + "norm2", x), w, p + "mlp.", layer["mlp"]))
        if streams is not None:
            streams.append(x.clone())
    return norm("final.norm", x) @ w["embed"].T
