"""The Nikonex design in the engine against the plain implementation: the new kernels alone (the pass over the stream with
a multiplier and with experts' outputs to add up, the norm of a stretch of columns and the product behind it, retention token by
token and in chunks, a router of sigmoid scores with groups by their best two and a shared expert, experts of two
matrices in every form), every mixer and feed-forward alone, whole prompts, tokens decoded one by one, portions down to two
tokens, mixed batches with pages and slots used again, keys far away under a sharp softmax, keys just inside and just
outside a window (in prompts and while decoding, at page borders), states that reach far, constants that carry
weight, the two sublayers on two streams, the first tokens of a request, long decoding, other sizes, and greedy
generation through the engine's own entry point and the command line."""

from __future__ import annotations

import copy
import json
import random
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import nikonex_util as nu
import replay_util as ru

pytestmark = pytest.mark.gpu

# Against the plain implementation (64-bit): 32-bit runs are held tightly.  In bfloat16 a run gets a loose bound there
# and a tight one against the engine's own whole-prompt run of the same requests (the same roundings; what differs
# between schedules is the cache and the batch: a lost key shows there in full).  All bounds are for a position that
# amplifies rounding as the median position does, and grow with a position's own amplification.  A position at which a
# router's choice may fall the other way under rounding is left out (`nikonex_util.close_calls`).
TOLERANCE = {"float32": 5e-5, "bfloat16": 0.1}
BETWEEN_SCHEDULES = 4e-2
DTYPES = ["float32", "bfloat16"]
F = torch.float64


def replayer(folder, dtype, prompts, live=4, block_size=16, graphs=True):
    from paged_llm_rs_amd.engine.replay import Replayer

    return Replayer(folder, dtype, max_tokens=ru.pool_tokens(prompts, live), block_size=block_size, max_live=live,
                    graphs=graphs)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name, dtype):
        if (name, dtype) not in made:
            made[name, dtype] = nu.write_model(tmp_path_factory.mktemp(f"nikonex_{name}_{dtype}"), nu.CONFIGS[name],
                                               seed=sorted(nu.CONFIGS).index(name) + 1, dtype=dtype)
        return made[name, dtype]
    return get


_whole: dict = {}
_factor: dict = {}
_plain: dict = {}
_close: dict = {}


def check(folder, dtype, prompts, steps, live=4, block_size=16, tolerance=None, between=BETWEEN_SCHEDULES, most_close=0.5):
    r = replayer(folder, dtype, prompts, live, block_size)
    got = ru.collect(r, steps)
    key = (str(folder), repr(sorted(prompts.items())))
    if key not in _plain:
        _plain[key] = nu.plain_logits(folder, prompts)
        _factor[key] = nu.sensitivity(folder, prompts)
    if (key, dtype) not in _close:
        _close[key, dtype] = nu.close_calls(folder, prompts, dtype)
    want, factor, close = _plain[key], _factor[key], _close[key, dtype]
    compared = {k: row for k, row in got.items() if not bool(close[k[0]][k[1]])}
    assert len(compared) >= (1 - most_close) * len(got), f"{len(got) - len(compared)} of {len(got)} positions are close calls of a router"
    scale = max(float(want[n][p].abs().max()) for (n, p) in got)
    bound = tolerance or TOLERANCE[dtype]
    worst = {}
    for (n, p), row in compared.items():
        ref = want[n][p].numpy()
        assert row.shape == ref.shape
        err = float(np.abs(row.astype(np.float64) - ref).max()) / scale
        if not err <= bound * float(factor[n][p]):
            worst[n, p] = err / (bound * float(factor[n][p]))
    # (in bfloat16 another token's close call may reach a position through what layers carry)
    spare = 0 if dtype == "float32" else max(1, len(got) // 50)
    assert len(worst) <= spare and all(x <= 4.0 for x in worst.values()), \
        f"over the bound by {sorted(worst.items(), key=lambda x: -x[1])[:5]} of {len(got)}"
    assert r.cache.manager.live_sequences == 0, "every request's pages came back"
    if dtype == "bfloat16":
        if key not in _whole:
            _whole[key] = ru.collect(replayer(folder, dtype, prompts, live), ru.whole(prompts))
        spread = float(np.mean([want[n][p].std() for (n, p) in got]))
        over = {}
        for (n, p), row in compared.items():
            gap = float(np.sqrt(np.mean((row - _whole[key][(n, p)]) ** 2))) / spread
            # (behind a close call that fell the other way, states and pages hold that token as another function made it)
            most = between * float(factor[n][p]) * (3 if bool(close[n][:p].any()) else 1)
            if not gap <= most:
                over[n, p] = gap / most
        assert len(over) <= max(1, len(got) // 50) and all(x <= 3.0 for x in over.values()), \
            f"between this schedule and the whole prompt, over the bound by {sorted(over.items(), key=lambda x: -x[1])[:5]} of {len(got)}"
    return r, got


# --- the new kernels alone --------------------------------------------------------------------------------------------

def dev(t, dtype=torch.float32):
    return t.to(dtype).cuda().contiguous()


class Step:
    """What a kernel reads of a step of requests that bring ``counts`` tokens, request i from position ``starts[i]`` on."""

    def __init__(self, counts, starts=None, slots=None, padding=0):
        starts = list(starts or [0] * len(counts))
        counts, slots = list(counts), list(slots if slots is not None else range(len(counts)))
        self.counts = list(counts)
        i32 = lambda x: torch.tensor(x, dtype=torch.int32).cuda()
        positions, seq_of, q_start, at = [], [], [], 0
        for s, (c, first) in enumerate(zip(counts, starts)):
            positions += list(range(first, first + c))
            seq_of += [s] * c
            q_start.append(at)
            at += c
        if padding:
            positions += [-1] * padding
            seq_of += [len(counts)] * padding
            counts, slots, q_start = counts + [padding], slots + [-1], q_start + [at]
        self.positions, self.seq_of, self.q_start, self.q_len = i32(positions), i32(seq_of), i32(q_start), i32(counts)
        self.state_slots = i32(slots)
        self.num_seqs, self.max_q_len = len(counts), max(counts)
        self.token_ids = i32([0] * len(positions))
        self.token_src = self.fed_tokens = None

    def tokens_of_short_requests(self, limit):
        return sum(c for c in self.counts if c < limit)


def close_to(got, want, tol):
    assert torch.isfinite(got).all()
    err = float((got.double().cpu() - want).abs().max()) / max(float(want.abs().max()), 1e-30)
    assert err <= tol, err


@pytest.mark.parametrize("width", [52, 200, 1024, 4100])
def test_the_pass_over_the_stream_with_a_multiplier_and_experts_to_add_up(width):
    from paged_llm_rs_amd import kernels

    g = torch.Generator().manual_seed(width)
    n, top, eps, mult = 23, 3, 1e-5, 0.37
    x, a, b = (torch.randn((n, width), generator=g, dtype=F) * s for s in (3, 1, 2))
    gain1, gain2 = (1 + 0.4 * torch.randn((width,), generator=g, dtype=F) for _ in range(2))
    norm = lambda u, gain: u / torch.sqrt((u * u).mean(-1, keepdim=True) + eps) * gain
    for dtype, tol in ((torch.float32, 2e-6), (torch.bfloat16, 8e-3)):
        stream = dev(x)
        rows1, rows2 = kernels.parallel_step(stream, a=dev(a), b=dev(b), mult=mult, gain1=dev(gain1), gain2=dev(gain2), eps=eps, out_dtype=dtype)
        close_to(stream, x + mult * (a + b), 2e-6)
        close_to(rows1, norm(x + mult * (a + b), gain1), tol)
        close_to(rows2, norm(x + mult * (a + b), gain2), tol)
    choice = torch.randint(0, 5, (n, top), generator=g).to(torch.int32)
    choice[4] = -1                                                    # (a row of padding)
    weight = torch.rand((n, top), generator=g)
    positions = torch.arange(n, dtype=torch.int32)
    positions[4] = -1
    for splits, dealt in ((1, False), (1, True), (3, True)):
        slots = torch.randperm(n * top + 40, generator=g)[:n * top].view(n, top).to(torch.int32) if dealt else torch.arange(n * top).view(n, top)
        y = torch.randn((splits, n * top + 40, width), generator=g)
        per_pair = y.double().sum(0)[slots.long()]                    # [n, top, width]
        per_pair[4] = 0
        if dealt:
            slots[4] = -1
        want = (per_pair * weight.double()[..., None]).sum(1)
        sums = kernels.ExpertSums(dev(y), dev(slots, torch.int32) if dealt else None, choice.cuda(), dev(weight), n, top, splits, dev(x), 5, 0, positions.cuda())
        close_to(sums.total(), want, 3e-6)
        stream = dev(x)
        rows1, rows2 = kernels.parallel_step(stream, a=dev(a), b=sums, mult=mult, gain1=dev(gain1), eps=eps)
        close_to(stream, x + mult * (a + want), 2e-6)
        close_to(rows1, norm(x + mult * (a + want), gain1), 3e-6)
        ls = 1 + 0.3 * torch.randn((width,), generator=g, dtype=F)
        assert rows2 is None and kernels.parallel_step(stream, b=sums, ls2=dev(ls)) == (None, None)
        close_to(stream, x + mult * (a + want) + want * ls, 3e-6)


@pytest.mark.parametrize("width,off,stride", [(44, 0, 72), (96, 4, 160), (512, 0, 768), (1536, 8, 1600), (3000, 0, 3004), (18, 3, 77)])
def test_the_norm_of_a_stretch_of_columns_and_the_product_behind_it(width, off, stride):
    from paged_llm_rs_amd import kernels

    g = torch.Generator().manual_seed(width)
    eps = 1e-5
    rows = torch.randn((40, stride), generator=g) * torch.rand((40, 1), generator=g) * 5
    gain = 1 + 0.3 * torch.randn((width,), generator=g)
    part = rows[:, off:off + width].double()
    want = part / torch.sqrt((part * part).mean(-1, keepdim=True) + eps) * gain.double()
    for dtype, tol in ((torch.float32, 2e-6), (torch.bfloat16, 8e-3)):
        got = kernels.rows_norm(dev(rows), off, dev(gain), eps, dtype)
        assert got.dtype == dtype
        close_to(got, want, tol)
    if width % 8 == 0 and off % 4 == 0 and stride % 4 == 0 and width <= kernels.FUSED_NORM_MAX_WIDTH:
        w = (torch.randn((200, width), generator=g) * width ** -0.5).bfloat16()
        for n in (1, 5, 16, 17, 32):
            got = kernels.gemm_skinny(dev(rows[:n]), w.cuda(), torch.float32, norm_gain=dev(gain), eps=eps, columns=(off, width))
            close_to(got, want[:n] @ w.double().T, 1e-2)


def test_the_norm_of_a_head_without_a_gain():
    from paged_llm_rs_amd import kernels

    g = torch.Generator().manual_seed(3)
    for n, group, groups in ((9, 40, 3), (5, 17, 2), (4, 600, 2), (3, 2500, 1), (6, 1, 5)):
        x = torch.randn((n, group * groups), generator=g) * 2
        gate = torch.randn((n, group * groups + 7), generator=g)
        part = x.double().view(n, groups, group)
        want = (part / torch.sqrt((part * part).mean(-1, keepdim=True) + 1e-5)).view(n, -1)
        z = gate[:, 7:].double()
        want = want * z * torch.sigmoid(z)
        for dtype, tol in ((torch.float32, 3e-6), (torch.bfloat16, 8e-3)):
            got = kernels.gated_group_norm(dev(x), group, None, 1e-5, dtype, gate=dev(gate), gate_off=7, gate_act="silu")
            close_to(got, want, tol)


def _retention64(q, k, v, decay, freq, amplitude, k_scale, positions, state):
    """Token by token in 64-bit: read-out [T, H, V]; ``state`` [H, D, V] is moved on."""
    half = len(freq)
    angle = positions.double()[:, None] * freq.double()[None, :]
    cos, sin = (angle.cos() * amplitude)[:, None, :], (angle.sin() * amplitude)[:, None, :]

    def turn(x):
        u, w = x[..., :half], x[..., half:2 * half]
        return torch.cat([u * cos - w * sin, w * cos + u * sin, x[..., 2 * half:]], -1)

    q, k = turn(q), turn(k) * k_scale
    out = torch.zeros(q.shape[0], v.shape[1], v.shape[2], dtype=F)
    for t in range(q.shape[0]):
        state.mul_(decay[:, None, None]).add_(k[t, :, :, None] * v[t, :, None, :])
        out[t] = (state * q[t, :, :, None]).sum(1)
    return out


@pytest.mark.parametrize("H,D,V,turned,decay", [(3, 24, 40, 24, "mild"), (2, 128, 160, 64, "mild"), (1, 2, 1, 2, "mild"), (4, 20, 12, 0, "wild"),
                                                (2, 150, 70, 100, "mild"), (5, 33, 64, 32, "wild"), (2, 256, 68, 256, "mild"), (3, 16, 17, 2, "none")])
def test_retention_over_steps_of_every_kind(H, D, V, turned, decay):
    """Long and short portions and single tokens side by side, from and into slots, against a loop over tokens in 64-bit;
    decays near one, from nothing to one beside each other, and (``none``) of zero, which keeps a layer out of chunks; padding rows; slots
    that nobody names stay."""
    from paged_llm_rs_amd import kernels

    g = torch.Generator().manual_seed(H * 1000 + D)
    decays = {"mild": torch.linspace(0.9, 0.9999, H), "wild": torch.tensor([1.0, 0.9, 1e-4, 0.5, 1e-20])[:H], "none": torch.tensor([0.0, 1.0, 0.5])[:H]}[decay]
    freq = torch.tensor([50.0 ** (-2.0 * i / max(turned, 2)) for i in range(turned // 2)]).float()
    amplitude, k_scale = 1.2, D ** -0.5
    for counts, starts in (([70, 3, 1, 200, 16, 15], [0, 5, 40, 64, 7, 0]), ([1, 1, 1], [0, 9, 700]), ([5, 2, 15], [3, 0, 100]), ([129], [10])):
        slots = [4, 0, 6, 2, 5, 3][:len(counts)]
        n = sum(counts)
        b = Step(counts, starts, slots, padding=3)
        off = 5 if V % 2 else 4
        width = off + H * (2 * D + V) + 3
        rows = torch.randn((n + 3, width), generator=g)
        rows[n:] = 0
        state = torch.randn((8, H * D * V), generator=g)
        on_gpu = dev(state)
        got = kernels.retention_scan(dev(rows), off, off + H * D, off + 2 * H * D, on_gpu, b, H, D, V, dev(decays), dev(freq) if turned else None,
                                     amplitude if turned else 1.0, k_scale, chunked=decay != "none")
        after, at = state.double().clone(), 0
        q, k, v = (rows[:, off + s:off + e].double().view(n + 3, H, -1) for s, e in ((0, H * D), (H * D, 2 * H * D), (2 * H * D, 2 * H * D + H * V)))
        want = torch.zeros((n, H * V), dtype=F)
        for c, first, slot in zip(counts, starts, slots):
            s = after[slot].view(H, D, V)
            want[at:at + c] = _retention64(q[at:at + c], k[at:at + c], v[at:at + c], decays.double(), freq, amplitude, k_scale,
                                           torch.arange(first, first + c), s).reshape(c, -1)
            at += c
        close_to(got[:n], want, 2e-5)
        close_to(on_gpu, after, 2e-5)
        others = [s for s in range(8) if s not in slots]
        assert torch.equal(on_gpu[others].cpu(), state[others]), "other requests' slots stay"


def _route64(z, top, groups, kept, best_of, scale):
    score = torch.sigmoid(z)
    pick = score
    if groups > 1:
        parts = score.view(z.shape[0], groups, -1)
        worth = parts.topk(min(best_of, parts.shape[-1]), -1).values.sum(-1)
        allowed = torch.zeros_like(worth, dtype=torch.bool).scatter_(1, worth.topk(kept, -1).indices, True)
        pick = score.masked_fill(~allowed.repeat_interleave(parts.shape[-1], 1), -1.0)
    chosen = pick.topk(top, -1).indices
    weight = score.gather(1, chosen)
    return chosen, weight / (weight.sum(-1, keepdim=True) + 1e-20) * scale


@pytest.mark.parametrize("total,top,groups,kept", [(10, 3, 5, 2), (9, 4, 3, 2), (1, 1, 1, 1), (4, 2, 4, 3), (64, 6, 8, 3), (256, 8, 8, 4), (300, 5, 10, 2),
                                                   (512, 9, 128, 70), (130, 2, 65, 3)])
@pytest.mark.parametrize("shared", [True, False])
def test_a_router_of_sigmoid_scores(total, top, groups, kept, shared):
    """Experts, their order and weights against 64-bit arithmetic over the same logits: groups by the sum of their two best, weights scaled,
    the shared expert behind the chosen ones with its own gate, rows of padding; and with the logits worked out by the kernel."""
    from paged_llm_rs_amd import kernels

    g = torch.Generator().manual_seed(total * 31 + top)
    n, scale, one = 150, 1.7, 1 if shared else 0
    z = (torch.randn((n, total + one), generator=g) * 2).float()
    positions = torch.arange(n, dtype=torch.int32)
    positions[17] = -1
    rows = [t for t in range(n) if t != 17]
    how = dict(score="sigmoid", group_best=2, scale=scale, shared=shared)

    def compare(chosen, weight, z, few):
        chosen, weight = chosen.cpu(), weight.cpu().double()
        assert chosen.shape == (n, top + one) and (chosen[17] == -1).all() and (weight[17] == 0).all()
        want_c, want_w = _route64(z.double()[:, :total], top, groups, kept, 2, scale)
        same = [t for t in rows if torch.equal(chosen[t, :top].long(), want_c[t])]
        assert len(same) >= len(rows) - few, "the same experts in the same order"
        assert (weight[same, :top] - want_w[same]).abs().max() <= 2e-5
        if shared:
            assert (chosen[rows, top] == total).all()
            assert (weight[rows, top] - torch.sigmoid(z.double()[rows, total])).abs().max() <= 2e-5

    compare(*kernels.router_select(z.cuda(), None, positions.cuda(), top, groups, kept, **how), z, few=1)
    width = 96
    for dtype in (torch.float32, torch.bfloat16):
        if not kernels.router_fuses(n - 30, total + one, width):
            continue
        x = torch.randn((n, width), generator=g).to(dtype)
        w = (torch.randn((total + one, width), generator=g) * 2 * width ** -0.5).to(dtype)
        compare(*kernels.router_select(None, None, positions.cuda(), top, groups, kept, x=x.cuda(), w=w.cuda(), **how), x.double() @ w.double().T, few=4)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,top,ff,size,width,rows,gated", [
    (8, 2, 64, 96, 160, 50, False), (3, 3, 44, 20, 52, 7, False), (1, 1, 32, 64, 96, 1, False), (16, 4, 96, 32, 256, 300, False),
    (4, 2, 160, 0, 512, 64, False), (5, 1, 32, 256, 64, 33, False), (12, 3, 64, 64, 192, 17, True), (6, 2, 128, 0, 96, 64, True),
    (9, 5, 64, 128, 320, 31, True), (40, 4, 32, 64, 64, 5, False), (2, 2, 32, 32, 1024, 64, False), (7, 3, 288, 544, 128, 129, False)])
def test_experts_with_a_shared_one_in_every_form(dtype, experts, top, ff, size, width, rows, gated):
    """A pair at a time, dealt to tiles, and by the kernels of few rows: every row against 64-bit arithmetic over its own chosen
    experts and the shared one, experts of two matrices and of three, pairs without an expert, rows of padding."""
    from paged_llm_rs_amd import kernels

    g = torch.Generator().manual_seed(experts * 100 + rows)
    act = "silu" if gated else "relu2"
    parts = 2 if gated else 1
    make = lambda *s: (torch.randn(s, generator=g) * s[-1] ** -0.5 * 1.3).to(dtype)
    w_first, w_down = make(experts, parts * ff, width), make(experts, width, ff)
    shared = (make(parts * size, width), make(width, size)) if size else None
    x = torch.randn((rows, width), generator=g).to(dtype)
    choice = torch.rand((rows, experts), generator=g).argsort(1)[:, :top].to(torch.int32)
    weight = torch.rand((rows, top), generator=g) + 0.1
    if size:
        choice = torch.cat([choice, torch.full((rows, 1), experts, dtype=torch.int32)], 1)
        weight = torch.cat([weight, torch.rand((rows, 1), generator=g)], 1)
    if rows > 4:
        choice[3, 0] = -1
    b = Step([rows])
    if rows > 2:
        b.positions[rows // 2] = -1
        choice[rows // 2] = -1

    def expert(first, down, v, F_):
        both = first.double() @ v
        h = torch.nn.functional.silu(both[:F_]) * both[F_:] if gated else torch.clamp(both, min=0) ** 2
        if dtype == torch.bfloat16:
            h = h.to(torch.bfloat16).double()            # (what lies between the two products is stored in the rows' type)
        return down.double() @ h

    want = torch.zeros((rows, width), dtype=F)
    for t in range(rows):
        for c, e in enumerate(choice[t].tolist()):
            if e >= 0:
                y = expert(*shared, x[t].double(), size) if e == experts else expert(w_first[e], w_down[e], x[t].double(), ff)
                want[t] += y * float(weight[t, c])
    both = (shared[0].cuda(), shared[1].cuda()) if size else None
    how = dict(choice=choice.cuda(), weight=dev(weight), gated=gated, shared=both)
    tol = 1e-5 if dtype == torch.float32 else 1.5e-2
    got = kernels.moe_rows(x.cuda(), b, None, w_first.cuda(), w_down.cuda(), act, **how)
    close_to(got, want, tol)
    sizes = [s for s in (ff, size) if s]
    if all(kernels.moe_grouped_applies(x.cuda(), width, s, gated) for s in sizes):
        close_to(kernels.moe_grouped(x.cuda(), b, None, w_first.cuda(), w_down.cuda(), act, **how), want, tol)
    if all(kernels.moe_few_applies(x.cuda(), width, s) for s in sizes):
        first = kernels.moe_few(x.cuda(), b, w_first.cuda(), w_down.cuda(), act, **how).total()
        close_to(first, want, tol)
        again = kernels.moe_few(x.cuda(), b, w_first.cuda(), w_down.cuda(), act, **how).total()
        assert torch.equal(first, again), "what a pair gives does not depend on the order in which a workgroup found it"
        if rows > 8:         # ... nor on the other rows of the step
            part = slice(0, rows // 3)
            few = Step([rows // 3])
            few.positions[:] = b.positions[part]
            how.update(choice=choice[part].cuda(), weight=dev(weight[part]))
            close_to(kernels.moe_few(x[part].cuda(), few, w_first.cuda(), w_down.cuda(), act, **how).total(), first[part].double().cpu(), 1e-6)


# --- every mixer and feed-forward alone, in 32-bit, the stream behind the layer against the plain implementation's ----

ALONE = {
    "latent, a window and a ramp": [nu.latent(3, 24, 8, 40, 36, 56, 0.3, window=11, base=300.0, ramp=(4.0, 64.0, 6.0, 1.0))],
    "latent, all keys": [nu.latent(2, 16, 16, 8, 12, 20, 0.4)],
    "latent, one of everything": [nu.latent(1, 1, 2, 1, 1, 1, 1.0, window=2)],
    "retention": [nu.retention(3, 24, 40, [0.5, 0.95, 0.999])],
    "retention, part of a head turns": [nu.retention(2, 30, 16, [0.9, 0.99], turned=14, base=40.0)],
    "retention, one of everything": [nu.retention(1, 2, 1, [0.7])],
    "experts, groups, a shared one": [nu.retention(1, 8, 4, [0.9], mlp=nu.moe(8, 3, 40, shared=56, groups=(4, 2), scale=2.2))],
    "experts alone": [nu.retention(1, 8, 4, [0.9], mlp=nu.moe(6, 2, 24))],
    "one expert": [nu.retention(1, 8, 4, [0.9], mlp=nu.moe(1, 1, 24, shared=8, scale=0.3))],
}


@pytest.mark.parametrize("which", sorted(ALONE))
def test_a_layer_alone_against_its_plain_function(tmp_path, which):
    """32-bit, the stream behind the layer against the plain implementation's: whole, and again in portions (the later
    portions read what the earlier ones left in pages and slots)."""
    layers = ALONE[which]
    config = nu.model(88, 61, layers, eps=1e-5, mult=0.45)
    folder = nu.write_model(tmp_path / "m", config, seed=7, std=0.2)
    tokens = [random.Random(3).randrange(61) for _ in range(45)]
    cfg, weights = nu.load_plain(folder)
    want = []
    nu.plain.forward(cfg, weights, tokens, want)
    r = replayer(folder, "float32", {"a": tokens}, graphs=False)
    rec = {}
    r.step([{"id": "a", "tokens": tokens, "want": []}], ["a"], trace=rec)
    assert (rec["l0.out"].double().cpu() - want[0]).abs().max() <= 5e-5 * want[0].abs().max(), which
    pieces, at = [], 0
    for n in (1, 2, 17, 3, 22):
        rec = {}
        r.step([{"id": "b", "tokens": tokens[at:at + n], "want": []}], ["b"] if at + n == 45 else [], trace=rec)
        pieces.append(rec["l0.out"].double().cpu())
        at += n
    assert (torch.cat(pieces) - want[0]).abs().max() <= 5e-5 * want[0].abs().max(), (which, "in portions")


# --- whole models of other sizes under every schedule ------------------------------------------------------------------

LENGTHS = [70, 3, 41, 18, 1, 33, 57]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(nu.CONFIGS))
def test_whole_prompts(folders, name, dtype):
    prompts = ru.make_prompts(nu.CONFIGS[name]["vocab"], LENGTHS, seed=1)
    check(folders(name, dtype), dtype, prompts, ru.whole(prompts))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(nu.CONFIGS))
def test_prefill_then_tokens_one_by_one(folders, name, dtype):
    prompts = ru.make_prompts(nu.CONFIGS[name]["vocab"], LENGTHS, seed=1)
    check(folders(name, dtype), dtype, prompts, ru.tail_decoded(prompts, tail=40))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(nu.CONFIGS))
@pytest.mark.parametrize("block_size", [16, 8])
def test_portions_down_to_two_tokens(folders, name, dtype, block_size):
    prompts = ru.make_prompts(nu.CONFIGS[name]["vocab"], LENGTHS, seed=1)
    check(folders(name, dtype), dtype, prompts, ru.portions(prompts), block_size=block_size)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(nu.CONFIGS))
@pytest.mark.parametrize("seed", [0, 1])
def test_unequal_requests_together_with_pages_and_slots_used_again(folders, name, dtype, seed):
    """Nine requests of unequal length through a pool and slots for four: portions of some beside single tokens of others,
    requests left out of steps, pages and slots of finished requests taken by the next."""
    prompts = ru.make_prompts(nu.CONFIGS[name]["vocab"], [70, 3, 41, 18, 1, 33, 57, 64, 22], seed=2 + seed)
    check(folders(name, dtype), dtype, prompts, ru.mixed(prompts, seed=seed, max_live=4, tail=14))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", range(12))
def test_drawn_configurations(tmp_path, seed, dtype):
    """Twelve drawn models (order of layers, sizes, head counts, windows, ramps, decays, experts, groups, constants;
    `nikonex_util.drawn_config`) under a mixed schedule and whole, over pages of 16, 8 and 32."""
    config = nu.drawn_config(100 + seed)
    folder = nu.write_model(tmp_path / "m", config, seed=seed, dtype=dtype)
    prompts = ru.make_prompts(config["vocab"], [75, 9, 130, 33, 2], seed=seed)
    block_size = (16, 8, 32)[seed % 3]
    check(folder, dtype, prompts, ru.mixed(prompts, seed=seed, max_live=3, tail=20), live=3, block_size=block_size, most_close=0.6)
    check(folder, dtype, prompts, ru.whole(prompts), live=3, block_size=block_size, most_close=0.6)


def test_schedules_agree_with_each_other_in_32_bit(folders):
    folder = folders("odd", "float32")
    prompts = ru.make_prompts(nu.ODD["vocab"], LENGTHS, seed=1)
    close, factor = nu.close_calls(folder, prompts, "float32"), nu.sensitivity(folder, prompts)
    whole = ru.collect(replayer(folder, "float32", prompts), ru.whole(prompts))
    scale = max(float(np.abs(row).max()) for row in whole.values())
    for steps in (ru.tail_decoded(prompts, tail=40), ru.portions(prompts), ru.mixed(prompts, seed=5)):
        for key, row in ru.collect(replayer(folder, "float32", prompts), steps).items():
            if not bool(close[key[0]][key[1]]):
                assert float(np.abs(row - whole[key]).max()) <= 2e-5 * scale * float(factor[key[0]][key[1]]), key


# --- keys far away, edges of windows, states that reach far ----------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
def test_one_key_among_hundreds_under_a_sharp_softmax(tmp_path, dtype):
    """Scales several times the usual make every softmax sharp: a key lost at a page border, at the edge of a tile of keys
    or between shares of the context moves the logits in full."""
    config = nu.model(64, 90, [nu.latent(8, 24, 16, 32, 40, 48, 0.9, base=1000.0, mlp=nu.moe(4, 2, 32, shared=32)),
                               nu.latent(3, 32, 8, 24, 48, 40, 0.9, window=400, ramp=(4.0, 128.0, 16.0, 1.0)),
                               nu.latent(16, 32, 16, 16, 32, 64, 0.8, window=300)])
    folder = nu.write_model(tmp_path / "m", config, seed=11, dtype=dtype, std=0.2)
    prompts = ru.make_prompts(90, [700, 333], seed=4)
    cfg, w = nu.load_plain(folder)
    # the test's own premise: the first layer's softmaxes are sharp and their heaviest keys lie far back
    m = cfg["layers"][0]["mixer"]
    positions = torch.arange(700)
    x = w["embed"][torch.tensor(prompts["r0"])]
    h = nu.plain.rms(x, 1e-6) * w["l0.norm1"]
    q = (nu.plain.rms(h @ w["l0.mix.dq"].T, 1e-6) * w["l0.mix.dq.norm"] @ w["l0.mix.uq"].T).view(700, 8, 40)
    both = h @ w["l0.mix.dkv"].T
    c = nu.plain.rms(both[:, :48], 1e-6) * w["l0.mix.dkv.norm"]
    k = (c @ w["l0.mix.uk"].T).view(700, 8, 24)
    turned_q, turned_k = nu.plain.rotate_neighbours(q[..., 24:], positions, m["rot"]), nu.plain.rotate_neighbours(both[:, 48:], positions, m["rot"])
    score = (torch.einsum("ihd,jhd->hij", q[..., :24], k) + torch.einsum("ihd,jd->hij", turned_q, turned_k)) * m["scale"]
    score = score.masked_fill(positions[:, None] < positions[None, :], -np.inf)
    far = (positions - score.argmax(-1))[:, 400:]
    assert (far > 100).double().mean() > 0.3 and torch.softmax(score, -1).max(-1).values[:, 400:].median() > 0.25
    steps = ru.tail_decoded(prompts, tail=48)
    for s in steps:            # every seventh position of the long first steps is compared, and every decoded token
        for e in s["entries"]:
            e["want"] = list(range(0, len(e["tokens"]), 7)) + ([len(e["tokens"]) - 1] if (len(e["tokens"]) - 1) % 7 else [])
    loose = 0.5 if dtype == "bfloat16" else 2e-4
    check(folder, dtype, prompts, steps, live=2, tolerance=loose, between=5 * BETWEEN_SCHEDULES, most_close=0.6)
    check(folder, dtype, prompts, ru.portions(prompts, sizes=(130, 2, 61, 16, 17, 300, 5)), live=2, tolerance=loose,
          between=5 * BETWEEN_SCHEDULES, most_close=0.6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 32, 33, 64])
def test_keys_just_inside_and_just_outside_a_window(tmp_path, dtype, window):
    """A layer whose scale is small, so that its softmax is flat and every key it sees carries its share of the
    weight: the engine's logits are the plain implementation's with this size of the window, and clearly not those with a window
    one token larger or smaller, in prompts, in portions and for tokens decoded one by one, with pages of 16 and of 4 tokens
    (edges at a page's border, before it and behind it)."""
    config = nu.model(48, 70, [nu.latent(8, 16, 8, 24, 24, 40, 0.01, window=window, ramp=(4.0, 64.0, 6.0, 1.0))], mult=1.0)

    def edit(tensors):
        nu.telling(tensors)
        tensors["embed"] = tensors["embed"] / 12

    folder = nu.write_model(tmp_path / "m", config, seed=20 + window, dtype=dtype, std=0.25, edit=edit)
    prompts = ru.make_prompts(70, [90, 49], seed=6)
    want = nu.plain_logits(folder, prompts)
    others = []
    for size in (window - 1, window + 1):
        if size >= 1:
            changed = copy.deepcopy(config)
            changed["layers"][0]["mixer"]["mask"]["size"] = size
            others.append(nu.plain_logits(folder, prompts, changed))
    for block_size in (16, 4):
        for steps in (ru.whole(prompts), ru.tail_decoded(prompts, tail=45), ru.portions(prompts, sizes=(18, 2, 15, 33, 3))):
            got = ru.collect(replayer(folder, dtype, prompts, live=2, block_size=block_size), steps)
            closer = total = 0
            for (n, p), row in got.items():
                err = float(np.sqrt(np.mean((row - want[n][p].numpy()) ** 2)))
                for o in others:
                    moved = float(((want[n][p] - o[n][p]) ** 2).mean().sqrt())
                    if moved < (1e-9 if dtype == "float32" else 2e-2) * float(want[n][p].std()):
                        continue          # (a position that sees the same keys under both, or whose difference is next to nothing)
                    total += 1
                    closer += err < (0.25 if dtype == "float32" else 0.5) * moved
            assert closer >= (total if dtype == "float32" else 0.9 * total), (block_size, closer, total)
            assert total > 8, "the edge has to be seen"


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_token_that_a_state_remembers(tmp_path, dtype):
    """Decays near one: changing the first tokens changes the logits hundreds of tokens later, and the engine follows the plain
    implementation there, whatever the schedule; a state that a slot's last owner left would show."""
    config = nu.model(64, 60, [nu.retention(4, 16, 24, [0.999, 0.9995, 0.9999, 1.0], mlp=nu.moe(3, 2, 32, shared=32)),
                               nu.retention(2, 40, 16, [0.9999, 0.998])])
    folder = nu.write_model(tmp_path / "m", config, seed=5, dtype=dtype, std=0.15)
    prompts = ru.make_prompts(60, [400, 150, 31, 260], seed=3)
    cfg, w = nu.load_plain(folder)
    base = nu.plain.forward(cfg, w, prompts["r0"])
    other = nu.plain.forward(cfg, w, [(t + 7) % 60 for t in prompts["r0"][:100]] + prompts["r0"][100:])
    assert float((base - other)[-1].std() / base[-1].std()) > 0.02
    check(folder, dtype, prompts, ru.tail_decoded(prompts, tail=60), live=1)
    check(folder, dtype, prompts, ru.mixed(prompts, seed=3, max_live=2, tail=30), live=2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_constants_and_tensors_that_carry_weight(tmp_path, dtype):
    """The engine agrees with the plain implementation, whose logits move by far more than the engine's error when the ramp, the
    groups, the shared expert's gate, the weights' scale or the multiplier is taken away, a decay or a base changes, or a norm's gain is
    set to one."""
    config = nu.model(64, 80, [nu.latent(8, 16, 16, 24, 40, 32, 0.5, window=20, base=200.0, ramp=(6.0, 64.0, 6.0, 0.5),
                                         mlp=nu.moe(8, 2, 32, shared=64, groups=(4, 1), scale=3.0)),
                               nu.retention(3, 24, 32, [0.9, 0.97, 0.6], base=100.0, mlp=nu.moe(6, 2, 32, shared=32, groups=(3, 2), scale=0.6))],
                      eps=1e-5, mult=0.6)
    folder = nu.write_model(tmp_path / "m", config, seed=31, dtype=dtype, std=0.2)
    prompts = ru.make_prompts(80, [60, 5], seed=8)
    _, got = check(folder, dtype, prompts, ru.tail_decoded(prompts, tail=20), live=2, most_close=0.6)
    cfg, weights = nu.load_plain(folder)
    close = nu.close_calls(folder, prompts, dtype)
    compared = [(n, p) for (n, p) in got if not bool(close[n][p])]
    want = {n: nu.plain.forward(cfg, weights, t) for n, t in prompts.items()}
    err = np.sqrt(np.median([np.mean((got[n, p] - want[n][p].numpy()) ** 2) for (n, p) in compared]))

    def changed(path, value):
        other = copy.deepcopy(cfg)
        at = other
        for key in path[:-1]:
            at = at[key]
        if value is None:
            at.pop(path[-1])
        else:
            at[path[-1]] = value
        return other

    first, second = ["layers", 0], ["layers", 1]
    configs = (changed(first + ["mixer", "rot", "scaling"], None), changed(first + ["mlp", "router", "groups"], None),
               changed(first + ["mlp", "router", "scale"], None), changed(second + ["mlp", "router", "scale"], 1.0),
               changed(first + ["mlp", "shared"], None), changed(["residual_mult"], 1.0), changed(first + ["mixer", "scale"], 0.4),
               changed(first + ["mixer", "rot", "base"], 100.0), changed(second + ["mixer", "decay"], [0.9, 0.9, 0.6]),
               changed(second + ["mixer", "rot", "base"], 400.0), changed(second + ["mixer", "rot", "dims"], 12))
    tensors = tuple((lambda k, v, end=end: torch.ones_like(v) if k.endswith(end) else v)
                    for end in ("dq.norm", "dkv.norm", "norm1", "norm2", "final.norm"))
    tensors += ((lambda k, v: torch.zeros_like(v) if k.endswith(".sg") else v), (lambda k, v: torch.zeros_like(v) if k.endswith(".g") else v))
    moved_all = [{n: nu.plain.forward(c, weights, t) for n, t in prompts.items()} for c in configs]
    moved_all += [{n: nu.plain.forward(cfg, {k: change(k, v) for k, v in weights.items()}, t) for n, t in prompts.items()} for change in tensors]
    for at, moved in enumerate(moved_all):
        part = 0.02 if dtype == "float32" else 0.6
        shift = np.sqrt(np.mean([float(((want[n][p] - moved[n][p]) ** 2).mean()) for (n, p) in compared]))
        assert err < part * shift, (at, err, shift)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_two_sublayers_on_two_streams_change_no_bit(folders, dtype, monkeypatch):
    """Mixer and feed-forward beside each other against one behind the other, kernel by kernel and from captured steps that are
    replayed with other work and synchronizations between them: the same bits at every position."""
    from paged_llm_rs_amd.parts.block import ParallelBlock

    folder = folders("plain", dtype)
    prompts = ru.make_prompts(nu.PLAIN["vocab"], [70, 30, 41], seed=21)
    steps = ru.mixed(prompts, seed=4, max_live=3, tail=24)

    def run(side, graphs):
        monkeypatch.setattr(ParallelBlock, "side_by_side", side)
        r = replayer(folder, dtype, prompts, live=3, graphs=graphs)
        passes = []
        for _ in range(3):
            got = ru.collect(r, steps)
            a = torch.randn((256, 256), device="cuda")
            float((a @ a).sum())
            torch.cuda.synchronize()
            passes.append(got)
        for later in passes[1:]:
            assert all(np.array_equal(later[k], passes[0][k]) for k in passes[0]), (side, graphs)
        return passes[0]

    want = run(False, False)
    for side, graphs in ((True, False), (True, True), (False, True)):
        got = run(side, graphs)
        assert got.keys() == want.keys() and all(np.array_equal(got[k], want[k]) for k in want), (side, graphs)


def test_the_first_tokens_of_a_request(folders):
    """Requests of one, two and three tokens, whole and token by token, in pages and slots that others have just left."""
    for name in ("ones", "odd"):
        folder = folders(name, "float32")
        prompts = ru.make_prompts(nu.CONFIGS[name]["vocab"], [1, 2, 3, 1, 2, 3, 1], seed=9)
        want, factor = nu.plain_logits(folder, prompts), nu.sensitivity(folder, prompts)
        r = replayer(folder, "float32", prompts, live=2)
        for steps in (ru.whole(prompts), ru.tail_decoded(prompts, tail=3), ru.whole(prompts)):
            for (n, p), row in ru.collect(r, steps).items():
                assert np.abs(row - want[n][p].numpy()).max() <= 5e-5 * float(want[n].abs().max()) * float(factor[n][p]), (n, p)


def test_long_decoding(folders):
    """Two hundred tokens decoded one by one from captured steps, beside a second request, past windows and page
    borders, against the plain implementation, in bfloat16 against the engine's own whole prompts as well."""
    for dtype in DTYPES:
        folder = folders("odd", dtype)
        prompts = ru.make_prompts(nu.ODD["vocab"], [230, 215], seed=12)
        steps = []
        for name, toks in prompts.items():
            steps.append({"step": len(steps), "entries": [{"id": name, "tokens": toks[:15], "want": [14]}], "end": []})
        for p in range(15, 230):
            entries = [{"id": n, "tokens": [t[p]], "want": [0]} for n, t in prompts.items() if p < len(t)]
            steps.append({"step": len(steps), "entries": entries, "end": [n for n, t in prompts.items() if p == len(t) - 1]})
        check(folder, dtype, prompts, steps, live=2)


# --- the engine's own entry point ------------------------------------------------------------------------------------------

@pytest.mark.parametrize("name", ["odd", "plain"])
@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_greedy_generation_through_the_engine(tmp_path, name, dtype):
    """Prompts of unequal length through Engine.generate (scheduler, portions of 8 tokens, batches, captured steps,
    steps queued ahead) against greedy decoding with the plain implementation."""
    from paged_llm_rs_amd import Engine

    folder = nu.write_model(tmp_path / "m", nu.CONFIGS[name], seed=3, dtype="float32" if dtype == "f32" else "bfloat16",
                            edit=nu.varied)
    prompts = list(ru.make_prompts(nu.CONFIGS[name]["vocab"], [5, 23, 1, 40, 12, 9], seed=10).values())
    engine = Engine(folder, dtype=dtype, block_size=16, num_blocks=24, max_batch=4, chunk=8)
    got = engine.generate(prompts, max_tokens=12, temperature=0.0, stop_tokens=[])
    cfg, weights = nu.load_plain(folder)
    for prompt, result in zip(prompts, got):
        # (the chosen token is the plain implementation's best or within rounding of it: a router's close call or a
        # near tie of two logits may fall either way, and from then on the two continue differently)
        logits = nu.plain.forward(cfg, weights, prompt + result["tokens"])[len(prompt) - 1:-1]
        chosen = logits[torch.arange(12), torch.tensor(result["tokens"])]
        bound = 1e-3 if dtype == "f32" else 0.1
        whole = {"a": prompt + result["tokens"]}
        close = nu.close_calls(folder, whole, "float32" if dtype == "f32" else "bfloat16")["a"][len(prompt) - 1:-1]
        behind = (logits.max(-1).values - chosen)[~close]
        assert (behind <= bound * logits.abs().max()).all(), prompt
        assert len(set(result["tokens"])) > 2, result["tokens"]
    if dtype == "f32":
        same = sum(result["tokens"] == nu.plain_greedy(folder, prompt, 12) for prompt, result in zip(prompts, got))
        assert same >= len(prompts) - 1
    assert engine.cache.manager.live_sequences == 0


def test_requests_that_give_way_are_computed_again(tmp_path):
    """A pool too small for all residents: the newest gives way, comes back and recomputes its prompt; the tokens are
    those of an engine with room to spare."""
    from paged_llm_rs_amd import Engine

    folder = nu.write_model(tmp_path / "m", nu.ODD, seed=3, edit=nu.varied)
    prompts = list(ru.make_prompts(nu.ODD["vocab"], [30, 28, 26, 31], seed=13).values())
    roomy = Engine(folder, dtype="f32", block_size=8, num_blocks=64, max_batch=4, chunk=16)
    want = roomy.generate(prompts, max_tokens=24, temperature=0.0, stop_tokens=[])
    tight = Engine(folder, dtype="f32", block_size=8, num_blocks=19, max_batch=4, chunk=16)
    got = tight.generate(prompts, max_tokens=24, temperature=0.0, stop_tokens=[])
    assert sum(r["preemptions"] for r in got) > 0, "the pool was meant to run dry"
    assert [r["tokens"] for r in got] == [r["tokens"] for r in want]
    assert all(len(set(r["tokens"])) > 4 for r in got)


def test_a_model_of_retention_layers_alone_generates(tmp_path):
    """No layer keeps pages: slots only."""
    from paged_llm_rs_amd import Engine

    folder = nu.write_model(tmp_path / "m", nu.model(64, 60, [nu.retention(4, 16, 32, [0.9, 0.99, 0.999, 0.5]),
                                                              nu.retention(2, 24, 16, [0.95, 0.8], mlp=nu.moe(3, 2, 48, shared=24))]),
                            seed=5, std=0.2, edit=nu.varied)
    prompts = list(ru.make_prompts(60, [5, 23, 1, 40, 12, 9], seed=10).values())
    engine = Engine(folder, dtype="f32", block_size=16, num_blocks=24, max_batch=3, chunk=8)
    got = engine.generate(prompts, max_tokens=8, temperature=0.0, stop_tokens=[])
    assert [r["tokens"] for r in got] == [nu.plain_greedy(folder, p, 8) for p in prompts]


def test_the_trace_runner_runs_the_design(tmp_path):
    folder = nu.write_model(tmp_path / "m", nu.ODD, seed=2, dtype="bfloat16")
    repo = Path(__file__).resolve().parent.parent
    prompts = ru.make_prompts(nu.ODD["vocab"], [20, 9], seed=3)
    steps = ru.mixed(prompts, seed=1, max_live=2, tail=4)
    out = tmp_path / "out"
    done = subprocess.run([sys.executable, str(repo / "bin" / "trace_run"), "--model", str(folder), "--dtype", "float32",
                           "--out", str(out), "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                          capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [line for line in done.stdout.splitlines() if line.startswith("done ")] == [f"done {s['step']}" for s in steps]
    want, factor = nu.plain_logits(folder, prompts), nu.sensitivity(folder, prompts)
    close = nu.close_calls(folder, prompts, "float32")
    fed: dict = {}
    for s in steps:
        rows = [(e["id"], fed.get(e["id"], 0) + w) for e in s["entries"] for w in e["want"]]
        for e in s["entries"]:
            fed[e["id"]] = fed.get(e["id"], 0) + len(e["tokens"])
        if rows:
            got = np.fromfile(out / f"{s['step']}.f32", dtype="<f4").reshape(len(rows), -1)
            for row, (n, p) in zip(got, rows):
                if not bool(close[n][p]):
                    assert np.abs(row - want[n][p].numpy()).max() <= 1e-4 * float(want[n][p].abs().max()) * float(factor[n][p])


def test_the_command_line_generates_with_the_design(tmp_path):
    config = tmp_path / "config.json"
    config.write_text(json.dumps(nu.ONES))
    root = Path(__file__).resolve().parent.parent
    done = subprocess.run([sys.executable, str(root / "bin" / "pagedllm"), "--model", str(tmp_path / "m"), "--random-weights",
                           str(config), "--dtype", "bf16", "--prompt-ids", "1,2,3,4,5", "--prompt-ids", "9,8",
                           "--max-tokens", "5", "--temperature", "0", "--stop-ids", ""],
                          capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-2000:]
    lines = [json.loads(x) for x in done.stdout.splitlines() if x.startswith("{")]
    assert len(lines) == 2 and all(len(x["tokens"]) == 5 for x in lines), done.stdout
