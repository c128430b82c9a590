"""Mixers that keep a matrix of state a head instead of keys and values in pages: linear attention with
a fixed decay (``lightning_attention``, and ``retention`` with rotated q and k), the matrix memory with exponential gates (mLSTM), the gated delta rule, and the state space
whose decay and step size come from the token (Mamba-2).

All of them are one product for every projection of the layer's input (32-bit sums out), the scan over
the step's tokens request by request (``kernels.recurrent_scan``: state, gates, decays and read-out in
32-bit, from and into the request's state slot), a norm over groups of the read-out times a gate, and
the output projection.  A request's state is one run of 32-bit floats in its slot; what a step's result
is does not depend on how the tokens were cut into steps, since the scan walks tokens one by one.
"""

from __future__ import annotations

import torch

from .. import kernels
from ..cache.layout import StateSpec
from ..errors import ConfigError, UnsupportedError
from ..weights.loader import ParamDecl
from .linear import Linear
from .registry import register_mixer
from .rotary import turning


def _f32(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.float32).contiguous()


class _ScanMixer:
    """What they have in common: the fused projection and where its pieces lie in a row."""

    graph_safe = True

    def _fuse(self, params: dict, names: list) -> None:
        self.columns, at = {}, 0
        for name in names:
            self.columns[name] = at
            at += params[name].shape[0]
        self.proj = Linear.fused([params[name] for name in names])

    @staticmethod
    def _sizes(spec, what: str) -> None:
        if spec.num_heads < 1 or not 1 <= spec.head_dim <= kernels.SCAN_MAX_DIM or spec.value_dim < 1:
            raise UnsupportedError(f"{what} of {spec.num_heads} heads of {spec.head_dim} by {spec.value_dim}: the scan "
                                   f"takes q and k up to {kernels.SCAN_MAX_DIM} a head")

    def cache_spec(self):
        return None


class LightningAttention(_ScanMixer):
    @staticmethod
    def declare(spec, hidden: int) -> list:
        qk, v = spec.num_heads * spec.head_dim, spec.num_heads * spec.value_dim
        return [ParamDecl("q", (qk, hidden)), ParamDecl("k", (qk, hidden)), ParamDecl("v", (v, hidden)),
                ParamDecl("g", (v, hidden)), ParamDecl("o", (hidden, v)), ParamDecl("norm", (v,), "gain")]

    def __init__(self, spec, hidden: int, params: dict, dtype, device, shared: dict):
        self._sizes(spec, "linear attention")
        if len(spec.decay) != spec.num_heads:
            raise ConfigError(f"{len(spec.decay)} decays for {spec.num_heads} heads")
        self.spec = spec
        self.H, self.D, self.V = spec.num_heads, spec.head_dim, spec.value_dim
        self._fuse(params, ["q", "k", "v", "g"])
        self.o_proj = Linear(params["o"])
        self.gain = _f32(params["norm"])
        self.decay = torch.tensor([float(d) for d in spec.decay], dtype=torch.float32, device=device)
        # (in chunks a decay enters through its logarithm)
        self.chunked = min(float(d) for d in spec.decay) > 0.0
        self.dtype = dtype

    def state_spec(self):
        return StateSpec((self.H * self.D * self.V,), torch.float32)

    def forward(self, x, ctx):
        c = self.columns
        rows = self.proj.forward(x, out_dtype=torch.float32)
        read = kernels.recurrent_scan("lightning", rows, c["q"], c["k"], c["v"], ctx.state(), ctx.batch,
                                      self.H, self.H, self.D, self.V, p1=self.decay, chunked=self.chunked)
        normed = kernels.gated_group_norm(read, self.H * self.V, self.gain, self.spec.eps, self.dtype,
                                          gate=rows, gate_off=c["g"], gate_act="sigmoid")
        return self.o_proj.forward(normed, out_dtype=torch.float32)


class Mlstm(_ScanMixer):
    @staticmethod
    def declare(spec, hidden: int) -> list:
        H = spec.num_heads
        qk, v = H * spec.head_dim, H * spec.value_dim
        return [ParamDecl("q", (qk, hidden)), ParamDecl("k", (qk, hidden)), ParamDecl("v", (v, hidden)),
                ParamDecl("g", (v, hidden)), ParamDecl("o", (hidden, v)), ParamDecl("norm", (v,), "gain"),
                ParamDecl("i", (H, hidden)), ParamDecl("i.b", (H,), "bias"),
                ParamDecl("f", (H, hidden)), ParamDecl("f.b", (H,), "bias")]

    def __init__(self, spec, hidden: int, params: dict, dtype, device, shared: dict):
        self._sizes(spec, "a matrix memory")
        if not spec.gate_cap > 0:
            raise ConfigError(f"a gate cap of {spec.gate_cap}")
        self.spec = spec
        self.H, self.D, self.V = spec.num_heads, spec.head_dim, spec.value_dim
        self._fuse(params, ["q", "k", "v", "g", "i", "f"])
        self.o_proj = Linear(params["o"])
        self.gain = _f32(params["norm"])
        self.bias_i, self.bias_f = _f32(params["i.b"]), _f32(params["f.b"])
        self.dtype = dtype

    def state_spec(self):
        # S, the normaliser n and the running maximum m (``kernels.scan_state_floats``)
        return StateSpec((kernels.scan_state_floats("mlstm", self.H, self.D, self.V),), torch.float32)

    def forward(self, x, ctx):
        c = self.columns
        rows = self.proj.forward(x, out_dtype=torch.float32)
        read = kernels.recurrent_scan("mlstm", rows, c["q"], c["k"], c["v"], ctx.state(), ctx.batch,
                                      self.H, self.H, self.D, self.V, gates=rows, g1_off=c["i"], g2_off=c["f"],
                                      p1=self.bias_i, p2=self.bias_f, cap=self.spec.gate_cap, chunked=True)
        normed = kernels.gated_group_norm(read, self.V, self.gain, self.spec.eps, self.dtype,
                                          gate=rows, gate_off=c["g"], gate_act="sigmoid")
        return self.o_proj.forward(normed, out_dtype=torch.float32)


class GatedDelta(_ScanMixer):
    @staticmethod
    def declare(spec, hidden: int) -> list:
        H, G, t = spec.num_heads, spec.num_qk_heads, spec.conv_taps
        qk, v = G * spec.head_dim, H * spec.value_dim
        return [ParamDecl("q", (qk, hidden)), ParamDecl("q.conv", (qk, t)),
                ParamDecl("k", (qk, hidden)), ParamDecl("k.conv", (qk, t)),
                ParamDecl("v", (v, hidden)), ParamDecl("v.conv", (v, t)),
                ParamDecl("b", (H, hidden)), ParamDecl("a", (H, hidden)),
                ParamDecl("A_log", (H,), "bias"), ParamDecl("dt_bias", (H,), "bias"),
                ParamDecl("norm", (spec.value_dim,), "gain"), ParamDecl("g", (v, hidden)), ParamDecl("o", (hidden, v))]

    def __init__(self, spec, hidden: int, params: dict, dtype, device, shared: dict):
        self._sizes(spec, "a delta rule")
        if spec.num_qk_heads < 1 or spec.num_heads % spec.num_qk_heads:
            raise UnsupportedError(f"{spec.num_heads} heads over {spec.num_qk_heads} heads of q and k, "
                                   "which do not group evenly")
        if not 1 <= spec.conv_taps <= 16:
            raise UnsupportedError(f"a convolution of {spec.conv_taps} taps (1 to 16)")
        self.spec = spec
        self.H, self.G, self.D, self.V = spec.num_heads, spec.num_qk_heads, spec.head_dim, spec.value_dim
        self._fuse(params, ["q", "k", "v", "g", "b", "a"])       # q | k | v first: the convolution's channels
        self.channels = 2 * self.G * self.D + self.H * self.V
        self.conv_w = torch.cat([_f32(params["q.conv"]), _f32(params["k.conv"]), _f32(params["v.conv"])], 0).t().contiguous()   # [taps, channels]
        self.o_proj = Linear(params["o"])
        self.gain = _f32(params["norm"])
        self.a_log, self.dt_bias = _f32(params["A_log"]), _f32(params["dt_bias"])
        self.dtype = dtype
        self.matrix = self.H * self.D * self.V

    def state_spec(self):
        # S [H, D, V], then the convolution's last taps - 1 inputs [taps - 1, channels]
        return StateSpec((self.matrix + (self.spec.conv_taps - 1) * self.channels,), torch.float32)

    def forward(self, x, ctx):
        c, G, D = self.columns, self.G, self.D
        state = ctx.state()
        history = state[:, self.matrix:]
        rows = self.proj.forward(x, out_dtype=torch.float32)
        mixed = kernels.short_conv(rows, c["q"], self.conv_w, history, ctx.batch, silu=True)
        kernels.conv_history(rows, c["q"], self.conv_w, history, ctx.batch)
        read = kernels.recurrent_scan("delta", mixed, 0, G * D, 2 * G * D, state[:, :self.matrix], ctx.batch,
                                      self.H, G, D, self.V, gates=rows, g1_off=c["b"], g2_off=c["a"],
                                      p1=self.a_log, p2=self.dt_bias, chunked=True)
        normed = kernels.gated_group_norm(read, self.V, self.gain, self.spec.eps, self.dtype,
                                          gate=rows, gate_off=c["g"], gate_act="silu")
        return self.o_proj.forward(normed, out_dtype=torch.float32)


class StateSpace(_ScanMixer):
    """One projection [z | x | B | C | dt]; x, B and C pass a short convolution with bias and silu together (channels of
    all heads side by side) and are v, k and q of the scan (``kernels.recurrent_scan``, kind ``ssd``).  The read-out is
    gated by silu(z) first and normed then, in equal parts of all heads' values together.
    Tensors: ``in``, ``conv`` [channels, taps], ``conv.b``, ``dt_bias``, ``A_log``, ``D`` (one a head), ``norm``, ``o``."""

    # requests that bring fewer tokens than this go through the scan token by token, which a step launches only where there are any
    short_portion = kernels.SCAN_CHUNKED_FROM

    @staticmethod
    def declare(spec, hidden: int) -> list:
        H, inner = spec.num_heads, spec.num_heads * spec.value_dim
        channels = inner + 2 * spec.groups * spec.state_dim
        return [ParamDecl("in", (inner + channels + H, hidden)), ParamDecl("conv", (channels, spec.conv_taps), "filter"),
                ParamDecl("conv.b", (channels,), "bias"), ParamDecl("dt_bias", (H,), "bias"), ParamDecl("A_log", (H,), "bias"),
                ParamDecl("D", (H,), "gain"), ParamDecl("norm", (inner,), "gain"), ParamDecl("o", (hidden, inner))]

    def __init__(self, spec, hidden: int, params: dict, dtype, device, shared: dict):
        H, G, N, V = spec.num_heads, spec.groups, spec.state_dim, spec.value_dim
        if H < 1 or V < 1 or not 1 <= N <= kernels.SCAN_MAX_DIM:
            raise UnsupportedError(f"a state space of {H} heads of {N} by {V}: the scan takes states up to {kernels.SCAN_MAX_DIM} rows")
        if G < 1 or H % G:
            raise UnsupportedError(f"{H} heads over {G} groups of B and C, which do not group evenly")
        if not 1 <= spec.conv_taps <= 16:
            raise UnsupportedError(f"a convolution of {spec.conv_taps} taps (1 to 16)")
        if spec.norm_groups < 1 or (H * V) % spec.norm_groups:
            raise UnsupportedError(f"a norm over {H * V} values in {spec.norm_groups} equal parts")
        self.spec, self.dtype = spec, dtype
        self.H, self.G, self.N, self.V = H, G, N, V
        self.inner = H * V
        self.channels = self.inner + 2 * G * N
        self.proj = Linear(params["in"])
        self.conv_w = _f32(params["conv"]).t().contiguous()                # [taps, channels]
        self.conv_b = _f32(params["conv.b"])
        self.o_proj = Linear(params["o"])
        self.gain, self.skip = _f32(params["norm"]), _f32(params["D"])
        self.a_log, self.dt_bias = _f32(params["A_log"]), _f32(params["dt_bias"])
        self.matrix = H * N * V
        self.history = (spec.conv_taps - 1) * self.channels

    def state_spec(self):
        # S [H, N, V], then the convolution's last taps - 1 inputs [taps - 1, channels]; a slot is a whole number of 16 bytes
        return StateSpec(((self.matrix + self.history + 3) // 4 * 4,), torch.float32)

    def forward(self, x, ctx):
        inner, G, N = self.inner, self.G, self.N
        state = ctx.state()
        rows = self.proj.forward(x, out_dtype=torch.float32)
        mixed = kernels.short_conv(rows, inner, self.conv_w, state[:, self.matrix:self.matrix + self.history], ctx.batch, silu=True,
                                   bias=self.conv_b,
                                   move_history=True)
        read = kernels.recurrent_scan("ssd", mixed, inner + G * N, inner, 0, state[:, :self.matrix], ctx.batch, self.H, G, N,
                                      self.V, gates=rows, g1_off=inner + self.channels, p1=self.a_log, p2=self.dt_bias,
                                      p3=self.skip, chunked=True)
        normed = kernels.gated_group_norm(read, inner // self.spec.norm_groups, self.gain, self.spec.eps, self.dtype,
                                          gate=rows, gate_off=0, gate_act="silu", gate_first=True)
        return self.o_proj.forward(normed, out_dtype=torch.float32)


class Retention(_ScanMixer):
    """Linear attention with a fixed decay a head and rotated queries and keys, no activations and no denominator; every head's read-out
    divided by its root mean square, times silu(gate).  Tensors: ``q``, ``k``, ``v``, ``g``, ``o``."""

    # requests that bring fewer tokens than this go token by token, which a step launches only where there are any
    short_portion = kernels.SCAN_CHUNKED_FROM

    @staticmethod
    def declare(spec, hidden: int) -> list:
        qk, v = spec.num_heads * spec.head_dim, spec.num_heads * spec.value_dim
        return [ParamDecl("q", (qk, hidden)), ParamDecl("k", (qk, hidden)), ParamDecl("v", (v, hidden)),
                ParamDecl("g", (v, hidden)), ParamDecl("o", (hidden, v))]

    def __init__(self, spec, hidden: int, params: dict, dtype, device, shared: dict):
        self._sizes(spec, "retention")
        if len(spec.decay) != spec.num_heads:
            raise ConfigError(f"{len(spec.decay)} decays for {spec.num_heads} heads")
        if spec.rotary_dims % 2 or not 0 <= spec.rotary_dims <= spec.head_dim:
            raise UnsupportedError(f"a rotation over {spec.rotary_dims} of {spec.head_dim} values")
        self.spec, self.dtype = spec, dtype
        self.H, self.D, self.V = spec.num_heads, spec.head_dim, spec.value_dim
        self._fuse(params, ["q", "k", "v", "g"])
        self.o_proj = Linear(params["o"])
        self.decay = torch.tensor([float(d) for d in spec.decay], dtype=torch.float32, device=device)
        # (in chunks a decay enters through its logarithm)
        self.chunked = min(float(d) for d in spec.decay) > 0.0
        self.freq, self.amplitude = None, 1.0
        if spec.rotary_dims:
            self.freq, self.amplitude = turning(spec.rotary_dims, spec.rotary_base, None, spec.rotary_ramp, device)
        self.key_scale = float(spec.key_scale) if spec.key_scale is not None else self.D ** -0.5

    def state_spec(self):
        return StateSpec((self.H * self.D * self.V,), torch.float32)

    def forward(self, x, ctx):
        c = self.columns
        rows = self.proj.forward(x, out_dtype=torch.float32)
        read = kernels.retention_scan(rows, c["q"], c["k"], c["v"], ctx.state(), ctx.batch, self.H, self.D, self.V, self.decay,
                                      self.freq, self.amplitude, self.key_scale, chunked=self.chunked)
        normed = kernels.gated_group_norm(read, self.V, None, self.spec.eps, self.dtype, gate=rows, gate_off=c["g"], gate_act="silu")
        return self.o_proj.forward(normed, out_dtype=torch.float32)


register_mixer("lightning_attention", LightningAttention)
register_mixer("retention", Retention)
register_mixer("mlstm", Mlstm)
register_mixer("gated_delta", GatedDelta)
register_mixer("state_space", StateSpace)
