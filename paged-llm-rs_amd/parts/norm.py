"""RMSNorm fused with the residual add (reference: model/layers.rs:40-65), and the layer norm with a bias."""

from __future__ import annotations

import torch

from .. import kernels
from ..errors import ConfigError
from ..weights.loader import ParamDecl
from .registry import register_norm


class PendingNorm:
    """A norm that has not run yet: the 32-bit stream it will read (every sum already in
    it), the norm, the type its output would have, and the rows wanted (all, or a list).

    A part that is handed one may pass it on to ``Linear.forward``, which runs norm and
    product as one kernel where that pays, or call ``materialize()`` for the normalised rows."""

    __slots__ = ("norm", "resid", "out_dtype", "rows", "handed")

    def __init__(self, norm, resid: torch.Tensor, out_dtype: torch.dtype, rows=None, handed=None):
        self.norm, self.resid, self.out_dtype, self.rows = norm, resid, out_dtype, rows
        # what the product that last added into the stream left of this norm's work (a filled
        # ``kernels.HandedNorm`` of this very norm, all rows), or None
        self.handed = handed if handed is not None and handed.filled and rows is None else None

    @property
    def num_rows(self) -> int:
        return self.resid.shape[0] if self.rows is None else self.rows.numel()

    @property
    def width(self) -> int:
        return self.resid.shape[1]

    def materialize(self) -> torch.Tensor:
        return self.norm.apply(self.resid, None, self.out_dtype, rows=self.rows)


def bare_names(norm, spec, width: int, stem: str) -> list:
    """[(a norm's local tensor name, its name under ``stem``)] where a gain is stored under the norm's own name: the one
    tensor of an RMS norm is ``stem``; a bias beside the gain is ``stem.b``."""
    names = [d.name for d in norm.declare(spec, width)]
    known = {"weight": stem, "bias": stem + ".b"}
    if names[0] != "weight" or any(n not in known for n in names):
        raise ConfigError(f"a norm of the tensors {', '.join(names)} cannot be stored under its own name")
    return [(n, known[n]) for n in names]


def bare_decls(norm, spec, width: int, stem: str, optional: bool = False) -> list:
    """A norm's tensors under the norm's own name (``bare_names``)."""
    names = dict(bare_names(norm, spec, width, stem))
    return [ParamDecl(names[d.name], d.shape, d.role, d.optional or optional) for d in norm.declare(spec, width)]


def bare_params(norm, spec, width: int, stem: str, params: dict) -> dict:
    return {local: params[name] for local, name in bare_names(norm, spec, width, stem)}


class RmsNorm:
    """x / sqrt(mean(x^2) + eps) * gain, statistic and product in 32-bit.  A spec with a ``gain_offset`` stores
    its gains as distances from that number (gains around zero for an offset of one): the sum is taken once,
    in 32-bit, when the norm is built."""

    # a product kernel can take this norm as its first stage: it needs ``gain32`` and ``eps`` only
    fuses_into_product = True

    @staticmethod
    def declare(spec, width: int) -> list:
        return [ParamDecl("weight", (width,), "gain_around_zero" if getattr(spec, "gain_offset", 0.0) else "gain")]

    def __init__(self, spec, width: int, params: dict, dtype, device):
        self.eps = float(spec.eps)
        self.width = width
        self.gain = params["weight"]
        offset = float(getattr(spec, "gain_offset", 0.0) or 0.0)
        if offset:
            self.gain = (self.gain.to(torch.float32) + offset).contiguous()
        # the product kernels that take the norm as their first stage read the gain in 32-bit
        self.gain32 = self.gain if self.gain.dtype == torch.float32 else self.gain.float()

    @property
    def sandwich(self) -> tuple:
        """(gain, bias, eps) for the pass over a layer whose sublayers stand between two norms."""
        return self.gain32, None, self.eps

    # what that pass is told: no mean is taken off
    centred = False

    def handoff(self, rows: int, device):
        """Room for this norm handed forward by a product that adds into the stream (``kernels.HandedNorm``),
        or None where no product would take it: many rows, a wide stream."""
        if rows > kernels.SKINNY_ROWS or self.width > kernels.FUSED_NORM_MAX_WIDTH or self.width % 8:
            return None
        return kernels.HandedNorm(self.gain32, self.eps, rows, self.width, device)

    def apply_onto(self, resid: torch.Tensor, y: torch.Tensor, rows_dtype=None):
        """resid += norm(y), for a layer that normalises a sublayer's output; ``y`` is 32-bit.  With
        ``rows_dtype`` the updated rows of the stream come back in that type too, otherwise None."""
        if not hasattr(self, "_gain32"):
            self._gain32 = self.gain if self.gain.dtype == torch.float32 else self.gain.float()
        return kernels.rmsnorm_onto(resid, y, self._gain32, self.eps, rows_dtype)

    def apply(self, resid: torch.Tensor, delta, out_dtype: torch.dtype, rows=None) -> torch.Tensor:
        n = resid.shape[0] if rows is None else rows.numel()
        out = torch.empty((n, self.width), dtype=out_dtype, device=resid.device)
        return kernels.add_rmsnorm(resid, delta, self.gain, self.eps, out, rows=rows)


register_norm("rms_norm", RmsNorm)


class LayerNorm:
    """(x - mean) / sqrt(mean((x - mean)^2) + eps) * gain + bias, all in 32-bit, rounded once at the store."""

    centred = True

    @staticmethod
    def declare(spec, width: int) -> list:
        return [ParamDecl("weight", (width,), "gain"), ParamDecl("bias", (width,), "bias")]

    def __init__(self, spec, width: int, params: dict, dtype, device):
        if width > kernels.SANDWICH_MAX_WIDTH:
            raise ConfigError(f"a layer norm over rows of {width} (up to {kernels.SANDWICH_MAX_WIDTH})")
        self.eps, self.width = float(spec.eps), width
        self.gain = params["weight"].to(torch.float32).contiguous()
        self.bias = params["bias"].to(torch.float32).contiguous()

    @property
    def sandwich(self) -> tuple:
        return self.gain, self.bias, self.eps

    def apply(self, resid: torch.Tensor, delta, out_dtype: torch.dtype, rows=None) -> torch.Tensor:
        if delta is not None:
            if rows is not None:
                raise ConfigError("a sum into the stream beside a list of rows")
            kernels.residual_add(resid, delta)
        return kernels.sandwich_step(resid, norm_x=self.sandwich, out_dtype=out_dtype, rows=rows)


register_norm("layer_norm", LayerNorm)
