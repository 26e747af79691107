"""RMSNorm and layer norm parts.  Reference: ``jllm/model/common.py:44-48``.

``y = x * rsqrt(mean(x^2, last axis) + eps) * weight`` with the mean square, the
inverse root and both products in float.  (The reference rounds the normalised value
to the activation type before the product with the weight; here it is rounded once,
after the product.)
"""
from __future__ import annotations

import torch

from ..ops import kernels as K
from .spec import TensorSpec, register_part


class RMSNorm:
    replayable = True
    may_leave_scale = True     # ``add_norm`` takes ``unscaled_ok`` (a norm part without this attribute is never asked)

    def __init__(self, size: int, eps: float, one_plus: bool = False, gain: float = 1.0):
        """``one_plus``: the stored weight lies around zero and the norm multiplies by 1 + weight.  ``gain``: a
        constant factor on the result (a residual multiplier folded into the norm of a sublayer's output)."""
        self.size, self.eps = int(size), float(eps)
        self.one_plus, self.gain = bool(one_plus), float(gain)
        self.weight = None

    def tensors(self) -> dict:
        return {"weight": TensorSpec((self.size,), role="vector", init="small" if self.one_plus else "norm")}

    def bind(self, tensors: dict, dtype: torch.dtype) -> None:
        w = tensors["weight"]
        if self.one_plus or self.gain != 1.0:
            w = ((w + 1.0 if self.one_plus else w) * self.gain).contiguous()     # float: the kernels see one weight
        self.weight = w
        self.dtype = dtype

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        """Norm over the last axis of an activation tensor (any leading shape)."""
        return K.rmsnorm(x, self.weight, self.eps)

    def add_norm(self, h: torch.Tensor, delta, rows=None, unscaled_ok: bool = False):
        """The residual step fused with the norm: ``h += delta`` in the float residual stream,
        returns ``norm(h)`` in the activation type.  ``delta`` may be a ``K.PendingNorm``: then what is
        added is its own norm of the sublayer's output.  With ``rows`` only those rows are normed
        and ``h`` is left alone.  With ``unscaled_ok`` the reader multiplies the rows by a matrix
        through ``K.linear`` and nothing else: for the few rows of a decode step whose ``delta``
        comes as partial products the result may then be ``K.UnscaledRows`` (``h * weight`` with
        the scale left to that product's epilogue), whose residual step is shared out to many blocks
        a row."""
        if isinstance(delta, K.PendingNorm):
            # a sublayer's output that is normed on its own before it joins the stream: both norms in one pass
            n_out = h.shape[0] if rows is None else rows.numel()
            out = torch.empty((n_out, self.size), dtype=self.dtype, device=h.device)
            K.postnorm_add_rmsnorm(h, delta.y, delta.parts, delta.weight, delta.eps, self.weight, out, rows, out_eps=self.eps,
                                   bias=delta.bias, plain_scale=delta.scale)
            return out
        if (unscaled_ok and rows is None and delta is not None and delta.dim() == 3
                and K.unscaled_rows_possible(self.dtype, h.shape[0], self.size)):
            return K.add_parts_unscaled(h, delta, self.weight, self.eps)
        n_out = h.shape[0] if rows is None else rows.numel()
        out = torch.empty((n_out, self.size), dtype=self.dtype, device=h.device)
        K.add_rmsnorm(h, delta, self.weight, out, self.eps, rows)
        return out


class LayerNorm:
    """``y = (x - mean(x)) / sqrt(mean((x - mean(x))^2) + eps) * weight + bias`` over the last axis, all in float."""

    replayable = True

    def __init__(self, size: int, eps: float):
        self.size, self.eps = int(size), float(eps)
        self.weight = self.bias = None

    def tensors(self) -> dict:
        return {"weight": TensorSpec((self.size,), role="vector", init="norm"),
                "bias": TensorSpec((self.size,), role="vector", init="small")}

    def bind(self, tensors: dict, dtype: torch.dtype) -> None:
        self.weight, self.bias = tensors["weight"], tensors["bias"]
        self.dtype = dtype

    def add_norm(self, h: torch.Tensor, delta, rows=None):
        """The residual step fused with the norm: ``h += delta`` in the float residual stream, returns ``norm(h)`` in the
        activation type.  ``delta`` is whatever a block hands on: rows, float partial results, a ``K.PendingNorm``, a
        ``K.PendingPair`` or None.  With ``rows`` only those rows are normed and ``h`` is left alone."""
        n_out = h.shape[0] if rows is None else rows.numel()
        out = torch.empty((n_out, self.size), dtype=self.dtype, device=h.device)
        K.add_layernorm(h, delta, self.weight, self.bias, self.eps, out, rows)
        return out


register_part("norm", "rmsnorm", RMSNorm)
register_part("norm", "layernorm", LayerNorm)
