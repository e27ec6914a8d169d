"""RMSNorm, alone or fused with the residual add that precedes it.

out = x * rsqrt(mean(x^2) + eps) * w, all in 32-bit; eps is added to the mean
inside the root and the weight multiplies after normalisation
(backend/model.cu:101-122; fused with the add: :144-165).

Parameters: ``size`` (channels), ``eps``, ``offset`` (added to the stored weight once, in 32-bit: 1 for
weights stored around zero), ``scale`` (a constant on the normed rows, taken into the weight).
Tensor: ``<prefix>.weight`` [size].
"""

from __future__ import annotations

import torch

from .. import kernels as K
from .base import Normed, NormRows, Part, ScaledSum, register_part
from .spec import WeightSpec


@register_part("norm", "rmsnorm")
class RMSNorm(Part):
    graph_safe = True
    records_launches = True
    fusable = True     # a product's epilogue may do the addition, its consumer the row scale

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        self.size = int(self.param("size"))
        self.eps = float(self.param("eps"))
        self.offset = float(self.param("offset", 0.0))
        self.scale = float(self.param("scale", 1.0))
        self.weight = None

    def weight_specs(self):
        return [WeightSpec(self.tensor_name("weight"), (self.size,), "vector")]

    def bind(self, weights):
        w = weights[self.tensor_name("weight")]
        self.weight = w if self.offset == 0.0 and self.scale == 1.0 else ((w + self.offset) * self.scale).contiguous()

    def forward(self, ctx, x, delta=None, rows=None, tag="xn", normed_ok=False):
        """Normalised rows in the compute dtype.  ``delta`` is added into x
        first (and x is updated) unless ``rows`` selects rows to read.  A
        ``delta`` that is a ``Normed`` says that x already holds the sum: it
        is handed on to a consumer that takes it (``normed_ok``), or the rows
        of x are normalised here.  ``NormRows`` made for this norm are its result."""
        if isinstance(delta, NormRows):
            if rows is None and delta.norm is self:
                return delta.rows
            delta = None
        if isinstance(delta, Normed):
            if delta.norm is not self:
                raise ValueError("norm: the residual product was made for another norm")
            if normed_ok and rows is None:
                return delta
            delta = None
        n = rows.numel() if rows is not None else x.shape[0]
        out = ctx.buf(tag, (n, self.size), self.runtime.dtype)
        if isinstance(delta, ScaledSum):
            K.group_norm_add(x, delta.deltas, bias=delta.bias, mult=delta.mult, weight=self.weight, out=out, rows=rows,
                             eps=self.eps)
            return out
        K.add_rmsnorm(x, delta=delta, weight=self.weight, out=out, rows=rows, eps=self.eps)
        return out

    def add(self, ctx, x, delta):
        if isinstance(delta, ScaledSum):
            K.group_norm_add(x, delta.deltas, bias=delta.bias, mult=delta.mult)
        elif not isinstance(delta, (Normed, NormRows)):        # their sums are in x already
            K.add_rmsnorm(x, delta=delta, write_x=True)
        return x


def pending_sums(delta):
    """What a norm is to add to the stream first, as arguments of ``K.group_norm_add``."""
    if delta is None:
        return {}
    if isinstance(delta, Normed):
        raise ValueError("a residual product cannot stand for this norm")
    if isinstance(delta, ScaledSum):
        return {"deltas": delta.deltas, "bias": delta.bias, "mult": delta.mult}
    return {"deltas": [delta]}


@register_part("norm", "group_rmsnorm")
class GroupRMSNorm(Part):
    """RMS norm in groups: the channels are cut into ``groups`` equal consecutive parts, each
    is divided by its own sqrt(mean(part^2) + eps), and the whole is multiplied by the weight
    (``groups`` = 1 is the plain RMS norm).  It also adds what is pending to the residual
    stream: a plain delta, or a ``ScaledSum`` of sub-layers that ran side by side.

    Parameters: ``size``, ``eps``, ``groups``.  Tensor: ``<prefix>.weight`` [size]."""
    graph_safe = True
    records_launches = True

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        self.size = int(self.param("size"))
        self.eps = float(self.param("eps"))
        self.groups = int(self.param("groups", 1))
        if self.groups < 1 or self.size % self.groups:
            raise ValueError(f"group_rmsnorm: {self.size} channels do not go into {self.groups} equal groups")
        self.weight = None

    def weight_specs(self):
        return [WeightSpec(self.tensor_name("weight"), (self.size,), "vector")]

    def bind(self, weights):
        self.weight = weights[self.tensor_name("weight")]

    def forward(self, ctx, x, delta=None, rows=None, tag="xn", normed_ok=False):
        n = rows.numel() if rows is not None else x.shape[0]
        out = ctx.buf(tag, (n, self.size), self.runtime.dtype)
        K.group_norm_add(x, weight=self.weight, out=out, rows=rows, groups=self.groups, eps=self.eps,
                         **pending_sums(delta))
        return out

    def add(self, ctx, x, delta):
        if delta is not None:
            K.group_norm_add(x, **pending_sums(delta))
        return x


@register_part("norm", "layer_norm")
class LayerNorm(Part):
    """Layer norm: (x - mean) / sqrt(mean((x - mean)^2) + eps) * w + b over the channels, in 32-bit.  It
    also adds what is pending to the residual stream: a plain delta, or a ``ScaledSum`` of
    sub-layers that ran side by side.

    Parameters: ``size``, ``eps``.  Tensors: ``<prefix>.weight`` [size], ``<prefix>.bias`` [size]."""
    graph_safe = True
    records_launches = True

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        self.size = int(self.param("size"))
        self.eps = float(self.param("eps"))
        self.weight = self.bias = None

    def weight_specs(self):
        return [WeightSpec(self.tensor_name("weight"), (self.size,), "vector"),
                WeightSpec(self.tensor_name("bias"), (self.size,), "vector")]

    def bind(self, weights):
        self.weight, self.bias = weights[self.tensor_name("weight")], weights[self.tensor_name("bias")]

    def forward(self, ctx, x, delta=None, rows=None, tag="xn", normed_ok=False):
        n = rows.numel() if rows is not None else x.shape[0]
        out = ctx.buf(tag, (n, self.size), self.runtime.dtype)
        K.group_norm_add(x, weight=self.weight, norm_bias=self.bias, out=out, rows=rows, eps=self.eps, **pending_sums(delta))
        return out

    def add(self, ctx, x, delta):
        if delta is not None:
            K.group_norm_add(x, **pending_sums(delta))
        return x
