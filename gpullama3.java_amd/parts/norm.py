"""RMSNorm: ``w * x / sqrt(mean(x^2) + eps)`` (J/inference/InferenceCore.java:47-56). A description with a
``weight_offset`` stores its weight around zero: the factor is ``weight_offset + w``, made once, in 32-bit, at load."""
from __future__ import annotations

import torch

from ..csrc import lib as K
from ..weights.loader import TensorSpec
from .base import register_part
from . import ops
from .ops import Normed



class RMSNorm:
    graph_safe = True      # kernel launches on the current stream only, sizes fixed by (T, B)
    folds = True           # a product can take over this norm's work (see ``ops.Normed``)
    takes_slices = True    # adds up the slices that the product before it left, while it reads the rows anyway

    def __init__(self, spec, dtype):
        self.dim, self.eps, self.dtype = spec.dim, spec.eps, dtype
        self.offset = float(getattr(spec, "weight_offset", 0.0))
        self.name = spec.names["weight"]
        self.weight = None

    def tensors(self):
        # (random weights: drawn around what makes the factor 1)
        return {self.name: TensorSpec((self.dim,), "vector", center=1.0 - self.offset if self.offset else None)}

    def load(self, weights):
        self.weight = weights[self.name]
        if self.offset:
            # the sum in 32-bit: 1 + w rounded to bfloat16 would lose most of a small w
            self.weight = (self.weight.float() + self.offset).contiguous()
        # the kernels that prepare a folded norm's rows read the weight as float (exact for 16-bit storage)
        self.weight_f32 = self.weight if self.weight.dtype == torch.float32 else self.weight.float()

    def __call__(self, ctx, x, rows=None, name="normed"):
        """The normalised rows, or a ``Normed`` when the next product can do the work itself (few
        rows, and the kernel that last wrote exactly this tensor prepared the rows for this norm)."""
        made = getattr(ctx, "normed", None)
        if made is not None and made[0] == x.data_ptr() and made[1] is self and rows is None and made[2].shape == x.shape:
            return made[2]                # (the kernel that completed the rows has made them already)
        rec = getattr(ctx, "ssq", None)
        if (getattr(ctx, "fuse", False) and rec is not None and rec[0] == x.data_ptr() and rec[4] is self
                and x.shape[0] <= ops.FUSE_ROWS and self.dtype == torch.bfloat16):
            return Normed(ctx, x, self.weight, self.eps, self.dtype, rec[3], rec[1], rec[2], rows, name)
        n = x.shape[0] if rows is None else rows.numel()
        out = ctx.buffer(name, (n, self.dim), self.dtype)
        pending = getattr(ctx, "pending", None)
        if pending is not None and pending[0] == x.data_ptr():
            # the product that last added to x left its sums in slices: add them up and normalise at once
            K.add_slices_rmsnorm(x, pending[1], self.weight, out, self.eps, rows)
            if rows is None:
                ctx.pending = None
            return out
        K.rmsnorm(x, self.weight, out, self.eps, rows)
        return out


class LayerNorm:
    """``(x - mean) / sqrt(var + eps) * w + b`` over the model width, statistics in 32-bit whatever the engine's type.
    As a norm in front of a part it hands out the normalised rows; a block whose norms stand behind its sublayers
    calls ``add_into`` instead: the residual rows take the norm of a sublayer's output."""
    graph_safe = True      # kernel launches on the current stream only

    def __init__(self, spec, dtype):
        self.dim, self.eps, self.dtype = spec.dim, spec.eps, dtype
        self.name, self.bias_name = spec.names["weight"], spec.names["bias"]
        self.weight = self.bias = None

    def tensors(self):
        return {self.name: TensorSpec((self.dim,), "vector"), self.bias_name: TensorSpec((self.dim,), "vector", 0.0, 0.1)}

    def load(self, weights):
        self.weight = weights[self.name].float().contiguous()
        self.bias = weights[self.bias_name].float().contiguous()

    def __call__(self, ctx, x, rows=None, name="normed"):
        n = x.shape[0] if rows is None else rows.numel()
        out = ctx.buffer(name, (n, self.dim), self.dtype)
        K.layernorm(x, self.weight, self.bias, out, self.eps, rows)
        return out

    def add_into(self, ctx, x, y, cast=None):
        """``x += norm(y)``; ``cast`` (the activations' type) receives the new rows of x."""
        K.layernorm_add(x, y, self.weight, self.bias, self.eps, cast)
        ops.residual_written(ctx, x)


register_part("norm", "rmsnorm", RMSNorm)
register_part("norm", "layernorm", LayerNorm)
