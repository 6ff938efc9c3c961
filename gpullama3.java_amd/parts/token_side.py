"""What a token's own row of a side table adds to the residual row behind a layer's sublayers.

    x += w * unit(W_proj g),   g = act(W_gate x) * e,   unit(y) = y over its root mean square (eps inside the root)

x is the residual row itself (whole: sums of the product before it are settled first), e the columns of this layer in the
token's row of a table that all layers share. Three launches: the first product reads the 32-bit rows and ends with
activation and e (``lib.side_gate``), the second is an ordinary product with 32-bit sums, and the norm's kernel
(``lib.norm_add_next``) also leaves what reads the completed rows next: the next norm's output as it is (``ops.normed_ahead``), or,
in front of the head, whose norm reads wanted rows only, what a product that takes the norm over needs.
"""
from __future__ import annotations

import torch

from ..csrc import lib as K
from ..weights.loader import TensorSpec
from . import ops
from .base import register_part


class TokenSide:
    graph_safe = True      # kernel launches on the current stream only, sizes fixed by the step's tokens

    def __init__(self, spec, dtype, device):
        self.spec, self.dtype, self.names = spec, dtype, spec.names
        self.d, self.dim = spec.hidden, spec.dim
        self.col = spec.index * spec.dim
        if spec.activation not in K.ACTIVATIONS:
            raise ValueError(f"activation {spec.activation!r} is not built ({sorted(K.ACTIVATIONS)})")
        if self.col + self.dim > spec.columns:
            raise ValueError(f"columns {self.col} .. {self.col + self.dim} of a side table of {spec.columns}")
        self.pad = -(-self.dim // 32) * 32         # whole steps of the second product
        self.table = self.w_gate = self.w_proj = self.norm_w = None

    def tensors(self):
        n = self.names
        return {n["embed"]: TensorSpec((self.spec.rows, self.spec.columns)), n["gate"]: TensorSpec((self.dim, self.d)),
                n["proj"]: TensorSpec((self.d, self.dim)), n["norm"]: TensorSpec((self.d,), "vector")}

    def load(self, weights):
        n = self.names
        self.table, gate, proj = weights[n["embed"]], weights[n["gate"]], weights[n["proj"]]
        self.w_gate = gate.to(self.table.dtype).contiguous()
        if self.pad != self.dim:
            padded = torch.zeros((self.d, self.pad), dtype=proj.dtype, device=proj.device)
            padded[:, :self.dim] = proj
            proj, weights[n["proj"]] = padded, padded[:, :self.dim]
        self.w_proj = ops.for_few_rows(proj, without=getattr(self, "without", frozenset()))
        self.norm_w = weights[n["norm"]].float().contiguous()

    def forward(self, ctx, x, norm_after=None):
        """Adds into the residual rows ``x``; ``norm_after``: the norm that reads them next, if known."""
        ops.settle_residual(ctx, x)
        T, d = x.shape
        g = ctx.buffer("side_gated", (T, self.pad), self.table.dtype)
        K.side_gate(x, self.w_gate, self.table, self.col, ctx.token_ids, g, act=self.spec.activation, mfma="mfma" not in ops._off(ctx))
        y = ctx.buffer("side_out", (T, d), torch.float32)
        ops.linear(g, self.w_proj, y, ops.EPI_STORE, ctx)
        if d % 4:
            K.sides_norm_add(x, y, None, self.norm_w, None, self.spec.norm_eps, 1.0)
            return ops.residual_written(ctx, x)
        ahead = ops.normed_ahead(ctx, norm_after, x)
        if ahead is not None:
            K.norm_add_next(x, y, self.norm_w, self.spec.norm_eps, norm_after.weight_f32, norm_after.eps, h=ahead)
            ops.residual_written(ctx, x)
            return ops.normed_is_ready(ctx, x, norm_after, ahead)
        ctx.next_norm, held = norm_after, getattr(ctx, "next_norm", None)
        norm, xg = (ops._next_norm(ctx, d) if getattr(ctx, "fuse", False) and "fused" not in ops._off(ctx)
                    and T == ctx.n_tokens <= ops.FUSE_ROWS and d % 16 == 0 else (None, None))
        ctx.next_norm = held
        if norm is not None:
            ssq = ctx.ssq_buffer(1)
            K.norm_add_next(x, y, self.norm_w, self.spec.norm_eps, norm.weight_f32, norm.eps, xg=xg, ssq=ssq)
            return ops.residual_written(ctx, x, ssq, 1, xg, norm)
        K.norm_add_next(x, y, self.norm_w, self.spec.norm_eps)
        ops.residual_written(ctx, x)


register_part("side", "token_side", TokenSide)
