"""Linear layers over unquantized weights (bfloat16 or float32, stored [out, in]) on the HIP library's dense kernels
(csrc/dense.hip), beside the quantized ExLlamaV2Linear.  No library GEMM: every row count goes to exl2_dense_linear."""
from __future__ import annotations

import torch


class DenseLinear:
    """y = epilogue(x . w^T).  `w` may hold several slabs ([slabs, out, in]): per-head projections run as one batched call,
    expert weights are picked per row (`w_sel`) or per group."""

    def __init__(self, ext, key: str, weight: torch.Tensor):
        if weight.dim() not in (2, 3):
            raise RuntimeError(f"{key}: a linear weight is [out, in] or [slabs, out, in]")
        self.ext, self.key = ext, key
        self.weight = weight.contiguous()
        self.out_features, self.in_features = weight.shape[-2], weight.shape[-1]
        self.slabs = weight.shape[0] if weight.dim() == 3 else 1

    @property
    def dtype(self):
        return self.weight.dtype

    def forward(self, x: torch.Tensor, rows: int, out_dtype=None, out: torch.Tensor | None = None, aux=None, epi: int = 0,
                limit: float = 0.0, ldx: int | None = None, x_off: int = 0, aux_ld: int = 0, aux_off: int = 0, bias=None) -> torch.Tensor:
        """Plain call on the first `rows` rows of x (leading dimension ldx, first value at element x_off); bias fp32 [out] or None."""
        n, k = self.out_features, self.in_features
        if out is None:
            out = torch.empty((rows, n), dtype=out_dtype or self.dtype, device=self.weight.device)
        self.ext.dense_linear(x, self.weight, out, rows, n, k, ldx or x.shape[-1], k, out.shape[-1], aux=aux, ldaux=aux_ld,
                              epi=epi, limit=limit, x_off=x_off, aux_off=aux_off, bias=bias)
        return out

    def weight_bytes(self) -> int:
        return self.weight.numel() * self.weight.element_size()


class JoinedFront:
    """ONE linear for everything that reads a layer's input: the members' projections (`member.front_part` = (weight [n, width], bias
    fp32 [n] | None), left by a module built with `joined=True`) stacked behind each other, every part starting at a multiple of four
    columns; a member learns where its columns start (`front_base`).  Plain (weight, bias) pairs may join; `bases` lists every
    member's first column in order.  A member may also leave `front_low` (weight [n, width]): the inner halves of low-rank projections,
    which the next linear reads -- they stand behind everything else (n a multiple of eight, so that it can be read in 16-byte pieces)
    and leave the same launch in the operand dtype, in rows of their own (`low_base` = the member's first column there)."""

    def __init__(self, ext, key: str, members):
        weights, biases, self.bases, at, low = [], [], [], 0, []
        self.low_columns = 0
        for m in members:
            w, b = m if isinstance(m, tuple) else m.front_part
            self.bases.append(at)
            if not isinstance(m, tuple):
                m.front_base, m.front_part = at, None
                if getattr(m, "front_low", None) is not None:
                    if m.front_low.shape[0] % 8:
                        raise RuntimeError(f"{key}: an inner projection of {m.front_low.shape[0]} columns")
                    low.append(m.front_low)
                    m.low_base, m.front_low = self.low_columns, None
                    self.low_columns += low[-1].shape[0]
            pad = -w.shape[0] % 4
            weights += [w] + ([w.new_zeros((pad, w.shape[1]))] if pad else [])
            bias = torch.zeros((w.shape[0] + pad,), dtype=torch.float32, device=w.device)
            if b is not None:
                bias[:w.shape[0]] = b.to(torch.float32)
            biases.append(bias)
            at += w.shape[0] + pad
        self.columns = at
        if low:
            biases.append(torch.zeros((self.low_columns,), dtype=torch.float32, device=low[0].device))
        self.linear = DenseLinear(ext, key, torch.cat(weights + low, 0))
        self.bias = torch.cat(biases, 0).contiguous()

    def weight_bytes(self) -> int:
        return self.linear.weight_bytes()

    def forward(self, xh: torch.Tensor, rows: int, model):
        """(fp32 rows of all members' projections, their leading dimension); with inner projections also (operand-dtype rows of those,
        their leading dimension)"""
        n = self.columns
        if self.low_columns:
            f = model.buf("layer.f", (rows, n), torch.float32)
            low = model.buf("layer.low", (rows, self.low_columns), model.dtype)
            self.linear.ext.dense_linear_split(xh, self.linear.weight, self.bias, f, low, rows, n)
            return f, n, low, self.low_columns
        return self.linear.forward(xh, rows, out=model.buf("layer.f", (rows, n), torch.float32), bias=self.bias), n


def front_rows(module, xh: torch.Tensor, rows: int, front):
    """(projections, leading dimension, first column) of a module that has a linear of its own or a share of a joined one"""
    if front is not None:
        return front[0], front[1], module.front_base
    n = module.front.out_features
    f = module.front.forward(xh, rows, out=module.model.buf("mix.f", (rows, n), torch.float32), bias=getattr(module, "front_bias", None))
    return f, n, 0
