"""Minimal gated recurrence (one number per channel, gates that read only the current token), beside the attention and state-space
mixers.

Per token, with h the layer input:
    z = sigmoid(W_z h + b_z);  u = W_x h + b_x;  c = u + 1/2 where u >= 0, sigmoid(u) elsewhere
    S <- (1 - z) S + z c  per channel;   out = W_o (S * silu(W_g h))                              (csrc/mingru.hip; S fp32 per slot)
The width of the recurrence is a constructor parameter.  `joined`: the projections are part of a linear the layer shares
(dense_linear.JoinedFront)."""
from __future__ import annotations

import torch

from .cache import SlotState
from .dense_linear import DenseLinear, front_rows


class MinimalGRU:
    CHUNKED_FROM = 33                                         # longest span of a step from which the chunked form is taken

    def __init__(self, model, key: str, layer_idx, *, width: int, out_tag: str = "mix.y", joined: bool = False):
        self.model, self.ext, self.key, self.layer_idx = model, model.ext, key, layer_idx
        self.inner, self.out_tag, self.joined = int(width), out_tag, joined
        if self.inner <= 0:
            raise ValueError(f"{key}: width {width}")
        self.kv_from = None
        self.front, self.front_base = None, 0

    def load(self, get):
        """`get(name)` returns the device tensor `<layer>.mix.<name>` in the model's operand dtype"""
        n, width, f32 = self.inner, self.model.width, torch.float32
        parts = [get("z"), get("x"), get("g")]
        bias = torch.zeros((3 * n,), dtype=f32, device=self.model.device)
        zb, xb = get("z.b"), get("x.b")
        self.o = DenseLinear(self.ext, self.key + ".o", get("o"))
        if any(tuple(p.shape) != (n, width) for p in parts) or zb.numel() != n or xb.numel() != n or tuple(self.o.weight.shape) != (width, n):
            raise RuntimeError(f"{self.key}: tensor shapes do not match the mixer's sizes")
        bias[:n], bias[n:2 * n] = zb.to(f32), xb.to(f32)
        self.front_part = (torch.cat(parts, 0), bias)
        if not self.joined:
            self.front, self.front_bias = DenseLinear(self.ext, self.key + ".front", self.front_part[0]), bias
            self.front_part = None
        return self

    def weight_bytes(self) -> int:
        return (self.front.weight_bytes() if self.front is not None else 0) + self.o.weight_bytes()

    def make_state(self, pool, dtype):
        return SlotState(pool, {"S": (self.inner,)})

    def forward(self, xh: torch.Tensor, rows: int, batch, cache, front=None) -> torch.Tensor:
        """xh: the normed layer input in the operand dtype [rows, width] (front: (rows of the layer's joined linear, their leading
        dimension)); returns the mixer's output, fp32 [rows, width]"""
        ext, m, n = self.ext, self.model, self.inner
        f, ld, base = front_rows(self, xh, rows, front)
        st = cache.layer(self.layer_idx)
        g = m.buf("gru.g", (rows, n), m.dtype)
        args = (f, ld, base, base + n, base + 2 * n, g, st["S"], batch.spans_dev, batch.row_seq, batch.row_pos, n)
        if batch.span_chunks is not None and batch.spans_dev[3] >= self.CHUNKED_FROM:
            # portions of prompts: every (chunk of tokens, channel) is independent work
            scratch = m.buf("gru.scratch", (2 * batch.span_chunks[2] + batch.spans_dev[2], n), torch.float32)
            ext.mingru_scan(*args, chunks=batch.span_chunks, scratch=scratch)
        else:
            ext.mingru_scan(*args)
        return self.o.forward(g, rows, out=m.buf(self.out_tag, (rows, m.width), torch.float32))
