"""Two mixers side by side on the same layer input: result = left_scale * left(h) + right_scale * right(h).

The halves are ordinary mixers of the stack's registry built with their own tensor prefix (`<layer>.mix.left.*`, `.right.*`), state
key ((layer, "left"), (layer, "right")) and result buffer; the weighted sum is not a launch of its own -- `forward` hands both fp32
results and their scales to the residual step that follows (rmsnorm.SandwichNorm), whose launch reads them.  `out_norms`: each result
is RMS-normed over the model width with a weight of its own (`.left.out`, `.right.out`) before the sum -- in that launch too
(rmsnorm.GatedResidualNorm reads `out_norms`)."""
from __future__ import annotations


class ParallelMixer:
    def __init__(self, model, key: str, layer_idx: int, left, right, left_scale: float, right_scale: float, out_norms: bool = False):
        self.model, self.ext, self.key, self.layer_idx = model, model.ext, key, layer_idx
        self.left, self.right, self.left_scale, self.right_scale = left, right, float(left_scale), float(right_scale)
        self.kv_from = None
        self.out_norms = (None, None) if out_norms else None
        if getattr(left, "kv_from", None) is not None or getattr(right, "kv_from", None) is not None:
            raise ValueError(f"{key}: a half of a parallel mixer keeps its own keys and values")
        if left.out_tag == right.out_tag:
            raise ValueError(f"{key}: the halves need result buffers of their own")

    def load(self, get):
        self.left.load(lambda n, optional=False: get("left." + n, optional))
        self.right.load(lambda n, optional=False: get("right." + n, optional))
        if self.out_norms is not None:
            self.out_norms = (get("left.out"), get("right.out"))
            if any(w.numel() != self.model.width for w in self.out_norms):
                raise RuntimeError(f"{self.key}: the norms behind the halves are over the model width")
        return self

    def weight_bytes(self) -> int:
        return self.left.weight_bytes() + self.right.weight_bytes()

    def make_states(self, pool, dtype) -> dict:
        return {self.left.layer_idx: self.left.make_state(pool, dtype), self.right.layer_idx: self.right.make_state(pool, dtype)}

    @property
    def front_members(self):
        return [self.left, self.right]

    def forward(self, xh, rows: int, batch, cache, front=None):
        """returns (left result, left scale, right result, right scale): fp32 [rows, width] each"""
        kw = dict(front=front) if front is not None else {}
        yl = self.left.forward(xh, rows, batch, cache, **kw)
        yr = self.right.forward(xh, rows, batch, cache, **kw)
        return yl, self.left_scale, yr, self.right_scale
