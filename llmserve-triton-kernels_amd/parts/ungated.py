"""Feed-forward of two matrices without a gate: down(act(up(x))), no biases.
Parameters: hidden, intermediate, activation ("squared_relu": max(u, 0)^2), result ("float32" leaves the result unrounded
for a caller that sums in 32-bit), names (local names of "up" and "down").
With few bfloat16 rows the activation is the first product's epilogue (ops.gemm_decode, in 32-bit, rounded once);
otherwise the product's result is replaced in place by a kernel of its own."""

from __future__ import annotations

import torch

from ..ops import library as ops
from .linear import decode_product, linear
from .registry import FeedForward, register_feed_forward
from .spec import ParamInfo


@register_feed_forward("ungated")
class Ungated(FeedForward):
    graph_safe = True

    def __init__(self, spec, ctx):
        super().__init__(spec, ctx)
        self.hidden = int(spec["hidden"])
        self.intermediate = int(spec["intermediate"])
        if spec["activation"] != "squared_relu":
            raise ValueError(f"activation={spec['activation']!r}; there is 'squared_relu'")
        names = spec.get("names") or {}
        self.names = {k: names.get(k, k) for k in ("up", "down")}
        self.result_dtype = torch.float32 if spec.get("result", "model") == "float32" else None
        self.up = self.down = None

    def param_infos(self):
        return {self.names["up"]: ParamInfo((self.intermediate, self.hidden)),
                self.names["down"]: ParamInfo((self.hidden, self.intermediate))}

    def load(self, tensors):
        self.up = tensors[self.names["up"]].contiguous()
        self.down = tensors[self.names["down"]].contiguous()

    def forward(self, x):
        if decode_product(x, self.up):
            act = torch.empty((x.shape[0], self.intermediate), dtype=x.dtype, device=x.device)
            ops.gemm_decode(act, x, self.up, squared_relu=True)
        else:
            act = ops.squared_relu(linear(x, self.up))
        return linear(act, self.down, out_dtype=self.result_dtype)
