"""Gated feed-forward: down(silu(gate(x)) * up(x)), no biases
(src/llmserve/model/llama.py:112-120).  Parameters: hidden, intermediate, and optionally unit ("silu"; "clamped" with
`limit`: down(g sigmoid(1.702 g) (u + 1)), g = min(gate(x), limit), u = clamp(up(x), -limit, limit); or "gelu_tanh":
down(gelu(gate(x)) * up(x)) with the tanh form of gelu).
gate_proj and up_proj are stacked into one [2I, H] matrix at load, so one product feeds
the activation.  With few bfloat16 rows that product also does the activation after it
(ops.gemm_stream); otherwise the product and the activation are kernels of their own."""

from __future__ import annotations

import torch

from ..ops import library as ops
from .linear import adds_residual_in_epilogue, decode_product, few_rows, linear, linear_partial_sums
from .registry import ADDED_IN_PLACE, DeferredNorm, FeedForward, register_feed_forward
from .spec import ParamInfo


@register_feed_forward("swiglu")
class SwiGLU(FeedForward):
    graph_safe = True
    accepts_deferred_norm = True

    def __init__(self, spec, ctx):
        super().__init__(spec, ctx)
        self.hidden = int(spec["hidden"])
        self.intermediate = int(spec["intermediate"])
        # `names`: local names of the three matrices; `result`: "float32" leaves the result unrounded for a caller
        # that sums in 32-bit
        names = spec.get("names") or {}
        self.names = {k: names.get(k, f"{k}_proj.weight") for k in ("gate", "up", "down")}
        self.result_dtype = torch.float32 if spec.get("result", "model") == "float32" else None
        self.unit = spec.get("unit", "silu")
        if self.unit not in ("silu", "clamped", "gelu_tanh"):
            raise ValueError(f"unit={self.unit!r}; choose 'silu', 'clamped' or 'gelu_tanh'")
        self.limit = float(spec["limit"]) if self.unit == "clamped" else None
        self.gelu = self.unit == "gelu_tanh"
        self.gate_up: torch.Tensor | None = None
        self.down: torch.Tensor | None = None

    def param_infos(self):
        h, i = self.hidden, self.intermediate
        return {self.names["gate"]: ParamInfo((i, h)), self.names["up"]: ParamInfo((i, h)),
                self.names["down"]: ParamInfo((h, i))}

    def load(self, tensors):
        self.gate_up = torch.cat([tensors[self.names["gate"]], tensors[self.names["up"]]], dim=0).contiguous()
        self.down = tensors[self.names["down"]].contiguous()

    def forward(self, x):
        deferred = isinstance(x, DeferredNorm)  # the caller hands the result to a norm, which takes partial sums
        rows = x.residual if deferred else x
        m = rows.shape[0]
        dtype, device = self.gate_up.dtype, self.gate_up.device
        act = torch.empty((m, self.intermediate), dtype=dtype, device=device)
        if decode_product(rows, self.gate_up):
            norm = x.fused() if deferred and m <= ops.GEMM_DECODE_NORM_ROWS else None
            if norm is not None:
                x.resolve(None)  # nothing is left to add: the kernel norms the residual rows as they are
            elif deferred:
                rows = x.materialize()
            ops.gemm_decode(act, rows, self.gate_up, swiglu=True, norm=norm, limit=self.limit, gelu=self.gelu)  # norm before, activation after the product
        else:
            if deferred:
                rows = x.materialize()
            few = dtype == torch.bfloat16 and few_rows(m, self.gate_up) and self.intermediate % 8 == 0
            if few and ops.gemm_bf16_supported(rows, self.gate_up):
                ops.gemm_stream(act, rows, self.gate_up, swiglu=True, limit=self.limit, gelu=self.gelu)  # activation in the product's epilogue
            else:
                ops.silu_mul(act, linear(rows, self.gate_up), self.limit, self.gelu)
        if deferred and x.may_add_in_place and adds_residual_in_epilogue(act, self.down):
            ops.gemm_decode(None, act, self.down, residual=x.residual)  # the residual sum in the product's epilogue
            return ADDED_IN_PLACE
        return (linear_partial_sums(act, self.down) if deferred else None) or linear(act, self.down,
                                                                                       out_dtype=self.result_dtype)


@register_feed_forward("none")
class NoFeedForward(FeedForward):
    """A layer without a feed-forward: nothing joins the stream."""

    graph_safe = True
    absent = True

    def forward(self, x):
        return None
