"""A state-space mixer with one decay per head and token, whose inputs and read-outs groups of heads share (Mamba-2).

Parameters (a `PartSpec` of kind "state_space"):
  hidden, num_heads (H), value_dim (P, columns of a head's state), states (N), groups (G), conv_taps
  norm_groups  equal parts of the heads' results that are normed by their own root mean square
  eps          of that norm (inside the root)
  result       "float32": the output projection's result stays unrounded (for a 32-bit residual stream)
  names        local tensor names (defaults: in, conv, conv.b, dt_bias, A_log, D, norm, o)

W_in h = [z: H P | x: H P | B: G N | C: G N | d: H].  x, B and C pass a causal convolution per channel (taps [channels,
conv_taps], the last column for the present token, a bias, zeros before the sequence) and SiLU.  dt = softplus(d + dt_bias),
a number per head.  Per head (with B and C of group h / (H / G)), S [N, P] zero before position 0:
    S <- exp(-exp(A_log_h) dt) S + dt B x^T,        y = S^T C + D_h x.
y silu(z) is normed part by part, multiplied by a weight of H P numbers; W_o follows.

A request keeps, in one state slot, S of every head (32-bit, column by column: [H, P, N]) and the last conv_taps - 1 rows of
[x | B | C] before the convolution (a ring indexed by position); a portion of a prompt starts from them and leaves them behind
its last token.  The projections take the model's dtype with 32-bit sums and leave 32-bit results; the convolution and SiLU
are computed in 32-bit and rounded once to the model's dtype; step sizes, decays, the recurrence, the gate and the norm are
32-bit, and the normed heads are rounded once as the operand of W_o.
"""

from __future__ import annotations

import torch

from ..ops import library as ops
from .attention_composed import _fill_taps
from .linear import linear
from .registry import Mixer, register_mixer
from .selective_scan import _fill_dt_bias, _fill_skip
from .spec import ParamInfo, StateCacheSpec

_DEFAULT_NAMES = {"in": "in", "conv": "conv", "conv_bias": "conv.b", "dt_bias": "dt_bias", "A_log": "A_log", "D": "D",
                  "norm": "norm", "o": "o"}


def _fill_rates(shape, generator, device, options):
    """log of decay rates between 1 and 16."""
    return 2.8 * torch.rand(shape, generator=generator, dtype=torch.float32, device=device)


@register_mixer("state_space")
class StateSpace(Mixer):
    graph_safe = True
    SCAN_UP_TO = 16  # new tokens of the longest portion up to which the recurrence runs token by token

    def __init__(self, spec, ctx):
        super().__init__(spec, ctx)
        self.hidden = int(spec["hidden"])
        self.heads = int(spec["num_heads"])
        self.p = int(spec["value_dim"])
        self.states = int(spec["states"])
        self.groups = int(spec["groups"])
        self.taps = int(spec["conv_taps"])
        self.norm_groups = int(spec.get("norm_groups", 1))
        self.eps = float(spec["eps"])
        self.result_dtype = torch.float32 if spec.get("result", "model") == "float32" else None
        self.names = dict(_DEFAULT_NAMES, **(spec.get("names") or {}))
        if min(self.hidden, self.heads, self.p, self.groups, self.taps, self.norm_groups) < 1 or self.heads % self.groups:
            raise ValueError("sizes must be positive and num_heads a multiple of groups")
        if not 1 <= self.states <= ops.SPACE_MAX_STATES:
            raise ValueError(f"1 to {ops.SPACE_MAX_STATES} states, got {self.states}")
        self.inner = self.heads * self.p
        if self.inner % self.norm_groups:
            raise ValueError(f"norm_groups={self.norm_groups} does not divide {self.inner}")
        self.channels = self.inner + 2 * self.groups * self.states
        self.dt_col = self.inner + self.channels
        self.scan_numbers = self.inner * self.states  # S first, then the ring
        self.w_in = self.w_o = self.taps_w = self.conv_bias = self.dt_bias = self.a_log = self.skip = self.norm_weight = None

    def libraries(self, dtype_name):
        return ("state_space",)

    def cache_spec(self):
        numbers = self.scan_numbers + (self.taps - 1) * self.channels
        return StateCacheSpec((numbers + -numbers % 4,), "float32")  # (slots at multiples of 16 bytes)

    def param_infos(self):
        n, h = self.names, self.hidden
        return {n["in"]: ParamInfo((self.dt_col + self.heads, h)), n["conv"]: ParamInfo((self.channels, self.taps), _fill_taps),
                n["conv_bias"]: ParamInfo((self.channels,), "around_zero"),
                n["dt_bias"]: ParamInfo((self.heads,), _fill_dt_bias, "stored"),
                n["A_log"]: ParamInfo((self.heads,), _fill_rates, "stored"), n["D"]: ParamInfo((self.heads,), _fill_skip, "stored"),
                n["norm"]: ParamInfo((self.inner,), "norm"), n["o"]: ParamInfo((h, self.inner))}

    def load(self, tensors):
        n = self.names
        w_in = tensors[n["in"]]
        # (rows of zeros up to a multiple of 8: every column of the products that a kernel reads in 16-byte pieces is aligned)
        self.w_in = torch.cat([w_in, w_in.new_zeros((-w_in.shape[0] % 8, w_in.shape[1]))], dim=0).contiguous()
        self.w_o = tensors[n["o"]].contiguous()
        self.taps_w = tensors[n["conv"]].float().contiguous()
        self.conv_bias, self.dt_bias, self.a_log, self.skip, self.norm_weight = (
            tensors[n[k]].float().contiguous() for k in ("conv_bias", "dt_bias", "A_log", "D", "norm"))

    def forward(self, x, batch, cache):
        rows, dev = x.shape[0], x.device
        u = linear(x, self.w_in, out_dtype=torch.float32)
        y = torch.empty((rows, self.inner), dtype=torch.float32, device=dev)
        self.recur(y, u, x.dtype, batch, cache.state)
        out = torch.empty((rows, self.inner), dtype=x.dtype, device=dev)
        ops.space_finish(out, y, u, self.norm_weight, parts=self.norm_groups, eps=self.eps, u=u, col=self.inner, taps=self.taps,
                         channels=self.channels, state=cache.state, ring_offset=self.scan_numbers, batch=batch)
        return linear(out, self.w_o, out_dtype=self.result_dtype)

    def recur(self, y, u, dtype, batch, state):
        """y from the products u of the step's tokens, and the requests' states brought up to date: token by token where every
        request brings few, in runs of 128 tokens on the matrix cores where one brings many (bfloat16)."""
        args = dict(col=self.inner, dt_col=self.dt_col, taps_w=self.taps_w, bias=self.conv_bias, dt_bias=self.dt_bias,
                    a_log=self.a_log, d_skip=self.skip, heads=self.heads, groups=self.groups, p=self.p, n_states=self.states,
                    state=state, scan_offset=0, ring_offset=self.scan_numbers, batch=batch)
        if batch.max_count > self.SCAN_UP_TO and ops.space_runs_supported(dtype, self.heads, self.groups, self.p, self.states, self.taps):
            ops.space_runs(y, u, **args)
        else:
            ops.space_scan(y, u, dtype=dtype, **args)
