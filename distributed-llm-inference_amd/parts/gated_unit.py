"""The gated unit recurrence as a mixer (``gated_unit``): a diagonal recurrence per channel whose decay and input
gate are block-diagonal maps of its own input, beside a second branch that gates its result.

From the rows ``h``, ``inner_size`` channels each: ``y = gelu(W_y h + b_y)`` (tanh form) and ``u``, ``W_x h + b_x`` behind a short
causal convolution per channel (``conv_taps`` taps with a bias, zeros before position 0, no activation). ``u`` is
split into ``blocks`` equal parts; in part ``b`` ``r = sigmoid(R_b u_b + r_b)`` and ``i = sigmoid(I_b u_b + i_b)``. Per channel
``log a = -decay_rate r softplus(lam)`` and ``S <- a S + sqrt(1 - a^2) i u`` from zero; the result is ``W_o (S y)``.

The request's state slot holds ``S`` and the convolution's last ``conv_taps - 1`` inputs, all 32-bit. The products
over the model width read the runtime's type and leave 32-bit sums; the convolution, the gates (their block
products included), the decays, the recurrence and the second branch's activation are 32-bit."""

from __future__ import annotations

from typing import Any, Mapping

import torch

from ..kernels import ops
from .base import Mixer, Runtime, StateSpec
from .linear import as_operand, linear_f32, stack_rows
from .registry import register_part
from .spec import WeightSpec


@register_part("mixer", "gated_unit")
class GatedUnit(Mixer):
    def __init__(self, runtime: Runtime, *, hidden_size: int, inner_size: int, blocks: int, conv_taps: int = 4,
                 decay_rate: float = 8.0) -> None:
        super().__init__(runtime)
        if min(hidden_size, inner_size, blocks) < 1 or inner_size % blocks or not 1 <= conv_taps <= 16:
            raise ValueError("sizes must be positive, the channels split evenly and the convolution have 1 to 16 taps")
        self.hidden_size, self.inner, self.blocks, self.taps = hidden_size, inner_size, blocks, conv_taps
        self.decay_rate = float(decay_rate)
        self.w_in = self.x_bias = self.y_bias = self.conv_w = self.conv_b = None
        self.w_r = self.w_i = self.r_bias = self.i_bias = self.decay = self.w_o = None

    def weight_specs(self) -> dict[str, WeightSpec]:
        h, c, b, s = self.hidden_size, self.inner, self.blocks, self.inner // self.blocks
        return {"y": WeightSpec((c, h)), "y.b": WeightSpec((c,), role="float32", init="zeros"),
                "x": WeightSpec((c, h)), "x.b": WeightSpec((c,), role="float32", init="zeros"),
                "conv": WeightSpec((c, self.taps), role="float32"), "conv.b": WeightSpec((c,), role="float32", init="zeros"),
                "ra": WeightSpec((b, s, s)), "ra.b": WeightSpec((b, s), role="float32", init="zeros"),
                "ri": WeightSpec((b, s, s)), "ri.b": WeightSpec((b, s), role="float32", init="zeros"),
                "lam": WeightSpec((c,), role="float32", init="zeros"), "o": WeightSpec((h, c))}

    def load_weights(self, tensors: Mapping[str, torch.Tensor]) -> None:
        # one product for both branches: the recurrence's input first (the convolution reads from column 0)
        self.w_in = stack_rows([tensors["x"], tensors["y"]])
        self.x_bias, self.y_bias = tensors["x.b"].contiguous(), tensors["y.b"].contiguous()
        self.conv_w, self.conv_b = tensors["conv"].contiguous(), tensors["conv.b"].contiguous()
        self.w_r, self.w_i = tensors["ra"].contiguous(), tensors["ri"].contiguous()
        self.r_bias, self.i_bias = tensors["ra.b"].reshape(-1).contiguous(), tensors["ri.b"].reshape(-1).contiguous()
        # a constant per channel: made once, rounded once
        lam = tensors["lam"].double()
        self.decay = (self.decay_rate * torch.nn.functional.softplus(lam, threshold=60.0)).float().contiguous()
        self.w_o = tensors["o"]

    def cache_spec(self) -> StateSpec:
        return StateSpec((self.taps * self.inner,), torch.float32)     # S, then taps - 1 inputs

    def graph_capturable(self, page_size: int) -> bool:
        return True  # kernels on the context's device arrays only; padding rows write the spare slot

    def forward(self, x: torch.Tensor, ctx: Any, cache: Any) -> torch.Tensor:
        if cache is None or cache.kind != "state" or not cache.writable:
            raise RuntimeError("gated_unit needs a state of its own")
        state = cache.state.view(cache.state.shape[0], -1)
        n, c = x.shape[0], self.inner
        proj = linear_f32(self.rt, as_operand(self.rt, x, ctx), self.w_in)          # x | y
        u = torch.empty(n, c, device=self.rt.device, dtype=torch.float32)
        ops.causal_conv(proj, self.conv_w, self.conv_b, state, c, ctx.q_start, ctx.positions, ctx.state_slots, u,
                        act="none", in_bias=self.x_bias)
        # a step of single tokens reads the context's device arrays alone
        tiles = None if ctx.num_decode == ctx.num_entries else ctx.q_tiles(ops.gated_unit_tile_rows())
        out = self.rt.empty(n, c)
        ops.gated_unit(u, self.w_r, self.w_i, self.r_bias, self.i_bias, self.decay, proj[:, c:2 * c], self.y_bias, state,
                       ctx.q_start, ctx.positions, ctx.state_slots, tiles, out)
        return linear_f32(self.rt, out, self.w_o)
