"""A state-space recurrence with a matrix state per head as a mixer (``state_space``): one step size and one decay a
head, input and output maps shared by the heads of a group.

From the rows ``h``, with ``inner = num_heads * value_dim``: ``W_in h`` is ``z`` (``inner``), ``x`` (``inner``), ``B`` and ``C``
(``groups * state_size`` each) and ``dt`` (``num_heads``). ``x``, ``B`` and ``C`` pass a short causal convolution per channel
(``conv_taps`` taps with a bias, zeros before position 0) and silu; ``dt = softplus(dt + dt_bias)``. Per head, which
reads ``B`` and ``C`` of group ``head // (num_heads / groups)``: ``S <- exp(-exp(A_log) dt) S + dt B x^T`` (``state_size x
value_dim``), ``y = S^T C + D x``. The heads side by side are multiplied by ``silu(z)``, each of ``norm_groups`` equal parts
is divided by its root mean square, the row is multiplied by ``norm``; then the output product.

The recurrence is the one of ``csrc/scalar_gate_scan.hip`` under a step size, with ``q = C``, ``k = B``, ``v = x``; the portions
of a bfloat16 step take ``csrc/state_space.hip``, tiles of tokens on the matrix cores. The request's state slot holds ``S``
and the convolution's last ``conv_taps - 1`` inputs, all 32-bit. Step sizes, decays, the recurrence, gate and norm are 32-bit; in
a bfloat16 runtime what leaves the convolution (``x``, ``B`` and ``C``) is rounded to bfloat16 once, for single tokens and
portions alike, where the sizes let the matrix cores take the portions."""

from __future__ import annotations

from typing import Any, Mapping, Optional

import torch

from ..kernels import ops
from .base import Mixer, Runtime, StateSpec
from .linear import as_operand, linear_f32, stack_rows
from .registry import register_part
from .spec import WeightSpec


@register_part("mixer", "state_space")
class StateSpace(Mixer):
    def __init__(self, runtime: Runtime, *, hidden_size: int, num_heads: int, value_dim: int, state_size: int, groups: int = 1,
                 norm_groups: int = 1, conv_taps: int = 4, norm_eps: float = 1e-6) -> None:
        super().__init__(runtime)
        if min(hidden_size, num_heads, value_dim, state_size, groups, norm_groups) < 1 or not 1 <= conv_taps <= 16:
            raise ValueError("sizes must be positive and the convolution have 1 to 16 taps")
        if num_heads % groups or num_heads * value_dim % norm_groups:
            raise ValueError(f"{num_heads} heads of {value_dim} do not split into {groups} groups or {norm_groups} normed parts")
        self.hidden_size, self.num_heads, self.value_dim, self.state_size = hidden_size, num_heads, value_dim, state_size
        self.groups, self.norm_groups, self.taps, self.norm_eps = groups, norm_groups, conv_taps, float(norm_eps)
        self.inner = num_heads * value_dim
        self.channels = self.inner + 2 * groups * state_size
        self.state_floats = self.inner * state_size
        self.w_in = self.conv_w = self.conv_b = self.dt_bias = self.a_log = self.d = self.norm_w = self.w_o = None

    def weight_specs(self) -> dict[str, WeightSpec]:
        h, H = self.hidden_size, self.num_heads
        return {"in": WeightSpec((self.inner + self.channels + H, h)), "conv": WeightSpec((self.channels, self.taps), role="float32"),
                "conv.b": WeightSpec((self.channels,), role="float32", init="zeros"),
                "dt_bias": WeightSpec((H,), role="float32", init="zeros"), "A_log": WeightSpec((H,), role="float32", init="zeros"),
                "D": WeightSpec((H,), role="float32", init="ones"), "norm": WeightSpec((self.inner,), role="float32", init="norm"),
                "o": WeightSpec((h, self.inner))}

    def load_weights(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.w_in = stack_rows([tensors["in"]])
        self.conv_w, self.conv_b = tensors["conv"].contiguous(), tensors["conv.b"].contiguous()
        self.dt_bias, self.a_log, self.d = (tensors[n].contiguous() for n in ("dt_bias", "A_log", "D"))
        self.norm_w, self.w_o = tensors["norm"].contiguous(), tensors["o"]

    def cache_spec(self) -> StateSpec:
        return StateSpec((-(-(self.state_floats + (self.taps - 1) * self.channels) // 4) * 4,), torch.float32)  # (slots begin on 16 bytes)

    def graph_capturable(self, page_size: int) -> bool:
        return True  # kernels on the context's device arrays only; padding rows write the spare slot

    def input_weight(self) -> Optional[torch.Tensor]:
        """The matrix of the one product that reads the rows, for whoever stacks it with others'
        (``forward`` then gets the product's result as ``proj``)."""
        return self.w_in

    def release_input_weight(self) -> None:
        self.w_in = None

    def forward(self, x: torch.Tensor, ctx: Any, cache: Any, proj: Optional[torch.Tensor] = None) -> torch.Tensor:
        if cache is None or cache.kind != "state" or not cache.writable:
            raise RuntimeError("state_space needs a state of its own")
        state = cache.state.view(cache.state.shape[0], -1)
        n, c, gn, dev = x.shape[0], self.inner, self.groups * self.state_size, self.rt.device
        if proj is None:
            proj = linear_f32(self.rt, as_operand(self.rt, x, ctx), self.w_in)          # z | x | B | C | dt
        tiled = self.rt.is_bf16 and ops.state_space_tiles_supports(self.state_size, self.value_dim)
        xbc = torch.empty(n, self.channels, device=dev, dtype=torch.bfloat16 if tiled else torch.float32)
        ops.causal_conv(proj[:, c:], self.conv_w, self.conv_b, state, self.state_floats, ctx.q_start, ctx.positions,
                        ctx.state_slots, None if tiled else xbc, rounded=xbc if tiled else None, act="silu")
        y = torch.empty(n, c, device=dev, dtype=torch.float32)
        C, B, v = xbc[:, c + gn:], xbc[:, c:c + gn], xbc[:, :c]
        step = proj[:, c + self.channels:c + self.channels + self.num_heads]
        sizes = (self.num_heads, self.state_size, self.value_dim)
        rule = dict(qk_heads=self.groups, step_bias=self.dt_bias, step_rate=self.a_log, skip=self.d)
        nd = ctx.num_decode if tiled else n     # (single tokens come first; without tiles the scan takes every entry)
        if nd == n or not tiled:
            ops.scalar_gate_scan(C, B, v, state, ctx.q_start, ctx.positions, ctx.state_slots, y, *sizes, step=step, **rule)
        else:
            if nd:
                ops.scalar_gate_scan(C[:nd], B[:nd], v[:nd], state, ctx.q_start[:nd + 1], ctx.positions[:nd], ctx.state_slots[:nd], y[:nd],
                                     *sizes, step=step[:nd], **rule)
            ops.state_space_tiles(C, B, v, state, ctx.q_start, ctx.positions, ctx.state_slots,
                                  ctx.q_tiles(ops.state_space_tile_rows(), first_entry=nd), y, *sizes, step=step, **rule)
        out = self.rt.empty(n, c)
        ops.head_norm_gate(y, proj[:, :c], self.norm_w, self.norm_eps, out, self.norm_groups, c // self.norm_groups,
                           gate="silu_first")
        return linear_f32(self.rt, out, self.w_o)
