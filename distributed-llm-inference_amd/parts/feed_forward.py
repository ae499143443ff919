"""Gated feed-forward: ``down(act(gate(x)) * up(x))`` with ``act = silu`` (SwiGLU; reference:
src/dli/model/llama.py:180-191), or ``down(g sigmoid(alpha g) (u + up_shift))`` with clamped halves
``g = min(gate(x), limit)``, ``u = clamp(up(x), -limit, limit)`` (``activation="clamped"``), or with the gate's gelu in its tanh form
(``activation="gelu_tanh"``). Gate and up matrices are stacked at load, so one product gives
both halves; the activation kernel reads them side by side."""

from __future__ import annotations

from typing import Any, Mapping, Optional

import torch

from ..kernels import ops
from .base import DecodeStream, FeedForward, Norm, Runtime
from .linear import decode_copy, finish_residual, linear, linear_f32
from .registry import register_part
from .spec import WeightSpec


@register_part("feed_forward", "gated_mlp")
class GatedMLP(FeedForward):
    NAMES = {"gate": "gate_proj.weight", "up": "up_proj.weight", "down": "down_proj.weight"}
    BIAS_NAMES = {"gate": "gate_proj.bias", "up": "up_proj.bias", "down": "down_proj.bias"}
    ACTIVATIONS = ("silu", "clamped", "gelu_tanh")

    def __init__(self, runtime: Runtime, *, hidden_size: int, intermediate_size: int,
                 activation: str = "silu", bias: bool = False, names: Optional[Mapping[str, str]] = None,
                 few_rows_fused: bool = False, limit: float = float("inf"), alpha: float = 1.0, up_shift: float = 0.0,
                 float32_out: bool = False, bias_names: Optional[Mapping[str, str]] = None, defer_output_bias: bool = False) -> None:
        """``limit``, ``alpha``, ``up_shift``: of the clamped activation. ``float32_out``: the result is the second product's
        32-bit sums (for a norm or a residual stream that is 32-bit). ``defer_output_bias``: the second product's bias is
        left to the block (``output_bias``)."""
        super().__init__(runtime)
        # forward() itself takes the few-row kernels (SwiGLU inside the first product) for up to 16
        # rows: for blocks that have no fused decode path of their own
        self.few_rows_fused = bool(few_rows_fused)
        # checkpoint names of the three matrices below the part's prefix, where they are not the usual ones
        self.names = {**self.NAMES, **dict(names or {})}
        self.bias_names = {**self.BIAS_NAMES, **dict(bias_names or {})}
        if bias and bool(names) != bool(bias_names):
            raise ValueError("gated_mlp: other tensor names are taken for the matrices and the biases alike")
        if activation not in self.ACTIVATIONS:
            raise ValueError(f"gated_mlp has no kernel for activation {activation!r} (only {', '.join(self.ACTIVATIONS)})")
        if bias and activation == "clamped":
            raise ValueError("gated_mlp: the clamped activation takes no biases")
        if defer_output_bias and not (bias and float32_out):
            raise ValueError("gated_mlp: a bias that the block adds belongs to a 32-bit result with biases")
        self.activation, self.defer_output_bias = activation, bool(defer_output_bias)
        self.clamped = (float(limit), float(alpha), float(up_shift)) if activation == "clamped" else None
        self.float32_out = bool(float32_out)
        self.hidden_size, self.intermediate_size, self.bias = hidden_size, intermediate_size, bias
        self.w_gate_up = self.b_gate_up = self.w_down = self.b_down = None
        self.w_gate_up_tiled = self.w_down_tiled = None

    def graph_capturable(self, page_size: int) -> bool:
        return True  # kernels on device arrays only

    def weight_specs(self) -> dict[str, WeightSpec]:
        h, i = self.hidden_size, self.intermediate_size
        specs = {self.names["gate"]: WeightSpec((i, h)), self.names["up"]: WeightSpec((i, h)),
                 self.names["down"]: WeightSpec((h, i))}
        if self.bias:
            n = self.bias_names
            specs.update({n["gate"]: WeightSpec((i,)), n["up"]: WeightSpec((i,)), n["down"]: WeightSpec((h,))})
        return specs

    def load_weights(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.w_gate_up = torch.cat([tensors[self.names["gate"]], tensors[self.names["up"]]], 0).contiguous()
        self.w_down = tensors[self.names["down"]]
        if self.bias:
            n = self.bias_names
            self.b_gate_up = torch.cat([tensors[n["gate"]], tensors[n["up"]]], 0).contiguous()
            self.b_down = tensors[n["down"]].contiguous()
            if self.defer_output_bias:
                self.output_bias, self.b_down = self.b_down, None

    def finalize(self) -> None:
        self.w_gate_up_tiled = decode_copy(self.rt, self.w_gate_up, ops.SKINNY_SWIGLU)
        self.w_down_tiled = decode_copy(self.rt, self.w_down, ops.SKINNY_RESIDUAL)

    def native_fields(self):
        from .native import _bf16_matrix, _bf16_vector

        h, i = self.hidden_size, self.intermediate_size
        if type(self) is not GatedMLP or self.activation != "silu" or self.float32_out:
            return None  # a subclass computes something else: it must describe itself
        if not (self.rt.is_bf16 and _bf16_matrix(self.w_gate_up, 2 * i, h) and _bf16_matrix(self.w_down, h, i)
                and _bf16_vector(self.b_gate_up, 2 * i) and _bf16_vector(self.b_down, h)):
            return None
        return {"kind": "gated_silu", "w_gate_up": self.w_gate_up, "b_gate_up": self.b_gate_up, "w_down": self.w_down, "b_down": self.b_down,
                "hidden": h, "intermediate": i}

    def _takes_few_rows(self, x: torch.Tensor) -> bool:
        n = x.shape[0]
        return (self.rt.is_bf16 and 0 < n <= self.FEW_ROWS and x.dtype == torch.bfloat16 and x.stride(0) % 8 == 0
                and x.data_ptr() % 16 == 0 and ops.skinny_gemm_supports(n, self.hidden_size, x.dtype)
                and ops.skinny_gemm_supports(n, self.intermediate_size, x.dtype))

    def forward(self, x: torch.Tensor, ctx: Any) -> torch.Tensor:
        n = x.shape[0]
        act = self.rt.empty(n, self.intermediate_size)
        if (self.few_rows_fused or self.float32_out) and self._takes_few_rows(x):
            # a few rows outside the fused decode path (a block that keeps its stream in 32-bit, say):
            # the few-row products, the activation inside the first
            ops.skinny_gemm(x, self.w_gate_up, w_tiled=self.w_gate_up_tiled, epilogue=ops.SKINNY_SWIGLU, out=act,
                            bias=self.b_gate_up, clamped=self.clamped, gelu=self.activation == "gelu_tanh")
            out = torch.empty(n, self.hidden_size, device=self.rt.device,
                              dtype=torch.float32 if self.float32_out else self.rt.dtype)
            ops.skinny_gemm(act, self.w_down, w_tiled=self.w_down_tiled, bias=self.b_down, out=out,
                            epilogue=ops.SKINNY_F32 if self.float32_out else ops.SKINNY_STORE)
            return out
        gate_up = linear(self.rt, x, self.w_gate_up, self.b_gate_up)
        if self.clamped is not None:
            ops.clamped_glu(gate_up, act, *self.clamped)
        elif self.activation == "gelu_tanh":
            ops.gelu_glu(gate_up, act)
        else:
            ops.silu_mul(gate_up, act)
        if self.float32_out:
            return linear_f32(self.rt, act, self.w_down, bias=self.b_down)
        return linear(self.rt, act, self.w_down, self.b_down)

    FEW_ROWS = 16  # the few-row product kernels; 17 to 64 rows take the one that shares activations

    def streams(self, ctx: Any) -> bool:
        n = ctx.num_tokens
        if self.activation != "silu" or self.float32_out or not (self.rt.is_bf16 and self.hidden_size % 8 == 0):
            return False
        if n > self.FEW_ROWS:
            return (self.w_gate_up_tiled is not None and self.w_down_tiled is not None
                    and ops.mid_gemm_supports(n, self.hidden_size, self.rt.dtype)
                    and ops.mid_gemm_supports(n, self.intermediate_size, self.rt.dtype))
        return (ops.skinny_gemm_supports(n, self.hidden_size, self.rt.dtype)
                and ops.skinny_gemm_supports(n, self.intermediate_size, self.rt.dtype))

    def forward_stream(self, stream: DecodeStream, norm: Norm, ctx: Any, following: Optional[Norm] = None) -> None:
        """``stream.x += mlp(norm(stream.x))``, norm and sum inside the two products' kernels.
        ``following``: the norm that the stream meets next; with 17 to 64 rows the kernel that makes
        the residual sum applies it as well, so that the next product reads normalised rows."""
        n = stream.x.shape[0]
        norm_w, eps = norm.fused_params()
        if n > self.FEW_ROWS:
            ready = stream.normed_by(norm)
            if ready is not None:
                act = ops.mid_gemm(ready, self.w_gate_up_tiled, tiled=True, n=self.intermediate_size,
                                   epilogue=ops.MID_SWIGLU, bias=self.b_gate_up)
            else:
                act = ops.mid_gemm(stream.x, self.w_gate_up_tiled, tiled=True, n=self.intermediate_size,
                                   epilogue=ops.MID_SWIGLU, bias=self.b_gate_up, norm_w=norm_w, eps=eps,
                                   ssq_in=stream.ssq)
            partial = ops.mid_gemm(act, self.w_down_tiled, tiled=True, n=self.hidden_size, epilogue=ops.MID_PARTIAL)
            finish_residual(self.rt, stream, partial, self.b_down, following)
            return
        act = self.rt.empty(n, self.intermediate_size)
        ops.skinny_gemm(stream.x, self.w_gate_up, w_tiled=self.w_gate_up_tiled, epilogue=ops.SKINNY_SWIGLU, out=act,
                        bias=self.b_gate_up, norm_w=norm_w, eps=eps, ssq_in=stream.ssq)
        stream.wrote(ops.skinny_gemm(act, self.w_down, w_tiled=self.w_down_tiled, epilogue=ops.SKINNY_RESIDUAL,
                                     stream=stream.x, bias=self.b_down))


@register_part("feed_forward", "poly_norm_mlp")
class PolyNormMLP(FeedForward):
    """``down(act(up(x)))`` with the polynomial activation ``act(z) = a N(z) + b N(z^2) + c N(z^3) + e``:
    powers element by element, ``N`` dividing a row of ``intermediate_size`` values by its root mean
    square (eps inside the root), and the four numbers ``(a, b, c, e)`` one tensor of the checkpoint.
    The first product leaves its 32-bit sums, the activation and its norms are 32-bit, and the result
    is the second product's 32-bit sums (a residual stream's next summand)."""

    def __init__(self, runtime: Runtime, *, hidden_size: int, intermediate_size: int, norm_eps: float = 1e-6,
                 names: Optional[Mapping[str, str]] = None) -> None:
        super().__init__(runtime)
        self.hidden_size, self.intermediate_size, self.norm_eps = hidden_size, intermediate_size, float(norm_eps)
        self.names = {"up": "up", "down": "down", "act": "act", **dict(names or {})}
        self.w_up = self.w_down = self.coef = None

    def graph_capturable(self, page_size: int) -> bool:
        return True  # kernels on device arrays only

    def weight_specs(self) -> dict[str, WeightSpec]:
        h, i = self.hidden_size, self.intermediate_size
        return {self.names["up"]: WeightSpec((i, h)), self.names["down"]: WeightSpec((h, i)),
                self.names["act"]: WeightSpec((4,), role="float32", init="norm")}

    def load_weights(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.w_up, self.w_down = tensors[self.names["up"]], tensors[self.names["down"]]
        self.coef = tensors[self.names["act"]].contiguous()

    def forward(self, x: torch.Tensor, ctx: Any) -> torch.Tensor:
        z = linear_f32(self.rt, x, self.w_up)
        act = self.rt.empty(x.shape[0], self.intermediate_size)
        ops.poly_norm(z, self.coef, self.norm_eps, act)
        return linear_f32(self.rt, act, self.w_down)
