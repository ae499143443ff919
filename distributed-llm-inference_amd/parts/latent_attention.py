"""Attention through a latent (``latent_attention``): per token one normalised vector ``c`` of ``kv_rank`` values
is cached, and every head's keys and values are linear maps of it; ``rot_dim`` > 0: a rotated key part shared by all
heads lies behind it.

From the rows ``h``: ``c_q = norm(W_dq h)`` (RMS norm with a weight), ``q = W_uq c_q`` (per head ``head_dim`` components and
``rot_dim`` more that are rotated by the position); ``c = norm`` of the first ``kv_rank`` rows of ``W_dkv h``, the other
``rot_dim``, rotated and not normed, are the shared key part ``e``. Head ``i`` has ``k = U_i c`` and ``v = V_i c`` (the rows of ``W_uk``
and ``W_uv`` that belong to it), scores ``scale (q_i . k + q_i,rot . e)`` over every earlier position and itself (``window``:
the last ``window`` of them), an ordinary softmax. With ``output_gate`` the concatenated heads are multiplied by
``sigmoid(W_g h)``, with ``head_gate`` each head by one number, ``sigmoid(W_g h)_i``, before the output product.
``own_kv=False``: the layer has no ``W_dkv`` and reads the latents and key parts of the schedule entry whose cache it is
given, with its own ``U``, ``V``, queries and window.

Since ``q_i . (U_i c) = (U_i^T q_i) . c`` and ``sum_j p_j V_i c_j = V_i (sum_j p_j c_j)``, the attention runs over the
cached latents themselves, as one kv head shared by all query heads whose values are the front of its keys,
between two small products per head: ``q'_i = U_i^T q_i`` before (``q_i``'s rotated part goes behind it) and ``V_i (.)`` after.
The cache is a group of pages of keys alone, one kv head of ``kv_rank + rot_dim``; the attention kernels are those of
:mod:`dli_amd.parts.scored_attention`.

Positions, angles, norms, scores, weights and gates are 32-bit; the products read the runtime's type with 32-bit sums."""

from __future__ import annotations

from typing import Any, Mapping, Optional

import torch

from ..kernels import ops
from .base import Mixer, PagedKVSpec, Runtime
from .linear import as_operand, linear_few, linear_f32, stack_rows
from .registry import build_part, register_part
from .scored_attention import paged_scored_attention
from .spec import PartSpec, WeightSpec


@register_part("mixer", "latent_attention")
class LatentAttention(Mixer):
    LONGEST_KEY = 1024   # what the attention kernels take where the values are the keys

    def __init__(self, runtime: Runtime, *, hidden_size: int, num_heads: int, head_dim: int, kv_rank: int, q_rank: int,
                 value_dim: Optional[int] = None, scale: Optional[float] = None, norm_eps: float = 1e-6,
                 output_gate: bool = False, head_gate: bool = False, window: int = 0, rot_dim: int = 0,
                 position: Optional[PartSpec] = None, own_kv: bool = True, cache_window: Optional[int] = None) -> None:
        """``position``: the rotary table of the ``rot_dim`` components (pairs half of them apart). ``cache_window``: how many of
        the latest latents the pages must keep where that is not this layer's own window (0: all): other layers that
        read them may look further back than it does."""
        super().__init__(runtime)
        value_dim = head_dim if value_dim is None else value_dim
        if min(num_heads, head_dim, value_dim, kv_rank, q_rank) < 1 or window < 0 or rot_dim < 0:
            raise ValueError("heads, sizes and ranks must be positive, the window and the rotated part not negative")
        if kv_rank + rot_dim > self.LONGEST_KEY:
            raise ops.KernelArgumentError(f"the attention kernels take latents with their rotated part of at most "
                                          f"{self.LONGEST_KEY} values, not {kv_rank + rot_dim}")
        if output_gate and head_gate:
            raise ValueError("latent_attention: a gate per component or per head")
        if cache_window is not None and cache_window and (not window or cache_window < window):
            raise ValueError("latent_attention: the pages must keep at least what this layer's own mask sees")
        self.position = build_part("position", position or PartSpec("none"), runtime)
        table = self.position.rotary_table()
        if (table.dim if table is not None else 0) != rot_dim or (table is not None and table.pairing != "half"):
            raise ops.KernelArgumentError("latent_attention needs a rotary table of rot_dim components, pairs half of them apart")
        self.hidden_size, self.num_heads, self.head_dim, self.value_dim = hidden_size, num_heads, head_dim, value_dim
        self.kv_rank, self.q_rank, self.window, self.rot_dim = kv_rank, q_rank, int(window), int(rot_dim)
        self.scale = float(scale) if scale is not None else (head_dim + rot_dim) ** -0.5
        self.norm_eps, self.output_gate, self.head_gate = float(norm_eps), bool(output_gate), bool(head_gate)
        self.own_kv, self.cache_window = bool(own_kv), cache_window
        self.w_in = self.w_uq = self.w_uk_t = self.w_uv = self.w_o = self.q_norm = self.c_norm = None

    def sub_parts(self) -> dict:
        return {"position": self.position}

    @property
    def _gates(self) -> int:
        return self.num_heads if self.head_gate else self.num_heads * self.value_dim if self.output_gate else 0

    def weight_specs(self) -> dict[str, WeightSpec]:
        h, H, d, dv = self.hidden_size, self.num_heads, self.head_dim, self.value_dim
        specs = {"dq": WeightSpec((self.q_rank, h)), "dq.norm": WeightSpec((self.q_rank,), role="float32", init="norm"),
                 "uq": WeightSpec((H * (d + self.rot_dim), self.q_rank)),
                 "uk": WeightSpec((H * d, self.kv_rank)), "uv": WeightSpec((H * dv, self.kv_rank)),
                 "o": WeightSpec((h, H * dv))}
        if self.own_kv:
            specs["dkv"] = WeightSpec((self.kv_rank + self.rot_dim, h))
            specs["dkv.norm"] = WeightSpec((self.kv_rank,), role="float32", init="norm")
        if self._gates:
            specs["g"] = WeightSpec((self._gates, h))
        return specs

    def load_weights(self, tensors: Mapping[str, torch.Tensor]) -> None:
        H, d, dv, r = self.num_heads, self.head_dim, self.value_dim, self.kv_rank
        # one product for everything that reads h: both latents (with the rotated key part) and the gate
        self.w_in = stack_rows([tensors[n] for n in ("dq", "dkv", "g") if n in tensors])
        self.q_norm = tensors["dq.norm"].contiguous()
        self.c_norm = tensors["dkv.norm"].contiguous() if self.own_kv else None
        self.w_uq = tensors["uq"]
        self.w_uk_t = tensors["uk"].view(H, d, r).transpose(1, 2).contiguous()    # per head [kv_rank, head_dim]
        self.w_uv = tensors["uv"].view(H, dv, r).contiguous()
        self.w_o = tensors["o"]

    def cache_spec(self) -> Optional[PagedKVSpec]:
        if not self.own_kv:
            return None   # the schedule hands this layer another entry's cache
        kept = self.cache_window if self.cache_window is not None else self.window
        return PagedKVSpec(1, self.kv_rank + self.rot_dim, kept, 0)

    def graph_capturable(self, page_size: int) -> bool:
        return True  # a step of single tokens is read through the context's device arrays alone

    def forward(self, x: torch.Tensor, ctx: Any, cache: Any) -> torch.Tensor:
        if cache is None or cache.kind != "paged" or cache.writable != self.own_kv:
            raise RuntimeError("latent_attention needs a paged cache: its own, or with own_kv=False another entry's")
        grp = ctx.groups[cache.group]
        n, H, r, e = x.shape[0], self.num_heads, self.kv_rank, self.rot_dim
        table = self.position.rotary_table()
        turn = dict(rot=e, inv_freq=table.inv_freq, positions=ctx.positions) if e else {}
        proj = linear_f32(self.rt, as_operand(self.rt, x, ctx), self.w_in)
        cq = self.rt.empty(n, self.q_rank)
        if self.own_kv:
            ops.latent_norm_cache(proj, 0, self.q_rank, self.q_rank, r, self.q_norm, self.c_norm, self.norm_eps, cq,
                                  grp.slots, cache.k_pages, **turn)
        else:
            ops.latent_norm_cache(proj, 0, self.q_rank, self.q_rank, 0, self.q_norm, None, self.norm_eps, cq, None, None)
        q = linear_few(self.rt, cq, self.w_uq)
        q_latent = self.rt.empty(n, H * (r + e))
        ops.head_products(q, self.w_uk_t, q_latent, **turn)
        mixed = self.rt.empty(n, H * r)
        paged_scored_attention(self.rt, ctx, cache, q_latent, mixed, H, r + e, r, self.scale, window=self.window)
        out = self.rt.empty(n, H * self.value_dim)
        g0 = self.q_rank + (r + e if self.own_kv else 0)
        ops.head_products(mixed, self.w_uv, out, gate=proj[:, g0:g0 + self._gates] if self._gates else None)
        return linear_f32(self.rt, out, self.w_o)
