"""Typed configuration of the Rurorax decoder: a list of layers, each ``x <- x + ls1 * mixer(h) + ls2 * ff(h)`` with
one ``h = tanh(alpha x) * w + b`` for both sublayers and a vector on each result. The mixer is a state-space
recurrence with one step size and decay a head (``mamba2``) or grouped rotary attention in chunks with norms over the
whole query and key projections (``attention``); the feed-forward is gated by a gelu, a mixture of experts whose
inputs are scaled by sigmoid scores, or absent. The head is the embedding table under a soft cap.

``config.json`` keys: ``vocab``, ``width``, ``norm.eps`` (of the norms inside the mixers), ``logit_softcap`` (absent: no cap)
and ``layers``: a list of ``{"type", "mixer": {...}, "mlp": {...} | null}``. Mixer keys by type:
``mamba2``: ``heads``, ``vdim``, ``state``, ``groups`` and ``norm_groups`` (absent: 1), ``conv``;
``attention``: ``heads``, ``kv_heads`` (absent: as many), ``dim``, ``vdim`` (absent: ``dim``), ``scale`` (absent:
``dim ** -0.5``), ``mask.size`` (absent: every earlier position is seen), ``rot.{dims, base, scaling.factor}`` (absent: no
rotation; absent ``scaling``: the plain frequencies).
``mlp``: ``{"kind": "dense", "ff"}`` or ``{"kind": "moe", "expert": {ff}, "router": {experts, top}}``.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional

from .betepel import _number
from .errors import UnsupportedModelError
from .makodra import _need, _positive
from .miberax import MiberaxAttention

LAYER_TYPES = ("mamba2", "attention")
MLP_KINDS = ("dense", "moe")


@dataclass(frozen=True)
class RuroraxStateSpace:
    heads: int
    vdim: int
    state: int
    groups: int
    norm_groups: int
    conv: int

    @staticmethod
    def parse(m: Mapping[str, Any], where: str) -> "RuroraxStateSpace":
        sizes = {k: _positive(_need(m, k, where), f"{where}.{k}") for k in ("heads", "vdim", "state", "conv")}
        sizes.update({k: _positive(m.get(k) or 1, f"{where}.{k}") for k in ("groups", "norm_groups")})
        if sizes["heads"] % sizes["groups"]:
            raise UnsupportedModelError(f"{where}: {sizes['heads']} heads do not split into {sizes['groups']} groups")
        if sizes["heads"] * sizes["vdim"] % sizes["norm_groups"]:
            raise UnsupportedModelError(f"{where}: {sizes['heads']} heads of {sizes['vdim']} do not split into "
                                        f"norm_groups={sizes['norm_groups']} equal parts")
        if sizes["conv"] > 16:
            raise UnsupportedModelError(f"{where}.conv={sizes['conv']}: the convolution kernel takes up to 16 taps")
        return RuroraxStateSpace(**sizes)


def _attention(m: Mapping[str, Any], where: str) -> MiberaxAttention:
    """Miberax's attention has these keys; here a scale may be left out."""
    if m.get("scale") is None:
        m = dict(m, scale=_positive(_need(m, "dim", where), where + ".dim") ** -0.5)
    return MiberaxAttention.parse(m, where)


@dataclass(frozen=True)
class RuroraxMLP:
    kind: str
    ff: int                     # dense: the hidden size; moe: an expert's
    experts: int = 0
    top: int = 0

    @staticmethod
    def parse(raw: Mapping[str, Any], where: str) -> "RuroraxMLP":
        kind = raw.get("kind", "dense")
        if kind not in MLP_KINDS:
            raise UnsupportedModelError(f"{where}.kind={kind!r}; known: {MLP_KINDS}")
        if kind == "dense":
            return RuroraxMLP(kind, _positive(_need(raw, "ff", where), where + ".ff"))
        expert, router = _need(raw, "expert", where), _need(raw, "router", where)
        experts = _positive(_need(router, "experts", where + ".router"), where + ".router.experts")
        top = _positive(_need(router, "top", where + ".router"), where + ".router.top")
        if top > min(experts, 64):
            raise UnsupportedModelError(f"{where}.router: {top} of {experts} experts cannot be chosen (at most 64)")
        return RuroraxMLP(kind, _positive(_need(expert, "ff", where + ".expert"), where + ".expert.ff"), experts, top)


@dataclass(frozen=True)
class RuroraxLayer:
    type: str
    mixer: Any                  # RuroraxStateSpace or MiberaxAttention
    mlp: Optional[RuroraxMLP] = None

    @staticmethod
    def parse(raw: Mapping[str, Any], index: int) -> "RuroraxLayer":
        where = f"layers[{index}]"
        kind = _need(raw, "type", where)
        if kind not in LAYER_TYPES:
            raise UnsupportedModelError(f"{where}.type={kind!r}; known: {LAYER_TYPES}")
        parse = {"mamba2": RuroraxStateSpace.parse, "attention": _attention}[kind]
        return RuroraxLayer(kind, parse(_need(raw, "mixer", where), where + ".mixer"),
                            RuroraxMLP.parse(raw["mlp"], where + ".mlp") if raw.get("mlp") is not None else None)


@dataclass(frozen=True)
class RuroraxConfig:
    vocab: int
    width: int
    norm_eps: float
    logit_softcap: float        # 0: no cap
    layers: tuple[RuroraxLayer, ...]

    architecture = "Rurorax"

    # the names under which the engine's tools ask any configuration for its common sizes
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "RuroraxConfig":
        layers = _need(raw, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise UnsupportedModelError("layers must be a list with at least one layer")
        cap = _number(raw.get("logit_softcap") or 0.0, "logit_softcap")
        if cap < 0:
            raise UnsupportedModelError(f"logit_softcap={cap} must not be negative")
        return cls(vocab=_positive(_need(raw, "vocab", ""), "vocab"), width=_positive(_need(raw, "width", ""), "width"),
                   norm_eps=_number(_need(_need(raw, "norm", ""), "eps", "norm"), "norm.eps"), logit_softcap=cap,
                   layers=tuple(RuroraxLayer.parse(l, i) for i, l in enumerate(layers)))
