"""Typed configuration of the Pibuvik decoder: a list of layers, each ``x <- x + m norm1b(mixer(norm1(x)))`` then
``x <- x + m norm2b(ff(norm2(x)))`` (norms before and after every sublayer, one constant ``m`` for the whole model), with
one of three mixers: attention through a latent with a rotated key part under a sliding window
(``latent_attention``, which may read an earlier layer's cached latents), a gated linear recurrence per channel
behind a short convolution (``rglru``), or attention whose values are its keys, with a sink per head and a
temperature on the queries (``attention``); and a dense feed-forward with clamped gates, or none. The embedded
rows are scaled by a constant, the head is the embedding table, its logits times another.

``config.json`` keys: ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``residual_mult``, ``logit_scale`` (the last three
absent: 1) and ``layers``: a list of ``{"type", "mixer": {...}, "mlp": {"kind": "dense", "ff", "limit"} | null}``.
Mixer keys by type:
``latent_attention``: ``heads``, ``dim``, ``rot_dim``, ``vdim`` (absent: ``dim``), ``kv_rank``, ``q_rank``, ``rot.{base, dims}``
(``dims`` equals ``rot_dim``), ``mask.size`` (absent: every earlier position), ``scale`` (absent: ``(dim + rot_dim) ** -0.5``),
``kv_from`` (an earlier layer of this type that has latents of its own, of equal ``kv_rank``, ``rot_dim`` and ``rot``);
``rglru``: ``width``, ``blocks``, ``conv``;
``attention``: ``heads``, ``kv_heads`` (absent: as many), ``dim``, ``vdim`` (equals ``dim``), ``scale`` (absent: ``dim ** -0.5``),
``q_temp.{coef, every}`` (absent: none).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional

from .betepel import _number, _unknown
from .errors import UnsupportedModelError
from .makodra import _need, _positive

LAYER_TYPES = ("latent_attention", "rglru", "attention")
MLP_KINDS = ("dense",)


@dataclass(frozen=True)
class PibuvikLatent:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    rot_base: float
    scale: float
    window: int = 0                  # mask.size (0: every earlier position is seen)
    kv_from: Optional[int] = None

    @staticmethod
    def parse(m: Mapping[str, Any], where: str) -> "PibuvikLatent":
        sizes = {k: _positive(_need(m, k, where), f"{where}.{k}") for k in ("heads", "dim", "rot_dim", "kv_rank", "q_rank")}
        rot = _need(m, "rot", where)
        _unknown(rot, ("base", "dims"), where + ".rot")
        if rot.get("dims", sizes["rot_dim"]) != sizes["rot_dim"] or sizes["rot_dim"] % 2:
            raise UnsupportedModelError(f"{where}.rot.dims={rot.get('dims')!r} must be rot_dim={sizes['rot_dim']}, an even number")
        mask = dict(m.get("mask") or {})
        _unknown(mask, ("size",), where + ".mask")
        kv_from = m.get("kv_from")
        if kv_from is not None and (isinstance(kv_from, bool) or not isinstance(kv_from, int) or kv_from < 0):
            raise UnsupportedModelError(f"{where}.kv_from={kv_from!r} must name a layer")
        return PibuvikLatent(
            **sizes, vdim=_positive(m.get("vdim") or sizes["dim"], where + ".vdim"),
            rot_base=_number(_need(rot, "base", where + ".rot"), where + ".rot.base"),
            scale=_number(m["scale"], where + ".scale") if m.get("scale") is not None else (sizes["dim"] + sizes["rot_dim"]) ** -0.5,
            window=_positive(mask["size"], where + ".mask.size") if mask.get("size") is not None else 0, kv_from=kv_from)


@dataclass(frozen=True)
class PibuvikRecurrence:
    width: int
    blocks: int
    conv: int

    @staticmethod
    def parse(m: Mapping[str, Any], where: str) -> "PibuvikRecurrence":
        sizes = {k: _positive(_need(m, k, where), f"{where}.{k}") for k in ("width", "blocks", "conv")}
        if sizes["width"] % sizes["blocks"]:
            raise UnsupportedModelError(f"{where}: {sizes['width']} channels do not split into {sizes['blocks']} equal blocks")
        return PibuvikRecurrence(**sizes)


@dataclass(frozen=True)
class PibuvikAttention:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    temp_coef: float = 0.0           # q_temp.coef (0: no temperature)
    temp_every: float = 1.0          # q_temp.every

    @staticmethod
    def parse(m: Mapping[str, Any], where: str) -> "PibuvikAttention":
        heads, dim = (_positive(_need(m, k, where), f"{where}.{k}") for k in ("heads", "dim"))
        kv = _positive(m.get("kv_heads") or heads, where + ".kv_heads")
        if heads % kv:
            raise UnsupportedModelError(f"{where}: {heads} heads do not group onto {kv} kv_heads")
        if (m.get("vdim") or dim) != dim:
            raise UnsupportedModelError(f"{where}.vdim={m['vdim']!r}: the values are the keys, of dim={dim}")
        temp = dict(m.get("q_temp") or {})
        _unknown(temp, ("coef", "every"), where + ".q_temp")
        coef = _number(_need(temp, "coef", where + ".q_temp"), where + ".q_temp.coef") if temp else 0.0
        every = _number(_need(temp, "every", where + ".q_temp"), where + ".q_temp.every") if temp else 1.0
        if not every > 0:
            raise UnsupportedModelError(f"{where}.q_temp.every={every!r} must be positive")
        return PibuvikAttention(heads=heads, kv_heads=kv, dim=dim, temp_coef=coef, temp_every=every,
                                scale=_number(m["scale"], where + ".scale") if m.get("scale") is not None else dim ** -0.5)


@dataclass(frozen=True)
class PibuvikMLP:
    ff: int
    limit: float

    @staticmethod
    def parse(raw: Mapping[str, Any], where: str) -> "PibuvikMLP":
        kind = raw.get("kind", "dense")
        if kind not in MLP_KINDS:
            raise UnsupportedModelError(f"{where}.kind={kind!r}; known: {MLP_KINDS}")
        limit = _number(_need(raw, "limit", where), where + ".limit")
        if not limit > 0:
            raise UnsupportedModelError(f"{where}.limit={limit!r} must be positive")
        return PibuvikMLP(ff=_positive(_need(raw, "ff", where), where + ".ff"), limit=limit)


@dataclass(frozen=True)
class PibuvikLayer:
    type: str
    mixer: Any                       # PibuvikLatent, PibuvikRecurrence or PibuvikAttention
    mlp: Optional[PibuvikMLP] = None

    @property
    def kv_from(self) -> Optional[int]:
        return self.mixer.kv_from if self.type == "latent_attention" else None

    @staticmethod
    def parse(raw: Mapping[str, Any], index: int) -> "PibuvikLayer":
        where = f"layers[{index}]"
        kind = _need(raw, "type", where)
        if kind not in LAYER_TYPES:
            raise UnsupportedModelError(f"{where}.type={kind!r}; known: {LAYER_TYPES}")
        parse = {"latent_attention": PibuvikLatent, "rglru": PibuvikRecurrence, "attention": PibuvikAttention}[kind].parse
        return PibuvikLayer(kind, parse(_need(raw, "mixer", where), where + ".mixer"),
                            PibuvikMLP.parse(raw["mlp"], where + ".mlp") if raw.get("mlp") is not None else None)


@dataclass(frozen=True)
class PibuvikConfig:
    vocab: int
    width: int
    norm_eps: float
    embed_scale: float
    residual_mult: float
    logit_scale: float
    layers: tuple[PibuvikLayer, ...]

    architecture = "Pibuvik"

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
    def from_dict(cls, raw: Mapping[str, Any]) -> "PibuvikConfig":
        layers = _need(raw, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise UnsupportedModelError("layers must be a list with at least one layer")
        parsed = tuple(PibuvikLayer.parse(l, i) for i, l in enumerate(layers))
        for i, layer in enumerate(parsed):
            j = layer.kv_from
            if j is None:
                continue
            if j >= i or parsed[j].type != "latent_attention" or parsed[j].kv_from is not None:
                raise UnsupportedModelError(f"layers[{i}].mixer.kv_from={j} must name an earlier latent_attention layer with "
                                            "latents of its own")
            a, b = layer.mixer, parsed[j].mixer
            if (a.kv_rank, a.rot_dim, a.rot_base) != (b.kv_rank, b.rot_dim, b.rot_base):
                raise UnsupportedModelError(f"layers[{i}] reads the latents of layers[{j}], whose kv_rank, rot_dim or rotation differ")
        return cls(vocab=_positive(_need(raw, "vocab", ""), "vocab"), width=_positive(_need(raw, "width", ""), "width"),
                   norm_eps=_number(_need(_need(raw, "norm", ""), "eps", "norm"), "norm.eps"),
                   embed_scale=_number((raw.get("embedding") or {}).get("scale", 1.0), "embedding.scale"),
                   residual_mult=_number(raw.get("residual_mult", 1.0), "residual_mult"),
                   logit_scale=_number(raw.get("logit_scale", 1.0), "logit_scale"), layers=parsed)
