"""``Pibuvik`` as a list of parts. Tensor names: ``embed``, ``final.norm``, and per layer ``i`` ``l<i>.norm1``, ``l<i>.norm1b``,
``l<i>.norm2``, ``l<i>.norm2b``, ``l<i>.mix.<name>`` and ``l<i>.mlp.<name>``; the head is the embedding table. Every layer is the
``sandwich_norms`` arrangement around a 32-bit residual stream; its mixer is attention through a latent (which may
read an earlier layer's latents), a gated unit recurrence, or attention whose values are its keys; its feed-forward
a gated product with clamped halves, or absent."""

from __future__ import annotations

from typing import Optional

from ..config.pibuvik import PibuvikAttention, PibuvikConfig, PibuvikLatent, PibuvikRecurrence
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

GATE_ALPHA, UP_SHIFT = 1.702, 1.0      # g sigmoid(1.702 g) (u + 1)
DECAY_RATE = 8.0                       # log a = -8 r softplus(lam)


def build_pibuvik_spec(cfg: PibuvikConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps

    def norm(name: str, prefix: str, scale: float = 1.0) -> tuple:
        return ("norm", PartSpec("rms_norm", dict(width=w, eps=eps, weight_name=name, weight_scale=scale), prefix))

    def kept_keys(i: int) -> Optional[int]:
        """What layer ``i``'s pages must keep for itself and for the layers that read them: every key (0) if one of
        them sees every earlier position, else the longest of their windows."""
        windows = [cfg.layers[i].mixer.window] + [l.mixer.window for l in cfg.layers if l.kv_from == i]
        return 0 if 0 in windows else max(windows)

    def mixer(i: int, m: object, prefix: str) -> PartSpec:
        if isinstance(m, PibuvikLatent):
            return PartSpec("latent_attention", dict(
                hidden_size=w, num_heads=m.heads, head_dim=m.dim, value_dim=m.vdim, kv_rank=m.kv_rank, q_rank=m.q_rank,
                scale=m.scale, norm_eps=eps, head_gate=True, window=m.window, rot_dim=m.rot_dim,
                position=PartSpec("rotary", dict(dim=m.rot_dim, theta=m.rot_base, pairing="half")),
                own_kv=m.kv_from is None, cache_window=kept_keys(i) if m.kv_from is None else None), prefix)
        if isinstance(m, PibuvikRecurrence):
            return PartSpec("gated_unit", dict(hidden_size=w, inner_size=m.width, blocks=m.blocks, conv_taps=m.conv,
                                               decay_rate=DECAY_RATE), prefix)
        assert isinstance(m, PibuvikAttention)
        return PartSpec("scored_attention", dict(
            hidden_size=w, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, scale=m.scale, qk_unit=False,
            keys_as_values=True, head_sink=True, query_temperature=(m.temp_coef, m.temp_every) if m.temp_coef else None), prefix)

    layers, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        parts = {"mixer_norm": norm("norm1", p), "mixer": ("mixer", mixer(i, layer.mixer, p + "mix.")),
                 "mixer_out_norm": norm("norm1b", p, cfg.residual_mult)}
        f = layer.mlp
        if f is not None:
            parts["feed_forward_norm"] = norm("norm2", p)
            parts["feed_forward"] = ("feed_forward", PartSpec("gated_mlp", dict(
                hidden_size=w, intermediate_size=f.ff, activation="clamped", limit=f.limit, alpha=GATE_ALPHA, up_shift=UP_SHIFT,
                float32_out=True, names={"gate": "gate", "up": "up", "down": "down"}), p + "mlp."))
            parts["feed_forward_out_norm"] = norm("norm2b", p, cfg.residual_mult)
        layers.append(LayerSpec(block=PartSpec("sandwich_norms"), parts=parts))
        schedule.append(ScheduleEntry(i, cache_of=layer.kv_from))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=w,
        embedding=PartSpec("token_embedding", dict(vocab_size=cfg.vocab, hidden_size=w, weight_name="embed",
                                                   float32_rows=True, scale=cfg.embed_scale)),
        layers=tuple(layers), schedule=tuple(schedule), final_norm=norm("norm", "final.")[1],
        head=PartSpec("linear_head", dict(vocab_size=cfg.vocab, hidden_size=w, tied=True, scale=cfg.logit_scale)))


register_architecture("Pibuvik", PibuvikConfig.from_dict, build_pibuvik_spec, model_types=("pibuvik",), replace=True)
