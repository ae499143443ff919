"""``Rurorax`` as a list of parts. Tensor names: ``embed``, ``final.norm``, and per layer ``i`` ``l<i>.norm1``, ``l<i>.ls1``,
``l<i>.ls2``, ``l<i>.mix.<name>`` and ``l<i>.mlp.<name>``; a norm's scalar and offset are ``<norm>.alpha`` and ``<norm>.b``, a
projection's bias is ``<name>.b``; the head is the embedding table. Every layer is the ``parallel_scaled``
arrangement around a 32-bit residual stream: one tanh in place of a norm, which mixer and feed-forward both read."""

from __future__ import annotations

from ..config.registry import register_architecture
from ..config.rurorax import RuroraxConfig
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry


def build_rurorax_spec(cfg: RuroraxConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps

    def norm(name: str, prefix: str) -> PartSpec:
        return PartSpec("tanh_norm", dict(width=w, weight_name=name), prefix)

    layers = []
    for i, layer in enumerate(cfg.layers):
        p, m, f = f"l{i}.", layer.mixer, layer.mlp
        if layer.type == "attention":
            position = None
            if m.rot_dims:
                position = PartSpec("rotary", dict(dim=m.rot_dims, theta=m.rot_base, pairing="half",
                                                   rope_type="linear" if m.rot_factor != 1.0 else "default", factor=m.rot_factor))
            mixer = PartSpec("scored_attention", dict(
                hidden_size=w, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim, scale=m.scale,
                qk_unit=False, qk_row_norm=True, norm_eps=eps, position=position, chunk=m.chunk, bias=True, out_bias=True,
                defer_output_bias=True), p + "mix.")
        else:
            mixer = PartSpec("state_space", dict(
                hidden_size=w, num_heads=m.heads, value_dim=m.vdim, state_size=m.state, groups=m.groups,
                norm_groups=m.norm_groups, conv_taps=m.conv, norm_eps=eps), p + "mix.")
        parts = {"mixer": ("mixer", mixer), "norm": ("norm", norm("norm1", p))}
        if f is not None and f.kind == "dense":
            parts["feed_forward"] = ("feed_forward", PartSpec("gated_mlp", dict(
                hidden_size=w, intermediate_size=f.ff, activation="gelu_tanh", bias=True, float32_out=True,
                names={"gate": "gate", "up": "up", "down": "down"}, bias_names={n: n + ".b" for n in ("gate", "up", "down")},
                defer_output_bias=True), p + "mlp."))
        elif f is not None:
            parts["feed_forward"] = ("feed_forward", PartSpec("routed_experts", dict(
                hidden_size=w, experts=f.experts, top=f.top, expert_size=f.ff, limit=float("inf"), alpha=1.0, up_shift=0.0,
                correction=False, scoring="sigmoid", normalize=False, weight_input=True), p + "mlp."))
        block = PartSpec("parallel_scaled", dict(hidden_size=w, scales={"mixer": "ls1", "feed_forward": "ls2"} if f is not None
                                                 else {"mixer": "ls1"}), p)
        layers.append(LayerSpec(block=block, parts=parts))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=w,
        embedding=PartSpec("token_embedding", dict(vocab_size=cfg.vocab, hidden_size=w, weight_name="embed", float32_rows=True)),
        layers=tuple(layers), schedule=tuple(ScheduleEntry(i) for i in range(len(layers))), final_norm=norm("norm", "final."),
        head=PartSpec("linear_head", dict(vocab_size=cfg.vocab, hidden_size=w, tied=True, softcap=cfg.logit_softcap)))


register_architecture("Rurorax", RuroraxConfig.from_dict, build_rurorax_spec, model_types=("rurorax",), replace=True)
