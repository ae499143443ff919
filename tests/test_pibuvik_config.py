"""Pibuvik without a GPU: the configuration's reader, its defaults and refusals, the list of parts it becomes, tensor
names and shapes against the plain implementation's own table, the layer that reads another's latents, and the
plain implementation's mechanisms against their definitions."""

from __future__ import annotations

import copy
import math

import pytest
import torch

import plain_pibuvik as P

F = torch.float64


def cfg_dict():
    latent = {"heads": 3, "dim": 8, "rot_dim": 6, "vdim": 12, "kv_rank": 20, "q_rank": 24, "scale": 0.3, "mask": {"size": 9},
              "rot": {"base": 1e4, "dims": 6}}
    reader = dict(latent, heads=2, dim=10, vdim=5, q_rank=7, scale=0.4, mask={"size": 15}, kv_from=0)
    mlp = {"kind": "dense", "ff": 20, "limit": 1.5}
    return {"architecture": "Pibuvik", "vocab": 50, "width": 48, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.5},
            "residual_mult": 0.4, "logit_scale": 0.7,
            "layers": [{"type": "latent_attention", "mixer": latent, "mlp": mlp},
                       {"type": "rglru", "mixer": {"width": 30, "blocks": 5, "conv": 4}, "mlp": None},
                       {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 10, "vdim": 10, "scale": 0.2,
                                                       "q_temp": {"coef": 0.6, "every": 11}}, "mlp": mlp},
                       {"type": "latent_attention", "mixer": reader, "mlp": dict(mlp, ff=33)}]}


def build(raw):
    from dli_amd.config.registry import resolve_architecture
    from dli_amd.parts import Runtime
    from dli_amd.parts.model import Model
    import dli_amd.architectures  # noqa: F401

    arch = resolve_architecture(raw)
    cfg = arch.parse_config(raw)
    return cfg, Model(arch.build_spec(cfg), Runtime(torch.device("cpu"), torch.float32))


def test_config_is_read_and_becomes_parts():
    from dli_amd.parts import PagedKVSpec, StateSpec

    cfg, model = build(cfg_dict())
    assert (cfg.architecture, cfg.vocab, cfg.width, cfg.norm_eps, cfg.embed_scale, cfg.residual_mult, cfg.logit_scale) == \
        ("Pibuvik", 50, 48, 1e-5, 2.5, 0.4, 0.7)
    assert [l.kv_from for l in cfg.layers] == [None, None, None, 0] and cfg.layers[1].mlp is None
    assert [l.parts["mixer"].kind for l in model.layers] == ["latent_attention", "gated_unit", "scored_attention", "latent_attention"]
    assert all(l.block.kind == "sandwich_norms" for l in model.layers)
    assert [e.cache_of for e in model.spec.schedule] == [None, None, None, 0]
    # the lender's pages keep what the reader's longer window sees; keys alone everywhere
    assert model.cache_specs() == [PagedKVSpec(1, 26, 15, 0), StateSpec((4 * 30,), torch.float32), PagedKVSpec(2, 10, 0, 0), None]
    a, b = model.layers[0].parts["mixer"], model.layers[3].parts["mixer"]
    assert (a.num_heads, a.head_dim, a.rot_dim, a.value_dim, a.kv_rank, a.q_rank, a.scale, a.window, a.own_kv) == (3, 8, 6, 12, 20, 24, 0.3, 9, True)
    assert (b.num_heads, b.head_dim, b.value_dim, b.q_rank, b.scale, b.window, b.own_kv) == (2, 10, 5, 7, 0.4, 15, False)
    att = model.layers[2].parts["mixer"]
    assert att.keys_as_values and att.head_sink and att.query_temperature == (0.6, 11.0) and (att.num_heads, att.num_kv_heads) == (4, 2)
    ff = model.layers[2].parts["feed_forward"]
    assert ff.clamped == (1.5, 1.702, 1.0) and ff.float32_out
    assert model.layers[2].parts["mixer_out_norm"].weight_scale == 0.4 and model.layers[2].parts["mixer_norm"].weight_scale == 1.0
    assert model.embedding.scale == 2.5 and model.head.tied and model.head.scale == 0.7
    assert "feed_forward" not in model.layers[1].parts and "feed_forward_out_norm" not in model.layers[1].parts


def test_what_is_left_out_has_its_plain_meaning():
    raw = cfg_dict()
    for key in ("embedding", "residual_mult", "logit_scale"):
        raw.pop(key)
    for l in raw["layers"]:
        l["mixer"] = dict(l["mixer"])
        for key in ("scale", "mask", "vdim", "q_temp", "kv_heads"):
            l["mixer"].pop(key, None)
    raw["layers"][0]["mixer"]["rot"] = {"base": 1e4}
    cfg, model = build(raw)
    assert (cfg.embed_scale, cfg.residual_mult, cfg.logit_scale) == (1.0, 1.0, 1.0)
    m = cfg.layers[0].mixer
    assert m.scale == (8 + 6) ** -0.5 and m.window == 0 and m.vdim == 8
    assert cfg.layers[2].mixer.kv_heads == 4 and cfg.layers[2].mixer.scale == 10 ** -0.5
    assert model.layers[2].parts["mixer"].query_temperature is None
    assert model.cache_specs()[0].window == 0


def test_a_lender_keeps_every_key_if_a_reader_sees_every_key():
    raw = cfg_dict()
    raw["layers"][3]["mixer"].pop("mask")
    _, model = build(raw)
    assert model.cache_specs()[0].window == 0 and model.layers[0].parts["mixer"].window == 9


def test_tensor_names_and_shapes_are_the_plain_table():
    raw = cfg_dict()
    _, model = build(raw)
    table = P.tensor_shapes(raw)
    specs = model.weight_specs()
    assert set(specs) == set(table)
    assert "l3.mix.dkv" not in specs and "l1.norm2" not in specs and "l2.mix.v" not in specs
    for name, shape in table.items():
        assert specs[name].fits(tuple(shape)), (name, shape, specs[name].shape)


def test_what_is_not_implemented_is_refused():
    from dli_amd.config.errors import ConfigError

    def broken(change):
        raw = copy.deepcopy(cfg_dict())
        change(raw)
        with pytest.raises(ConfigError):
            build(raw)

    broken(lambda r: r["layers"][0].__setitem__("type", "mla"))
    broken(lambda r: r["layers"][0]["mixer"].pop("kv_rank"))
    broken(lambda r: r["layers"][0]["mixer"].pop("rot"))
    broken(lambda r: r["layers"][0]["mixer"]["rot"].__setitem__("dims", 4))          # not the rotated part's size
    broken(lambda r: r["layers"][0]["mixer"]["rot"].__setitem__("scaling", {"factor": 2}))
    broken(lambda r: r["layers"][0]["mixer"]["mask"].__setitem__("keep_first", 2))
    broken(lambda r: r["layers"][1]["mixer"].__setitem__("blocks", 4))               # 30 channels in 4 parts
    broken(lambda r: r["layers"][2]["mixer"].__setitem__("vdim", 8))                 # the values are the keys
    broken(lambda r: r["layers"][2]["mixer"].__setitem__("kv_heads", 3))
    broken(lambda r: r["layers"][2]["mixer"]["q_temp"].__setitem__("every", 0))
    broken(lambda r: r["layers"][0]["mlp"].__setitem__("kind", "moe"))
    broken(lambda r: r["layers"][0]["mlp"].pop("limit"))
    broken(lambda r: r["layers"][3]["mixer"].__setitem__("kv_from", 3))              # itself
    broken(lambda r: r["layers"][3]["mixer"].__setitem__("kv_from", 1))              # a layer of another kind
    broken(lambda r: r["layers"][3]["mixer"].__setitem__("kv_rank", 16))             # another size than the lender's
    broken(lambda r: r["layers"][3]["mixer"].__setitem__("rot", {"base": 2e4, "dims": 6}))
    broken(lambda r: r["layers"].append(dict(r["layers"][3], mixer=dict(r["layers"][3]["mixer"], kv_from=3))))   # a borrower
    broken(lambda r: r.pop("norm"))


def test_sizes_that_no_kernel_takes_are_refused_when_the_model_is_built():
    from dli_amd.kernels.ops import KernelArgumentError

    raw = cfg_dict()
    raw["layers"][0]["mixer"]["kv_rank"] = raw["layers"][3]["mixer"]["kv_rank"] = 1020
    with pytest.raises(KernelArgumentError):
        build(raw)


def test_plain_mechanisms_agree_with_their_definitions():
    torch.manual_seed(0)
    # rotation: component i turns with i + dims/2; position 0 stays
    x = torch.randn(2, 4, dtype=F)
    y = P.rotate_half(x, torch.tensor([0, 3]), 100.0)
    assert torch.equal(y[0], x[0])
    a = 3 * 100.0 ** (-2 / 4)
    assert abs(y[1, 1] - (x[1, 1] * math.cos(a) - x[1, 3] * math.sin(a))) < 1e-12
    assert abs(y[1, 3] - (x[1, 3] * math.cos(a) + x[1, 1] * math.sin(a))) < 1e-12
    # a window of 4 sees itself and three before
    assert list(P.visible(9, 4)) == [6, 7, 8, 9] and list(P.visible(2, 4)) == [0, 1, 2] and list(P.visible(2, 0)) == [0, 1, 2]
    # the sink takes its share of the weight
    w = P.softmax_with_sink(torch.zeros(1, 3, dtype=F), torch.tensor([math.log(5.0)], dtype=F))
    assert torch.allclose(w, torch.full((1, 3), 1 / 8, dtype=F))
    # the temperature steps where p + 1 is a multiple
    t = P.query_temperature(torch.tensor([0, 9, 10, 18, 19]), 0.5, 10)
    assert torch.allclose(t, torch.tensor([1, 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(2),
                                           1 + 0.5 * math.log(3)], dtype=F))
    # the convolution's last column belongs to the current token, zeros (not biases) before the start
    x, w, b = torch.randn(4, 2, dtype=F), torch.randn(2, 3, dtype=F), torch.randn(2, dtype=F)
    st = {}
    y = P.causal_conv(x, w, b, st)
    assert torch.allclose(y[0], w[:, 2] * x[0] + b) and torch.allclose(y[2], w[:, 2] * x[2] + w[:, 1] * x[1] + w[:, 0] * x[0] + b)
    # a block maps its own part alone
    u, m = torch.randn(1, 4, dtype=F), torch.randn(2, 2, 2, dtype=F)
    assert torch.allclose(P.block_diagonal(u, m)[0], torch.cat([m[0] @ u[0, :2], m[1] @ u[0, 2:]]))
    # the recurrence's first token has no special case: sqrt(1 - a^2) i u
    u, r, i, lam = torch.randn(2, 1, dtype=F), torch.tensor([[0.5], [0.2]], dtype=F), torch.tensor([[0.3], [0.9]], dtype=F), torch.zeros(1, dtype=F)
    a = torch.exp(-8 * r * math.log(2.0))
    out, S = P.gated_unit(u, r, i, lam, None)
    s0 = torch.sqrt(1 - a[0] ** 2) * i[0] * u[0]
    assert torch.allclose(out[0], s0) and torch.allclose(S, a[1] * s0 + torch.sqrt(1 - a[1] ** 2) * i[1] * u[1])
    # clamps: the gate from above alone, the other half from both sides
    eye = torch.eye(3, dtype=F)
    h = torch.tensor([[5.0, -5.0, 1.0]], dtype=F)
    y = P.clamped_mlp(h, {"gate": eye, "up": eye, "down": eye}, 2.0)
    g, u = torch.tensor([2.0, -5.0, 1.0], dtype=F), torch.tensor([2.0, -2.0, 1.0], dtype=F)
    assert torch.allclose(y[0], g * P.sigmoid(1.702 * g) * (u + 1))


def test_the_plain_model_stepped_is_the_plain_model_whole():
    raw = cfg_dict()
    W = P.random_weights(raw, 3)
    toks = [(7 * i + 3) % 50 for i in range(33)]
    m = P.PlainPibuvik(raw, W)
    whole = m.forward(toks)
    st = m.new_state()
    parts, at = [], 0
    for n in (1, 2, 5, 1, 1, 23):
        parts.append(m.forward(toks[at:at + n], st))
        at += n
    assert (torch.cat(parts) - whole).abs().max() < 1e-9
