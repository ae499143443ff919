"""Rurorax without a GPU: the configuration's reader, its defaults and refusals, the list of parts it becomes, tensor
names and shapes against the plain implementation's own table, and the plain implementation's mechanisms
against their definitions."""

from __future__ import annotations

import copy
import math

import pytest
import torch

import plain_rurorax as P

F = torch.float64


def cfg_dict():
    att = {"heads": 6, "kv_heads": 3, "dim": 10, "vdim": 7, "scale": 0.3, "mask": {"size": 9},
           "rot": {"dims": 6, "base": 1e4, "scaling": {"factor": 4.0}}}
    ssm = {"heads": 6, "vdim": 5, "state": 12, "groups": 2, "norm_groups": 3, "conv": 3}
    dense = {"kind": "dense", "ff": 20}
    moe = {"kind": "moe", "expert": {"ff": 14}, "router": {"experts": 5, "top": 2}}
    return {"architecture": "Rurorax", "vocab": 50, "width": 48, "norm": {"eps": 1e-5}, "logit_softcap": 12.0,
            "layers": [{"type": "mamba2", "mixer": ssm, "mlp": dense}, {"type": "attention", "mixer": att, "mlp": moe},
                       {"type": "mamba2", "mixer": dict(ssm, heads=3, groups=1, norm_groups=1, conv=1), "mlp": None}]}


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
    assert (cfg.architecture, cfg.vocab, cfg.width, cfg.norm_eps, cfg.logit_softcap, cfg.num_layers) == ("Rurorax", 50, 48, 1e-5, 12.0, 3)
    assert [l.parts["mixer"].kind for l in model.layers] == ["state_space", "scored_attention", "state_space"]
    assert all(l.block.kind == "parallel_scaled" and l.parts["norm"].kind == "tanh_norm" for l in model.layers)
    # S (heads x state x vdim), then taps - 1 inputs of x, B and C
    assert model.cache_specs() == [StateSpec((6 * 12 * 5 + 2 * (30 + 48),), torch.float32), PagedKVSpec(3, 10, 0, 7),
                                   StateSpec((3 * 12 * 5,), torch.float32)]
    s = model.layers[0].parts["mixer"]
    assert (s.num_heads, s.value_dim, s.state_size, s.groups, s.norm_groups, s.taps, s.norm_eps) == (6, 5, 12, 2, 3, 3, 1e-5)
    a = model.layers[1].parts["mixer"]
    assert (a.num_heads, a.num_kv_heads, a.head_dim, a.value_dim, a.scale, a.chunk, a.norm_eps) == (6, 3, 10, 7, 0.3, 9, 1e-5)
    assert a.qk_row_norm and a.bias and a.out_bias and a.defer_output_bias and not a.qk_unit
    table = a.position.rotary_table()
    want = [1e4 ** (-2 * i / 6) / 4 for i in range(3)]
    assert table.dim == 6 and table.pairing == "half" and torch.allclose(table.inv_freq.double(), torch.tensor(want, dtype=F), rtol=1e-6)
    f = model.layers[0].parts["feed_forward"]
    assert f.activation == "gelu_tanh" and f.bias and f.float32_out and f.defer_output_bias
    e = model.layers[1].parts["feed_forward"]
    assert (e.experts, e.top, e.expert_size, e.scoring, e.normalize, e.weight_input, e.has_correction) == (5, 2, 14, "sigmoid", False, True, False)
    assert "feed_forward" not in model.layers[2].parts and set(model.layers[2].block.scale_names) == {"mixer"}
    assert model.head.tied and model.head.softcap == 12.0


def test_what_is_left_out_has_its_plain_meaning():
    raw = cfg_dict()
    raw.pop("logit_softcap")
    for key in ("kv_heads", "vdim", "scale", "mask", "rot"):
        raw["layers"][1]["mixer"].pop(key)
    for key in ("groups", "norm_groups"):
        raw["layers"][0]["mixer"].pop(key)
    cfg, model = build(raw)
    a, s = cfg.layers[1].mixer, cfg.layers[0].mixer
    assert cfg.logit_softcap == 0.0 and model.head.softcap == 0.0
    assert (a.kv_heads, a.vdim, a.scale, a.chunk, a.rot_dims) == (6, 10, 10 ** -0.5, 0, 0) and (s.groups, s.norm_groups) == (1, 1)
    assert model.layers[1].parts["mixer"].position.rotary_table() is None
    raw["layers"][1]["mixer"]["rot"] = {"dims": 4, "base": 50.0}
    _, model = build(raw)
    assert torch.allclose(model.layers[1].parts["mixer"].position.rotary_table().inv_freq, torch.tensor([1.0, 50.0 ** -0.5]))


def test_tensor_names_and_shapes_are_the_plain_table():
    raw = cfg_dict()
    _, model = build(raw)
    table, specs = P.tensor_shapes(raw), model.weight_specs()
    assert set(specs) == set(table)
    assert "l2.ls2" not in specs and "l1.mix.o.b" in specs and "l0.mix.o.b" not in specs and "final.norm.alpha" in specs
    for name, shape in table.items():
        assert specs[name].fits(tuple(shape)), (name, shape, specs[name].shape)


def test_what_is_not_implemented_is_refused():
    from dli_amd.config.errors import ConfigError

    def broken(change):
        raw = copy.deepcopy(cfg_dict())
        change(raw)
        with pytest.raises(ConfigError):
            build(raw)

    broken(lambda r: r["layers"][0].__setitem__("type", "mamba3"))
    broken(lambda r: r["layers"][0]["mixer"].pop("state"))
    broken(lambda r: r["layers"][0]["mixer"].__setitem__("groups", 4))            # 6 heads in 4 groups
    broken(lambda r: r["layers"][0]["mixer"].__setitem__("norm_groups", 4))       # 30 values in 4 parts
    broken(lambda r: r["layers"][0]["mixer"].__setitem__("conv", 17))
    broken(lambda r: r["layers"][0]["mixer"].__setitem__("heads", True))
    broken(lambda r: r["layers"][1]["mixer"].__setitem__("kv_heads", 4))
    broken(lambda r: r["layers"][1]["mixer"]["rot"].__setitem__("dims", 5))
    broken(lambda r: r["layers"][1]["mixer"]["rot"].__setitem__("dims", 12))      # more than a head has
    broken(lambda r: r["layers"][1]["mixer"]["rot"]["scaling"].__setitem__("low", 1.0))
    broken(lambda r: r["layers"][1]["mixer"]["mask"].__setitem__("keep_first", 2))
    broken(lambda r: r["layers"][1]["mlp"]["router"].__setitem__("top", 6))
    broken(lambda r: r["layers"][1]["mlp"].__setitem__("kind", "table"))
    broken(lambda r: r["layers"][0]["mlp"].pop("ff"))
    broken(lambda r: r.__setitem__("logit_softcap", -1.0))
    broken(lambda r: r.__setitem__("layers", []))
    broken(lambda r: r.pop("norm"))


def test_parts_refuse_what_no_kernel_computes():
    from dli_amd.parts import PartSpec, Runtime, build_part

    rt = Runtime(torch.device("cpu"), torch.float32)
    attention = dict(hidden_size=16, num_heads=2, num_kv_heads=1, head_dim=8, qk_unit=False)
    for family, kind, params in (
            ("mixer", "scored_attention", dict(attention, qk_unit=True, qk_row_norm=True)),
            ("mixer", "scored_attention", dict(attention, qk_row_norm=True, own_kv=False)),
            ("mixer", "scored_attention", dict(attention, defer_output_bias=True)),
            ("feed_forward", "gated_mlp", dict(hidden_size=16, intermediate_size=8, activation="relu")),
            ("feed_forward", "gated_mlp", dict(hidden_size=16, intermediate_size=8, activation="clamped", bias=True)),
            ("feed_forward", "gated_mlp", dict(hidden_size=16, intermediate_size=8, bias=True, names={"gate": "g"})),
            ("feed_forward", "gated_mlp", dict(hidden_size=16, intermediate_size=8, defer_output_bias=True)),
            ("feed_forward", "routed_experts", dict(hidden_size=16, experts=4, top=1, expert_size=8, limit=1.0, scoring="tanh")),
            ("feed_forward", "routed_experts", dict(hidden_size=16, experts=4, top=1, expert_size=8, limit=1.0, identity=1, weight_input=True)),
            ("mixer", "state_space", dict(hidden_size=16, num_heads=3, value_dim=4, state_size=8, groups=2)),
            ("mixer", "state_space", dict(hidden_size=16, num_heads=3, value_dim=4, state_size=8, conv_taps=17)),
            ("block", "parallel_scaled", dict(hidden_size=16, scales={"norm": "s"}))):
        with pytest.raises(ValueError):
            build_part(family, PartSpec(kind, params), rt)


def test_plain_mechanisms_agree_with_their_definitions():
    torch.manual_seed(0)
    # rotation: component i turns with i + dims/2, slowed by the factor; position 0 stays, the rest of the head passes
    x = torch.randn(2, 1, 5, dtype=F)
    y = P.rotate(x, torch.tensor([0, 3]), {"dims": 4, "base": 100.0, "scaling": {"factor": 2.0}})
    assert torch.equal(y[0], x[0]) and y[1, 0, 4] == x[1, 0, 4]
    a = 3 * 100.0 ** (-2 / 4) / 2
    assert abs(y[1, 0, 1] - (x[1, 0, 1] * math.cos(a) - x[1, 0, 3] * math.sin(a))) < 1e-12
    assert abs(y[1, 0, 3] - (x[1, 0, 3] * math.cos(a) + x[1, 0, 1] * math.sin(a))) < 1e-12
    # chunks are counted from position 0
    assert [j for j in range(12) if P.visible(9, j, 4)] == [8, 9] and [j for j in range(12) if P.visible(11, j, 4)] == [8, 9, 10, 11]
    assert [j for j in range(5) if P.visible(3, j, None)] == [0, 1, 2, 3]
    # the convolution's last column belongs to the current token, zeros before the start
    x, w, b = torch.randn(4, 2, dtype=F), torch.randn(2, 3, dtype=F), torch.randn(2, dtype=F)
    y, kept = P.convolve(x, w, b, None)
    assert torch.allclose(y[0], w[:, 2] * x[0] + b) and torch.allclose(y[2], w[:, 2] * x[2] + w[:, 1] * x[1] + w[:, 0] * x[0] + b)
    assert torch.equal(kept, x[2:]) and P.convolve(x, w[:, :1], b, None)[1].shape == (0, 2)
    # the recurrence: two heads on one group, the second token's decay is the step size times exp(a_log)
    x, B, C = torch.randn(2, 2, 3, dtype=F), torch.randn(2, 1, 4, dtype=F), torch.randn(2, 1, 4, dtype=F)
    dt, a_log, d = torch.tensor([[0.3, 0.7], [0.2, 0.5]], dtype=F), torch.tensor([0.1, -0.4], dtype=F), torch.tensor([2.0, 0.0], dtype=F)
    y, S = P.state_space(x, B, C, dt, a_log, d, None)
    s0 = 0.7 * torch.outer(B[0, 0], x[0, 1])
    s1 = math.exp(-math.exp(-0.4) * 0.5) * s0 + 0.5 * torch.outer(B[1, 0], x[1, 1])
    assert torch.allclose(S[1], s1) and torch.allclose(y[1, 1], s1.t() @ C[1, 0])
    assert torch.allclose(y[0, 0], 0.3 * (B[0, 0] @ C[0, 0]) * x[0, 0] + 2 * x[0, 0])
    # the gate comes before the norm, each part by its own root mean square
    v, z, w = torch.randn(1, 6, dtype=F), torch.randn(1, 6, dtype=F), torch.rand(6, dtype=F)
    g = v * z * P.sigmoid(z)
    assert torch.allclose(P.gated_parts_norm(v, z, w, 2, 0.0)[0, 3:], g[0, 3:] / g[0, 3:].pow(2).mean().sqrt() * w[3:])
    # scores are not divided by their sum, and they scale what an expert reads
    ids, s = P.choose(torch.tensor([[0.0, 2.0, -1.0, 1.0]], dtype=F), 2)
    assert ids.tolist() == [[1, 3]] and torch.allclose(s, P.sigmoid(torch.tensor([[2.0, 1.0]], dtype=F)))
    eye = torch.eye(2, dtype=F)
    p = {"router": torch.tensor([[1.0, 0.0], [0.0, 1.0]], dtype=F), **{f"e{e}.{n}": (e + 1) * eye for e in (0, 1) for n in ("gate", "up", "down")}}
    h = torch.tensor([[0.5, 3.0]], dtype=F)
    u = 2 * P.sigmoid(torch.tensor(3.0, dtype=F)) * h
    assert torch.allclose(P.experts(h, p, {"router": {"top": 1}}), 2 * u * P.sigmoid(u) * u)
    assert abs(P.gelu_tanh(torch.tensor(1.0, dtype=F)) - 0.8411919906) < 1e-9
    assert torch.allclose(P.softplus(torch.tensor([-40.0, 0.0, 50.0], dtype=F)), torch.tensor([math.exp(-40), math.log(2), 50.0], dtype=F))


def test_the_plain_model_stepped_is_the_plain_model_whole():
    raw = cfg_dict()
    W = P.random_weights(raw, 3)
    toks = [(7 * i + 3) % 50 for i in range(33)]
    m = P.PlainRurorax(raw, W)
    whole = m.forward(toks)
    st = m.new_state()
    parts, at = [], 0
    for n in (1, 2, 5, 1, 1, 23):
        parts.append(m.forward(toks[at:at + n], st, start=at))
        at += n
    assert (torch.cat(parts) - whole).abs().max() < 1e-9
