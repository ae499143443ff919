"""Rurorax on the GPU against the plain float64 implementation of ``plain_rurorax.py``: every mechanism's kernel
alone, then whole models of several small shapes through the engine's step function, cache manager, scheduler
and entry points, however the requests are cut and batched.
"""

from __future__ import annotations

import math
import random

import pytest
import torch

import plain_rurorax as P

pytestmark = pytest.mark.gpu
F = torch.float64


def i32(values):
    return torch.tensor(list(values), dtype=torch.int32).cuda()


@pytest.fixture(scope="module")
def ops():
    from dli_amd.kernels import ops as o

    o.library()
    return o


def step_arrays(entries):
    """``entries``: (slot, first position, rows) of a step -> q_start, positions, state_slots on the device."""
    starts, pos = [0], []
    for _, p0, n in entries:
        starts.append(starts[-1] + n)
        pos += list(range(p0, p0 + n))
    return i32(starts), i32(pos), i32([e[0] for e in entries])


def in_steps(requests, plan, run):
    """Walks ``plan`` (steps of (request, rows)) over ``requests`` (name -> (slot, rows tensor)): ``run(rows,
    q_start, positions, slots)`` gets the step's stacked rows and returns the step's results, which are
    handed back request by request, in order."""
    at = {r: 0 for r in requests}
    got = {r: [] for r in requests}
    for step in plan:
        entries, rows = [], []
        for r, n in step:
            slot, x = requests[r]
            entries.append((slot, at[r], n))
            rows.append(x[at[r]:at[r] + n])
        out = run(torch.cat(rows).cuda(), *step_arrays(entries))
        r0 = 0
        for r, n in step:
            got[r].append(out[r0:r0 + n].cpu())
            r0 += n
            at[r] += n
    assert all(at[r] == requests[r][1].shape[0] for r in requests)
    return {r: torch.cat(v) for r, v in got.items()}


# a plan over three requests through two slots: "c" starts in "a"'s slot once "a" has ended
PLAN = [[("a", 3), ("b", 1)], [("a", 1), ("b", 4)], [("b", 1), ("a", 2)], [("a", 17), ("b", 2)], [("a", 1)], [("a", 40), ("b", 30)],
        [("c", 1), ("b", 1)], [("c", 1)], [("c", 2), ("b", 35)], [("c", 60)]]
LENGTHS = {"a": 64, "b": 74, "c": 64}
SLOTS = {"a": 1, "b": 0, "c": 1}


# ------------------------------------------------------------------------------ small kernels

@pytest.mark.parametrize("width", [5, 64, 260, 1030, 5000])
def test_sums_into_the_stream_and_the_tanh_that_follows(ops, width):
    torch.manual_seed(width)
    n = 7
    x, a, b = torch.randn(n, width), torch.randn(n, width + 4), torch.randn(n, width)
    s1, s2, c, w, o = (torch.randn(width) for _ in range(5))
    alpha = 0.63
    D = lambda t: t.double()
    for dtype, tol in ((torch.float32, 5e-6), (torch.bfloat16, 6e-3)):
        for first, second, scaled, const in ((True, True, True, True), (True, False, True, False), (True, True, False, True), (False, False, False, False)):
            ref = D(x)
            if first:
                ref = ref + D(a[:, 4:]) * (D(s1) if scaled else 1) + (D(b) * (D(s2) if scaled else 1) if second else 0) + (D(c) if const else 0)
            want = P.tanh_norm(ref, torch.tensor(alpha, dtype=F), D(w), D(o))
            xs, out = x.cuda(), torch.empty(n, width, dtype=dtype).cuda()
            kw = dict(a=a.cuda()[:, 4:], b=b.cuda() if second else None, a_scale=s1.cuda() if scaled else None,
                      b_scale=s2.cuda() if scaled and second else None, constant=c.cuda() if const else None) if first else {}
            ops.tanh_norm_stream(xs, norm=(alpha, w.cuda(), o.cuda()), out=out, **kw)
            assert (xs.cpu().double() - ref).abs().max() < 2e-6 * ref.abs().max()
            assert (out.cpu().double() - want).abs().max() < tol * want.abs().max(), (dtype, first, second)
            if first:
                alone = x.cuda()
                ops.tanh_norm_stream(alone, **kw)                      # the sum without a norm: the same bits
                assert torch.equal(alone, xs)
            else:
                assert torch.equal(xs.cpu(), x)


def test_the_norm_part_applies_itself(ops):
    from dli_amd.parts.base import Runtime
    from dli_amd.parts.norm import TanhNorm

    torch.manual_seed(1)
    norm = TanhNorm(Runtime(torch.device("cuda"), torch.float32), width=70, weight_name="w")
    w, b, alpha = torch.randn(70), torch.randn(70), torch.tensor(1.7)
    norm.load_weights({"w": w.cuda(), "w.b": b.cuda(), "w.alpha": alpha.cuda()})
    x, delta = 2 * torch.randn(3, 70), torch.randn(3, 70)
    xs = x.cuda()
    ref = P.tanh_norm(x.double() + delta.double(), alpha.double(), w.double(), b.double())
    assert (norm.forward(xs, delta.cuda()).cpu().double() - ref).abs().max() < 1e-5
    assert torch.equal(xs.cpu(), x + delta)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 5e-6), (torch.bfloat16, 8e-3)])
@pytest.mark.parametrize("at", [3, 4], ids=["unaligned", "aligned"])
@pytest.mark.parametrize("parts,size", [(1, 40), (3, 24), (2, 96), (1, 300), (4, 520), (5, 1), (2, 2052), (1, 4096), (1, 4100)])
def test_gate_before_the_norm_in_parts(ops, parts, size, at, dtype, tol):
    torch.manual_seed(parts * 7 + size)
    n, width = 6, parts * size
    y, z, w = 2 * torch.randn(n, width), 2 * torch.randn(n, width + 4), 1 + 0.3 * torch.randn(width)
    ref = P.gated_parts_norm(y.double(), z.double()[:, at:at + width], w.double(), parts, 1e-4)
    out = torch.empty(n, width, dtype=dtype).cuda()
    ops.head_norm_gate(y.cuda(), z.cuda()[:, at:at + width], w.cuda(), 1e-4, out, parts, size, gate="silu_first")
    assert (out.cpu().double() - ref).abs().max() < tol * ref.abs().max()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [9, 150])
@pytest.mark.parametrize("more", [3, 4], ids=["rows_unaligned", "rows_aligned"])
@pytest.mark.parametrize("qh,kh,d,dv,rot_dims", [(6, 2, 24, 10, 16), (3, 1, 5, 8, 2), (4, 4, 64, 80, 64), (6, 3, 24, 16, 8), (8, 2, 40, 40, 0),
                                                 (4, 2, 20, 12, 12), (1, 1, 130, 3, 128)])
def test_norms_over_whole_projections_before_the_rotation(ops, dtype, n, more, qh, kh, d, dv, rot_dims):
    """q and k, heads of very different size, each by one root mean square over all heads; biases first, rotation last, v untouched."""
    g = torch.Generator().manual_seed(qh * 10 + d)
    cols, ps = (qh + kh) * d + kh * dv, 4
    size = torch.cat([torch.linspace(0.1, 3.0, cols), torch.ones(more)])
    proj, bias = torch.randn(n, cols + more, generator=g) * size, torch.randn(cols + more, generator=g)
    qw, kw = 1 + 0.3 * torch.randn(qh * d, generator=g), 1 + 0.3 * torch.randn(kh * d, generator=g)
    rot = {"dims": rot_dims, "base": 100.0, "scaling": {"factor": 3.0}} if rot_dims else None
    pos = torch.tensor([0, 1, 2, 700, 701, 5, 9000, 3, 4] + list(range(9, n)))
    slots = torch.randperm(4 * n, generator=g)[:n]
    slots[7] = -1
    kp, vp = torch.zeros(n, kh, ps, d, dtype=dtype).cuda(), torch.zeros(n, kh, dv, ps, dtype=dtype).cuda()
    q = torch.empty(n, qh * d, dtype=dtype).cuda()
    inv = P.rotary_frequencies(rot).float().cuda() if rot else None
    ops.rotary_cache(proj.cuda(), 0, qh * d, (qh + kh) * d, i32(pos.tolist()), inv, rot_dims, False, q, i32(slots.tolist()), kp, vp,
                     qh, bias=bias.cuda(), row_norm=(qw.cuda(), kw.cuda(), 1e-4))
    full = proj.double() + bias.double()
    q_ref = P.rotate((P.rms(full[:, :qh * d], 1e-4) * qw.double()).view(n, qh, d), pos, rot)
    k_ref = P.rotate((P.rms(full[:, qh * d:(qh + kh) * d], 1e-4) * kw.double()).view(n, kh, d), pos, rot)
    v_ref = full[:, (qh + kh) * d:cols].view(n, kh, dv)
    tol = 1e-4 if dtype == torch.float32 else 2e-2    # (32-bit frequencies: an angle at position 9000 is good to 1e-3)
    assert (q.cpu().double().view(n, qh, d) - q_ref).abs().max() < tol * q_ref.abs().max()
    for t in range(n):
        s = int(slots[t])
        if s < 0:
            continue
        assert (kp[s // ps, :, s % ps].cpu().double() - k_ref[t]).abs().max() < tol * k_ref.abs().max()
        assert (vp[s // ps, :, :, s % ps].cpu().double() - v_ref[t]).abs().max() < tol * v_ref.abs().max()
    unused = [s for s in range(4 * n) if s not in slots.tolist()]
    assert all(not kp[s // ps, :, s % ps].any() and not vp[s // ps, :, :, s % ps].any() for s in unused[:20])


@pytest.mark.parametrize("rows", [1, 3, 8, 16, 40, 300])
@pytest.mark.parametrize("width,ff", [(64, 96), (128, 256), (256, 40), (40, 20)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_gelu_gate_with_biases(ops, rows, width, ff, dtype):
    """The part itself, few rows (the activation inside the product) and many; the output bias added here or left to the block."""
    from dli_amd.parts import PartSpec, Runtime, build_part

    torch.manual_seed(rows + width)
    t = torch.float32 if dtype == "float32" else torch.bfloat16
    rt = Runtime(torch.device("cuda"), t)
    W = {"g": torch.randn(ff, width) / width ** 0.5 * 2, "u": torch.randn(ff, width) / width ** 0.5, "d": torch.randn(width, ff) / ff ** 0.5,
         "g.b": torch.randn(ff), "u.b": torch.randn(ff), "d.b": torch.randn(width)}
    W = {k: v.to(torch.bfloat16) for k, v in W.items()}
    h = (2 * torch.randn(rows, width)).to(torch.bfloat16)
    p = {("gate" if k[0] == "g" else "up" if k[0] == "u" else "down") + k[1:]: v.double() for k, v in W.items()}
    ref = P.dense(h.double(), p)
    for defer in (False, True):
        names = {"gate": "g", "up": "u", "down": "d"}
        mlp = build_part("feed_forward", PartSpec("gated_mlp", dict(
            hidden_size=width, intermediate_size=ff, activation="gelu_tanh", bias=True, float32_out=True, names=names,
            bias_names={k: v + ".b" for k, v in names.items()}, defer_output_bias=defer)), rt)
        mlp.load_weights({k: v.to(t).cuda() for k, v in W.items()})
        mlp.finalize()
        got = mlp.forward(h.to(t).cuda(), None)
        assert got.dtype == torch.float32 and (mlp.output_bias is not None) == defer
        got = got.cpu().double() + (p["down.b"] if defer else 0)
        assert (got - ref).abs().max() < (1e-5 if dtype == "float32" else 2e-2) * ref.abs().max()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n,experts,top,width,ff", [(1, 4, 1, 64, 32), (9, 5, 2, 40, 12), (70, 12, 3, 64, 96), (33, 3, 3, 96, 64), (200, 70, 1, 32, 32),
                                                      (300, 4, 2, 256, 128), (513, 5, 3, 128, 64), (260, 5, 1, 384, 192)])
def test_sigmoid_scores_scale_what_the_experts_read(ops, dtype, n, experts, top, width, ff):
    """Scores as they are, largest first, on the experts' inputs: with weights below one half of the result that
    a weight on the output would give differs, since the activation bends."""
    torch.manual_seed(n + experts)
    h = (2 * torch.randn(n, width)).to(torch.bfloat16)
    z = torch.randn(n, experts)
    gate, up, down = ((torch.randn(experts, *s) / s[1] ** 0.5 * 2).to(torch.bfloat16) for s in ((ff, width), (ff, width), (width, ff)))
    ids, w = torch.empty(n, top, dtype=torch.int32).cuda(), torch.empty(n, top).cuda()
    wide = torch.cat([z, 99 * torch.ones(n, 2)], dim=1).cuda()                        # (columns past the router's are not its own)
    ops.router_choose(wide, experts, None, 1, 1, top, 1.0, ids, w, sigmoid=True, normalize=False)
    want_ids, want_w = P.choose(z.double(), top)
    assert torch.equal(ids.cpu().long(), want_ids) and (w.cpu().double() - want_w).abs().max() < 1e-6
    args = [t.to(dtype).cuda() for t in (h, gate, up, down)]
    zs = ops.expert_products(ids, *args, float("inf"), 1.0, 0.0, in_weights=w)
    out = torch.empty(n, width).cuda()
    ops.expert_combine(ids, None, zs, args[0], experts, out)
    p = {f"e{e}.{k}": m[e].double() for e in range(experts) for k, m in (("gate", gate), ("up", up), ("down", down))}
    ref = torch.zeros(n, width, dtype=F)
    on_outputs = torch.zeros(n, width, dtype=F)
    for t in range(n):
        for e, s in zip(want_ids[t].tolist(), want_w[t]):
            mine = (p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"])
            ref[t] += P.expert(s * h[t:t + 1].double(), *mine)[0]
            on_outputs[t] += s * P.expert(h[t:t + 1].double(), *mine)[0]
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert (out.cpu().double() - ref).abs().max() < tol * ref.abs().max()
    assert (on_outputs - ref).abs().max() > 0.05 * ref.abs().max()


def test_softmax_scores_without_their_sum(ops):
    torch.manual_seed(4)
    z = torch.randn(11, 6)
    ids, w = torch.empty(11, 2, dtype=torch.int32).cuda(), torch.empty(11, 2).cuda()
    ops.router_choose(z.cuda(), 6, None, 1, 1, 2, 1.5, ids, w, normalize=False)
    s = torch.softmax(z.double(), dim=1)
    assert (w.cpu().double() - 1.5 * s.gather(1, ids.cpu().long())).abs().max() < 1e-6
    ops.router_choose(z.cuda(), 6, None, 1, 1, 2, 1.5, ids, w, sigmoid=True)
    s = P.sigmoid(z.double()).gather(1, ids.cpu().long())
    assert (w.cpu().double() - 1.5 * s / s.sum(1, keepdim=True)).abs().max() < 1e-6


# ------------------------------------------------------------------------------ the state-space recurrence

def scan(ops, rows, state, q_start, positions, slots, H, G, N, V, p, **kw):
    """rows ``[n, x | B | C | dt]`` -> y ``[n, H * V]``."""
    x1, b1, c1 = H * V, H * V + G * N, H * V + 2 * G * N
    o = torch.empty(rows.shape[0], H * V).cuda()
    ops.scalar_gate_scan(rows[:, b1:c1], rows[:, x1:b1], rows[:, :x1], state, q_start, positions, slots, o, H, N, V, qk_heads=G,
                         step=rows[:, c1:c1 + H], step_bias=p["bias"].cuda(), step_rate=p["a_log"].cuda(), skip=p["d"].cuda(), **kw)
    return o


def plain_scan(x, H, G, N, V, p):
    x = x.double()
    n, x1, b1, c1 = x.shape[0], H * V, H * V + G * N, H * V + 2 * G * N
    y, S = P.state_space(x[:, :x1].reshape(n, H, V), x[:, x1:b1].reshape(n, G, N), x[:, b1:c1].reshape(n, G, N),
                         P.softplus(x[:, c1:] + p["bias"].double()), p["a_log"].double(), p["d"].double(), None)
    return y.reshape(n, H * V), S


def scan_params(H, g):
    """Decays from a token to thousands of tokens, step sizes around a tenth."""
    return {"bias": -2 + torch.randn(H, generator=g), "a_log": torch.linspace(-6.0, 2.0, H) if H > 1 else torch.tensor([-3.0]),
            "d": torch.randn(H, generator=g)}


SHAPES = [(2, 1, 8, 6), (4, 2, 32, 48), (6, 3, 16, 20), (1, 1, 64, 16), (8, 1, 64, 64), (3, 3, 20, 70), (4, 2, 128, 64), (2, 2, 128, 3),
          (5, 1, 48, 1), (2, 1, 96, 40), (4, 4, 80, 33), (3, 1, 200, 9), (2, 1, 112, 100)]


@pytest.mark.parametrize("chunked", [True, False])
@pytest.mark.parametrize("H,G,N,V", SHAPES)
def test_state_space_in_steps_against_whole(ops, H, G, N, V, chunked):
    """Three requests through two slots that held rubbish, steps of every kind."""
    g = torch.Generator().manual_seed(H * 100 + N + V)
    p, width = scan_params(H, g), H * V + 2 * G * N + H
    reqs = {r: (SLOTS[r], torch.randn(n, width, generator=g)) for r, n in LENGTHS.items()}
    floats = H * V * N
    state = torch.full((3, floats + 5), 55.0).cuda()
    got = in_steps(reqs, PLAN, lambda rows, qs, pos, sl: scan(ops, rows, state, qs, pos, sl, H, G, N, V, p, chunked=chunked))
    for r, (slot, x) in reqs.items():
        ref, S = plain_scan(x, H, G, N, V, p)
        assert (got[r].double() - ref).abs().max() < 1e-5 * max(1.0, ref.abs().max()), (r, (got[r].double() - ref).abs().max())
        if r != "a":                                                        # ("c" holds "a"'s slot by now); kept column by column
            held = state[slot, :floats].cpu().double().view(H, V, N).transpose(1, 2)
            assert (held - S).abs().max() < 1e-5 * max(1.0, S.abs().max())
    assert (state[:, floats:] == 55.0).all()


@pytest.mark.parametrize("H,G,N,V", [(4, 2, 32, 48), (2, 1, 128, 64), (3, 3, 16, 20), (2, 1, 20, 7), (4, 1, 96, 33)])
def test_state_space_over_long_portions(ops, H, G, N, V):
    """Portions of many chunks beside short ones and single tokens, one of them on top of an earlier state."""
    g = torch.Generator().manual_seed(N + V)
    p, width = scan_params(H, g), H * V + 2 * G * N + H
    lengths = {"a": 1300, "b": 700, "c": 3}
    reqs = {r: (i, torch.randn(n, width, generator=g)) for i, (r, n) in enumerate(lengths.items())}
    state = torch.full((3, H * V * N), -9.0).cuda()
    plan = [[("a", 131), ("b", 1)], [("b", 1), ("a", 1029), ("c", 2)], [("c", 1), ("a", 64), ("b", 513)], [("a", 1), ("b", 128)], [("b", 57), ("a", 75)]]
    got = in_steps(reqs, plan, lambda rows, qs, pos, sl: scan(ops, rows, state, qs, pos, sl, H, G, N, V, p))
    for r, (slot, x) in reqs.items():
        ref, S = plain_scan(x, H, G, N, V, p)
        assert (got[r].double() - ref).abs().max() < 2e-5 * max(1.0, ref.abs().max()), r
        held = state[slot].cpu().double().view(H, V, N).transpose(1, 2)
        assert (held - S).abs().max() < 2e-5 * max(1.0, S.abs().max())


def scan_tiles(ops, rows, state, q_start, positions, slots, H, G, N, V, p, singles_scanned=False):
    """The same with x, B and C rounded to bfloat16, in tiles on the matrix cores (``singles_scanned``: entries of one row,
    which must come first, by the scan)."""
    x1, b1, c1 = H * V, H * V + G * N, H * V + 2 * G * N
    n = rows.shape[0]
    xbc = torch.empty(n, c1, dtype=torch.bfloat16).cuda()
    xbc.copy_(rows[:, :c1])
    o = torch.full((n, H * V), 77.0).cuda()
    starts = q_start.tolist()
    lengths = [b - a for a, b in zip(starts, starts[1:])]
    step, rule = rows[:, c1:c1 + H], dict(qk_heads=G, step_bias=p["bias"].cuda(), step_rate=p["a_log"].cuda(), skip=p["d"].cuda())
    nd = next((i for i, m in enumerate(lengths) if m > 1), len(lengths)) if singles_scanned else 0
    if nd:
        ops.scalar_gate_scan(xbc[:nd, b1:], xbc[:nd, x1:b1], xbc[:nd, :x1], state, q_start[:nd + 1], positions[:nd], slots[:nd], o[:nd],
                             H, N, V, step=step[:nd], **rule)
    tile = ops.state_space_tile_rows()
    ent = [e for e in range(nd, len(lengths)) for _ in range(0, lengths[e], tile)]
    q0 = [q for e in range(nd, len(lengths)) for q in range(0, lengths[e], tile)]
    if ent:
        ops.state_space_tiles(xbc[:, b1:], xbc[:, x1:b1], xbc[:, :x1], state, q_start, positions, slots, (i32(ent), i32(q0)), o, H, N, V,
                              step=step, **rule)
    return o


def rounded_inputs(x, H, G, N, V):
    c1 = H * V + 2 * G * N
    return torch.cat([x[:, :c1].to(torch.bfloat16).float(), x[:, c1:]], dim=1)


@pytest.mark.parametrize("singles_scanned", [False, True])
@pytest.mark.parametrize("H,G,N,V", [(2, 1, 32, 8), (4, 2, 32, 48), (8, 1, 64, 64), (4, 2, 128, 64), (2, 1, 96, 40), (3, 3, 128, 104), (2, 2, 64, 136)])
def test_state_space_in_tiles_against_whole(ops, H, G, N, V, singles_scanned):
    """Portions shorter and longer than a tile and a tile's block, on fresh and on earlier states, beside single tokens."""
    g = torch.Generator().manual_seed(N + V)
    p, width = scan_params(H, g), H * V + 2 * G * N + H
    lengths = {"a": 1300, "b": 700, "c": 5, "d": 64}
    reqs = {r: (i, torch.randn(n, width, generator=g)) for i, (r, n) in enumerate(lengths.items())}
    floats = H * V * N
    state = torch.full((4, floats + 4), -9.0).cuda()
    plan = [[("b", 1), ("a", 131)], [("b", 1), ("a", 1029), ("c", 2)], [("c", 1), ("a", 63), ("b", 513)], [("a", 1), ("c", 2), ("b", 128)],
            [("b", 57), ("a", 76), ("d", 64)]]
    got = in_steps(reqs, plan, lambda rows, qs, pos, sl: scan_tiles(ops, rows, state, qs, pos, sl, H, G, N, V, p, singles_scanned))
    for r, (slot, x) in reqs.items():
        ref, S = plain_scan(rounded_inputs(x, H, G, N, V), H, G, N, V, p)
        # (the results' second operands are sums of two bfloat16 numbers: 2^-17; the state itself is 32-bit)
        assert (got[r].double() - ref).abs().max() < 5e-5 * max(1.0, ref.abs().max()), (r, (got[r].double() - ref).abs().max())
        held = state[slot, :floats].cpu().double().view(H, V, N).transpose(1, 2)
        assert (held - S).abs().max() < 1e-5 * max(1.0, S.abs().max()), (r, (held - S).abs().max())
    assert (state[:, floats:] == -9.0).all()


def test_tiles_forget_and_remember(ops):
    """Pre-activations of -60 and +60 token by token, a head that hardly decays and one that forgets within a token: the
    factors span what 32-bit holds, and a value written 700 tokens ago is found again."""
    H, G, N, V, n = 2, 1, 32, 8, 900
    g = torch.Generator().manual_seed(3)
    p = {"bias": torch.zeros(H), "a_log": torch.tensor([-30.0, 3.0]), "d": torch.tensor([0.0, 0.5])}
    rows = torch.randn(n, H * V + 2 * G * N + H, generator=g)
    rows[:, -H:] = torch.where(torch.rand(n, H, generator=g) < 0.7, torch.tensor(-60.0), torch.tensor(60.0))
    rows[200:, H * V:H * V + N] = 0.0                           # nothing is written from here on
    ref, S = plain_scan(rounded_inputs(rows, H, G, N, V), H, G, N, V, p)
    state = torch.full((1, H * V * N), 5.0).cuda()
    got = in_steps({"a": (0, rows)}, [[("a", 500)], [("a", 1)], [("a", 399)]],
                   lambda r, qs, pos, sl: scan_tiles(ops, r, state, qs, pos, sl, H, G, N, V, p, True))["a"]
    assert ref[700:, :V].abs().max() > 10
    assert (got.double() - ref).abs().max() < 5e-5 * ref.abs().max()
    assert (state[0].cpu().double().view(H, V, N).transpose(1, 2) - S).abs().max() < 1e-5 * S.abs().max()


@pytest.mark.parametrize("N", [16, 128, 20])
def test_a_state_written_long_ago_is_still_there(ops, N):
    """A head that hardly decays: what the first token wrote answers a query 900 tokens later, over portions and single
    tokens; the head that decays fast has forgotten it."""
    H, G, V, n = 2, 1, 8, 900
    p = {"bias": torch.zeros(H), "a_log": torch.tensor([-30.0, 3.0]), "d": torch.zeros(H)}
    rows = torch.zeros(n, H * V + 2 * G * N + H)
    rows[:, -H:] = 1.0
    rows[0, H * V + 3] = 1.0                                    # B
    rows[0, 5], rows[0, V + 5] = 2.0, 2.0                       # value 5 of both heads
    rows[n - 1, H * V + N + 3] = 1.0                            # the last C asks for it
    state = torch.full((2, H * V * N), 3.0).cuda()
    got = in_steps({"a": (1, rows)}, [[("a", 500)], *[[("a", 1)]] * 20, [("a", 370)], *[[("a", 1)]] * 10],
                   lambda r, qs, pos, sl: scan(ops, r, state, qs, pos, sl, H, G, N, V, p))["a"]
    dt = math.log1p(math.e)
    assert abs(float(got[n - 1, 5]) - 2 * dt) < 1e-5 and abs(float(got[n - 1, V + 5])) < 1e-30
    assert float(got[n - 1].abs().sum()) - 2 * dt < 1e-5


def test_step_sizes_at_both_ends(ops):
    """Pre-activations of -60 and +60: a step of nearly nothing leaves the state, a step of 60 forgets it."""
    H, G, N, V, n = 2, 1, 16, 4, 70
    g = torch.Generator().manual_seed(9)
    p = {"bias": torch.zeros(H), "a_log": torch.zeros(H), "d": torch.tensor([0.0, 1.5])}
    rows = torch.randn(n, H * V + 2 * G * N + H, generator=g)
    rows[:, -H:] = torch.where(torch.rand(n, H, generator=g) < 0.5, torch.tensor(-60.0), torch.tensor(60.0))
    ref, _ = plain_scan(rows, H, G, N, V, p)
    for plan in ([[("a", n)]], [[("a", 1)]] * n):
        state = torch.zeros(1, H * V * N).cuda()
        got = in_steps({"a": (0, rows)}, plan, lambda r, qs, pos, sl: scan(ops, r, state, qs, pos, sl, H, G, N, V, p))["a"]
        assert (got.double() - ref).abs().max() < 1e-5 * ref.abs().max()


# ------------------------------------------------------------------------------ attention in chunks

def paged(x, page_size, dtype, order, transposed):
    """``x [tokens, heads, dim]`` into pages in the order of ``order`` (a shuffled list of page numbers)."""
    n, heads, dim = x.shape
    pages = max(order) + 1
    out = torch.zeros(pages, heads, dim, page_size, dtype=dtype) if transposed else torch.zeros(pages, heads, page_size, dim, dtype=dtype)
    for t in range(n):
        if transposed:
            out[order[t // page_size], :, :, t % page_size] = x[t].to(dtype)
        else:
            out[order[t // page_size], :, t % page_size] = x[t].to(dtype)
    return out.cuda()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("qh,kh,d,dv,size,ps", [(4, 2, 16, 32, 24, 4), (8, 2, 48, 16, 65, 16), (2, 2, 32, 32, 9, 4), (3, 1, 20, 12, 30, 4),
                                                (4, 4, 64, 80, 64, 8), (6, 1, 64, 64, 128, 16), (2, 1, 128, 96, 1, 4), (5, 1, 64, 48, 100, 16)])
def test_planted_keys_at_the_edges_of_chunks(ops, dtype, qh, kh, d, dv, size, ps):
    """One direction stands out for the queries around a chunk's edge: a query must find the planted keys of its own
    chunk (its first, its own place) and none of the chunk before; through the tile kernel, the matrix-core kernel and
    the single-token kernel, with pages in shuffled order."""
    n = 150
    g = torch.Generator().manual_seed(qh * 31 + size)
    order = torch.randperm(-(-n // ps) + 3, generator=g).tolist()
    scale = 0.5
    k, v, q = 0.3 * torch.randn(n, kh, d, generator=g), torch.randn(n, kh, dv, generator=g), 0.3 * torch.randn(n, qh, d, generator=g)
    edge = size * (140 // size)                             # a chunk begins here
    edge = edge if edge >= 5 else n - 10                    # (a chunk longer than the sequence: nothing is hidden)
    direction = torch.randn(d, generator=g)
    direction /= direction.norm()
    planted = [0, edge - size, edge - 1, edge, edge + 2]
    for i in (edge - 1, edge, edge + 1, min(edge + size - 1, n - 1), min(edge + size, n - 1), n - 1):
        q[i] = 6.0 * direction
    for c, j in enumerate(p for p in planted if 0 <= p < n):
        k[j] = 3.0 * direction * (1 + 0.1 * c)
        v[j] = 5.0 + c
    q, k, v = (t.to(torch.bfloat16).double() for t in (q, k, v))
    ref = P.chunked_attention(q, k, v, 0, scale, size)
    if size > 1 and edge % size == 0:
        assert ref[edge, :, 0].min() > 7.9                 # its own key, at least: none of the 5 to 7 from before
    kp, vp = paged(k, ps, dtype, order, False), paged(v, ps, dtype, order, True)
    table = i32(order + [0, 0]).view(1, -1)
    tol = 2e-5 if dtype == torch.float32 else 3e-2

    def check(out, rows, what):
        err = (out.cpu().double().view(-1, qh, dv) - ref[rows]).abs().max()
        assert err < tol * ref.abs().max(), (what, float(err))

    qd = q.reshape(n, qh * d).to(dtype).cuda()
    for first in (0, 120):
        rows, m = slice(first, n), n - first
        tile_rows = ops.attention_generic_tile_rows(max(d, dv))
        ent, q0 = i32([0] * len(range(0, m, tile_rows))), i32(range(0, m, tile_rows))
        out = torch.empty(m, qh * dv, dtype=dtype).cuda()
        ops.attention_scored(qd[rows], kp, vp, out, i32([0, m]), i32([n]), table, ent, q0, qh, scale, chunk=size)
        check(out, rows, ("tiles", first))
        if dtype == torch.bfloat16 and ops.attention_scored_mfma_supports(d, dv, ps, dtype):
            ent, q0 = i32([0] * len(range(0, m, 64))), i32(range(0, m, 64))
            out = torch.empty(m, qh * dv, dtype=dtype).cuda()
            ops.attention_scored_mfma(qd[rows], kp, vp, out, i32([0, m]), i32([n]), table, ent, q0, qh, scale, chunk=size)
            check(out, rows, ("matrix cores", first))
        if dtype == torch.bfloat16 and ops.attention_grouped_supports(d, dv, ps, dtype):
            tokens = ops.attention_grouped_tile_tokens(qh, kh)
            ent, q0 = i32([0] * len(range(0, m, tokens))), i32(range(0, m, tokens))
            out = torch.empty(m, qh * dv, dtype=dtype).cuda()
            ops.attention_grouped(qd[rows], kp, vp, out, i32([0, m]), i32([n]), table, ent, q0, qh, scale, chunk=size)
            check(out, rows, ("grouped", first))
    for t in range(100, n, 3):
        rows = [t, min(t + 1, n - 1), min(t + 2, n - 1)]
        out = torch.empty(3, qh * dv, dtype=dtype).cuda()
        ops.attention_scored(qd[rows], kp, vp, out, i32([0, 1, 2, 3]), i32([r + 1 for r in rows]), table.repeat(3, 1).contiguous(),
                             None, None, qh, scale, chunk=size)
        check(out, rows, ("single", t))


def plain_masked(q, k, v, first, scale, low, keep, sink, v_heads):
    """Softmax over ``low(i) <= j <= i`` and ``j < keep``, ``exp(sink[h])`` more in the denominator; key head ``g`` reads value head
    ``g % v_heads``."""
    n, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(n, H, v.shape[2], dtype=F)
    for t in range(n):
        i = first + t
        seen = [j for j in range(i + 1) if j >= low(i) or j < keep]
        for h in range(H):
            g = h // (H // G)
            w = torch.exp(k[seen, g] @ q[t, h] * scale)
            out[t, h] = (w @ v[seen, g % v_heads]) / (w.sum() + (math.exp(sink[h]) if sink is not None else 0.0))
    return out


@pytest.mark.parametrize("out32", [False, True])
@pytest.mark.parametrize("qh,kh,vh,d,dv,window,chunk,keep,sink,gated,ps", [
    (4, 2, 2, 64, 64, 70, 0, 0, True, False, 16), (8, 4, 2, 40, 128, 33, 0, 70, False, False, 8), (6, 2, 1, 128, 20, 64, 90, 5, True, True, 16),
    (3, 3, 3, 8, 4, 0, 0, 0, False, True, 8), (66, 1, 1, 16, 48, 0, 50, 0, True, False, 16), (5, 1, 1, 104, 112, 1, 0, 1, False, False, 32),
    (4, 4, 2, 24, 100, 100, 64, 3, True, True, 8), (2, 1, 1, 96, 96, 200, 0, 130, False, False, 16)])
def test_grouped_attention_with_every_change(ops, qh, kh, vh, d, dv, window, chunk, keep, sink, gated, ps, out32):
    """Windows, kept first positions, chunks, sinks, gates, shared value heads, in two entries on one list of tiles (one a
    portion on top of earlier keys), against the plain softmax; a negative scale once."""
    g = torch.Generator().manual_seed(qh * 7 + d)
    lens, news = [190, 75], [97, 75]
    scale = (-1 if kh == 3 else 1) * d ** -0.5
    need = [-(-n // ps) for n in lens]
    order = torch.randperm(sum(need) + 2, generator=g).tolist()
    orders = [order[:need[0]], order[need[0]:need[0] + need[1]]]
    kp, vp = torch.zeros(len(order), kh, ps, d, dtype=torch.bfloat16).cuda(), torch.zeros(len(order), vh, dv, ps, dtype=torch.bfloat16).cuda()
    sinks = torch.randn(qh, generator=g) if sink else None
    qs, refs = [], []
    low = lambda i: max(i - window + 1 if window else 0, i // chunk * chunk if chunk else 0)
    for n, m, o in zip(lens, news, orders):
        q, k, v = (torch.randn(n, h, s, generator=g).to(torch.bfloat16) for h, s in ((qh, d), (kh, d), (vh, dv)))
        for t in range(n):
            kp[o[t // ps], :, t % ps] = k[t].cuda()
            vp[o[t // ps], :, :, t % ps] = v[t].cuda()
        qs.append(q[n - m:])
        ref = torch.zeros(m, qh, dv, dtype=F)
        for t in range(m):                                     # (kept positions count within the query's own chunk alone)
            i = n - m + t
            start = i // chunk * chunk if chunk else 0
            ref[t] = plain_masked(q[i:i + 1].double(), k[start:].double(), v[start:].double(), i - start, scale, lambda x: low(x + start) - start,
                                  max(0, keep - start) if window else 0, sinks, vh)[0]
        refs.append(ref)
    q = torch.cat(qs).reshape(sum(news), qh * d).cuda()
    gate = torch.randn(sum(news), qh * dv, generator=g) if gated else None
    ref = torch.cat(refs).reshape(sum(news), qh * dv)
    if gated:
        ref = ref * P.sigmoid(gate.double())
    table = i32([p for o in orders for p in (o + [0] * max(need))[:max(need)]]).view(2, max(need))
    tokens = ops.attention_grouped_tile_tokens(qh, kh)
    ent = [e for e, m in enumerate(news) for _ in range(0, m, tokens)]
    q0 = [x for m in news for x in range(0, m, tokens)]
    out = torch.empty(sum(news), qh * dv, dtype=torch.float32 if out32 else torch.bfloat16).cuda()
    ops.attention_grouped(q, kp, vp, out, i32([0, news[0], sum(news)]), i32(lens), table, i32(ent), i32(q0), qh, scale, window=window,
                          chunk=chunk, keep_first=keep, sinks=sinks.cuda() if sink else None, gate=gate.cuda() if gated else None)
    assert (out.cpu().double() - ref).abs().max() < 2e-2 * ref.abs().max()


# ------------------------------------------------------------------------------ whole models

def attention(heads, kv, dim, vdim, size, rot=None, factor=None, base=1000.0, scale=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}
    if size:
        m["mask"] = {"size": size}
    if rot:
        m["rot"] = {"dims": rot, "base": base, **({"scaling": {"factor": factor}} if factor else {})}
    return {"type": "attention", "mixer": m}


def mamba(heads, vdim, state, groups, norm_groups, conv):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(width, vocab, cap, layers, eps=1e-5):
    return {"architecture": "Rurorax", "vocab": vocab, "width": width, "norm": {"eps": eps}, **({"logit_softcap": cap} if cap else {}),
            "layers": [dict(mixer, mlp=mlp) for mixer, mlp in layers]}


CONFIGS = {
    "varied": config(48, 50, 8.0, [(mamba(4, 6, 8, 2, 2, 4), dense(20)), (attention(4, 2, 8, 12, 11, 4, 4.0), moe(5, 2, 20)),
                                   (mamba(3, 10, 12, 1, 1, 2), moe(3, 1, 12)), (attention(6, 3, 6, 6, 25, 6), dense(28)),
                                   (mamba(4, 6, 8, 4, 4, 3), dense(12))]),
    # sizes that the matrix-core kernels take, chunks longer than a tile of keys
    "aligned": config(64, 90, 20.0, [(attention(4, 2, 32, 16, 130, 16, 2.0), dense(96)), (mamba(4, 32, 16, 2, 1, 4), moe(4, 1, 32)),
                                     (attention(8, 2, 16, 32, 64, 16), moe(6, 3, 32)), (mamba(2, 64, 64, 1, 2, 4), dense(64)),
                                     (mamba(2, 16, 128, 2, 2, 4), None)]),
}
MORE_CONFIGS = {
    # sizes that nothing aligns, one head, no mask, no rotation, no cap, no feed-forward, one tap, all experts chosen
    "odd": config(40, 33, None, [(attention(1, 1, 12, 5, None), None), (mamba(1, 7, 5, 1, 1, 1), moe(2, 2, 10)),
                                 (attention(3, 3, 6, 7, 200, 2, 3.0, 3.0), dense(9)), (mamba(5, 3, 20, 5, 3, 7), None),
                                 (attention(2, 1, 10, 10, 1, 10), moe(6, 1, 8))], eps=1e-3),
}
CONFIGS_ALL = {**CONFIGS, **MORE_CONFIGS}
_MODELS: dict = {}


def model(name: str, tmp_root):
    if name not in _MODELS:
        cfg = CONFIGS_ALL[name]
        W = P.random_weights(cfg, seed=len(name) * 7 + 1)
        if name == "aligned":                                   # sharp attention: a query's weight lies on few keys, near or far
            W = {k: (v * 2).to(torch.bfloat16).double() if k.endswith((".q.norm", ".k.norm")) else v for k, v in W.items()}
        _MODELS[name] = (cfg, W, P.write_folder(tmp_root / name, cfg, W))
    return _MODELS[name]


@pytest.fixture(scope="module")
def tmp_root(tmp_path_factory):
    return tmp_path_factory.mktemp("rurorax")


def session(folder, dtype, pages=40, page_size=16, max_seqs=4, graphs=False):
    from dli_amd.engine.core import build_core
    from dli_amd.trace import TraceSession

    class Session(TraceSession):
        """Logits of a replayed graph are a view of its output buffer, good until the next step:
        the tests keep every step's rows, so they take copies."""

        def step(self, entries, end=()):
            return super().step(entries, end).clone()

    core = build_core(folder, num_pages=pages, page_size=page_size, max_seqs=max_seqs, dtype=dtype,
                      enable_prefix_caching=False, watermark=0.0)
    if graphs:
        core.step.enable_decode_graphs(max_seqs, pages * page_size)
    return Session(core)


_REFS: dict = {}


def reference(name, W, cfg, toks, dtype):
    """The plain logits; how far each row moves when the matrices are jittered by bfloat16's rounding (the larger of
    two draws): what rounding of that size may do to the row; and the closest choice of experts of each row and the
    three before it (which it reads through a convolution)."""
    key = (name, tuple(toks))
    if key not in _REFS:
        margins = [torch.full((len(toks),), math.inf, dtype=F)]
        ref = P.PlainRurorax(cfg, W).forward(toks, margins=margins)
        moved = [(P.PlainRurorax(cfg, P.jittered(W, seed=j)).forward(toks) - ref).abs().max(dim=-1, keepdim=True).values for j in (0, 5)]
        closest = torch.stack(margins).min(dim=0).values
        closest = torch.stack([closest[max(0, t - 3):t + 1].min() for t in range(len(toks))])
        _REFS[key] = (ref, torch.maximum(*moved), closest[:, None])
    return _REFS[key]


def rows_of(ref, rows):
    return tuple(r[rows] for r in ref)


def close(got: torch.Tensor, ref, dtype: str, what) -> None:
    """In 32-bit every row is held, and that is where a fault of the cache, the state or a chunk's edge shows. In bfloat16 a
    row may be off by bfloat16's usual share of its largest logit and a few times what a jitter of the matrices by
    bfloat16's rounding does to it; a row whose router's last choice was closer than rounding may decide is let go."""
    ref, moved, margin = ref
    got, ref = got.double().cpu(), ref.double()
    assert got.shape == ref.shape, what
    err = (got - ref).abs()
    top = ref.abs().max(dim=-1, keepdim=True).values.clamp(min=1.0)
    if dtype == "bfloat16":
        bad = (err > 5e-2 * top + 6 * moved).any(dim=-1) & (margin[:, 0] > 0.05)
        assert not bad.any(), (what, bad.nonzero().flatten().tolist(), float((err / top).max()))
        assert len(err) < 8 or (err / top).max(dim=-1).values.median() < 3e-2, (what, (err / top).max(dim=-1).values.median())
        return
    assert (err <= 1e-4 * top + 1e-3 * moved).all(), (what, (err / top).max())
    assert (err / top).max(dim=-1).values.median() < 2e-5, (what, (err / top).max(dim=-1).values.median())


def prompt(cfg, n, seed):
    return [random.Random(seed * 1000 + i).randrange(cfg["vocab"]) for i in range(n)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS_ALL))
def test_whole_prompt_and_the_first_tokens_alone(name, dtype, tmp_root):
    cfg, W, folder = model(name, tmp_root)
    toks = prompt(cfg, 70, 1)
    ref = reference(name, W, cfg, toks, dtype)
    s = session(folder, dtype)
    got = s.step([{"id": "a", "tokens": toks, "want": list(range(len(toks)))}], end=["a"])
    close(got, ref, dtype, name)
    one = s.step([{"id": "b", "tokens": toks[:1], "want": [0]}], end=["b"])   # the first token alone, in a's slot
    close(one, rows_of(ref, slice(0, 1)), dtype, name)
    two = s.step([{"id": "c", "tokens": toks[:2], "want": [0, 1]}], end=["c"])
    close(two, rows_of(ref, slice(0, 2)), dtype, name)
    s.core.manager.check_invariants()


def test_every_layer_against_the_plain_model(tmp_root):
    """The residual stream after each layer, in 32-bit, through a step of two portions."""
    cfg, W, folder = model("varied", tmp_root)
    toks = prompt(cfg, 40, 4)
    plain, layers = P.PlainRurorax(cfg, W), []
    plain.forward(toks, layers_out=layers)
    s = session(folder, "float32")
    seen = []
    m = s.core.model
    for built in m.layers:
        fwd = built.block.forward

        def spy(x, delta, ctx, cache, parts, following=None, fwd=fwd):
            out = fwd(x, delta, ctx, cache, parts, following=following)
            seen.append(out[0].clone())
            return out

        built.block.forward = spy
    s.step([{"id": "a", "tokens": toks[:25], "want": []}])
    s.step([{"id": "a", "tokens": toks[25:], "want": []}], end=["a"])
    n = len(cfg["layers"])
    for i in range(n):
        got = torch.cat([seen[i], seen[n + i]]).cpu().double()
        assert (got - layers[i]).abs().max() < 2e-5 * layers[i].abs().max(), i


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_prompt_whose_queries_look_far_back(dtype, tmp_root):
    """Sharp attention over 330 positions and twenty pages, chunks that begin and end inside pages, whole and with its last tokens one by one."""
    cfg, W, folder = model("aligned", tmp_root)
    toks = prompt(cfg, 330, 5)
    ref = reference("aligned", W, cfg, toks, dtype)
    s = session(folder, dtype, pages=48)
    got = s.step([{"id": "a", "tokens": toks, "want": list(range(len(toks)))}], end=["a"])
    close(got, ref, dtype, "whole")
    rows = [s.step([{"id": "b", "tokens": toks[:101], "want": [100]}])]
    for t in range(101, len(toks)):
        rows.append(s.step([{"id": "b", "tokens": toks[t:t + 1], "want": [0]}]))
    close(torch.cat(rows), rows_of(ref, slice(100, None)), dtype, "decoded")


@pytest.mark.parametrize("graphs", [False, True])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prefill_then_long_decoding_token_by_token(name, dtype, graphs, tmp_root):
    """A long run of single tokens crosses pages and chunks; with graphs they are replayed."""
    if graphs and dtype == "float32":
        pytest.skip("decode graphs are recorded in bfloat16")
    cfg, W, folder = model(name, tmp_root)
    toks = prompt(cfg, 150, 2)
    ref = reference(name, W, cfg, toks, dtype)
    s = session(folder, dtype, graphs=graphs)
    rows = [s.step([{"id": "a", "tokens": toks[:19], "want": [0, 18]}])]
    for t in range(19, len(toks)):
        rows.append(s.step([{"id": "a", "tokens": toks[t:t + 1], "want": [0]}], end=["a"] if t + 1 == len(toks) else []))
    close(torch.cat(rows), rows_of(ref, [0] + list(range(18, len(toks)))), dtype, name)
    if graphs:
        assert s.core.step.graphs is not None and s.core.step.graphs.replays > 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS_ALL))
def test_decoding_from_the_first_token_on(name, dtype, tmp_root):
    """No prompt to speak of: one token, then single tokens across the first chunks."""
    cfg, W, folder = model(name, tmp_root)
    toks = prompt(cfg, 90, 6)
    ref = reference(name, W, cfg, toks, dtype)
    s = session(folder, dtype, graphs=dtype == "bfloat16")
    rows = [s.step([{"id": "a", "tokens": toks[t:t + 1], "want": [0]}]) for t in range(len(toks))]
    close(torch.cat(rows), ref, dtype, name)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS_ALL))
def test_portions_of_every_size(name, dtype, tmp_root):
    cfg, W, folder = model(name, tmp_root)
    toks = prompt(cfg, 131, 3)
    ref = reference(name, W, cfg, toks, dtype)
    for sizes in ([2, 2, 3, 17, 2, 40, 1, 1, 5, 33, 2, 23], [64, 64, 3], [1] * 9 + [2] * 5 + [112]):
        assert sum(sizes) == len(toks)
        s = session(folder, dtype, pages=12, page_size=16, max_seqs=1)
        at, rows = 0, []
        for n in sizes:
            rows.append(s.step([{"id": 7, "tokens": toks[at:at + n], "want": list(range(n))}]))
            at += n
        close(torch.cat(rows), ref, dtype, (name, sizes))


@pytest.mark.parametrize("page_size", [16, 4])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS_ALL))
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype, page_size, tmp_root):
    """Five unequal requests through two state slots and a pool that holds two of them at a time:
    portions of some beside single tokens of others, a request left out of steps; every request against
    itself alone."""
    cfg, W, folder = model(name, tmp_root)
    reqs = {i: prompt(cfg, n, 10 + i) for i, n in enumerate([90, 37, 1, 64, 55])}
    refs = {i: reference(name, W, cfg, t, dtype) for i, t in reqs.items()}
    s = session(folder, dtype, pages=192 // page_size, page_size=page_size, max_seqs=2, graphs=dtype == "bfloat16")
    plan = [[(0, 30), (1, 5)], [(0, 1), (1, 30)], [(0, 2), (1, 1)], [(1, 1), (0, 40)], [(0, 1)], [(0, 16), (2, 1)],
            [(3, 33)], [(3, 1)], [(3, 30), (4, 2)], [(4, 1)], [(4, 1)], [(4, 50)], [(4, 1)]]
    at = {i: 0 for i in reqs}
    got = {i: [] for i in reqs}
    for step in plan:
        entries, end = [], []
        for i, n in step:
            entries.append({"id": f"r{i}", "tokens": reqs[i][at[i]:at[i] + n], "want": list(range(n))})
            at[i] += n
            if at[i] == len(reqs[i]):
                end.append(f"r{i}")
        out = s.step(entries, end=end)
        r0 = 0
        for i, n in step:
            got[i].append(out[r0:r0 + n])
            r0 += n
        s.core.manager.check_invariants()
    for i in reqs:
        assert at[i] == len(reqs[i])
        close(torch.cat(got[i]), refs[i], dtype, (name, i))


def drawn_config(seed: int) -> dict:
    """A model whose sizes, order of layers, chunks and constants are drawn from ``seed``."""
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randrange(3, 7)):
        if rng.random() < 0.5:
            kv = rng.choice([1, 2, 3])
            dim = rng.choice([16, 24, 32, 48, 64])
            m = attention(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([16, 32, 40, 64, 80]), rng.choice([None, 1, 7, 16, 33, 64, 90, 128]),
                          rng.choice([None, 2, 8, 16, dim]), rng.choice([None, 2.0, 8.0]), rng.choice([100.0, 1e4, 5e5]), dim ** -0.5 * rng.choice([1, 1.5]))
        else:
            groups, heads = rng.choice([1, 2, 3]), rng.choice([1, 2, 3])
            vdim = rng.choice([8, 16, 24, 40, 64])
            m = mamba(groups * heads, vdim, rng.choice([16, 24, 32, 64, 96, 128]), groups, rng.choice([1, 2, groups * heads]) if vdim % 2 == 0 else 1,
                      rng.choice([1, 2, 4, 5]))
        experts = rng.randrange(1, 9)
        layers.append((m, rng.choice([None, dense(rng.choice([16, 40, 96])), dense(rng.choice([32, 64])),
                                      moe(experts, rng.randrange(1, min(experts, 3) + 1), rng.choice([16, 24, 32, 64]))])))
    return config(rng.choice([96, 128, 160, 192, 256]), rng.randrange(150, 700), rng.choice([None, 10.0, 30.0]), layers, eps=rng.choice([1e-5, 1e-6]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(8))
def test_models_of_drawn_sizes_whole_in_portions_decoded_and_mixed(seed, dtype, tmp_root):
    """Sizes, order of layers, chunks, rotations and constants drawn at random: whole prompts, portions that change in size, a
    decoded tail, and two requests beside each other, each against the plain model."""
    name = f"drawn{seed}"
    if name not in _MODELS:
        cfg = drawn_config(seed)
        W = P.random_weights(cfg, seed=100 + seed)
        _MODELS[name] = (cfg, W, P.write_folder(tmp_root / name, cfg, W))
    cfg, W, folder = _MODELS[name]
    a, b = prompt(cfg, 170, 40 + seed), prompt(cfg, 61, 60 + seed)
    ra, rb = reference(name, W, cfg, a, dtype), reference(name, W, cfg, b, dtype)
    s = session(folder, dtype, pages=24, graphs=dtype == "bfloat16")
    close(s.step([{"id": "w", "tokens": a, "want": list(range(len(a)))}], end=["w"]), ra, dtype, (name, "whole"))
    rows, at = {"a": [], "b": []}, {"a": 0, "b": 0}
    toks = {"a": a, "b": b}
    plan = [[("a", 37)], [("a", 2), ("b", 30)], [("b", 1), ("a", 64)], [("a", 3), ("b", 1)], [("a", 40), ("b", 2)], [("b", 27)]]
    plan += [[("a", 1)]] * 24
    for step in plan:
        entries, end = [], []
        for r, n in step:
            entries.append({"id": r, "tokens": toks[r][at[r]:at[r] + n], "want": list(range(n))})
            at[r] += n
            if at[r] == len(toks[r]):
                end.append(r)
        out = s.step(entries, end=end)
        r0 = 0
        for r, n in step:
            rows[r].append(out[r0:r0 + n])
            r0 += n
    assert at == {"a": len(a), "b": len(b)}
    close(torch.cat(rows["a"]), ra, dtype, (name, "a"))
    close(torch.cat(rows["b"]), rb, dtype, (name, "b"))
    s.core.manager.check_invariants()


def test_a_row_does_not_depend_on_its_batch(tmp_root):
    """In 32-bit the logits of a request's rows are the same bits alone and beside others."""
    cfg, W, folder = model("varied", tmp_root)
    a, b, c = prompt(cfg, 40, 31), prompt(cfg, 23, 32), prompt(cfg, 9, 33)
    s = session(folder, "float32")
    alone = s.step([{"id": "a", "tokens": a, "want": list(range(40))}], end=["a"])
    s.step([{"id": "b", "tokens": b[:20], "want": []}])
    both = s.step([{"id": "b", "tokens": b[20:21], "want": [0]}, {"id": "a2", "tokens": a, "want": list(range(40))},
                   {"id": "c", "tokens": c, "want": [8]}], end=["a2", "b", "c"])
    assert torch.equal(alone, both[1:41])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(dtype, tmp_root):
    """The engine's own entry points and scheduler: one request, then several at once."""
    from dli_amd.engine.generate import generate, greedy_generate
    from dli_amd.sampling import SamplingParams

    cfg, W, folder = model("varied", tmp_root)
    prompts = [prompt(cfg, n, 20 + n) for n in (9, 30, 3)]
    want = [P.greedy_generate(cfg, W, p, 12) for p in prompts]

    def same(got, ref, p):
        if got == ref:
            return
        # tokens may part only where the plain logits of the engine's own tokens are close
        logits = P.PlainRurorax(cfg, W).forward(list(p) + got[:-1])
        for j, g in enumerate(got):
            row = logits[len(p) - 1 + j]
            assert (row.max() - row[g]).item() < (1e-3 if dtype == "float32" else 0.05) * row.abs().max().item(), (j, got, ref)

    same(greedy_generate(str(folder), prompts[0], 12, dtype=dtype, block_size=16), want[0], prompts[0])
    outs = generate(str(folder), prompts, SamplingParams(max_tokens=12), dtype=dtype, num_blocks=24, block_size=8,
                    max_num_seqs=2, max_num_batched_tokens=16, enable_prefix_caching=False)
    for got, ref, p in zip(outs, want, prompts):
        assert len(got) == 12
        same(got, ref, p)
