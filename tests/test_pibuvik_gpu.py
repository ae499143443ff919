"""Pibuvik on the GPU against the plain float64 implementation of ``plain_pibuvik.py``: every mechanism's kernel
alone, then whole models of several small shapes through the engine's step function, cache manager, scheduler
and entry points, however the requests are cut and batched."""

from __future__ import annotations

import random

import pytest
import torch

import plain_pibuvik as P

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


def tiles_of(lengths, rows):
    ent, q0 = [], []
    for e, n in enumerate(lengths):
        for a in range(0, n, rows):
            ent.append(e)
            q0.append(a)
    return i32(ent), i32(q0)


TOL = {torch.float32: 5e-6, torch.bfloat16: 6e-3}


# ------------------------------------------------------------------------------ norms, embedding, feed-forward

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [5, 40, 258, 1024, 1040, 2048, 4096, 5000])
def test_out_norm_sum_and_next_norm_in_one_kernel(ops, width, dtype):
    torch.manual_seed(width)
    n = 6
    wide, x = 3 * torch.randn(n, width + 4), torch.randn(n, width)
    w1, w2 = torch.randn(width), 1 + 0.2 * torch.randn(width)
    y = wide[:, :width]
    xs, out = x.cuda(), torch.empty(n, width, dtype=dtype).cuda()
    ops.norm_stream_norm(wide.cuda()[:, :width], w1.cuda(), 1e-3, xs, w2.cuda(), 1e-5, out)
    stream = x.double() + P.rms_norm(y.double(), w1.double(), 1e-3)
    normed = P.rms_norm(stream, w2.double(), 1e-5)
    assert (xs.cpu().double() - stream).abs().max() < 5e-6 * stream.abs().max()
    assert (out.cpu().double() - normed).abs().max() < TOL[dtype] * normed.abs().max()


def test_scaled_rows_of_the_table(ops):
    table = torch.randn(30, 50).to(torch.bfloat16)
    ids = torch.randint(0, 30, (9,), dtype=torch.int32)
    out = torch.empty(9, 50).cuda()
    ops.embed_sinusoid(table.cuda(), ids.cuda(), i32(range(9)), None, out, scale=2.75)
    assert torch.equal(out.cpu(), table[ids.long()].float() * 2.75)


@pytest.mark.parametrize("rows", [1, 3, 8, 16])
@pytest.mark.parametrize("ff,width", [(48, 64), (256, 128), (80, 96)])
def test_clamped_activation_inside_the_few_row_product(ops, rows, ff, width):
    """Halves far beyond the clamp on both sides: only the gate's upper side and both sides of the other are cut."""
    torch.manual_seed(rows + ff)
    x = torch.randn(rows, width).to(torch.bfloat16)
    w = (3 * torch.randn(2 * ff, width) / width ** 0.5).to(torch.bfloat16)
    both = (x.double() @ w.double().t()).to(torch.bfloat16).double()
    g, u = both[:, :ff].clamp(max=1.5), both[:, ff:].clamp(-1.5, 1.5)
    assert (both[:, :ff] > 1.5).any() and (both[:, :ff] < -1.5).any() and (both[:, ff:] < -1.5).any()
    ref = g * P.sigmoid(1.702 * g) * (u + 1)
    out = torch.empty(rows, ff, dtype=torch.bfloat16).cuda()
    ops.skinny_gemm(x.cuda(), w.cuda(), epilogue=ops.SKINNY_SWIGLU, out=out, clamped=(1.5, 1.702, 1.0))
    assert (out.cpu().double() - ref).abs().max() < 2e-2 * ref.abs().max()
    plain = torch.empty(rows, ff, dtype=torch.bfloat16).cuda()
    ops.skinny_gemm(x.cuda(), w.cuda(), epilogue=ops.SKINNY_SWIGLU, out=plain)
    ref = both[:, :ff] * P.sigmoid(both[:, :ff]) * both[:, ff:]
    assert (plain.cpu().double() - ref).abs().max() < 2e-2 * ref.abs().max()


# ------------------------------------------------------------------------------ the gated unit recurrence

# a plan over three requests through two slots: "c" starts in "a"'s slot once "a" has ended
PLAN = [[("a", 3), ("b", 1)], [("a", 1), ("b", 4)], [("b", 1), ("a", 2)], [("a", 17), ("b", 2)], [("a", 1)], [("a", 140), ("b", 64)],
        [("c", 1), ("b", 1)], [("c", 1)], [("c", 2), ("b", 35)], [("c", 129)]]
SLOTS = {"a": 1, "b": 0, "c": 1}
LENGTHS = {r: sum(n for step in PLAN for q, n in step if q == r) for r in SLOTS}


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("blocks,s,taps", [(2, 8, 4), (3, 5, 2), (1, 48, 3), (2, 136, 4), (4, 32, 1), (1, 1, 3), (5, 40, 6), (1, 260, 4)])
def test_recurrence_behind_its_convolution_cut_into_steps(ops, dtype, blocks, s, taps):
    """Three requests through two slots that held rubbish; decays from a few tokens to thousands."""
    C = blocks * s
    g = torch.Generator().manual_seed(10 * blocks + s)
    rnd = lambda *shape: torch.randn(*shape, generator=g)
    lam = -9.0 + 11.0 * torch.rand(C, generator=g)
    p = {"conv": 0.6 * rnd(C, taps), "conv.b": 0.5 * rnd(C), "x.b": rnd(C), "y.b": 0.5 * rnd(C), "ra.b": rnd(C), "ri.b": rnd(C)}
    p.update(ra=rnd(blocks, s, s) / s ** 0.5, ri=rnd(blocks, s, s) / s ** 0.5)
    p = {k: v.to(torch.bfloat16).float() for k, v in p.items()}
    decay = (8.0 * torch.nn.functional.softplus(lam.double())).float()
    xs = {r: rnd(n, 2 * C) for r, n in LENGTHS.items()}          # the recurrence's input, then the other branch
    state = torch.full((3, taps * C), 77.0).cuda()
    dev = {k: v.cuda() for k, v in p.items()}
    wr, wi = dev["ra"].to(dtype), dev["ri"].to(dtype)
    at, got = {r: 0 for r in xs}, {r: [] for r in xs}
    for step in PLAN:
        entries = [(SLOTS[r], at[r], n) for r, n in step]
        rows = torch.cat([xs[r][at[r]:at[r] + n] for r, n in step]).cuda()
        q_start, pos, slots = step_arrays(entries)
        u = torch.empty(rows.shape[0], C).cuda()
        ops.causal_conv(rows, dev["conv"], dev["conv.b"], state, C, q_start, pos, slots, u, act="none", in_bias=dev["x.b"])
        out = torch.empty(rows.shape[0], C, dtype=dtype).cuda()
        lengths = [n for _, n in step]
        tiles = None if max(lengths) == 1 else tiles_of(lengths, ops.gated_unit_tile_rows())
        ops.gated_unit(u, wr, wi, dev["ra.b"], dev["ri.b"], decay.cuda(), rows[:, C:], dev["y.b"], state, q_start, pos, slots, tiles, out)
        r0 = 0
        for r, n in step:
            got[r].append(out[r0:r0 + n].cpu().double())
            r0 += n
            at[r] += n
    d = {k: v.double() for k, v in p.items()}
    for r, x in xs.items():
        x = x.double()
        u = P.causal_conv(x[:, :C] + d["x.b"], d["conv"], d["conv.b"], {})
        rg, ig = P.sigmoid(P.block_diagonal(u, d["ra"]) + d["ra.b"]), P.sigmoid(P.block_diagonal(u, d["ri"]) + d["ri.b"])
        S, last = P.gated_unit(u, rg, ig, lam.double(), None)
        ref = S * P.gelu_tanh(x[:, C:] + d["y.b"])
        err = (torch.cat(got[r]) - ref).abs()
        assert (err < TOL[dtype] * ref.abs() + (2e-5 if dtype == torch.float32 else 5e-5) * ref.abs().max()).all(), (r, err.max())
        if r != "a":                                              # ("c" has "a"'s slot)
            assert (state[SLOTS[r], :C].cpu().double() - last).abs().max() < 2e-5 * last.abs().max()


def test_a_state_that_hardly_decays_is_still_there(ops):
    """One loud token, then 900 of silence (portions and single tokens) under a decay of almost one."""
    C, n = 16, 900
    z = torch.zeros
    u = z(n, C)
    u[3] = 1.0
    state = torch.full((1, C), 5.0).cuda()
    w = z(1, C, C).to(torch.bfloat16).cuda()
    bias, decay = z(C).cuda(), torch.full((C,), 1e-4).cuda()      # r = 1/2: a = exp(-5e-5)
    y = torch.full((n, C), 20.0)                                  # gelu(20) = 20
    at, got = 0, []
    for k in (1, 1, 64, 130, 1, 200, 1, 1, 501):
        q_start, pos, slots = step_arrays([(0, at, k)])
        out = torch.empty(k, C, dtype=torch.bfloat16).cuda()
        ops.gated_unit(u[at:at + k].cuda(), w, w, bias, bias, decay, y[at:at + k].cuda(), None, state, q_start, pos, slots,
                       None if k == 1 else tiles_of([k], ops.gated_unit_tile_rows()), out)
        got.append(out.cpu().double())
        at += k
    assert at == n
    got = torch.cat(got)[:, 0] / 20.0
    a = torch.exp(torch.tensor(-5e-5, dtype=F))
    ref = torch.sqrt(1 - a * a) * 0.5 * a ** (torch.arange(n, dtype=F) - 3)
    assert (got[:3] == 0).all() and (got[3:] - ref[3:]).abs().max() < 6e-3 * ref[3]
    # (the step of a decay this close to one: sqrt(1 - a^2) must not come from a rounded a)
    assert (state[0].cpu().double() - ref[-1]).abs().max() < 1e-5 * ref[-1]


# ------------------------------------------------------------------------------ products per head, latents, queries

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,m,k,rot", [(3, 40, 16, 8), (2, 128, 72, 0), (1, 20, 24, 6), (4, 64, 56, 16), (2, 7, 9, 2), (5, 4, 8, 0)])
@pytest.mark.parametrize("rows", [1, 16, 17, 70, 300])
def test_products_per_head_with_a_rotated_tail_and_gates(ops, dtype, H, m, k, rot, rows):
    torch.manual_seed(rows + m)
    x = torch.randn(rows, H * (k + rot)).to(dtype)
    w = (torch.randn(H, m, k) / k ** 0.5).to(dtype)
    pos = torch.randint(0, 400, (rows,), dtype=torch.int32)
    base = 1000.0
    inv = torch.tensor([base ** (-2.0 * i / max(rot, 2)) for i in range(rot // 2)], dtype=torch.float32)
    turn = dict(rot=rot, inv_freq=inv.cuda(), positions=pos.cuda()) if rot else {}
    xh = x.double().view(rows, H, k + rot)
    ref = torch.einsum("nhk,hmk->nhm", xh[..., :k], w.double())
    tol = TOL[dtype] * 4
    out = torch.full((rows, H * (m + rot)), 9.0, dtype=dtype).cuda()
    ops.head_products(x.cuda(), w.cuda(), out, **turn)
    got = out.cpu().double().view(rows, H, m + rot)
    assert (got[..., :m] - ref).abs().max() < tol * ref.abs().max()
    if rot:
        tail = P.rotate_half(xh[..., k:], pos, base)
        assert (got[..., m:] - tail).abs().max() < (5e-5 if dtype == torch.float32 else 2e-2) * tail.abs().max()
    gates = torch.randn(rows, H * m + H + 3).cuda()
    out = torch.empty(rows, H * m, dtype=dtype).cuda()
    ops.head_products(x.cuda(), w.cuda(), out, gate=gates[:, 2:2 + H])
    per = P.sigmoid(gates[:, 2:2 + H].cpu().double())[:, :, None]
    assert (out.cpu().double().view(rows, H, m) - ref * per).abs().max() < tol * ref.abs().max()
    if m > 1:
        ops.head_products(x.cuda(), w.cuda(), out, gate=gates[:, :H * m])
        each = P.sigmoid(gates[:, :H * m].cpu().double()).view(rows, H, m)
        assert (out.cpu().double().view(rows, H, m) - ref * each).abs().max() < tol * ref.abs().max()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("q_rank,r,rot", [(12, 20, 6), (40, 300, 16), (1100, 8, 2), (24, 32, 0)])
def test_latents_and_their_rotated_part_reach_their_page(ops, dtype, q_rank, r, rot):
    torch.manual_seed(r)
    n, ps = 9, 4
    proj = 2 * torch.randn(n, 3 + q_rank + r + rot)
    wq, wc = 1 + 0.2 * torch.randn(q_rank), 1 + 0.2 * torch.randn(r)
    pos = torch.tensor([0, 1, 7, 100, 3000, 5, 6, 8, 9], dtype=torch.int32)
    inv = torch.tensor([500.0 ** (-2.0 * i / max(rot, 2)) for i in range(rot // 2)], dtype=torch.float32)
    slots = [13, 0, 5, -1, 22, 23, 1, 2, 3]                        # (the fourth row is not cached)
    kp = torch.full((6, 1, ps, r + rot), 3.0, dtype=dtype).cuda()
    cq = torch.empty(n, q_rank, dtype=dtype).cuda()
    turn = dict(rot=rot, inv_freq=inv.cuda(), positions=pos.cuda()) if rot else {}
    ops.latent_norm_cache(proj.cuda(), 3, q_rank, 3 + q_rank, r, wq.cuda(), wc.cuda(), 1e-4, cq, i32(slots), kp, **turn)
    d = proj.double()
    ref = P.rms_norm(d[:, 3:3 + q_rank], wq.double(), 1e-4)
    assert (cq.cpu().double() - ref).abs().max() < TOL[dtype] * ref.abs().max()
    key = P.rms_norm(d[:, 3 + q_rank:3 + q_rank + r], wc.double(), 1e-4)
    if rot:
        key = torch.cat([key, P.rotate_half(d[:, 3 + q_rank + r:], pos, 500.0)], dim=-1)
    flat = kp.cpu().double().view(-1, r + rot)
    for t, slot in enumerate(slots):
        if slot >= 0:
            assert (flat[slot] - key[t]).abs().max() < (2e-5 if dtype == torch.float32 else 8e-3) * key.abs().max()
    untouched = [s for s in range(flat.shape[0]) if s not in slots]
    assert (flat[untouched] == 3.0).all()
    only = torch.empty(n, q_rank, dtype=dtype).cuda()              # a layer that reads another's latents
    ops.latent_norm_cache(proj.cuda(), 3, q_rank, 3 + q_rank, 0, wq.cuda(), None, 1e-4, only, None, None)
    assert torch.equal(only, cq)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_query_temperature_and_keys_without_values(ops, dtype):
    torch.manual_seed(3)
    H, G, dim, ps, coef, every = 4, 2, 10, 4, 0.7, 13
    pos = torch.tensor([0, 11, 12, 13, 24, 25, 38, 1299, 100000], dtype=torch.int32)
    n = len(pos)
    proj = torch.randn(n, (H + G) * dim)
    q = torch.empty(n, H * dim, dtype=dtype).cuda()
    kp = torch.zeros(3, G, ps, dim, dtype=dtype).cuda()
    ops.rotary_cache(proj.cuda(), 0, H * dim, (H + G) * dim, pos.cuda(), None, 0, False, q, i32(range(n)), kp, None, H,
                     query_temperature=(coef, every))
    ref = proj.double()[:, :H * dim] * P.query_temperature(pos, coef, every)[:, None]
    assert (q.cpu().double() - ref).abs().max() < TOL[dtype] * ref.abs().max()
    keys = proj.double()[:, H * dim:].view(n, G, dim)
    for t in range(n):
        assert (kp[t // ps, :, t % ps].cpu().double() - keys[t]).abs().max() < TOL[dtype] * keys.abs().max()


# ------------------------------------------------------------------------------ attention whose values are its keys

def paged(k, ps, dtype, seed):
    """Keys ``[n, G, D]`` of one request in shuffled pages -> (pages, table)."""
    n, G, D = k.shape
    used = -(-n // ps)
    order = list(range(used + 3))
    random.Random(seed).shuffle(order)
    kp = torch.zeros(used + 3, G, ps, D, dtype=dtype)
    for t in range(n):
        kp[order[t // ps], :, t % ps] = k[t].to(dtype)
    return kp.cuda(), order[:used]


def dense(q, k, V, scale, window, sinks, rows):
    """The plain attention of the last tokens ``rows`` (positions): q ``[len(rows), H, D]``, k ``[n, G, D]``, float64."""
    H, G = q.shape[1], k.shape[1]
    kk = k.repeat_interleave(H // G, dim=1)
    out = torch.zeros(len(rows), H, V, dtype=F)
    for i, p in enumerate(rows):
        js = list(P.visible(p, window))
        w = P.softmax_with_sink((q[i][None] * kk[js]).sum(-1).t() * scale, sinks)
        out[i] = (w.t()[:, :, None] * kk[js][:, :, :V]).sum(0)
    return out


KV_CASES = [  # H, G, D, V
    (4, 1, 96, 64), (8, 2, 64, 64), (3, 3, 24, 16), (16, 1, 288, 256), (5, 1, 576, 512), (70, 1, 40, 32), (12, 4, 104, 104),
    (2, 1, 640, 600), (1, 1, 8, 8), (6, 2, 192, 160), (24, 1, 320, 320), (130, 1, 32, 24), (2, 1, 20, 12), (2, 1, 700, 650), (9, 3, 33, 33)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("case", KV_CASES)
def test_one_key_stands_out_for_every_query_that_sees_it(ops, dtype, case):
    """A key far longer than the others, in the direction that all queries share, planted at a page's and a block's
    border and in between: rows whose window just holds it differ from rows whose window just does not. Through the
    portions' kernel and the single-token kernel (keys cut over workgroups and not), with and without sinks; the
    matrix-core kernel where it takes the sizes, else the vector-unit ones."""
    H, G, D, V = case
    mfma = ops.attention_keyvalue_supports(D, V, dtype)
    assert mfma == (dtype == torch.bfloat16 and D % 8 == 0 and V % 8 == 0 and D <= 640)
    g = torch.Generator().manual_seed(sum(case))
    n, ps = 150, 16
    for planted, window, sink in ((0, 0, True), (31, 32, False), (32, 33, True), (47, 64, False), (64, 17, True), (79, 1, False)):
        k = torch.randn(n, G, D, generator=g) * 0.5
        k[planted, :, 0] += 6.0
        q = torch.randn(n, H, D, generator=g) * 0.5
        scale = 1.0 / max(1.0, D ** 0.5 / 4)
        q[..., 0] += 1.3 / scale                                # (a score of about 8)
        q, k = q.to(dtype).double(), k.to(dtype).double()
        sinks = torch.randn(H, generator=g).double() * 2 if sink else None
        first = 90 if planted < 90 and window else 3            # the portion's first position: inside a page and a block
        if window:
            first = max(0, min(first, planted + window - 4))    # rows on both sides of the window's edge
        rows = list(range(first, n))
        ref = dense(q[rows], k, V, scale, window, sinks, rows)
        kp, table = paged(k, ps, dtype, planted)
        tables = i32(table).reshape(1, -1)
        dev = lambda t: t.reshape(t.shape[0], -1).to(dtype).cuda()
        sk = sinks.float().cuda() if sink else None
        out = torch.empty(len(rows), H * V, dtype=dtype).cuda()
        if mfma:
            te, tq = tiles_of([len(rows)], ops.attention_keyvalue_tile_tokens(H, G))
            ops.attention_keyvalue(dev(q[rows]), kp, out, i32([0, len(rows)]), i32([n]), tables, te, tq, H, scale, window=window, sinks=sk)
        else:
            te, tq = tiles_of([len(rows)], ops.attention_generic_tile_rows(D))
            ops.attention_scored(dev(q[rows]), kp, None, out, i32([0, len(rows)]), i32([n]), tables, te, tq, H, scale, window=window, sinks=sk)
        tol = 1e-4 if dtype == torch.float32 else 2e-2
        err = (out.cpu().double().view(ref.shape) - ref).abs()
        assert err.max() < tol * ref.abs().max(), (planted, window, sink, err.max())
        # single tokens at both sides of the edge, as entries of one step
        edge = [p for p in ((planted + window - 1, planted + window) if window else (planted, n - 1)) if p < n] + [planted, 0]
        ref1 = dense(q[edge], k, V, scale, window, sinks, edge)
        rows1 = torch.cat([i32(table)[None]] * len(edge)).contiguous()
        for splits in ((1, 3, None) if mfma else (None,)):
            out = torch.empty(len(edge), H * V, dtype=dtype).cuda()
            args = (i32(range(len(edge) + 1)), i32([p + 1 for p in edge]), rows1, None, None, H, scale)
            if mfma:
                ops.attention_keyvalue(dev(q[edge]), kp, out, *args, window=window, sinks=sk, splits=splits)
            else:
                ops.attention_scored(dev(q[edge]), kp, None, out, *args, window=window, sinks=sk)
            err = (out.cpu().double().view(ref1.shape) - ref1).abs()
            assert err.max() < tol * ref1.abs().max(), (planted, window, sink, splits, err.max())
        if window > 1 and len(edge) == 4:
            assert (ref1[0, :, 0] - ref1[1, :, 0]).abs().max() > 0.5   # the edge shows


def test_sinks_per_head_in_the_kernels_with_value_pages(ops):
    torch.manual_seed(5)
    H, G, D, n, ps = 4, 2, 32, 70, 16
    q, k, v = torch.randn(n, H, D), torch.randn(n, G, D), torch.randn(n, G, D)
    sinks = torch.tensor([-3.0, 0.0, 2.0, 5.0])
    for dtype in (torch.float32, torch.bfloat16):
        qd, kd, vd = (t.to(dtype).double() for t in (q, k, v))
        kk, vv = kd.repeat_interleave(H // G, 1), vd.repeat_interleave(H // G, 1)
        ref = torch.zeros(n, H, D, dtype=F)
        for t in range(n):
            w = P.softmax_with_sink((qd[t][None] * kk[:t + 1]).sum(-1).t() * 0.2, sinks.double())
            ref[t] = (w.t()[:, :, None] * vv[:t + 1]).sum(0)
        kp, table = paged(kd, ps, dtype, 1)
        vp = torch.zeros(kp.shape[0], G, D, ps, dtype=dtype)
        for t in range(n):
            vp[table[t // ps], :, :, t % ps] = vd[t].to(dtype)
        vp = vp.cuda()
        kinds = ["tiles", "single"] + (["mfma"] if dtype == torch.bfloat16 else [])
        for kind in kinds:
            if kind == "single":
                rows = [0, 20, n - 1]
                out = torch.empty(3, H * D, dtype=dtype).cuda()
                ops.attention_scored(qd[rows].reshape(3, -1).to(dtype).cuda(), kp, vp, out, i32(range(4)), i32([r + 1 for r in rows]),
                                     torch.cat([i32(table)[None]] * 3).contiguous(), None, None, H, 0.2, sinks=sinks.cuda())
            else:
                rows = list(range(n))
                out = torch.empty(n, H * D, dtype=dtype).cuda()
                fn, step = (ops.attention_scored, ops.attention_generic_tile_rows(D)) if kind == "tiles" else (ops.attention_scored_mfma, ops.SCORED_MFMA_TILE_ROWS)
                te, tq = tiles_of([n], step)
                fn(qd.reshape(n, -1).to(dtype).cuda(), kp, vp, out, i32([0, n]), i32([n]), i32(table).reshape(1, -1), te, tq, H, 0.2, sinks=sinks.cuda())
            err = (out.cpu().double().view(len(rows), H, D) - ref[rows]).abs().max()
            assert err < (1e-5 if dtype == torch.float32 else 2e-2) * ref.abs().max(), (dtype, kind)


# ------------------------------------------------------------------------------ whole models through the engine

def config(width, vocab, layers, *, eps=1e-5, scale=1.0, mult=0.5, logit=1.0):
    return {"architecture": "Pibuvik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "residual_mult": mult, "logit_scale": logit, "layers": layers}


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def dense_mlp(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def latent(heads, dim, rot, vdim, r, q_rank, window=None, base=1e4, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": r, "q_rank": q_rank, "rot": {"base": base, "dims": rot},
         "scale": scale if scale is not None else (dim + rot) ** -0.5}
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def rglru(width, blocks, conv):
    return {"width": width, "blocks": blocks, "conv": conv}


def att(heads, kv, dim, scale=None, temp=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale if scale is not None else dim ** -0.5}
    if temp:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return m


def varied():
    """Nothing aligned; a borrower that looks further back than its lender, one that looks less far; two lenders."""
    return config(46, 51, [
        layer("latent_attention", latent(3, 10, 6, 7, 21, 13, window=9), dense_mlp(27, 1.1)),
        layer("rglru", rglru(33, 3, 4), None),
        layer("latent_attention", latent(2, 5, 6, 9, 21, 18, window=23, kv_from=0), dense_mlp(31, 3.0)),
        layer("attention", att(6, 3, 9, temp=(0.8, 7)), dense_mlp(20, 0.7)),
        layer("latent_attention", latent(1, 4, 2, 3, 11, 5, base=300.0), None),
        layer("rglru", rglru(14, 14, 1), dense_mlp(9, 2.0)),
        layer("latent_attention", latent(4, 4, 2, 6, 11, 8, window=5, base=300.0, kv_from=4), dense_mlp(16, 2.0))],
        eps=1e-4, scale=1.7, mult=0.6, logit=1.3)


def aligned():
    """Sizes that the matrix-core kernels take, windows longer and shorter than a block of 32 keys, sharp queries."""
    return config(64, 90, [
        layer("latent_attention", latent(4, 16, 8, 24, 80, 32, window=70), dense_mlp(96, 2.5)),
        layer("attention", att(8, 2, 32, temp=(0.4, 50)), dense_mlp(64, 2.5)),
        layer("rglru", rglru(96, 2, 3), dense_mlp(64, 1.0)),
        layer("latent_attention", latent(6, 8, 8, 16, 80, 48, window=19, kv_from=0), dense_mlp(64, 2.5))], scale=2.0, mult=0.4, logit=0.8)


def plain_ends():
    """Every earlier position seen, one kv head, as many kv heads as heads, values of one, no temperature, no constants."""
    return config(40, 33, [
        layer("attention", att(5, 1, 16), None), layer("rglru", rglru(40, 1, 2), None),
        layer("attention", att(3, 3, 8), dense_mlp(24, 50.0)), layer("latent_attention", latent(2, 8, 8, 1, 8, 8), dense_mlp(8, 0.2))],
        mult=1.0)


CONFIGS = {"varied": varied(), "aligned": aligned(), "plain_ends": plain_ends()}
_MODELS: dict = {}


def model(name, tmp_root, cfg=None):
    if name not in _MODELS:
        cfg = cfg or CONFIGS[name]
        W = P.random_weights(cfg, seed=len(name) * 7 + 1, sharp=3.0 if name == "aligned" else 2.0)
        _MODELS[name] = (cfg, W, P.write_folder(tmp_root / name, cfg, W))
    return _MODELS[name]


@pytest.fixture(scope="module")
def tmp_root(tmp_path_factory):
    return tmp_path_factory.mktemp("pibuvik")


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


def reference(W, cfg, toks):
    """The plain logits, and how far each row moves when the matrices are jittered by bfloat16's rounding (the larger of
    two draws): what rounding of that size may do to the row."""
    key = (id(W), tuple(toks))
    if key not in _REFS:
        run = lambda t: P.PlainPibuvik(cfg, t).forward(toks)
        ref = run(W)
        moved = [(run(P.jittered(W, seed=j)) - ref).abs().max(dim=-1, keepdim=True).values for j in (0, 5)]
        _REFS[key] = (ref, torch.maximum(*moved))
    return _REFS[key]


def rows_of(ref, rows):
    return tuple(r[rows] for r in ref)


def close(got, ref, dtype, what):
    """In 32-bit every row is held closely, and that is where a fault of the cache, the state or a window shows (it
    moves rows by 1e-2 and more). In bfloat16 a row may be off by bfloat16's usual share of its largest logit and a
    few times what a jitter of that size on the matrices does to it."""
    ref, moved = ref
    got, ref = got.double().cpu(), ref.double()
    assert got.shape == ref.shape, what
    err = (got - ref).abs()
    top = ref.abs().max(dim=-1, keepdim=True).values.clamp(min=1.0)
    if dtype == "bfloat16":
        bad = (err > 4e-2 * top + 6 * moved).any(dim=-1)
        assert not bad.any(), (what, bad.nonzero().flatten().tolist())
        assert (err / top).max(dim=-1).values.median() < 4e-2, (what, (err / top).max(dim=-1).values.median())
        return
    assert (err <= 1e-4 * top + 1e-3 * moved).all(), (what, (err / top).max())
    assert (err / top).max(dim=-1).values.median() < 2e-5, (what, (err / top).max(dim=-1).values.median())


def prompt(cfg, n, seed):
    return [random.Random(seed * 1000 + i).randrange(cfg["vocab"]) for i in range(n)]


def run_plan(s, toks, plan):
    """Steps of (request, tokens); a request ends with its last token -> rows of every request."""
    at, got = {r: 0 for r in toks}, {r: [] for r in toks}
    for step in plan:
        entries, end = [], []
        for r, n in step:
            entries.append({"id": f"r{r}", "tokens": toks[r][at[r]:at[r] + n], "want": list(range(n))})
            at[r] += n
            if at[r] == len(toks[r]):
                end.append(f"r{r}")
        out = s.step(entries, end=end)
        r0 = 0
        for r, n in step:
            got[r].append(out[r0:r0 + n])
            r0 += n
        s.core.manager.check_invariants()
    assert all(at[r] == len(toks[r]) for r in toks)
    return {r: torch.cat(v) for r, v in got.items()}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_the_first_tokens_alone(name, dtype, tmp_root):
    cfg, W, folder = model(name, tmp_root)
    toks = prompt(cfg, 70, 1)
    ref = reference(W, cfg, toks)
    s = session(folder, dtype)
    close(s.step([{"id": "a", "tokens": toks, "want": list(range(len(toks)))}], end=["a"]), ref, dtype, name)
    for n in (1, 2):                                              # in a's slot and pages
        got = s.step([{"id": n, "tokens": toks[:n], "want": list(range(n))}], end=[n])
        close(got, rows_of(ref, slice(0, n)), dtype, (name, n))
    s.core.manager.check_invariants()


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_stream_after_every_layer(name, tmp_root):
    cfg, W, folder = model(name, tmp_root)
    toks = prompt(cfg, 40, 8)
    want: list = []
    P.PlainPibuvik(cfg, W).forward(toks, layers_out=want)
    for dtype, tol in (("float32", 2e-5), ("bfloat16", 5e-2)):
        s = session(folder, dtype)
        seen = []
        for l in s.core.model.layers:
            def spy(x, delta, ctx, cache, parts, following=None, forward=l.block.forward):
                x, delta = forward(x, delta, ctx, cache, parts, following=following)
                seen.append(x.double().cpu())
                return x, delta
            l.block.forward = spy
        s.step([{"id": "a", "tokens": toks, "want": [0]}], end=["a"])
        assert len(seen) == len(want)
        for i, (g, w) in enumerate(zip(seen, want)):
            assert (g - w).abs().max() < tol * w.abs().max(), (dtype, i)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_prompt_and_long_decoding_with_sharp_queries(dtype, tmp_root):
    """330 positions over twenty pages, past the windows and over several blocks of keys, whole and with the last 230
    decoded one by one (replayed from graphs in bfloat16)."""
    cfg, W, folder = model("aligned", tmp_root)
    toks = prompt(cfg, 330, 5)
    ref = reference(W, cfg, toks)
    s = session(folder, dtype, pages=48, graphs=dtype == "bfloat16")
    close(s.step([{"id": "a", "tokens": toks, "want": list(range(len(toks)))}], end=["a"]), ref, dtype, "whole")
    got = run_plan(s, {"b": toks}, [[("b", 100)]] + [[("b", 1)]] * 230)
    close(got["b"], ref, dtype, "decoded")
    if dtype == "bfloat16":
        assert s.core.step.graphs is not None and s.core.step.graphs.replays > 0


@pytest.mark.parametrize("graphs", [False, True])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_token_by_token_from_the_first_on(name, dtype, graphs, tmp_root):
    if graphs and dtype == "float32":
        pytest.skip("decode graphs are recorded in bfloat16")
    cfg, W, folder = model(name, tmp_root)
    toks = prompt(cfg, 90, 2)
    s = session(folder, dtype, graphs=graphs)
    got = run_plan(s, {"a": toks}, [[("a", 1)]] * 90)
    close(got["a"], reference(W, cfg, toks), dtype, name)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_portions_of_every_size(name, dtype, tmp_root):
    cfg, W, folder = model(name, tmp_root)
    toks = prompt(cfg, 131, 3)
    ref = reference(W, cfg, toks)
    for sizes in ([2, 2, 3, 17, 2, 40, 1, 1, 5, 33, 2, 23], [64, 64, 3], [1] * 9 + [2] * 5 + [112], [65, 66]):
        s = session(folder, dtype, pages=12, page_size=16, max_seqs=1)
        got = run_plan(s, {7: toks}, [[(7, n)] for n in sizes])
        close(got[7], ref, dtype, (name, sizes))


@pytest.mark.parametrize("page_size", [16, 4])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype, page_size, tmp_root):
    """Five unequal requests through two state slots and a pool that holds two of them at a time: portions of some
    beside single tokens of others, a request left out of steps; every request against itself alone."""
    cfg, W, folder = model(name, tmp_root)
    reqs = {i: prompt(cfg, n, 10 + i) for i, n in enumerate([90, 37, 1, 64, 55])}
    s = session(folder, dtype, pages=192 // page_size, page_size=page_size, max_seqs=2, graphs=dtype == "bfloat16")
    plan = [[(0, 30), (1, 5)], [(0, 1), (1, 30)], [(0, 2), (1, 1)], [(1, 1), (0, 40)], [(0, 1)], [(0, 16), (2, 1)],
            [(3, 33)], [(3, 1)], [(3, 30), (4, 2)], [(4, 1)], [(4, 1)], [(4, 50)], [(4, 1)]]
    got = run_plan(s, reqs, plan)
    for i in reqs:
        close(got[i], reference(W, cfg, reqs[i]), dtype, (name, i))


def drawn_config(seed):
    rng = random.Random(seed)
    dims = (lambda: rng.choice([8, 16, 24, 32, 40])) if seed % 2 else (lambda: rng.randrange(2, 30))
    layers, lenders = [], []
    for i in range(rng.randrange(3, 6)):
        mlp = dense_mlp(dims(), rng.choice([0.5, 1.5, 4.0])) if rng.random() < 0.8 else None
        kind = rng.choice(["latent_attention", "latent_attention", "rglru", "attention"])
        if kind == "rglru":
            blocks = rng.randrange(1, 5)
            mixer = rglru(blocks * dims(), blocks, rng.randrange(1, 6))
        elif kind == "attention":
            kv = rng.randrange(1, 4)
            mixer = att(kv * rng.randrange(1, 5), kv, dims(), temp=(rng.choice([0.3, 1.0]), rng.randrange(3, 60)) if rng.random() < 0.7 else None)
        else:
            window = rng.choice([None, rng.randrange(1, 12), rng.randrange(12, 100)])
            src = rng.choice(lenders) if lenders and rng.random() < 0.6 else None
            r, rot, base = (layers[src]["mixer"][k] for k in ("kv_rank", "rot_dim", "rot")) if src is not None else \
                (dims() * rng.randrange(1, 5), 2 * rng.randrange(1, 9), {"base": rng.choice([50.0, 1e4])})
            mixer = latent(rng.randrange(1, 6), dims(), rot, dims(), r, dims(), window, base["base"], kv_from=src)
            if src is None:
                lenders.append(i)
        layers.append(layer(kind, mixer, mlp))
    return config(8 * rng.randrange(3, 10) if seed % 2 else rng.randrange(24, 70), rng.randrange(20, 80), layers,
                  eps=rng.choice([1e-6, 1e-4]), scale=rng.choice([1.0, 2.5]), mult=rng.choice([0.25, 1.0]), logit=rng.choice([0.5, 1.0, 2.0]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(10))
def test_models_of_drawn_sizes_whole_in_portions_decoded_and_mixed(seed, dtype, tmp_root):
    """Sizes, order of layers, lenders, windows, periods and constants drawn at random: whole prompts, portions that
    change in size, a decoded tail, and two requests beside each other, each against the plain model."""
    cfg, W, folder = model(f"drawn{seed}", tmp_root, drawn_config(seed))
    toks = {"a": prompt(cfg, 150, 40 + seed), "b": prompt(cfg, 61, 60 + seed)}
    refs = {r: reference(W, cfg, t) for r, t in toks.items()}
    s = session(folder, dtype, pages=24, graphs=dtype == "bfloat16")
    close(s.step([{"id": "w", "tokens": toks["a"], "want": list(range(150))}], end=["w"]), refs["a"], dtype, (seed, "whole"))
    plan = [[("a", 37)], [("a", 2), ("b", 30)], [("b", 1), ("a", 64)], [("a", 3), ("b", 1)], [("a", 20), ("b", 2)], [("b", 27)]]
    got = run_plan(s, toks, plan + [[("a", 1)]] * 24)
    for r in toks:
        close(got[r], refs[r], dtype, (seed, r))


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
        logits = P.PlainPibuvik(cfg, W).forward(list(p) + got[:-1])
        for j, g in enumerate(got):
            row = logits[len(p) - 1 + j]
            assert (row.max() - row[g]).item() < (1e-3 if dtype == "float32" else 0.05) * row.abs().max().item(), (j, got, ref)

    same(greedy_generate(str(folder), prompts[0], 12, dtype=dtype, block_size=16), want[0], prompts[0])
    outs = generate(str(folder), prompts, SamplingParams(max_tokens=12), dtype=dtype, num_blocks=24, block_size=8,
                    max_num_seqs=2, max_num_batched_tokens=16, enable_prefix_caching=False)
    for got, ref, p in zip(outs, want, prompts):
        assert len(got) == 12
        same(got, ref, p)
