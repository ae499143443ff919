"""A plain, slow Pibuvik in float64: whole sequences, no cache pages, no batching, one function per
mechanism. It takes the configuration as the dictionary that ``config.json`` holds and the tensors by
their checkpoint names, and shares no code with the engine.

A layer is ``x <- x + m norm1b(mixer(norm1(x)))`` then ``x <- x + m norm2b(ff(norm2(x)))`` with one constant ``m``;
the mixers are attention through a latent under a window (``latent_attention``, which may read an earlier
layer's latents), a gated linear recurrence per channel behind a short convolution (``rglru``) and attention
whose values are its keys, with a sink and a temperature on the queries (``attention``). ``states`` carry what a
sequence keeps from one call to the next, so that the same functions also step token by token.
"""

from __future__ import annotations

import math
from typing import Any, Mapping, Optional

import torch

F = torch.float64


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.where(x > 30.0, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rotate_half(x: torch.Tensor, positions: torch.Tensor, base: float) -> torch.Tensor:
    """``x [tokens, ..., dims]``: component ``i`` turns with ``i + dims/2`` by ``p base^(-2i/dims)``."""
    dims = x.shape[-1]
    half = dims // 2
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=F)
    angle = positions.to(F).view(-1, *([1] * (x.dim() - 1))) * freq
    u, v = x[..., :half], x[..., half:]
    return torch.cat([u * torch.cos(angle) - v * torch.sin(angle), v * torch.cos(angle) + u * torch.sin(angle)], dim=-1)


def visible(p: int, window: int) -> range:
    """The positions that position ``p`` sees (``window`` 0: all up to itself)."""
    return range(max(0, p - window + 1) if window else 0, p + 1)


def softmax_with_sink(scores: torch.Tensor, sink: Optional[torch.Tensor]) -> torch.Tensor:
    """Weights over the last axis; ``sink`` (a number per row): one more term of the denominator, ``exp(sink)``."""
    if sink is None:
        return torch.softmax(scores, dim=-1)
    return torch.softmax(torch.cat([scores, sink[:, None]], dim=-1), dim=-1)[:, :-1]


def query_temperature(positions: torch.Tensor, coef: float, every: int) -> torch.Tensor:
    return torch.tensor([1.0 + coef * math.log((int(p) + 1) // every + 1) for p in positions], dtype=F)


def causal_conv(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, state: dict) -> torch.Tensor:
    """Per channel, ``y[t] = b + sum_j w[:, taps-1-j] x[t-j]``; ``state['conv']`` holds the last ``taps-1`` inputs."""
    taps = w.shape[1]
    kept = state.get("conv")
    if kept is None:
        kept = torch.zeros(taps - 1, x.shape[1], dtype=F)
    full = torch.cat([kept, x], dim=0)
    out = torch.stack([(full[t:t + taps] * w.t()).sum(0) for t in range(x.shape[0])]) + b
    state["conv"] = full[full.shape[0] - (taps - 1):].clone()
    return out


def block_diagonal(u: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """``w [blocks, out, in]``: block ``b`` maps the b-th equal part of every row."""
    blocks, size = w.shape[0], w.shape[1]
    return torch.cat([u[:, b * size:(b + 1) * size] @ w[b].t() for b in range(blocks)], dim=-1)


def gated_unit(u: torch.Tensor, r: torch.Tensor, i: torch.Tensor, lam: torch.Tensor, S: Optional[torch.Tensor]) -> tuple:
    """``S <- a S + sqrt(1 - a^2) i u``, ``log a = -8 r softplus(lam)``, token by token from zero."""
    S = torch.zeros(u.shape[1], dtype=F) if S is None else S
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        log_a = -8.0 * r[t] * softplus(lam)
        S = torch.exp(log_a) * S + torch.sqrt(-torch.expm1(2.0 * log_a)) * i[t] * u[t]
        out[t] = S
    return out, S


def rglru(h: torch.Tensor, p: Mapping[str, torch.Tensor], state: dict) -> torch.Tensor:
    y = gelu_tanh(h @ p["y"].t() + p["y.b"])
    u = causal_conv(h @ p["x"].t() + p["x.b"], p["conv"], p["conv.b"], state)
    r = sigmoid(block_diagonal(u, p["ra"]) + p["ra.b"].reshape(-1))
    i = sigmoid(block_diagonal(u, p["ri"]) + p["ri.b"].reshape(-1))
    S, state["S"] = gated_unit(u, r, i, p["lam"], state.get("S"))
    return (S * y) @ p["o"].t()


def key_value_attention(h: torch.Tensor, p: Mapping[str, torch.Tensor], m: Mapping[str, Any], state: dict) -> torch.Tensor:
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    n = h.shape[0]
    k = (h @ p["k"].t()).view(n, G, d)
    k = k if state.get("k") is None else torch.cat([state["k"], k], dim=0)
    state["k"] = k
    first = k.shape[0] - n
    q = (h @ p["q"].t()).view(n, H, d)
    if m.get("q_temp"):
        q = q * query_temperature(torch.arange(first, first + n), m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    kv = k.repeat_interleave(H // G, dim=1)
    out = torch.zeros(n, H, d, dtype=F)
    for t in range(n):
        seen = kv[:first + t + 1]
        w = softmax_with_sink((q[t][None] * seen).sum(-1).t() * m["scale"], p["sink"])
        out[t] = (w.t()[:, :, None] * seen).sum(0)
    return out.reshape(n, H * d) @ p["o"].t()


def latent_attention(h: torch.Tensor, p: Mapping[str, torch.Tensor], m: Mapping[str, Any], eps: float, state: dict,
                     lender: Optional[dict]) -> torch.Tensor:
    """``lender``: the state of the layer whose latents and rotated keys this one reads (it has taken the step)."""
    H, d, rd, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    n = h.shape[0]
    if lender is None:
        low = h @ p["dkv"].t()
        past = state.get("c")
        first = 0 if past is None else past.shape[0]
        c = rms_norm(low[:, :m["kv_rank"]], p["dkv.norm"], eps)
        kr = rotate_half(low[:, m["kv_rank"]:], torch.arange(first, first + n), m["rot"]["base"])
        state["c"] = c if past is None else torch.cat([past, c], dim=0)
        state["kr"] = kr if past is None else torch.cat([state["kr"], kr], dim=0)
        lender = state
    c, kr = lender["c"], lender["kr"]
    first = c.shape[0] - n
    q = (rms_norm(h @ p["dq"].t(), p["dq.norm"], eps) @ p["uq"].t()).view(n, H, d + rd)
    qn, qr = q[..., :d], rotate_half(q[..., d:], torch.arange(first, first + n), m["rot"]["base"])
    k = (c @ p["uk"].t()).view(-1, H, d)
    v = (c @ p["uv"].t()).view(-1, H, dv)
    gate = sigmoid(h @ p["g"].t())
    out = torch.zeros(n, H, dv, dtype=F)
    window = (m.get("mask") or {}).get("size") or 0
    for t in range(n):
        js = list(visible(first + t, window))
        s = ((qn[t][None] * k[js]).sum(-1) + (qr[t][None] * kr[js][:, None]).sum(-1)) * m["scale"]   # [keys, H]
        w = torch.softmax(s, dim=0)
        out[t] = (w[:, :, None] * v[js]).sum(0) * gate[t][:, None]
    return out.reshape(n, H * dv) @ p["o"].t()


def clamped_mlp(h: torch.Tensor, p: Mapping[str, torch.Tensor], limit: float) -> torch.Tensor:
    g = torch.clamp(h @ p["gate"].t(), max=limit)
    u = torch.clamp(h @ p["up"].t(), -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ p["down"].t()


def sub_tensors(tensors: Mapping[str, torch.Tensor], prefix: str) -> dict:
    return {k[len(prefix):]: v.to(F) for k, v in tensors.items() if k.startswith(prefix)}


class PlainPibuvik:
    def __init__(self, config: Mapping[str, Any], tensors: Mapping[str, torch.Tensor]) -> None:
        self.cfg, self.t = config, {k: v.to(F) for k, v in tensors.items()}
        self.eps, self.m = float(config["norm"]["eps"]), float(config["residual_mult"])

    def new_state(self) -> list:
        return [{} for _ in self.cfg["layers"]]

    def layer(self, i: int, x: torch.Tensor, states: list) -> torch.Tensor:
        entry = self.cfg["layers"][i]
        own, mix = sub_tensors(self.t, f"l{i}."), sub_tensors(self.t, f"l{i}.mix.")
        kind, m = entry["type"], entry["mixer"]
        h = rms_norm(x, own["norm1"], self.eps)
        if kind == "rglru":
            y = rglru(h, mix, states[i])
        elif kind == "attention":
            y = key_value_attention(h, mix, m, states[i])
        else:
            lender = m.get("kv_from")
            y = latent_attention(h, mix, m, self.eps, states[i], None if lender is None else states[lender])
        x = x + self.m * rms_norm(y, own["norm1b"], self.eps)
        if entry.get("mlp") is not None:
            f = clamped_mlp(rms_norm(x, own["norm2"], self.eps), sub_tensors(self.t, f"l{i}.mlp."), entry["mlp"]["limit"])
            x = x + self.m * rms_norm(f, own["norm2b"], self.eps)
        return x

    def forward(self, tokens, states: Optional[list] = None, layers_out: Optional[list] = None) -> torch.Tensor:
        """Logits ``[tokens, vocab]``; ``states`` (from :meth:`new_state`) carries the sequence from call to call."""
        states = self.new_state() if states is None else states
        x = self.t["embed"][torch.as_tensor(tokens, dtype=torch.long)] * self.cfg["embedding"]["scale"]
        for i in range(len(self.cfg["layers"])):
            x = self.layer(i, x, states)
            if layers_out is not None:
                layers_out.append(x.clone())
        x = rms_norm(x, self.t["final.norm"], self.eps)
        return x @ self.t["embed"].t() * self.cfg["logit_scale"]


def greedy_generate(cfg: Mapping[str, Any], tensors: Mapping[str, torch.Tensor], prompt, n_new: int) -> list:
    m, out = PlainPibuvik(cfg, tensors), []
    states = m.new_state()
    row = m.forward(prompt, states)[-1]
    for _ in range(n_new):
        out.append(int(row.argmax()))
        row = m.forward(out[-1:], states)[-1]
    return out


# ------------------------------------------------------------------------------ weights of a test model

def tensor_shapes(cfg: Mapping[str, Any]) -> dict:
    """Name -> shape of every tensor of a model of this configuration."""
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out.update({p + "norm1": (w,), p + "norm1b": (w,)})
        if layer["type"] == "rglru":
            c, b = m["width"], m["blocks"]
            s = c // b
            out.update({p + "mix.y": (c, w), p + "mix.y.b": (c,), p + "mix.x": (c, w), p + "mix.x.b": (c,),
                        p + "mix.conv": (c, m["conv"]), p + "mix.conv.b": (c,), p + "mix.ra": (b, s, s), p + "mix.ra.b": (b, s),
                        p + "mix.ri": (b, s, s), p + "mix.ri.b": (b, s), p + "mix.lam": (c,), p + "mix.o": (w, c)})
        elif layer["type"] == "attention":
            H, G, d = m["heads"], m["kv_heads"], m["dim"]
            out.update({p + "mix.q": (H * d, w), p + "mix.k": (G * d, w), p + "mix.sink": (H,), p + "mix.o": (w, H * d)})
        else:
            H, d, rd, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            out.update({p + "mix.dq": (m["q_rank"], w), p + "mix.dq.norm": (m["q_rank"],),
                        p + "mix.uq": (H * (d + rd), m["q_rank"]), p + "mix.uk": (H * d, r), p + "mix.uv": (H * dv, r),
                        p + "mix.g": (H, w), p + "mix.o": (w, H * dv)})
            if m.get("kv_from") is None:
                out.update({p + "mix.dkv": (r + rd, w), p + "mix.dkv.norm": (r,)})
        f = layer.get("mlp")
        if f is not None:
            out.update({p + "norm2": (w,), p + "norm2b": (w,), p + "mlp.gate": (f["ff"], w), p + "mlp.up": (f["ff"], w),
                        p + "mlp.down": (w, f["ff"])})
    return out


def random_weights(cfg: Mapping[str, Any], seed: int, sharp: float = 2.0) -> dict:
    """Random tensors whose values are exactly representable in bfloat16 (float64 here), drawn so that every
    mechanism matters: queries ``sharp`` enough that a key counts, sinks of the size of a score, decays from a
    few tokens to a few hundred, activations beyond the clamp."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".", 1)[1] if name.startswith("l") and "." in name else name
        if "norm" in leaf:
            t = 1.0 + 0.2 * torch.randn(shape, generator=g)
        elif leaf in ("mix.y.b", "mix.x.b", "mix.conv.b", "mix.ra.b", "mix.ri.b"):
            t = 0.5 * torch.randn(shape, generator=g)
        elif leaf == "mix.conv":
            t = 0.6 * torch.randn(shape, generator=g)
        elif leaf == "mix.lam":
            t = -6.0 + 4.0 * torch.rand(shape, generator=g)
        elif leaf == "mix.sink":
            t = 1.5 * torch.randn(shape, generator=g)
        elif name == "embed":
            t = 0.5 * torch.randn(shape, generator=g)
        else:
            t = torch.randn(shape, generator=g) / math.sqrt(shape[-1])
            t = t * {"mix.q": sharp, "mix.uq": sharp, "mlp.gate": 2.0, "mlp.up": 2.0}.get(leaf, 1.0)
        out[name] = t.to(torch.bfloat16).to(F)
    return out


def jittered(tensors: Mapping[str, torch.Tensor], seed: int = 0, size: float = 2.0 ** -8) -> dict:
    """Every matrix with relative noise of the size of bfloat16's rounding: how far the logits of a position
    move under it says how far rounding may move them."""
    g = torch.Generator().manual_seed(seed)
    return {n: t * (1 + size * torch.randn(t.shape, generator=g, dtype=F)) if t.dim() >= 2 else t for n, t in tensors.items()}


def write_folder(folder, cfg: Mapping[str, Any], tensors: Mapping[str, torch.Tensor]):
    """``config.json`` and ``model.safetensors`` (bfloat16) of ``tensors``, written byte by byte here."""
    import json
    import struct

    import numpy as np

    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    header, blobs, at = {}, [], 0
    for name in sorted(tensors):
        bits = (tensors[name].to(torch.float32).contiguous().view(torch.int32).numpy().astype(np.uint32) >> 16).astype("<u2")
        raw = bits.tobytes()
        header[name] = {"dtype": "BF16", "shape": list(tensors[name].shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(header).encode()
    head += b" " * (-len(head) % 8)
    with open(folder / "model.safetensors", "wb") as f:
        f.write(struct.pack("<Q", len(head)))
        f.write(head)
        for raw in blobs:
            f.write(raw)
    return folder
