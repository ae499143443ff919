"""A plain, slow Rurorax in float64: one sequence at a time, no cache, no batching, one function per
mechanism. It takes the configuration as the dictionary that ``config.json`` holds and the tensors by
their checkpoint names, and shares no code with the engine.

A layer reads its stream once, through a tanh in place of a norm, and adds both sublayers' results, each
times a vector of its own: ``x <- x + s1 * mixer(h) + s2 * ff(h)``, ``h = tanh(alpha x) * w + b``. The mixer is
a state-space recurrence with one decay and step size a head and maps shared by groups of heads
(``mamba2``), or grouped attention in chunks with norms over the whole query and key projections
(``attention``). The feed-forward is gated by a gelu, or a mixture of experts under sigmoid scores which
scale the experts' inputs. ``states`` carry what a sequence keeps from one call to the next, so that the same
functions also step token by token.
"""

from __future__ import annotations

import math
from typing import Any, Mapping, Optional

import torch

F = torch.float64


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * sigmoid(x)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z * z * z)))


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def tanh_norm(x: torch.Tensor, alpha: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    return torch.tanh(alpha * x) * w + b


def linear(h: torch.Tensor, p: Mapping[str, torch.Tensor], name: str) -> torch.Tensor:
    y = h @ p[name].t()
    return y + p[name + ".b"] if name + ".b" in p else y


# ------------------------------------------------------------------------------ attention

def rotary_frequencies(rot: Mapping[str, Any]) -> torch.Tensor:
    """``base^(-2i/dims)``, all divided by ``scaling.factor``."""
    dims, factor = rot["dims"], float((rot.get("scaling") or {}).get("factor", 1.0))
    return torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) / factor for i in range(dims // 2)], dtype=F)


def rotate(x: torch.Tensor, positions: torch.Tensor, rot: Optional[Mapping[str, Any]]) -> torch.Tensor:
    """``x [n, heads, dim]``: component ``i`` turns with component ``i + dims/2`` for ``i < dims/2``; the rest stays."""
    if not rot:
        return x
    dims = rot["dims"]
    half = dims // 2
    angle = positions.to(F)[:, None, None] * rotary_frequencies(rot)
    c, s = torch.cos(angle), torch.sin(angle)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


def visible(i: int, j: int, size: Optional[int]) -> bool:
    return j <= i and (not size or i // size == j // size)


def attention_sizes(m: Mapping[str, Any]) -> tuple:
    """heads, kv heads (absent: as many), key size, value size (absent: the key's), scale (absent: dim^-1/2)."""
    H, d = m["heads"], m["dim"]
    scale = m.get("scale")
    return H, m.get("kv_heads") or H, d, m.get("vdim") or d, float(scale) if scale is not None else d ** -0.5


def chunked_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, first: int, scale: float, size: Optional[int]) -> torch.Tensor:
    """``q [n, heads, d]`` at positions ``first ..``; ``k [total, kv, d]``, ``v [total, kv, dv]`` from position 0;
    query head ``h`` reads kv head ``h // (heads / kv)``. Returns ``[n, heads, dv]``."""
    n, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(n, H, v.shape[2], dtype=F)
    for t in range(n):
        seen = [j for j in range(first + t + 1) if visible(first + t, j, size)]
        for g in range(G):
            heads = [h for h in range(H) if h // (H // G) == g]
            s = q[t, heads] @ k[seen, g].t() * scale
            out[t, heads] = torch.softmax(s, dim=-1) @ v[seen, g]
    return out


def attention(h: torch.Tensor, p: Mapping[str, torch.Tensor], m: Mapping[str, Any], eps: float, first: int, state: dict) -> torch.Tensor:
    n = h.shape[0]
    H, G, d, dv, scale = attention_sizes(m)
    pos = torch.arange(first, first + n)
    q = rotate((rms(linear(h, p, "q"), eps) * p["q.norm"]).view(n, H, d), pos, m.get("rot"))
    k = rotate((rms(linear(h, p, "k"), eps) * p["k.norm"]).view(n, G, d), pos, m.get("rot"))
    v = linear(h, p, "v").view(n, G, dv)
    if "k" in state:
        k, v = torch.cat([state["k"], k]), torch.cat([state["v"], v])
    state["k"], state["v"] = k, v
    o = chunked_attention(q, k, v, first, scale, (m.get("mask") or {}).get("size"))
    return linear(o.reshape(n, H * dv), p, "o")


# ------------------------------------------------------------------------------ the state-space recurrence

def convolve(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, kept: Optional[torch.Tensor]) -> tuple:
    """A causal convolution per channel: ``y_t = b + sum_j w[:, taps - 1 - j] x_(t - j)``; ``kept [taps - 1, channels]`` are
    the inputs before the first row (``None``: zeros). Returns the result and what is kept for the next call."""
    taps = w.shape[1]
    full = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=F) if kept is None else kept, x])
    out = torch.stack([b + sum(w[:, i] * full[t + i] for i in range(taps)) for t in range(x.shape[0])])
    return out, full[full.shape[0] - (taps - 1):]


def state_space(x: torch.Tensor, B: torch.Tensor, C: torch.Tensor, dt: torch.Tensor, a_log: torch.Tensor, d: torch.Tensor,
                S: Optional[torch.Tensor]) -> tuple:
    """``x [n, H, V]``, ``B, C [n, G, N]``, ``dt [n, H]``: per head ``S <- exp(-exp(a_log) dt) S + dt B x^T`` (``S [H, N, V]``),
    ``y = S^T C + d x``; head ``h`` reads B and C of group ``h // (H / G)``."""
    n, H, V = x.shape
    G, N = B.shape[1], B.shape[2]
    S = torch.zeros(H, N, V, dtype=F) if S is None else S.clone()
    y = torch.zeros(n, H, V, dtype=F)
    for t in range(n):
        for h in range(H):
            g = h // (H // G)
            S[h] = torch.exp(-torch.exp(a_log[h]) * dt[t, h]) * S[h] + dt[t, h] * torch.outer(B[t, g], x[t, h])
            y[t, h] = S[h].t() @ C[t, g] + d[h] * x[t, h]
    return y, S


def gated_parts_norm(y: torch.Tensor, z: torch.Tensor, w: torch.Tensor, parts: int, eps: float) -> torch.Tensor:
    """The gate first, then each of ``parts`` equal parts of the row by its own root mean square, then the weight."""
    n, width = y.shape
    return rms((y * silu(z)).view(n, parts, width // parts), eps).reshape(n, width) * w


def mamba2(h: torch.Tensor, p: Mapping[str, torch.Tensor], m: Mapping[str, Any], eps: float, state: dict) -> torch.Tensor:
    n, H, V, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m.get("groups") or 1
    inner, channels = H * V, H * V + 2 * G * N
    z, xbc, dt = (h @ p["in"].t()).split([inner, channels, H], dim=1)
    xbc, state["kept"] = convolve(xbc, p["conv"], p["conv.b"], state.get("kept"))
    x, B, C = silu(xbc).split([inner, G * N, G * N], dim=1)
    y, state["S"] = state_space(x.reshape(n, H, V), B.reshape(n, G, N), C.reshape(n, G, N), softplus(dt + p["dt_bias"]), p["A_log"],
                                p["D"], state.get("S"))
    return gated_parts_norm(y.reshape(n, inner), z, p["norm"], m.get("norm_groups") or 1, eps) @ p["o"].t()


# ------------------------------------------------------------------------------ feed-forward

def dense(h: torch.Tensor, p: Mapping[str, torch.Tensor]) -> torch.Tensor:
    return linear(gelu_tanh(linear(h, p, "gate")) * linear(h, p, "up"), p, "down")


def choose(z: torch.Tensor, top: int) -> tuple:
    """The ``top`` largest sigmoid scores of each row, as they are: ids and scores."""
    s = sigmoid(z)
    ids = torch.argsort(s, dim=-1, descending=True, stable=True)[:, :top]
    return ids, s.gather(1, ids)


def expert(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor) -> torch.Tensor:
    return (silu(h @ gate.t()) * (h @ up.t())) @ down.t()


def call_margins(z: torch.Tensor, top: int) -> torch.Tensor:
    """How far each row's last chosen logit lies above the first that is not chosen (all chosen: infinity)."""
    if top >= z.shape[1]:
        return torch.full((z.shape[0],), math.inf, dtype=F)
    best = torch.sort(z, dim=1, descending=True).values
    return best[:, top - 1] - best[:, top]


def experts(h: torch.Tensor, p: Mapping[str, torch.Tensor], f: Mapping[str, Any], margins: Optional[list] = None) -> torch.Tensor:
    z = h @ p["router"].t()
    if margins is not None:
        margins.append(call_margins(z, f["router"]["top"]))
    ids, s = choose(z, f["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(ids[t].tolist(), s[t]):
            out[t] += expert((w * h[t])[None], p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"])[0]
    return out


# ------------------------------------------------------------------------------ the model

def sub_tensors(tensors: Mapping[str, torch.Tensor], prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


class PlainRurorax:
    def __init__(self, config: Mapping[str, Any], tensors: Mapping[str, torch.Tensor]) -> None:
        self.cfg = config
        self.t = {k: v.to(F) for k, v in tensors.items()}
        self.eps = float(config["norm"]["eps"])

    def new_state(self) -> list:
        return [{} for _ in self.cfg["layers"]]

    def norm(self, name: str, x: torch.Tensor) -> torch.Tensor:
        return tanh_norm(x, self.t[name + ".alpha"], self.t[name], self.t[name + ".b"])

    def layer(self, i: int, x: torch.Tensor, first: int, states: list, margins: Optional[list] = None) -> torch.Tensor:
        entry, p = self.cfg["layers"][i], f"l{i}."
        h, mix = self.norm(p + "norm1", x), sub_tensors(self.t, p + "mix.")
        if entry["type"] == "mamba2":
            y = mamba2(h, mix, entry["mixer"], self.eps, states[i])
        elif entry["type"] == "attention":
            y = attention(h, mix, entry["mixer"], self.eps, first, states[i])
        else:
            raise ValueError(entry["type"])
        out = x + self.t[p + "ls1"] * y
        f = entry.get("mlp")
        if f is not None:
            own = sub_tensors(self.t, p + "mlp.")
            out = out + self.t[p + "ls2"] * (dense(h, own) if f["kind"] == "dense" else experts(h, own, f, margins))
        return out

    def forward(self, tokens, states: Optional[list] = None, start: int = 0, layers_out: Optional[list] = None,
                margins: Optional[list] = None) -> torch.Tensor:
        """Logits ``[tokens, vocab]`` of ``tokens`` at positions ``start, start+1, ...``; ``states`` (from
        :meth:`new_state`) carries the sequence from call to call. ``margins`` receives, per mixture of
        experts, how close each token's choice was."""
        states = self.new_state() if states is None else states
        x = self.t["embed"][torch.as_tensor(tokens, dtype=torch.long)]
        for i in range(len(self.cfg["layers"])):
            x = self.layer(i, x, start, states, margins)
            if layers_out is not None:
                layers_out.append(x.clone())
        logits = self.norm("final.norm", x) @ self.t["embed"].t()
        cap = self.cfg.get("logit_softcap")
        return float(cap) * torch.tanh(logits / float(cap)) if cap else logits


def greedy_generate(cfg: Mapping[str, Any], tensors: Mapping[str, torch.Tensor], prompt, n_new: int) -> list:
    m = PlainRurorax(cfg, tensors)
    states = m.new_state()
    logits = m.forward(list(prompt), states)
    out, at = [], len(prompt)
    for _ in range(n_new):
        nxt = int(logits[-1].argmax())
        out.append(nxt)
        logits = m.forward([nxt], states, start=at)
        at += 1
    return out


# ------------------------------------------------------------------------------ weights of a test model

def tensor_shapes(cfg: Mapping[str, Any]) -> dict:
    """Name -> shape of every tensor of a model of this configuration."""
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "final.norm.b": (w,), "final.norm.alpha": ()}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out.update({p + "norm1": (w,), p + "norm1.b": (w,), p + "norm1.alpha": (), p + "ls1": (w,)})
        if layer["type"] == "attention":
            H, G, d, dv, _ = attention_sizes(m)
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                out.update({p + "mix." + n: (rows, w), p + f"mix.{n}.b": (rows,)})
            out.update({p + "mix.q.norm": (H * d,), p + "mix.k.norm": (G * d,), p + "mix.o": (w, H * dv), p + "mix.o.b": (w,)})
        else:
            H, V, N, G = m["heads"], m["vdim"], m["state"], m.get("groups") or 1
            inner, channels = H * V, H * V + 2 * G * N
            out.update({p + "mix.in": (inner + channels + H, w), p + "mix.conv": (channels, m["conv"]), p + "mix.conv.b": (channels,),
                        p + "mix.dt_bias": (H,), p + "mix.A_log": (H,), p + "mix.D": (H,), p + "mix.norm": (inner,),
                        p + "mix.o": (w, inner)})
        f = layer.get("mlp")
        if f is not None:
            out[p + "ls2"] = (w,)
            if f["kind"] == "dense":
                for n, shape in (("gate", (f["ff"], w)), ("up", (f["ff"], w)), ("down", (w, f["ff"]))):
                    out.update({p + "mlp." + n: shape, p + f"mlp.{n}.b": shape[:1]})
            else:
                out[p + "mlp.router"] = (f["router"]["experts"], w)
                for e in range(f["router"]["experts"]):
                    out.update({p + f"mlp.e{e}.gate": (f["expert"]["ff"], w), p + f"mlp.e{e}.up": (f["expert"]["ff"], w),
                                p + f"mlp.e{e}.down": (w, f["expert"]["ff"])})
    return out


def random_weights(cfg: Mapping[str, Any], seed: int) -> dict:
    """Random tensors whose values are exactly representable in bfloat16 (float64 here), drawn so that every
    mechanism matters: projections of unit-size outputs, weights around one, decays from a few tokens to hundreds, routers
    that rarely come close to a tie, biases that count."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        parts = name.split(".")
        leaf = ".".join(parts[-2:]) if parts[-1] in ("b", "norm", "alpha") and len(parts) > 2 else parts[-1]
        r = torch.randn(shape, generator=g)
        if leaf.endswith("alpha"):
            t = 0.6 + 0.1 * r
        elif leaf.endswith("norm.b") or leaf.endswith("norm1.b"):
            t = 0.2 * r
        elif leaf in ("ls1", "ls2"):
            t = 0.5 + 0.2 * r
        elif leaf.endswith("norm") or leaf == "norm1":
            t = 1.0 + 0.2 * r
        elif leaf == "A_log":
            t = -1.0 + 1.0 * r
        elif leaf == "dt_bias":
            t = -2.0 + 1.0 * r
        elif leaf == "D":
            t = 0.7 + 0.4 * r
        elif leaf == "conv":
            t = 0.6 * r
        elif leaf.endswith(".b"):
            t = 0.3 * r
        elif name == "embed":
            t = 0.7 * r
        else:
            t = r / math.sqrt(shape[-1]) * (3.0 if leaf == "router" else 1.5)
        out[name] = t.to(torch.bfloat16).to(F)
    return out


def jittered(tensors: Mapping[str, torch.Tensor], seed: int = 0, size: float = 2.0 ** -8) -> dict:
    """Every matrix with relative noise of the size of bfloat16's rounding: how far the logits of a position
    move under it says how far rounding may move them. (The routers stay: no test rests on a close call.)"""
    g = torch.Generator().manual_seed(seed)
    return {n: t * (1 + size * torch.randn(t.shape, generator=g, dtype=F)) if t.dim() == 2 and not n.endswith("router") else t
            for n, t in tensors.items()}


def write_folder(folder, cfg: Mapping[str, Any], tensors: Mapping[str, torch.Tensor]):
    """``config.json`` and ``model.safetensors`` (bfloat16) of ``tensors``, written byte by byte here."""
    import json
    import struct

    import numpy as np

    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    header, blobs, at = {}, [], 0
    for name in sorted(tensors):
        t = tensors[name].to(torch.float32).contiguous()
        raw = (t.view(torch.int32).numpy().astype(np.uint32) >> 16).astype("<u2").tobytes()
        header[name] = {"dtype": "BF16", "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
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
