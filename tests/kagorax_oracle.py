"""Plain, slow oracle of the Kagorax design: one function per mechanism, whole sequences only, no cache, no batching.

Written from the design's equations in float64 and shares no code with the package: the tests compare the engine (its
kernels, cache, scheduler) with this.  Inputs: the configuration as the dictionary a checkpoint's ``config.json`` holds,
and the weights as {tensor name: tensor}.

Notation: ``x`` is the residual stream [T, W].  A layer is ``h = n(x) * w; x += mixer(h) + ff(h)`` with
``n(v) = v / sqrt(mean(v^2) + eps)``.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms(v, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def position_vector(p: int, width: int):
    """(sin, cos) pairs: entry 2i turns with 10000^(-2i / width) per position."""
    out = torch.zeros(width, dtype=F64)
    for c in range(width):
        ang = p * 10000.0 ** (-(c - c % 2) / width)
        out[c] = math.sin(ang) if c % 2 == 0 else math.cos(ang)
    return out


def embedding(cfg: dict, w: dict, tokens):
    scale = float((cfg.get("embedding") or {}).get("scale", 1.0))
    W = w["embed"].shape[1]
    return w["embed"][tokens] * scale + torch.stack([position_vector(t, W) for t in range(len(tokens))])


def bucket(n: int, B: int, D: float) -> int:
    """Distances below B/2 have a row each; the rest share logarithmic rows up to the distance D, then the last one.
    A tiny nudge keeps distances that lie exactly on a row's edge on the upper side whatever the logarithm rounds to."""
    half = B // 2
    if n < half:
        return n
    return min(B - 1, half + math.floor(math.log(n / half) / math.log(D / half) * (B - half) + 1e-9))


def visible(i: int, j: int, mask: dict | None) -> bool:
    if j > i:
        return False
    if not mask or "size" not in mask:
        return True
    return i - j < int(mask["size"]) or j < int(mask.get("keep_first", 0))


def keys_values(h, m: dict, w: dict, eps: float):
    T, G = h.shape[0], int(m["kv_heads"])
    k = rms((h @ w["k"].T + w["k.b"]).view(T, G, int(m["dim"])), eps)
    v = (h @ w["v"].T + w["v.b"]).view(T, G, int(m["vdim"]))
    return k, v


def attention(h, m: dict, w: dict, eps: float, kv):
    """kv: the keys and values this layer attends to -- its own, or those of the layer it takes them from."""
    T, H, G, D, V = h.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = rms((h @ w["q"].T + w["q.b"]).view(T, H, D), eps)
    k, v = kv
    rel = w["rel"]
    B = rel.shape[0]
    row_of = torch.tensor([bucket(n, B, float(m["bias_max"])) for n in range(T)])
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    dist = (i - j).clamp(min=0)
    seen = torch.tensor([[visible(a, b, m.get("mask")) for b in range(T)] for a in range(T)])
    o = torch.zeros(T, H, V, dtype=h.dtype)
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * float(m["scale"]) + rel[row_of[dist], hd]
        o[:, hd] = torch.softmax(s.masked_fill(~seen, float("-inf")), dim=-1) @ v[:, g]
    return (o.reshape(T, H * V) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(z, top: int):
    """The experts with the largest sigmoid scores; the scores themselves are the weights."""
    s = torch.sigmoid(z)
    idx = s.topk(top, dim=-1).indices
    return idx, s.gather(1, idx)


def feed_forward(h, f: dict, w: dict):
    idx, wt = route(h @ w["router"].T, int(f["router"]["top"]))
    out = torch.zeros(h.shape[0], w["e0.down"].shape[0], dtype=h.dtype)
    for t in range(h.shape[0]):
        for e, c in zip(idx[t].tolist(), wt[t]):
            out[t] += expert(c * h[t:t + 1], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])[0]
    if f.get("shared"):
        out = out + torch.sigmoid(h @ w["shared.sg"].T) * expert(h, w["shared.gate"], w["shared.up"], w["shared.down"])
    return out


def sub(w: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def layer(x, i: int, cfg: dict, w: dict, kvs: dict):
    """kvs: {layer: its (keys, values)}, filled here by the layers that make their own."""
    L, eps = cfg["layers"][i], float(cfg["norm"]["eps"])
    lw = sub(w, f"l{i}.")
    m, mw = L["mixer"], sub(lw, "mix.")
    h = rms(x, eps) * lw["norm1"]
    src = m.get("kv_from")
    if src is None:
        kvs[i] = keys_values(h, m, mw, eps)
    y = attention(h, m, mw, eps, kvs[i if src is None else int(src)])
    if L.get("mlp"):
        y = y + feed_forward(h, L["mlp"], sub(lw, "mlp."))
    return x + y


def forward(cfg: dict, weights: dict, tokens, trace: list | None = None):
    """Logits [T, vocab] of one sequence; `trace` receives the stream after every layer."""
    w = {k: v.to(F64) if v.is_floating_point() else v for k, v in weights.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x, kvs = embedding(cfg, w, tokens), {}
    for i in range(len(cfg["layers"])):
        x = layer(x, i, cfg, w, kvs)
        if trace is not None:
            trace.append(x.clone())
    return (rms(x, float(cfg["norm"]["eps"])) * w["final.norm"]) @ w["embed"].T
