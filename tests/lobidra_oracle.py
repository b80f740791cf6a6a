"""Plain, slow oracle of the Lobidra design: one function per mechanism, whole sequences only, no cache, no batching.

Written from the design's equations in float64 and shares no code with the package: the tests compare the engine (its
kernels, caches, state slots and scheduler) with this.  Inputs: the configuration as the dictionary a checkpoint's
``config.json`` holds, and the weights as {tensor name: tensor}.

Notation: ``x`` is the residual stream [T, W], ``n(v, g) = v / sqrt(mean(v^2) + eps) * (1 + g)``.  A layer is
``x += n(mixer(n(x, a1)), b1); x += n(ff(n(x, a2)), b2)``.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def rms(v, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def offset_norm(v, gain, eps):
    """RMS norm whose stored gain sits around zero."""
    return rms(v, eps) * (1.0 + gain)


def short_conv(u, taps):
    """y[t] = sum_j taps[:, j] u[t - K + 1 + j] per channel; nothing before the start."""
    T, K = u.shape[0], taps.shape[1]
    y = torch.zeros_like(u)
    for j in range(K):
        back = K - 1 - j
        if back < T:
            y[back:] = y[back:] + taps[:, j] * u[:T - back]
    return y


def frequencies(rot: dict):
    """One frequency per pair; long wavelengths are slowed by `factor`, a band between two limits is blended."""
    out = []
    for i in range(int(rot["dims"]) // 2):
        f = float(rot["base"]) ** (-2.0 * i / int(rot["dims"]))
        s = rot.get("scaling")
        if s:
            factor, low, high, orig = (float(s[k]) for k in ("factor", "low", "high", "original"))
            wave = 2.0 * math.pi / f
            if wave > orig / low:
                f = f / factor
            elif wave >= orig / high:
                mix = (orig / wave - low) / (high - low)
                f = (1.0 - mix) * f / factor + mix * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate(v, rot: dict | None):
    """Neighbouring coordinates (2i, 2i + 1) of v [T, heads, D] turn by position * frequency i."""
    if not rot or not int(rot["dims"]):
        return v
    T, n = v.shape[0], int(rot["dims"])
    ang = torch.arange(T, dtype=F64)[:, None] * frequencies(rot)[None, :]
    cos, sin = ang.cos()[:, None, :], ang.sin()[:, None, :]
    out = v.clone()
    a, b = v[..., 0:n:2], v[..., 1:n:2]
    out[..., 0:n:2] = a * cos - b * sin
    out[..., 1:n:2] = b * cos + a * sin
    return out


def sink_softmax(q, k, v, scale: float, sink):
    """Causal attention of q [T, H, D] over k [T, G, D], v [T, G, V]; exp(sink[h]) joins head h's denominator."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    o = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    unseen = torch.arange(T)[None, :] > torch.arange(T)[:, None]
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(unseen, float("-inf"))
        top = torch.maximum(s.max(-1, keepdim=True).values, sink[h])
        e = torch.exp(s - top)
        o[:, h] = (e @ v[:, g]) / (e.sum(-1, keepdim=True) + torch.exp(sink[h] - top))
    return o


def conv_attention(h, m: dict, w: dict):
    """Keys that are also the values (before they are rotated), a sink of score zero, one gate per head."""
    T, H, G, D = h.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q, k = h @ w["q"].T, h @ w["k"].T
    if "q.conv" in w:
        q, k = short_conv(q, w["q.conv"]), short_conv(k, w["k.conv"])
    q, k = q.view(T, H, D), k.view(T, G, D)
    o = sink_softmax(rotate(q, m.get("rot")), rotate(k, m.get("rot")), k, float(m["scale"]), torch.zeros(H, dtype=F64))
    return (o * torch.sigmoid(h @ w["g"].T)[:, :, None]).reshape(T, -1) @ w["o"].T


def temperature(p: int, t: dict | None) -> float:
    return 1.0 if not t else 1.0 + float(t["coef"]) * math.log(math.floor((p + 1) / t["every"]) + 1)


def warm_attention(h, m: dict, w: dict):
    """No rotation; queries grow with their position; a learned sink per head; a gate per output element."""
    T, H, G, D, V = h.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    temp = torch.tensor([temperature(p, m.get("q_temp")) for p in range(T)], dtype=F64)
    q = (h @ w["q"].T).view(T, H, D) * temp[:, None, None]
    k, v = (h @ w["k"].T).view(T, G, D), (h @ w["v"].T).view(T, G, V)
    o = sink_softmax(q, k, v, float(m["scale"]), w["sink"]).reshape(T, H * V)
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def matrix_memory(q, k, v, ig, fg):
    """q, k [T, H, D], v [T, H, V], log gates ig, fg [T, H] -> read-outs [T, H, V]; the running maximum starts at zero."""
    T, H, D = k.shape
    S = torch.zeros(H, D, v.shape[2], dtype=k.dtype)
    n, m = torch.zeros(H, D, dtype=k.dtype), torch.zeros(H, dtype=k.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        new = torch.maximum(fg[t] + m, ig[t])
        keep, put = torch.exp(fg[t] + m - new), torch.exp(ig[t] - new)
        S = keep[:, None, None] * S + put[:, None, None] * (k[t][:, :, None] * v[t][:, None, :])
        n = keep[:, None] * n + put[:, None] * k[t]
        m = new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = torch.einsum("hdv,hd->hv", S, q[t]) / den[:, None]
    return out


def memory_mixer(h, m: dict, w: dict, eps: float):
    T, H, D, V = h.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    cap = float(m["gate_cap"])
    q = (h @ w["q"].T).view(T, H, D) * D ** -0.5
    k, v = (h @ w["k"].T).view(T, H, D), (h @ w["v"].T).view(T, H, V)
    ig = cap * torch.tanh((h @ w["i"].T + w["i.b"]) / cap)
    fg = torch.nn.functional.logsigmoid(cap * torch.tanh((h @ w["f"].T + w["f.b"]) / cap))
    o = rms(matrix_memory(q, k, v, ig, fg), eps).reshape(T, H * V) * w["norm"]
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def sub(w: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def parallel(h, m: dict, w: dict, eps: float):
    left = warm_attention(h, m["left"], sub(w, "left."))
    right = memory_mixer(h, m["right"], sub(w, "right."), eps)
    return float(m["left_scale"]) * left + float(m["right_scale"]) * right


def gated_expert(h, w: dict):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def feed_forward(h, f: dict, w: dict, tokens):
    if f.get("kind") == "dense":
        return gelu_tanh(h @ w["up"].T) @ w["down"].T
    top = int(f["router"]["top"])
    out = torch.zeros_like(h)
    for t, tok in enumerate(tokens.tolist()):
        for e in w["table"][tok].tolist():
            out[t] += gated_expert(h[t:t + 1], sub(w, f"e{e}."))[0] / top
    if f.get("shared"):
        out = out + gated_expert(h, sub(w, "shared."))
    return out


def layer(x, L: dict, w: dict, eps: float, tokens):
    h = offset_norm(x, w["norm1"], eps)
    mw = sub(w, "mix.")
    y = conv_attention(h, L["mixer"], mw) if L["type"] == "attention" else parallel(h, L["mixer"], mw, eps)
    x = x + offset_norm(y, w["norm1b"], eps)
    if L.get("mlp"):
        y = feed_forward(offset_norm(x, w["norm2"], eps), L["mlp"], sub(w, "mlp."), tokens)
        x = x + offset_norm(y, w["norm2b"], eps)
    return x


def forward(cfg: dict, weights: dict, tokens, trace: list | None = None):
    """Logits [T, vocab] of one sequence; `trace` receives the stream after every layer."""
    w = {k: v.to(F64) if v.is_floating_point() else v for k, v in weights.items()}
    eps = float(cfg["norm"]["eps"])
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x = w["embed"][tokens] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    for i, L in enumerate(cfg["layers"]):
        owner = i
        while cfg["layers"][owner].get("weights_of") is not None:  # the layer that has the tensors
            owner = int(cfg["layers"][owner]["weights_of"])
        x = layer(x, L, sub(w, f"l{owner}."), eps, tokens)
        if trace is not None:
            trace.append(x.clone())
    return offset_norm(x, w["final.norm"], eps) @ w["head"].T
