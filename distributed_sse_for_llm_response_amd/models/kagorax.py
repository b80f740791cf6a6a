"""Kagorax: a decoder-only family whose mixer and feed-forward read ONE norm side by side, with distance-biased window
attention and layers that attend to another layer's keys and values; its layer list comes from ``config.json``.

The embedding output is ``x = embed[token] * scale + s(p)`` with the sinusoidal position vector ``s(p)[2i] =
sin(p 10000^(-2i/W))``, ``s(p)[2i + 1]`` the cosine of the same angle.  Every layer is

    h = n(x) * w;   x += attention(h) + ff(h)

on an fp32 residual stream, ``n(v) = v / sqrt(mean(v^2) + eps)``.  Mixer and feed-forward:

* ``attention`` -- grouped key/value heads; q, k and v projected with biases; q and k divided by their root mean square
  per head (no gain, no rotation); score ``scale q.k + rel[bucket(i - j), head]``: a learned bias per bucket of
  distances (one row per distance below half the table, then logarithmic rows up to ``bias_max``, the last row for
  everything farther; a table per layer); a sliding window of ``mask.size`` keys that also keeps the sequence's first
  ``mask.keep_first`` keys visible; the concatenated heads multiplied element by element with ``sigmoid(g h)`` before
  the output projection.  A layer with ``kv_from: j`` has no key / value projections: it attends, with its own queries,
  bias, mask and gate, to the keys and values that layer j keeps in its pages.
* routed experts -- gated-SiLU experts, the ``top`` largest ``sigmoid(router h)``, used as weights as they are and
  applied to the expert's INPUT, ``sum_k expert_k(s_k h)``; plus a shared expert for every token, multiplied by one
  number ``sigmoid(sg h)``.

The head is the embedding table itself (without its scale) behind the final norm.

This module holds the configuration (parsed from / written to the ``config.json`` dictionary), the checkpoint's tensor
naming, the distance buckets, random initialisation for tests and benchmarks, and named configurations.  The forward
pass lives in ``engine/layered_runner.py`` on the kernels of ``ops/layers.py``.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field

import torch

from .surodra import ANY, NO_WINDOW

POSITION_BASE = 10000.0


@dataclass(frozen=True)
class BiasedAttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: float           # distances from here on share the bias table's last row
    window: int = NO_WINDOW
    keep_first: int = 0       # first keys of the sequence that stay visible beyond the window
    kv_from: int = ANY        # layer whose keys and values this layer attends to (ANY: its own)


@dataclass(frozen=True)
class InputWeightedMoeSpec:
    experts: int
    top: int
    ff: int
    shared_ff: int = 0        # 0 = no shared expert


@dataclass(frozen=True)
class LayerSpec:
    kind: str                 # "attention"
    mixer: BiasedAttentionSpec
    mlp: InputWeightedMoeSpec | None


@dataclass(frozen=True)
class KagoraxConfig:
    vocab_size: int
    width: int
    eps: float
    layers: tuple
    embed_scale: float = 1.0
    name: str = "kagorax"
    max_position: int = 32768
    bos_token_id: int = 1
    eos_token_id: int = 2
    raw: dict = field(default=None, compare=False, hash=False, repr=False)

    family = "kagorax"

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def kv_layer(self, i: int) -> int:
        """The layer whose pages layer i attends to."""
        src = self.layers[i].mixer.kv_from
        return i if src == ANY else src

    # ---- config.json <-> dataclasses
    @classmethod
    def from_dict(cls, d: dict, name: str = "kagorax") -> "KagoraxConfig":
        layers = []
        for i, L in enumerate(d["layers"]):
            if L["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer type {L['type']!r}")
            m = L["mixer"]
            mask, src = m.get("mask") or {}, m.get("kv_from")
            mixer = BiasedAttentionSpec(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])),
                                        dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]),
                                        bias_max=float(m["bias_max"]), window=int(mask.get("size", NO_WINDOW)),
                                        keep_first=int(mask.get("keep_first", 0)),
                                        kv_from=ANY if src is None else int(src))
            f = L.get("mlp")
            mlp = None
            if f:
                if f.get("kind", "moe") != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward kind {f['kind']!r}")
                r = f["router"]
                mlp = InputWeightedMoeSpec(experts=int(r["experts"]), top=int(r["top"]), ff=int(f["expert"]["ff"]),
                                           shared_ff=int((f.get("shared") or {}).get("ff", 0)))
            layers.append(LayerSpec(kind=L["type"], mixer=mixer, mlp=mlp))
        cfg = cls(vocab_size=int(d["vocab"]), width=int(d["width"]), eps=float(d["norm"]["eps"]), layers=tuple(layers),
                  embed_scale=float((d.get("embedding") or {}).get("scale", 1.0)), name=name, raw=d)
        cfg.validate()
        return cfg

    def to_dict(self) -> dict:
        out = {"architecture": "Kagorax", "vocab": self.vocab_size, "width": self.width, "norm": {"eps": self.eps},
               "embedding": {"scale": self.embed_scale}, "layers": []}
        for L in self.layers:
            m, f = L.mixer, L.mlp
            mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale,
                     "bias_max": m.bias_max}
            if m.window != NO_WINDOW:
                mixer["mask"] = {"size": m.window, "keep_first": m.keep_first}
            if m.kv_from != ANY:
                mixer["kv_from"] = m.kv_from
            mlp = None
            if f is not None:
                mlp = {"kind": "moe", "expert": {"ff": f.ff}, "router": {"experts": f.experts, "top": f.top}}
                if f.shared_ff:
                    mlp["shared"] = {"ff": f.shared_ff}
            out["layers"].append({"type": L.kind, "mixer": mixer, "mlp": mlp})
        return out

    def validate(self, tp: int = 1) -> None:
        if tp != 1:
            raise ValueError("Kagorax runs on one GPU per replica (no tensor-parallel sharding of its layers)")
        for i, L in enumerate(self.layers):
            m, f = L.mixer, L.mlp
            if m.kv_heads < 1 or m.heads % m.kv_heads or max(m.dim, m.vdim) > 512:
                raise ValueError(f"layer {i}: heads must be a multiple of kv_heads, head widths at most 512")
            if m.window < 1 or m.keep_first < 0 or m.bias_max <= 0:
                raise ValueError(f"layer {i}: mask.size >= 1, mask.keep_first >= 0, bias_max > 0")
            if m.kv_from != ANY:
                if not 0 <= m.kv_from < i:
                    raise ValueError(f"layer {i}: kv_from must name an earlier layer, not {m.kv_from}")
                src = self.layers[m.kv_from].mixer
                if src.kv_from != ANY:
                    raise ValueError(f"layer {i}: kv_from names layer {m.kv_from}, which has no keys and values of its own")
                if (src.kv_heads, src.dim, src.vdim) != (m.kv_heads, m.dim, m.vdim):
                    raise ValueError(f"layer {i}: its key/value heads differ from those of layer {m.kv_from}")
            if f is not None and not (1 <= f.top <= f.experts <= 256):
                raise ValueError(f"layer {i}: 1 <= top <= experts <= 256")

    def num_params(self) -> int:
        return sum(math.prod(max(x, 1) for x in s) for s in tensor_shapes(self).values())

    def cache_bytes_per_token(self, elem_bytes: int = 2) -> int:
        """Paged cache bytes per token: keys and values of the layers that have their own."""
        return sum(L.mixer.kv_heads * (L.mixer.dim + L.mixer.vdim) * elem_bytes for L in self.layers
                   if L.mixer.kv_from == ANY)


def distance_bucket(n: int, rows: int, far: float) -> int:
    """Row of the bias table for the distance n >= 0: n itself below half = rows / 2, then `rows - half` logarithmic
    rows that end at the distance `far`, then the last row.  A distance that lies exactly on a row's edge belongs to the
    row that starts there, whatever the logarithms round to."""
    half = rows // 2
    if n < half:
        return n
    if n >= far or half < 1:
        return rows - 1
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half) + 1e-9))


def bias_by_distance(rel: torch.Tensor, far: float) -> torch.Tensor:
    """The bias table [rows, heads] laid out per head and distance, [heads, distances] fp32: entry n is the bias of the
    distance n, the last entry that of every larger one."""
    rows = rel.shape[0]
    last = 0  # first distance of the last row: later entries would all repeat it
    while distance_bucket(last, rows, far) < rows - 1:
        last += 1
    idx = torch.tensor([distance_bucket(n, rows, far) for n in range(last + 1)], device=rel.device)
    return rel.float()[idx].t().contiguous()


def position_table(positions: int, width: int, device=None) -> torch.Tensor:
    """fp32 [positions, width] sinusoidal position vectors, made in float64."""
    i = torch.arange((width + 1) // 2, dtype=torch.float64)
    out = torch.empty(positions, 2 * i.numel(), dtype=torch.float32, device=device)
    f = (POSITION_BASE ** (-2.0 * i / width)).to(out.device)
    step = max(1, (1 << 24) // max(1, width))  # bounds the float64 temporaries
    for p0 in range(0, positions, step):
        ang = torch.arange(p0, min(positions, p0 + step), dtype=torch.float64, device=out.device)[:, None] * f[None, :]
        out[p0:p0 + ang.shape[0], 0::2] = ang.sin().float()
        out[p0:p0 + ang.shape[0], 1::2] = ang.cos().float()
    return out[:, :width].contiguous()


def layer_tensor_shapes(cfg: KagoraxConfig, i: int) -> dict:
    """{tensor name: shape} of layer i (checkpoint naming, linear weights [out, in]); ANY = the checkpoint decides (the
    number of bias rows)."""
    L, W, p = cfg.layers[i], cfg.width, f"l{i}."
    m, f = L.mixer, L.mlp
    s = {p + "norm1": (W,), p + "mix.q": (m.heads * m.dim, W), p + "mix.q.b": (m.heads * m.dim,)}
    if m.kv_from == ANY:
        s.update({p + "mix.k": (m.kv_heads * m.dim, W), p + "mix.k.b": (m.kv_heads * m.dim,),
                  p + "mix.v": (m.kv_heads * m.vdim, W), p + "mix.v.b": (m.kv_heads * m.vdim,)})
    s.update({p + "mix.rel": (ANY, m.heads), p + "mix.g": (m.heads * m.vdim, W), p + "mix.o": (W, m.heads * m.vdim)})
    if f is not None:
        for e in range(f.experts):
            s.update({f"{p}mlp.e{e}.gate": (f.ff, W), f"{p}mlp.e{e}.up": (f.ff, W), f"{p}mlp.e{e}.down": (W, f.ff)})
        s[p + "mlp.router"] = (f.experts, W)
        if f.shared_ff:
            s.update({p + "mlp.shared.gate": (f.shared_ff, W), p + "mlp.shared.up": (f.shared_ff, W),
                      p + "mlp.shared.down": (W, f.shared_ff), p + "mlp.shared.sg": (1, W)})
    return s


def tensor_shapes(cfg: KagoraxConfig) -> dict:
    s = {"embed": (cfg.vocab_size, cfg.width)}
    for i in range(len(cfg.layers)):
        s.update(layer_tensor_shapes(cfg, i))
    s["final.norm"] = (cfg.width,)
    return s


@torch.no_grad()
def init_weights(cfg: KagoraxConfig, seed: int = 0, device="cpu", dtype=torch.bfloat16, rows: int = 32) -> dict:
    """Random weights in the checkpoint's naming: projections ~ N(0, 1 / fan-in), gains near 1, biases ~ N(0, 0.3),
    distance biases ~ N(0, 1) in tables of `rows` rows."""
    dev = torch.device(device)
    gdev = dev if dev.type == "cuda" else torch.device("cpu")
    g = torch.Generator(device=gdev).manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        shape = tuple(rows if x == ANY else x for x in shape)
        t = torch.randn(shape, generator=g, device=gdev)
        if leaf == "norm1" or name == "final.norm":
            t = 1.0 + 0.2 * t
        elif leaf == "b":
            t = 0.3 * t
        elif name != "embed" and leaf != "rel":
            t = t / math.sqrt(shape[-1])
        out[name] = t.to(dtype).to(dev)
    return out


def _named(name: str, vocab: int, width: int, n_layers: int, sharing: int, heads: int, kv_heads: int, dim: int, vdim: int,
           window: int, keep_first: int, experts: int, top: int, ff: int, shared_ff: int, bias_max: float = 128,
           max_position: int = 32768) -> KagoraxConfig:
    """`n_layers` layers of which the last `sharing` attend to the keys and values of the layer before them."""
    own = n_layers - sharing
    mlp = InputWeightedMoeSpec(experts=experts, top=top, ff=ff, shared_ff=shared_ff)
    layers = tuple(
        LayerSpec("attention", BiasedAttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim,
                                                   scale=1.0 / math.sqrt(dim), bias_max=bias_max, window=window,
                                                   keep_first=keep_first, kv_from=ANY if i < own else own - 1), mlp)
        for i in range(n_layers))
    cfg = KagoraxConfig(vocab_size=vocab, width=width, eps=1e-6, layers=layers, embed_scale=math.sqrt(width), name=name,
                        max_position=max_position)
    cfg.validate()
    return cfg


# Named configurations (random weights): a toy for smoke runs and sizes that resemble real models' layers for the
# benchmark -- "mid" has 2048-wide layers, "wide" the 4096-wide layers of a 7B-class model; six layers each, experts and
# shared expert of the sizes that the muderax-mid / -wide models have.
TINY = _named("kagorax-tiny", vocab=512, width=128, n_layers=3, sharing=1, heads=4, kv_heads=2, dim=32, vdim=32,
              window=24, keep_first=3, experts=6, top=2, ff=80, shared_ff=112, bias_max=60, max_position=4096)
MID = _named("kagorax-mid", vocab=32768, width=2048, n_layers=6, sharing=2, heads=16, kv_heads=8, dim=128, vdim=128,
             window=1024, keep_first=4, experts=16, top=2, ff=1408, shared_ff=2816)
WIDE = _named("kagorax-wide", vocab=32768, width=4096, n_layers=6, sharing=2, heads=32, kv_heads=8, dim=128, vdim=128,
              window=1024, keep_first=4, experts=16, top=2, ff=3584, shared_ff=7168)

CONFIGS = {c.name: c for c in (TINY, MID, WIDE)}
