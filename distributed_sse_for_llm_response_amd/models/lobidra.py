"""Lobidra: a decoder-only family of convolved softmax attention, layers that run attention and a matrix memory side by
side, and experts chosen by token id; its layer list comes from ``config.json``.

The embedding output is ``x = embed[token] * scale``.  Every layer is

    x += n(mixer(n(x, a1)), b1);   x += n(ff(n(x, a2)), b2)

on an fp32 residual stream, ``n(v, a) = v / sqrt(mean(v^2) + eps) * (1 + a)``.  Mixers:

* ``attention`` -- grouped key/value heads; q and k run through a short causal convolution over time per channel; the
  values ARE the convolved keys before rotation (no value projection); interleaved rotary pairs on the leading
  coordinates with Llama-3.1 frequency scaling; a constant sink (score 0) in the softmax's denominator; one sigmoid gate
  per head.
* ``parallel`` -- two mixers on the same input, ``left_scale * left + right_scale * right``.  Left: grouped attention
  without rotation whose queries grow with the position (``1 + coef ln(floor((p + 1) / every) + 1)``), a learned sink per
  head and a gate per output element.  Right: a matrix memory with exponential input gate and log-sigmoid forget gate
  (both soft-capped), a running maximum that starts at 0 and a normaliser vector:
  ``m' = max(f + m, i); S = e^(f + m - m') S + e^(i - m') k v^T; n likewise; o = S^T q / (max(|n.q|, e^-m') + 1e-6)``;
  RMS norm per head, one gain per output element, a sigmoid gate.

Feed-forward: dense (up, gelu, down), or gated-SiLU experts whose choice is a table row per token id (weight 1 / top
each) beside an always-on shared expert.  A layer may use another layer's tensors (``weights_of``) with a cache and state
of its own.  The head is a matrix of its own behind the final norm.

This module holds the configuration (parsed from / written to the ``config.json`` dictionary), the checkpoint's tensor
naming, random initialisation for tests and benchmarks, and named configurations.  The forward pass lives in
``engine/layered_runner.py`` on the kernels of ``ops/layers.py``.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field, replace

import torch

from .surodra import LayerRun

MEMORY_EPS = 1e-6  # added to the matrix memory's denominator


@dataclass(frozen=True)
class BandScaling:
    """Llama-3.1 frequency scaling: wavelengths beyond original / low are slowed by `factor`, those below
    original / high keep their frequency, the band between is blended."""
    factor: float
    low: float
    high: float
    original: float


@dataclass(frozen=True)
class PairRotarySpec:
    """Interleaved rotary: coordinates (2i, 2i + 1) of a head's first `dims` turn by pos * f_i."""
    dims: int
    base: float
    scaling: BandScaling | None = None

    def frequencies(self) -> torch.Tensor:
        f = self.base ** (-2.0 * torch.arange(self.dims // 2, dtype=torch.float64) / self.dims)
        s = self.scaling
        if s is None:
            return f
        wave = 2.0 * math.pi / f
        mix = (s.original / wave - s.low) / (s.high - s.low)
        band = (1.0 - mix) * f / s.factor + mix * f
        return torch.where(wave < s.original / s.high, f, torch.where(wave > s.original / s.low, f / s.factor, band))

    def table(self, max_pos: int, device=None) -> torch.Tensor:
        """fp32 [max_pos, dims / 2, 2] (cos, sin), made in float64."""
        ang = torch.arange(max_pos, dtype=torch.float64)[:, None] * self.frequencies()[None, :]
        return torch.stack([ang.cos(), ang.sin()], dim=-1).float().to(device)

    @classmethod
    def from_dict(cls, r: dict | None) -> "PairRotarySpec | None":
        if not r or not int(r["dims"]):
            return None
        s = r.get("scaling")
        sc = BandScaling(*(float(s[k]) for k in ("factor", "low", "high", "original"))) if s else None
        return cls(dims=int(r["dims"]), base=float(r["base"]), scaling=sc)

    def to_dict(self) -> dict:
        d = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            s = self.scaling
            d["scaling"] = {"factor": s.factor, "low": s.low, "high": s.high, "original": s.original}
        return d


@dataclass(frozen=True)
class QueryTemperature:
    """Queries at position p are multiplied by 1 + coef ln(floor((p + 1) / every) + 1)."""
    coef: float
    every: float

    def table(self, max_pos: int, device=None) -> torch.Tensor:
        """fp32 [max_pos], made in float64."""
        p = torch.arange(1, max_pos + 1, dtype=torch.float64)
        return (1.0 + self.coef * torch.log(torch.floor(p / self.every) + 1.0)).float().to(device)


@dataclass(frozen=True)
class ConvAttentionSpec:
    heads: int
    kv_heads: int
    dim: int                  # also the value width: the values are the unrotated keys
    conv: int                 # taps of the convolution over q and k (0: none)
    scale: float
    rot: PairRotarySpec | None = None

    @property
    def vdim(self) -> int:
        return self.dim


@dataclass(frozen=True)
class WarmAttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    temp: QueryTemperature | None = None


@dataclass(frozen=True)
class MatrixMemorySpec:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass(frozen=True)
class TwinSpec:
    left: WarmAttentionSpec
    right: MatrixMemorySpec
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class DenseGeluSpec:
    ff: int


@dataclass(frozen=True)
class TableMoeSpec:
    experts: int
    top: int
    ff: int
    shared_ff: int = 0        # 0 = no shared expert


@dataclass(frozen=True)
class LayerSpec:
    kind: str                 # "conv_attention" or "twin"
    mixer: ConvAttentionSpec | TwinSpec
    mlp: DenseGeluSpec | TableMoeSpec | None
    weights_of: int           # the layer whose tensors it uses (its own index when it has its own)


KINDS = {"attention": "conv_attention", "parallel": "twin"}  # config.json type -> mixer kind


def _attention_from(m: dict, i: int) -> ConvAttentionSpec:
    if int(m.get("vdim", m["dim"])) != int(m["dim"]):
        raise ValueError(f"layer {i}: values that are the keys have their width, vdim must equal dim")
    return ConvAttentionSpec(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])), dim=int(m["dim"]),
                             conv=int(m.get("conv") or 0), scale=float(m["scale"]), rot=PairRotarySpec.from_dict(m.get("rot")))


def _twin_from(m: dict) -> TwinSpec:
    a, r, t = m["left"], m["right"], m["left"].get("q_temp")
    left = WarmAttentionSpec(heads=int(a["heads"]), kv_heads=int(a.get("kv_heads", a["heads"])), dim=int(a["dim"]),
                             vdim=int(a["vdim"]), scale=float(a["scale"]),
                             temp=QueryTemperature(float(t["coef"]), float(t["every"])) if t else None)
    right = MatrixMemorySpec(heads=int(r["heads"]), dim=int(r["dim"]), vdim=int(r["vdim"]), gate_cap=float(r["gate_cap"]))
    return TwinSpec(left=left, right=right, left_scale=float(m["left_scale"]), right_scale=float(m["right_scale"]))


@dataclass(frozen=True)
class LobidraConfig:
    vocab_size: int
    width: int
    eps: float
    layers: tuple
    embed_scale: float = 1.0
    name: str = "lobidra"
    max_position: int = 32768
    bos_token_id: int = 1
    eos_token_id: int = 2
    raw: dict = field(default=None, compare=False, hash=False, repr=False)

    family = "lobidra"
    # parts of the bracket-norm walk that this family does not have
    bigram = None
    side_dim = 0
    loop_times = 0

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> list:
        """One run per layer, with the layer whose tensors it uses; caches and state are kept per run."""
        return [LayerRun(layer=L.weights_of, index=i, pass_no=-1) for i, L in enumerate(self.layers)]

    # ---- config.json <-> dataclasses
    @classmethod
    def from_dict(cls, d: dict, name: str = "lobidra") -> "LobidraConfig":
        layers = []
        for i, L in enumerate(d["layers"]):
            if L["type"] not in KINDS:
                raise ValueError(f"layer {i}: unknown mixer type {L['type']!r}")
            m, f = L["mixer"], L.get("mlp")
            mixer = _attention_from(m, i) if L["type"] == "attention" else _twin_from(m)
            mlp = None
            if f and f["kind"] == "dense":
                mlp = DenseGeluSpec(ff=int(f["ff"]))
            elif f and f["kind"] == "moe":
                r = f["router"]
                mlp = TableMoeSpec(experts=int(r["experts"]), top=int(r["top"]), ff=int(f["expert"]["ff"]),
                                   shared_ff=int((f.get("shared") or {}).get("ff", 0)))
            elif f:
                raise ValueError(f"layer {i}: unknown feed-forward kind {f['kind']!r}")
            own = L.get("weights_of")
            layers.append(LayerSpec(kind=KINDS[L["type"]], mixer=mixer, mlp=mlp, weights_of=i if own is None else int(own)))
        for i, L in enumerate(layers):  # follow chains to the layer that has the tensors
            j, hops = L.weights_of, 0
            while 0 <= j < len(layers) and layers[j].weights_of != j and hops < len(layers):
                j, hops = layers[j].weights_of, hops + 1
            layers[i] = replace(L, weights_of=j)
        cfg = cls(vocab_size=int(d["vocab"]), width=int(d["width"]), eps=float(d["norm"]["eps"]), layers=tuple(layers),
                  embed_scale=float((d.get("embedding") or {}).get("scale", 1.0)), name=name, raw=d)
        cfg.validate()
        return cfg

    def to_dict(self) -> dict:
        out = {"architecture": "Lobidra", "vocab": self.vocab_size, "width": self.width, "norm": {"eps": self.eps},
               "embedding": {"scale": self.embed_scale}, "layers": []}
        for i, L in enumerate(self.layers):
            m, f = L.mixer, L.mlp
            if L.kind == "conv_attention":
                e = {"type": "attention", "mixer": {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim,
                                                    "conv": m.conv, "scale": m.scale}}
                if m.rot is not None:
                    e["mixer"]["rot"] = m.rot.to_dict()
            else:
                a, r = m.left, m.right
                left = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale}
                if a.temp is not None:
                    left["q_temp"] = {"coef": a.temp.coef, "every": a.temp.every}
                e = {"type": "parallel", "mixer": {
                    "left": left, "right": {"heads": r.heads, "dim": r.dim, "vdim": r.vdim, "gate_cap": r.gate_cap},
                    "left_scale": m.left_scale, "right_scale": m.right_scale}}
            e["mlp"] = None
            if isinstance(f, DenseGeluSpec):
                e["mlp"] = {"kind": "dense", "ff": f.ff}
            elif f is not None:
                e["mlp"] = {"kind": "moe", "expert": {"ff": f.ff}, "router": {"experts": f.experts, "top": f.top}}
                if f.shared_ff:
                    e["mlp"]["shared"] = {"ff": f.shared_ff}
            if L.weights_of != i:
                e["weights_of"] = L.weights_of
            out["layers"].append(e)
        return out

    def validate(self, tp: int = 1) -> None:
        if tp != 1:
            raise ValueError("Lobidra runs on one GPU per replica (no tensor-parallel sharding of its layers)")
        for i, L in enumerate(self.layers):
            m, f = L.mixer, L.mlp
            a = m if L.kind == "conv_attention" else m.left
            if a.kv_heads < 1 or a.heads % a.kv_heads or max(a.dim, a.vdim) > 512:
                raise ValueError(f"layer {i}: heads must be a multiple of kv_heads, head widths at most 512")
            if L.kind == "conv_attention":
                if not 0 <= m.conv <= 16 or (m.rot is not None and (m.rot.dims % 2 or m.rot.dims > m.dim)):
                    raise ValueError(f"layer {i}: conv in 0..16, rot.dims even and at most dim")
                s = m.rot.scaling if m.rot is not None else None
                if s is not None and (s.factor <= 0 or s.low <= 0 or s.high <= s.low or s.original <= 0):
                    raise ValueError(f"layer {i}: rot.scaling needs factor, low, original > 0 and high > low")
            else:
                r = m.right
                if r.heads < 1 or not 1 <= r.dim <= 512 or not 1 <= r.vdim <= 512 or r.gate_cap <= 0:
                    raise ValueError(f"layer {i}: matrix memory head widths in 1..512, gate_cap > 0")
                if a.temp is not None and a.temp.every <= 0:
                    raise ValueError(f"layer {i}: q_temp.every > 0")
            if isinstance(f, TableMoeSpec) and not 1 <= f.top <= f.experts <= 4095:
                raise ValueError(f"layer {i}: 1 <= top <= experts <= 4095")
            j = L.weights_of
            if not 0 <= j < len(self.layers) or self.layers[j].weights_of != j:
                raise ValueError(f"layer {i}: weights_of names no layer with tensors of its own")
            if (self.layers[j].kind, self.layers[j].mixer, self.layers[j].mlp) != (L.kind, m, f):
                raise ValueError(f"layer {i} uses the tensors of layer {j} but differs from it")

    def num_params(self) -> int:
        return sum(math.prod(s) for s in tensor_shapes(self).values())

    def cache_bytes_per_token(self, elem_bytes: int = 2) -> int:
        """Paged cache bytes per token: keys and values of every layer's attention (the values of a convolved layer are
        kept beside its rotated keys)."""
        atts = [L.mixer if L.kind == "conv_attention" else L.mixer.left for L in self.layers]
        return sum(a.kv_heads * (a.dim + a.vdim) * elem_bytes for a in atts)


def layer_tensor_shapes(cfg: LobidraConfig, i: int) -> dict:
    """{tensor name: shape} of layer i (checkpoint naming, linear weights [out, in]); nothing for a layer that uses
    another one's tensors."""
    L, W, p = cfg.layers[i], cfg.width, f"l{i}."
    m, f = L.mixer, L.mlp
    if L.weights_of != i:
        return {}
    s = {p + "norm1": (W,), p + "norm1b": (W,)}
    if L.kind == "conv_attention":
        nq, nk = m.heads * m.dim, m.kv_heads * m.dim
        s.update({p + "mix.q": (nq, W), p + "mix.k": (nk, W)})
        if m.conv > 0:
            s.update({p + "mix.q.conv": (nq, m.conv), p + "mix.k.conv": (nk, m.conv)})
        s.update({p + "mix.g": (m.heads, W), p + "mix.o": (W, m.heads * m.vdim)})
    else:
        a, r, pl, pr = m.left, m.right, p + "mix.left.", p + "mix.right."
        no, nr = a.heads * a.vdim, r.heads * r.vdim
        s.update({pl + "q": (a.heads * a.dim, W), pl + "k": (a.kv_heads * a.dim, W), pl + "v": (a.kv_heads * a.vdim, W),
                  pl + "sink": (a.heads,), pl + "g": (no, W), pl + "o": (W, no),
                  pr + "q": (r.heads * r.dim, W), pr + "k": (r.heads * r.dim, W), pr + "v": (nr, W), pr + "g": (nr, W),
                  pr + "o": (W, nr), pr + "norm": (nr,), pr + "i": (r.heads, W), pr + "i.b": (r.heads,),
                  pr + "f": (r.heads, W), pr + "f.b": (r.heads,)})
    if f is not None:
        s.update({p + "norm2": (W,), p + "norm2b": (W,)})
    if isinstance(f, DenseGeluSpec):
        s.update({p + "mlp.up": (f.ff, W), p + "mlp.down": (W, f.ff)})
    elif f is not None:
        for e in range(f.experts):
            s.update({f"{p}mlp.e{e}.gate": (f.ff, W), f"{p}mlp.e{e}.up": (f.ff, W), f"{p}mlp.e{e}.down": (W, f.ff)})
        s[p + "mlp.table"] = (cfg.vocab_size, f.top)
        if f.shared_ff:
            s.update({p + "mlp.shared.gate": (f.shared_ff, W), p + "mlp.shared.up": (f.shared_ff, W),
                      p + "mlp.shared.down": (W, f.shared_ff)})
    return s


def tensor_shapes(cfg: LobidraConfig) -> dict:
    s = {"embed": (cfg.vocab_size, cfg.width)}
    for i in range(len(cfg.layers)):
        s.update(layer_tensor_shapes(cfg, i))
    s["final.norm"] = (cfg.width,)
    s["head"] = (cfg.vocab_size, cfg.width)
    return s


@torch.no_grad()
def init_weights(cfg: LobidraConfig, seed: int = 0, device="cpu", dtype=torch.bfloat16) -> dict:
    """Random weights in the checkpoint's naming: projections ~ N(0, 1 / fan-in), stored gains near 0, the memory's
    output gains near 1, forget gates that remember, sinks ~ N(0, 1), tables of distinct experts."""
    dev = torch.device(device)
    gdev = dev if dev.type == "cuda" else torch.device("cpu")
    g = torch.Generator(device=gdev).manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf == "table":
            experts = cfg.layers[int(name[1:name.index(".")])].mlp.experts
            t = torch.rand(shape[0], experts, generator=g, device=gdev).argsort(dim=-1)[:, :shape[1]]
            out[name] = t.to(torch.int32).contiguous().to(dev)
            continue
        t = torch.randn(shape, generator=g, device=gdev)
        if leaf.startswith("norm"):
            t = 0.2 * t + (1.0 if name.endswith("right.norm") else 0.0)
        elif name.endswith("f.b"):
            t = 3.0 + t
        elif leaf == "conv":
            t = t / math.sqrt(max(1, shape[-1]))
        elif leaf not in ("b", "sink") and name != "embed":
            t = t / math.sqrt(shape[-1])
        out[name] = t.to(dtype).to(dev)
    return out


def _named(name: str, vocab: int, width: int, pattern: tuple, heads: int, kv_heads: int, dim: int, vdim: int, mem_heads: int,
           mem_dim: int, mem_vdim: int, ff: int, experts: int, top: int, expert_ff: int, shared_ff: int, rot_dims: int,
           shared_last: bool = True, max_position: int = 32768) -> LobidraConfig:
    """Layers of the given kinds; the first feed-forward is dense, the last layer uses the tensors of the latest layer of
    its kind before it."""
    rot = PairRotarySpec(dims=rot_dims, base=500000.0, scaling=BandScaling(8.0, 1.0, 4.0, 8192.0))
    att = ConvAttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, conv=4, scale=1.0 / math.sqrt(dim), rot=rot)
    twin = TwinSpec(left=WarmAttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=1.0 / math.sqrt(dim),
                                           temp=QueryTemperature(0.1, 8192.0)),
                    right=MatrixMemorySpec(heads=mem_heads, dim=mem_dim, vdim=mem_vdim, gate_cap=15.0), left_scale=1.0,
                    right_scale=1.0)
    moe = TableMoeSpec(experts=experts, top=top, ff=expert_ff, shared_ff=shared_ff)
    layers = [LayerSpec(kind=k, mixer=att if k == "conv_attention" else twin, mlp=DenseGeluSpec(ff) if i == 0 else moe,
                        weights_of=i) for i, k in enumerate(pattern)]
    if shared_last:
        j = max(i for i, L in enumerate(layers[:-1]) if L.kind == layers[-1].kind and L.mlp is moe)
        layers[-1] = replace(layers[-1], weights_of=j)
    cfg = LobidraConfig(vocab_size=vocab, width=width, eps=1e-5, layers=tuple(layers), embed_scale=math.sqrt(width),
                        name=name, max_position=max_position)
    cfg.validate()
    return cfg


# Named configurations (random weights): a toy for smoke runs and sizes that resemble real models' layers for the
# benchmark -- "mid" has 2048-wide layers, "wide" the 4096-wide layers of a 7B-class model; six layers each.
PATTERN = ("conv_attention", "conv_attention", "twin", "conv_attention", "twin", "conv_attention")
TINY = _named("lobidra-tiny", vocab=512, width=128, pattern=("conv_attention", "conv_attention", "twin", "conv_attention"),
              heads=4, kv_heads=2, dim=32, vdim=48, mem_heads=2, mem_dim=32, mem_vdim=64, ff=192, experts=6, top=2,
              expert_ff=80, shared_ff=112, rot_dims=16, max_position=4096)
MID = _named("lobidra-mid", vocab=32768, width=2048, pattern=PATTERN, heads=16, kv_heads=8, dim=128, vdim=128, mem_heads=16,
             mem_dim=128, mem_vdim=128, ff=8192, experts=16, top=2, expert_ff=1408, shared_ff=2816, rot_dims=64)
WIDE = _named("lobidra-wide", vocab=32768, width=4096, pattern=PATTERN, heads=32, kv_heads=8, dim=128, vdim=128,
              mem_heads=32, mem_dim=128, mem_vdim=128, ff=14336, experts=16, top=2, expert_ff=3584, shared_ff=7168,
              rot_dims=64)

CONFIGS = {c.name: c for c in (TINY, MID, WIDE)}
