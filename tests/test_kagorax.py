"""Kagorax on the engine against the plain oracle (tests/kagorax_oracle.py).

Every test builds its own small configuration and random weights, drives the engine through its own entry points
(LLMEngine.force_step for given tokens, add_request + step for generation) and compares the logits with the oracle's
whole-sequence forward in float64.  The same tests run on the CPU (PyTorch reference ops: scheduler, cache and batch
plumbing) and, marked ``gpu``, on the HIP kernels in fp32 (every row, tight tolerance) and bf16 (the bulk of the rows: a
close router call flips under bf16 rounding in these tiny random models and moves single rows).  Where a test asserts
that something matters, the mistake is planted in the oracle.
"""
from __future__ import annotations

import copy
import json

import pytest
import torch

import kagorax_oracle as oracle
from distributed_sse_for_llm_response_amd import ops
from distributed_sse_for_llm_response_amd.engine.engine import LLMEngine, SamplingParams
from distributed_sse_for_llm_response_amd.engine.model_runner import PrefillSeq
from distributed_sse_for_llm_response_amd.engine.weights import convert_kagorax
from distributed_sse_for_llm_response_amd.models import registry
from distributed_sse_for_llm_response_amd.models.kagorax import (KagoraxConfig, bias_by_distance, distance_bucket,
                                                                 init_weights, position_table, tensor_shapes)

GPU = pytest.param("cuda", marks=pytest.mark.gpu)
DEVICES = ["cpu", GPU]
VOCAB = 53


def moe(experts=5, top=2, ff=9, shared=7):
    f = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def att(heads=4, kv_heads=2, dim=10, vdim=6, window=9, keep=3, scale=0.4, far=40, kv_from=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": far}
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mlp": mlp, "mixer": m}


def config(layers, width=26, vocab=VOCAB, eps=3e-6, scale=3.0):
    return {"architecture": "Kagorax", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": copy.deepcopy(layers)}


STACK = config([att(mlp=moe()), att(heads=3, kv_heads=3, dim=8, vdim=8, window=33, keep=5, far=90, mlp=moe(top=1)),
                att(heads=3, kv_heads=3, dim=8, vdim=8, window=12, keep=1, far=20, kv_from=1, mlp=moe(shared=0)),
                att(kv_from=0, heads=6, mlp=None), att(heads=3, kv_heads=3, dim=8, vdim=8, window=None, kv_from=1,
                                                       mlp=moe(experts=3, top=3))], width=40)


def settled(cfgd):
    """The same model with as many experts as each token uses: the weighted paths without a choice to flip."""
    d = copy.deepcopy(cfgd)
    for L in d["layers"]:
        if L.get("mlp"):
            L["mlp"]["router"]["experts"] = L["mlp"]["router"]["top"]
    return d


def stack_for(dtype):
    """The tests of cuts, batches and pools judge every row: in bf16 they run the stack with nothing to choose (a close
    router call that flips under bf16 rounding moves the row); the choice in bf16 is judged in the other tests."""
    return STACK if dtype == torch.float32 else settled(STACK)


class Model:
    """Configuration + random weights + an engine on `device` in `dtype`."""

    def __init__(self, cfg_dict, device, dtype=torch.float32, seed=0, max_tokens=256, max_seqs=4, tweak=None, rows=12):
        self.cfg_dict = cfg_dict
        self.cfg = KagoraxConfig.from_dict(cfg_dict)
        self.weights = init_weights(self.cfg, seed=seed, rows=rows)
        if tweak:
            tweak(self.weights)
        self.device, self.dtype = torch.device(device), dtype
        w = convert_kagorax(self.cfg, self.weights, device=self.device, dtype=dtype)
        fam = registry.family_of(self.cfg)
        assert fam.name == "kagorax"
        self.runner = registry.make_runner(fam, w, num_blocks=-(-max_tokens // 32), max_batch=max_seqs,
                                           max_model_len=max_tokens, max_prefill_tokens=max_tokens, device=self.device,
                                           use_graphs=False)
        self.engine = LLMEngine(self.runner, eos_id=-1)
        self.engine.watermark = 0

    def expect(self, tokens, cfg_dict=None, weights=None):
        return oracle.forward(cfg_dict or self.cfg_dict, weights or self.weights, tokens).float()

    def check(self, got, want, what=""):
        """Row-wise: rms of the difference (mean taken off) over the rms of the expected logits.  fp32 judges every
        row; bf16 every row but one in ten where there is nothing to choose, else seven rows in ten."""
        got, want = got.detach().float().cpu(), want.float()
        assert got.shape == want.shape, (got.shape, want.shape)
        assert torch.isfinite(got).all(), what
        d = got - want
        d = d - d.mean(-1, keepdim=True)
        err = d.pow(2).mean(-1).sqrt() / (want - want.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt().clamp_min(1e-6)
        if self.dtype == torch.float32:
            assert float(err.max()) < 2e-4, f"{what}: worst row {int(err.argmax())} error {float(err.max()):.3g}"
        else:
            routers = [L["mlp"]["router"] for L in self.cfg_dict["layers"] if L.get("mlp")]
            part = 0.7 if any(r["experts"] > r["top"] for r in routers) else 0.9
            assert float((err < 4e-2).float().mean()) >= part and float(err.median()) < 2e-2, \
                f"{what}: median {float(err.median()):.3g}, {int((err >= 4e-2).sum())} of {err.numel()} rows off"

    def run_cut(self, cid, tokens, cuts, end=True):
        """Feed `tokens` in portions of the given sizes (the last size repeats), all logits wanted."""
        out, at, k = [], 0, 0
        while at < len(tokens):
            n = min(cuts[min(k, len(cuts) - 1)], len(tokens) - at)
            last = at + n == len(tokens)
            out.append(self.engine.force_step([(cid, tokens[at:at + n], list(range(n)))], [cid] if last and end else []))
            at, k = at + n, k + 1
        return torch.cat(out)


def toks(n, vocab=VOCAB, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def modes(device):
    return [torch.float32] if device == "cpu" else [torch.float32, torch.bfloat16]


def gap(a, b, rows=slice(None)):
    """Median over rows of |a - b| rms relative to b's rms: how far a variant of the design is from the design."""
    a, b = a[rows], b[rows]
    return float(((a - b).pow(2).mean(-1).sqrt() / b.pow(2).mean(-1).sqrt().clamp_min(1e-6)).median())


def gap_max(a, b, rows=slice(None)):
    a, b = a[rows], b[rows]
    return float(((a - b).pow(2).mean(-1).sqrt() / b.pow(2).mean(-1).sqrt().clamp_min(1e-6)).max())


def changed(weights, fn):
    """A copy of the weights with fn(name, tensor) -> tensor or None (unchanged) applied."""
    out = {}
    for k, v in weights.items():
        r = fn(k, v)
        out[k] = v if r is None else r
    return out


def tweak_of(fn):
    def tweak(w):
        w.update(changed(w, fn))
    return tweak


# ---------------------------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name,cfgd", [
    ("grouped heads, window, kept keys", config([att()])),
    ("a key head per head, no mask", config([att(heads=3, kv_heads=3, dim=8, vdim=8, window=None)])),
    ("one key head, window of one, nothing kept", config([att(heads=3, kv_heads=1, window=1, keep=0)])),
    ("one kept key", config([att(window=4, keep=1)])),
    ("more keys kept than the sequence has", config([att(window=5, keep=100)])),
    ("one-wide values, one-wide queries", config([att(heads=2, kv_heads=1, dim=1, vdim=1)])),
    ("keys and values of an earlier layer", config([att(), att(kv_from=0)])),
    ("keys and values of an earlier layer, other mask, bias, scale and head count", config(
        [att(), att(heads=2, kv_heads=2, dim=4, vdim=4), att(heads=8, kv_heads=2, window=20, keep=0, scale=1.0, far=90, kv_from=0)])),
    ("routed experts with a shared one", config([att(heads=1, kv_heads=1, mlp=moe())])),
    ("one expert per token, no shared one", config([att(mlp=moe(top=1, shared=0))])),
    ("every expert", config([att(mlp=moe(experts=4, top=4))])),
    ("a single expert", config([att(mlp=moe(experts=1, top=1))])),
    ("shared expert wider than the routed ones", config([att(mlp=moe(ff=3, shared=31))])),
    ("embedding without a scale", {k: v for k, v in config([att(mlp=moe())]).items() if k != "embedding"}),
])
def test_mechanism_alone(device, name, cfgd):
    for dtype in modes(device):
        m = Model(cfgd, device, dtype)
        t = toks(47, seed=1)
        m.check(m.run_cut("a", t, [len(t)]), m.expect(t), name + ", whole")
        m.check(m.run_cut("b", t, [9, 1]), m.expect(t), name + ", decoding")


def test_each_op_against_its_oracle_function():
    """The reference ops the CPU engine runs on, one mechanism at a time, against the oracle's functions."""
    g = torch.Generator().manual_seed(5)
    # routing: sigmoid scores as they are, and the shared expert's gate as one more logit
    z = torch.randn(40, 9, generator=g) * 2
    idx, w = oracle.route(z[:, :8].double(), 3)
    ti, tw = torch.zeros(40, 3, dtype=torch.int32), torch.zeros(40, 4)
    ops.moe_route(z, None, ti, tw, 1, 1, 1.0, 2)
    assert torch.equal(ti.long(), idx) and torch.allclose(tw[:, :3], w.float(), atol=1e-6)
    assert torch.allclose(tw[:, 3], torch.sigmoid(z[:, 8]), atol=1e-6)
    # experts: the weight on the input, the shared expert's on the output
    x = torch.randn(40, 10, generator=g)
    shapes = {"gate": (6, 10), "up": (6, 10), "down": (10, 6)}
    ew = {f"e{e}.{k}": torch.randn(s, generator=g) for e in range(8) for k, s in shapes.items()}
    ew.update({f"shared.{k}": torch.randn(s, generator=g) for k, s in shapes.items()})
    stack = {k: torch.stack([ew[f"e{e}.{k}"] for e in range(8)]) for k in shapes}
    o = torch.zeros(160, 10)
    none = torch.zeros(1)
    ops.moe_grouped(x, ti, tw, stack["gate"], stack["up"], stack["down"], ew["shared.gate"], ew["shared.up"],
                    ew["shared.down"], none, none, none, none, o, True)
    d = {k: v.double() for k, v in ew.items()}
    for t in range(40):
        want = sum(oracle.expert(tw[t, k].double() * x[t:t + 1].double(), *(d[f"e{int(ti[t, k])}.{n}"] for n in shapes))
                   for k in range(3))
        want = want + tw[t, 3].double() * oracle.expert(x[t:t + 1].double(), *(d[f"shared.{n}"] for n in shapes))
        assert torch.allclose(o.view(40, 4, 10)[t].sum(0), want[0].float(), atol=1e-4, rtol=1e-4)
    # the embedding's rows
    cfgd = config([att()])
    e = torch.randn(VOCAB, 27, generator=g)
    t = toks(9, seed=3)
    want = oracle.embedding(cfgd, {"embed": e.double()}, torch.tensor(t))
    resid = torch.zeros(9, 27)
    ids, table = torch.tensor(t, dtype=torch.int32), position_table(12, 27)
    ops.embed_rows(ids, e, resid, None, 3.0, torch.arange(9, dtype=torch.int32), table)
    assert torch.allclose(resid, want.float(), atol=1e-5)
    ops.embed_rows(ids[4:], e, resid[:5], None, 3.0, torch.arange(4, 9, dtype=torch.int32), table)
    assert torch.allclose(resid[:5], want[4:].float(), atol=1e-5), "the position decides, not the row's place in the step"
    # both sublayers into the stream, then the norm
    y, y2, res = (torch.randn(s, generator=g) for s in ((10, 8), (5, 8), (5, 8)))
    go = torch.randn(8, generator=g)
    want_res = res.double() + y.double().view(5, 2, 8).sum(1) + y2.double()
    out, out32 = torch.zeros(5, 8, dtype=torch.bfloat16), torch.zeros(5, 8)
    ops.add_norm_rows(y, 2, None, res, go, 1e-5, out, out32, y2)
    assert torch.allclose(res, want_res.float(), atol=1e-5)
    assert torch.allclose(out32, (oracle.rms(want_res, 1e-5) * go.double()).float(), atol=1e-5)
    assert torch.equal(out, out32.to(torch.bfloat16))
    # the attention's operands: bias first, then the per-head norm of q and k; v as it is
    m = att()["mixer"]
    H, G, D, V = 4, 2, 10, 6
    x, b = torch.randn(7, H * D + G * (D + V) + 5, generator=g), torch.randn(H * D + G * (D + V), generator=g)
    eye = {"k": torch.eye(G * D), "k.b": b[H * D:(H + G) * D], "v": torch.eye(G * V), "v.b": b[(H + G) * D:]}
    k, _ = oracle.keys_values(x[:, H * D:(H + G) * D].double(), m, {**{n: v.double() for n, v in eye.items()},
                              "v": torch.zeros(G * V, G * D, dtype=torch.float64)}, 1e-5)
    v = (x[:, (H + G) * D:(H + G) * D + G * V] + b[(H + G) * D:]).view(7, G, V)
    q = torch.zeros(7, H, D)
    kc, vc, vt = torch.zeros(2, 32, G, D), torch.zeros(2, 32, G, V), torch.zeros(2, G, V, 32)
    rows = torch.tensor([3, 40, -1, 63, 0, 1, 2], dtype=torch.int32)
    ops.qkv_rows(x, b, H, G, D, V, 1e-5, rows, q, kc, vc, vt)
    assert torch.allclose(q, oracle.rms((x[:, :H * D] + b[:H * D]).double().view(7, H, D), 1e-5).float(), atol=1e-5)
    for t, r in enumerate(rows.tolist()):
        if r >= 0:
            assert torch.allclose(kc.view(64, G, D)[r], k[t].float(), atol=1e-5) and torch.equal(vc.view(64, G, V)[r], v[t])
    assert int((kc.view(64, -1).abs().sum(-1) > 0).sum()) == 6
    q2 = torch.zeros(7, H, D)
    ops.qkv_rows(x[:, :H * D + 3], b[:H * D], H, G, D, V, 1e-5, rows, q2)   # a layer without keys of its own
    assert torch.equal(q, q2)


def test_distance_buckets():
    """Every distance's row against the oracle's function, edges that are exact powers, and the table laid out per
    distance (its last entry serves everything farther)."""
    for rows, far in ((2, 5), (8, 64), (16, 72), (12, 40), (32, 128), (16, 2048), (32, 4096), (7, 50), (10, 7.5)):
        got = [distance_bucket(n, rows, far) for n in range(5000)]
        assert got == [oracle.bucket(n, rows, far) for n in range(5000)]
        assert got[:rows // 2] == list(range(rows // 2)) and got[-1] == rows - 1 and sorted(got) == got
        rel = torch.randn(rows, 3)
        table = bias_by_distance(rel, far)
        for n in (0, 1, rows // 2, int(far) - 1, int(far), int(far) + 1, 4999):
            assert torch.equal(table[:, min(n, table.shape[1] - 1)], rel[got[n]]), (rows, far, n)
        assert table.shape[1] <= max(far, rows) + 1
    # 4 rows of one distance each, then [4, 8), [8, 16), [16, 32), [32, ..): the edges belong to the row that starts there
    assert [distance_bucket(n, 8, 64) for n in (3, 4, 7, 8, 15, 16, 31, 32, 63, 64, 1000)] == [3, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7]
    # thirds of a cube: 27 = 3^3 over three rows from 5 on
    assert [distance_bucket(n, 6, 81) for n in (3, 8, 9, 26, 27, 80, 81)] == [3, 3, 4, 4, 5, 5, 5]
    assert torch.allclose(position_table(40, 9), torch.stack([oracle.position_vector(p, 9) for p in range(40)]).float(), atol=1e-6)


@pytest.mark.parametrize("device", DEVICES)
def test_layer_trace(device):
    """The engine's layer trace (the stream after every layer) against the oracle's."""
    for dtype in modes(device):
        m = Model(stack_for(dtype), device, dtype)
        t = toks(21, seed=2)
        got, want = [], []
        m.runner.prefill([PrefillSeq(slot=0, tokens=t, start_pos=0, block_table=[0], last_chunk=False)], 0, trace=got)
        oracle.forward(m.cfg_dict, m.weights, t, want)
        assert len(got) == len(want) == 5
        for i, (a, b) in enumerate(zip(got, want)):
            err = (a.cpu().double() - b).abs().amax(-1) / b.abs().max()
            assert float(err.max()) < (1e-4 if dtype == torch.float32 else 3e-2), f"layer {i}"


# ---------------------------------------------------------------------------------------------- cuts, batches, pools
@pytest.mark.parametrize("device", DEVICES)
def test_prefill_against_token_by_token(device):
    t = toks(45, seed=3)
    for dtype in modes(device):
        m = Model(stack_for(dtype), device, dtype)
        want = m.expect(t)
        whole = m.run_cut("w", t, [len(t)])
        single = m.run_cut("s", t, [1])
        m.check(whole, want, "whole prompt")
        m.check(single, want, "token by token")
        if dtype == torch.float32:
            m.check(single, whole.cpu(), "token by token against the whole prompt")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[2], [3, 2, 7], [5, 1, 1, 2, 11], [31, 2, 1], [33, 1], [64, 2]])
def test_portions(device, cuts):
    """Portions cut inside pages and windows, down to two tokens."""
    t = toks(70, seed=4)
    for dtype in modes(device):
        m = Model(stack_for(dtype), device, dtype)
        m.check(m.run_cut("p", t, cuts), m.expect(t), f"portions {cuts}")


@pytest.mark.parametrize("device", DEVICES)
def test_unequal_batch_against_each_alone(device):
    """Four requests of unequal length in one batch: portions of some beside single tokens of others, one sits out
    steps, one ends early and its slot and pages go to a newcomer."""
    seqs = {"a": toks(50, seed=5), "b": toks(9, seed=6), "c": toks(34, seed=7), "d": toks(1, seed=8), "e": toks(40, seed=9)}
    plan = [{"a": 7, "b": 2, "c": 20}, {"a": 1, "b": 1, "d": 1}, {"a": 1, "c": 2, "b": 1}, {"a": 30, "b": 1, "e": 3},
            {"a": 1, "b": 1, "c": 1, "e": 33}, {"a": 1, "b": 1, "c": 11, "e": 1}, {"a": 9, "b": 2, "e": 3}]
    for dtype in modes(device):
        m = Model(stack_for(dtype), device, dtype, max_tokens=256)
        at = {k: 0 for k in seqs}
        got = {k: [] for k in seqs}
        for step in plan:
            entries, end = [], []
            for k, n in step.items():
                n = min(n, len(seqs[k]) - at[k])
                entries.append((k, seqs[k][at[k]:at[k] + n], list(range(n))))
                at[k] += n
                if at[k] == len(seqs[k]):
                    end.append(k)
            out = m.engine.force_step(entries, end)
            o = 0
            for k, tk, _ in entries:
                got[k].append(out[o:o + len(tk)])
                o += len(tk)
        for k, t in seqs.items():
            assert at[k] == len(t), k
            m.check(torch.cat(got[k]), m.expect(t), f"request {k} in the batch")
        assert m.engine.alloc.num_free == m.engine.alloc.num_blocks


@pytest.mark.parametrize("device", DEVICES)
def test_pages_and_slots_used_again(device):
    """A pool of three pages and two slots: every later request runs in pages and slots that held another one, in
    prompts and in decoding."""
    for dtype in modes(device):
        m = Model(stack_for(dtype), device, dtype, max_tokens=96, max_seqs=2)
        for i, (n, cuts) in enumerate([(60, [60]), (64, [33, 1]), (40, [2, 30, 1]), (64, [64]), (5, [1])]):
            t = toks(n, seed=30 + i)
            keep = toks(20, seed=40 + i)
            first = m.engine.force_step([(f"k{i}", keep[:10], list(range(10)))])
            got = m.run_cut(f"r{i}", t, cuts)
            rest = m.engine.force_step([(f"k{i}", keep[10:], list(range(10)))], [f"k{i}"])
            m.check(got, m.expect(t), f"request {i}")
            m.check(torch.cat([first, rest]), m.expect(keep), f"neighbour of request {i}")
        assert m.engine.alloc.num_free == m.engine.alloc.num_blocks
    m.engine.force_step([("held", toks(64, seed=1), [])])
    with pytest.raises(MemoryError):
        m.engine.force_step([("late", toks(64, seed=2), [])])


# ---------------------------------------------------------------------------------------------- far keys and edges
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dim,vdim", [(8, 6), (32, 16)])
def test_far_key_among_hundreds(device, dim, vdim):
    """Attention without a mask, every query pointing (through its bias) at the key of one token that occurs once, as the
    sequence's second: one far key carries the weight.  Another token in its place moves the logits 250 tokens later in
    the oracle, and the engine agrees with it in prompts cut at page borders and in decoding."""
    cfgd = config([att(heads=2, kv_heads=1, dim=dim, vdim=vdim, window=None, scale=1.0 * (8 / dim) ** 0.5, far=64)], width=40)

    def planted(w):
        w.update(changed(w, farsighted))
        u = torch.ones(dim)
        w["l0.mix.q.b"] = (4.0 * u).repeat(2).to(torch.bfloat16)
        e = torch.linalg.pinv(w["l0.mix.k"].float()) @ u
        w["embed"][VOCAB - 1] = (e / e.norm() * 30 / w["l0.norm1"].float()).to(torch.bfloat16)

    t = toks(300, vocab=VOCAB - 1, seed=10)
    t[1] = VOCAB - 1
    for dtype in modes(device):
        m = Model(cfgd, device, dtype, max_tokens=320, tweak=planted)
        want = m.expect(t)
        moved = list(t)
        moved[1] = 7
        assert gap(m.expect(moved), want, slice(250, None)) > 5e-2, "the far key does not matter in this construction"
        m.check(m.run_cut("a", t, [256, 1]), want, "prompt to a page border, then decoding")
        m.check(m.run_cut("b", t, [32, 64, 33, 2, 97, 1]), want, "portions on and off page borders")


def farsighted(k, v):
    """Distance biases that grow with the distance, and heads that count three times as much in the stream."""
    if k.endswith("rel"):
        return torch.linspace(0.0, 3.0, v.shape[0])[:, None].expand_as(v).to(v.dtype).contiguous()
    return (v.float() * 3).to(v.dtype) if k.endswith("mix.o") else None


WIDTHS = [(8, 6), (32, 16)]  # head widths of the row form and of the MFMA form


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dim,vdim", WIDTHS)
@pytest.mark.parametrize("window,keep", [(1, 0), (2, 1), (31, 2), (32, 0), (33, 5), (40, 32), (17, 33), (70, 4)])
def test_window_and_kept_key_edges(device, dim, vdim, window, keep):
    """Sharp windowed attention: the key just inside the window counts and the one just outside does not; the last kept
    key stays visible from afar and the next one does not, in prompts and in decoding.  The oracle with a window or a
    number of kept keys that is one off is far from the design in some row."""
    def cfg_w(w, k):
        return config([att(heads=2, kv_heads=1, dim=dim, vdim=vdim, window=w, keep=k, scale=1.6 * (8 / dim) ** 0.5, far=24)])

    t = toks(110, seed=11)
    for dtype in modes(device):
        m = Model(cfg_w(window, keep), device, dtype, tweak=tweak_of(farsighted))
        want = m.expect(t)
        for w, k in ((window + 1, keep), (window - 1, keep), (window, keep + 1), (window, keep - 1)):
            if w >= 1 and k >= 0:
                assert gap_max(m.expect(t, cfg_w(w, k)), want, slice(window + 1, None)) > 1e-2, (w, k)
        m.check(m.run_cut("p", t, [len(t)]), want, "prompt")
        m.check(m.run_cut("d", t, [max(1, window - 1), 1]), want, "decoding over the edge")
        m.check(m.run_cut("c", t, [window + 1, 2, 31, 1]), want, "portions over the edge")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dim,vdim", WIDTHS)
def test_kept_keys_carry_the_weight(device, dim, vdim):
    """The bias of the farthest distances made large: far behind the window's reach the kept keys hold nearly all of the
    weight, with their true distances.  The oracle that forgets them, or that lets their distances start anew at the
    window's edge, is far away."""
    def cfg_k(keep):
        return config([att(heads=2, kv_heads=2, dim=dim, vdim=vdim, window=20, keep=keep, far=60, scale=0.3),
                       att(heads=2, kv_heads=2, dim=dim, vdim=vdim, window=20, keep=keep, far=60, scale=0.3, kv_from=0)])

    def heavy(k, v):
        if k.endswith("rel"):
            v = v.clone()
            v[-1] = 6.0
            return v

    t = toks(150, seed=12)
    for dtype in modes(device):
        m = Model(cfg_k(4), device, dtype, tweak=tweak_of(heavy))
        want = m.expect(t)
        assert gap(m.expect(t, cfg_k(0)), want, slice(70, None)) > 5e-2
        light = changed(m.weights, lambda k, v: torch.cat([v[:-1], v[-2:-1]]) if k.endswith("rel") else None)
        assert gap(m.expect(t, weights=light), want, slice(70, None)) > 5e-2
        m.check(m.run_cut("w", t, [len(t)]), want, "prompt")
        m.check(m.run_cut("d", t, [96, 1]), want, "decoding from a page's edge")
        m.check(m.run_cut("c", t, [3, 2, 64, 2, 1]), want, "portions, the first ones inside the kept keys")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dim,vdim", WIDTHS)
def test_every_distance_has_its_bias(device, dim, vdim):
    """Flat scores under steep distance biases: the weights are the biases' alone.  The oracle with two neighbouring rows
    exchanged anywhere, with the table of another layer, with another reach, or with the score's scale on the bias is
    far away."""
    L = [att(heads=2, kv_heads=1, dim=dim, vdim=vdim, window=None, far=70, scale=0.01),
         att(heads=2, kv_heads=1, dim=dim, vdim=vdim, window=None, far=70, scale=0.01)]
    cfgd = config(L)

    def steep(k, v):
        return (v.float() * 2.5).to(v.dtype) if k.endswith("rel") else None

    t = toks(130, seed=13)
    for dtype in modes(device):
        m = Model(cfgd, device, dtype, tweak=tweak_of(steep), rows=12)
        want = m.expect(t)
        for r in range(11):
            order = list(range(12))
            order[r], order[r + 1] = r + 1, r
            assert gap_max(m.expect(t, weights=changed(m.weights, lambda k, v: v[order] if k.endswith("rel") else None)), want) > 1e-2, r
        swapped = dict(m.weights)
        swapped["l0.mix.rel"], swapped["l1.mix.rel"] = m.weights["l1.mix.rel"], m.weights["l0.mix.rel"]
        assert gap(m.expect(t, weights=swapped), want) > 1e-2
        assert gap(m.expect(t, weights=changed(m.weights, lambda k, v: v * 0.01 if k.endswith("rel") else None)), want) > 1e-2
        other = copy.deepcopy(cfgd)
        other["layers"][0]["mixer"]["bias_max"] = other["layers"][1]["mixer"]["bias_max"] = 100
        assert gap_max(m.expect(t, other), want) > 1e-2
        m.check(m.run_cut("w", t, [len(t)]), want, "prompt")
        m.check(m.run_cut("d", t, [30, 1]), want, "decoding over every row of the table")
        m.check(m.run_cut("c", t, [2, 33, 31, 2]), want, "portions")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("rows,far", [(2, 3), (24, 2000), (8, 9)])
def test_bias_tables_short_and_long(device, rows, far):
    """A table of two rows, one that reaches beyond every key (more distances than the attention kernel stages), and one
    whose logarithmic part is squeezed into a distance; on the MFMA form's widths, without a window."""
    cfgd = config([att(heads=4, kv_heads=2, dim=32, vdim=32, window=None, far=far, scale=0.02)], width=32)
    t = toks(600 if far == 2000 and device != "cpu" else 100, seed=14)
    for dtype in modes(device):
        m = Model(cfgd, device, dtype, rows=rows, max_tokens=640,
                  tweak=tweak_of(lambda k, v: (v.float() * 2).to(v.dtype) if k.endswith("rel") else None))
        m.check(m.run_cut("w", t, [len(t) - 20, 1]), m.expect(t), f"{rows} rows to {far}")


# ---------------------------------------------------------------------------------------------- shared keys and values
@pytest.mark.parametrize("device", DEVICES)
def test_layers_share_keys_and_values(device):
    """Three layers over the pages of two others: the oracle that takes another layer's keys and values is far away; the
    engine keeps pages for the owners alone."""
    kw = dict(heads=2, kv_heads=1, dim=8, vdim=8)
    cfgd = config([att(**kw), att(**kw), att(kv_from=0, **kw), att(kv_from=1, **kw), att(kv_from=0, window=30, **kw)])
    t = toks(60, seed=15)
    for dtype in modes(device):
        m = Model(cfgd, device, dtype)
        want = m.expect(t)
        assert sorted(m.runner.kv.k) == sorted(m.runner.kv.v) == [0, 1]
        other = copy.deepcopy(cfgd)
        other["layers"][2]["mixer"]["kv_from"] = 1
        assert gap(m.expect(t, other), want) > 1e-2
        m.check(m.run_cut("k", t, [25, 2, 1]), want, "shared pages")
    assert not [n for n in tensor_shapes(m.cfg) if n.startswith(("l2.mix.k", "l2.mix.v", "l4.mix.k"))]
    assert m.cfg.cache_bytes_per_token(2) == 2 * (8 + 8) * 2


# ---------------------------------------------------------------------------------------------- feed-forward, positions
@pytest.mark.parametrize("device", DEVICES)
def test_weights_enter_the_experts(device, monkeypatch):
    """Scores well away from 0 and 1 on experts that are far from linear: the oracle with the weight on the output, with
    renormalised weights, or with an ungated shared expert is far away."""
    cfgd = config([att(mlp=moe(top=2))], scale=1.0)
    big = tweak_of(lambda k, v: (v.float() * 2).to(v.dtype) if k.endswith((".gate", ".up", ".down")) else None)
    t = toks(40, seed=16)
    plain = oracle.feed_forward

    def variant(mode):
        def ff(h, f, w):
            idx, wt = oracle.route(h @ w["router"].T, int(f["router"]["top"]))
            if mode == "renormalised":
                wt = wt / wt.sum(-1, keepdim=True)
            out = torch.zeros(h.shape[0], w["e0.down"].shape[0], dtype=h.dtype)
            for r in range(h.shape[0]):
                for e, c in zip(idx[r].tolist(), wt[r]):
                    mats = (w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])
                    out[r] += (c * oracle.expert(h[r:r + 1], *mats) if mode == "output" else oracle.expert(c * h[r:r + 1], *mats))[0]
            g = 1.0 if mode == "ungated" else torch.sigmoid(h @ w["shared.sg"].T)
            return out + g * oracle.expert(h, w["shared.gate"], w["shared.up"], w["shared.down"])
        return ff

    for dtype in modes(device):
        m = Model(cfgd, device, dtype, tweak=big)
        want = m.expect(t)
        for mode in ("output", "renormalised", "ungated"):
            monkeypatch.setattr(oracle, "feed_forward", variant(mode))
            assert gap(m.expect(t), want) > 2e-2, mode
        monkeypatch.setattr(oracle, "feed_forward", plain)
        m.check(m.run_cut("f", t, [17, 2, 1]), want, "weights on the inputs")


@pytest.mark.parametrize("device", DEVICES)
def test_both_sublayers_read_the_same_norm(device, monkeypatch):
    """The oracle in which the feed-forward sees what the mixer added is far away."""
    cfgd = config([att(mlp=moe()), att(mlp=moe())], scale=1.0)
    t = toks(30, seed=17)

    def in_turn(x, i, cfg, w, kvs):
        L, eps = cfg["layers"][i], float(cfg["norm"]["eps"])
        lw = oracle.sub(w, f"l{i}.")
        h = oracle.rms(x, eps) * lw["norm1"]
        kvs[i] = oracle.keys_values(h, L["mixer"], oracle.sub(lw, "mix."), eps)
        x = x + oracle.attention(h, L["mixer"], oracle.sub(lw, "mix."), eps, kvs[i])
        return x + oracle.feed_forward(oracle.rms(x, eps) * lw["norm1"], L["mlp"], oracle.sub(lw, "mlp."))

    for dtype in modes(device):
        m = Model(cfgd, device, dtype)
        want = m.expect(t)
        with monkeypatch.context() as mp:
            mp.setattr(oracle, "layer", in_turn)
            assert gap(m.expect(t), want) > 5e-2
        m.check(m.run_cut("n", t, [len(t)]), want, "side by side")


@pytest.mark.parametrize("device", DEVICES)
def test_positions_reach_every_row(device, monkeypatch):
    """A small embedding scale makes the position vectors count: the oracle whose positions start at one is far away; a
    portion in the middle of a sequence, a decoded token and a reused slot all take their own position."""
    cfgd = config([att(mlp=moe())], scale=0.3, width=25)
    t = toks(60, seed=18)
    for dtype in modes(device):
        m = Model(cfgd, device, dtype, max_seqs=2)
        want = m.expect(t)
        plain = oracle.position_vector
        with monkeypatch.context() as mp:
            mp.setattr(oracle, "position_vector", lambda p, width: plain(p + 1, width))
            assert gap(m.expect(t), want) > 5e-2
        m.run_cut("warm", toks(40, seed=19), [40])
        m.check(m.run_cut("p", t, [13, 1, 2, 30, 1]), want, "positions")


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens(device):
    """Positions 0, 1, 2 as a one-token request, as single tokens from the start, and in a slot that held another
    sequence."""
    for dtype in modes(device):
        m = Model(stack_for(dtype), device, dtype, max_seqs=1)
        m.run_cut("warm", toks(40, seed=15), [40])
        for n in (1, 2, 3):
            t = toks(n, seed=16 + n)
            m.check(m.run_cut(f"n{n}", t, [1]), m.expect(t), f"{n} first tokens, one by one")
            m.check(m.run_cut(f"w{n}", t, [n]), m.expect(t), f"{n} first tokens, at once")


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(device):
    """Decoding runs over several pages and past the windows."""
    t = toks(150, seed=20)
    for dtype in modes(device):
        m = Model(stack_for(dtype), device, dtype)
        m.check(m.run_cut("l", t, [5, 1]), m.expect(t), "long decoding")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name,cfgd,rows", [
    ("all ones", config([att(heads=1, kv_heads=1, dim=1, vdim=1, window=1, keep=1, far=2, mlp=moe(experts=1, top=1, ff=1, shared=1))],
                        width=2, vocab=7, scale=1.0), 2),
    ("odd sizes", config([att(heads=6, kv_heads=3, dim=14, vdim=11, window=13, keep=7, mlp=moe(experts=9, top=4, ff=7, shared=5)),
                          att(heads=9, kv_heads=3, dim=14, vdim=11, window=21, keep=2, kv_from=0)], width=19, vocab=23), 10),
    ("sizes that vector loads and the MFMA attention like", config(
        [att(heads=8, kv_heads=2, dim=64, vdim=32, window=48, keep=5, scale=0.2, mlp=moe(experts=8, top=2, ff=64, shared=32)),
         att(heads=2, kv_heads=1, dim=32, vdim=64, window=None, mlp=moe(experts=4, top=1, ff=32, shared=0)),
         att(heads=6, kv_heads=2, dim=64, vdim=32, window=20, keep=40, scale=0.2, kv_from=0)], width=64, vocab=96), 32),
    ("wide heads on the row form", config([att(heads=2, kv_heads=1, dim=136, vdim=72, window=20, scale=0.1)], width=48, vocab=50), 12),
    ("wide heads on the MFMA form", config([att(heads=5, kv_heads=5, dim=256, vdim=160, window=40, scale=0.1),
                                            att(heads=4, kv_heads=1, dim=512, vdim=128, window=40, scale=0.1)], width=48, vocab=50), 12),
    ("projections on the tiled-layout GEMMs", config(
        [att(heads=8, kv_heads=4, dim=128, vdim=128, window=40, scale=0.1, mlp=moe(experts=4, top=2, ff=256, shared=512)),
         att(heads=8, kv_heads=4, dim=128, vdim=128, window=30, keep=0, scale=0.1, kv_from=0,
             mlp=moe(experts=4, top=1, ff=256, shared=128))], width=1024, vocab=1024), 16),
])
def test_other_sizes(device, name, cfgd, rows):
    vocab = cfgd["vocab"]
    t = toks(61, vocab=vocab, seed=21)
    for dtype in modes(device):
        m = Model(cfgd, device, dtype, rows=rows)
        m.check(m.run_cut("x", t, [len(t)]), m.expect(t), name + ", whole")
        m.check(m.run_cut("y", t, [7, 2, 1]), m.expect(t), name + ", portions and decoding")


@pytest.mark.gpu
def test_long_prompt_of_many_tiles():
    """Six hundred tokens on the GPU: prompt-sized expert tiles, attention tiles over many pages, a window and kept keys
    far apart."""
    cfgd = config([att(heads=4, kv_heads=2, dim=32, vdim=32, window=100, keep=40, far=300, mlp=moe(experts=8, top=2, ff=64, shared=128)),
                   att(heads=4, kv_heads=2, dim=32, vdim=32, window=64, keep=3, far=50, kv_from=0, mlp=moe(experts=3, top=1, ff=64, shared=0))],
                  width=64, vocab=200)
    t = toks(600, vocab=200, seed=22)
    for dtype in (torch.float32, torch.bfloat16):
        m = Model(cfgd, "cuda", dtype, max_tokens=640)
        want = m.expect(t)
        m.check(m.run_cut("a", t, [560, 1]), want, "prompt, then decoding")
        m.check(m.run_cut("b", t, [300, 3, 257, 1]), want, "portions")


# ---------------------------------------------------------------------------------------------- generation
@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_scheduler(device):
    """add_request + step: admission, chunked prompt passes (a 16-token budget), mixed steps, decode with sampling at
    temperature 0, slot release.  Each generated token is the oracle's argmax given the tokens before it (a step whose two
    best logits are closer than the tolerance is not judged)."""
    m = Model(STACK, device, torch.float32, max_tokens=512, max_seqs=3)
    eng = LLMEngine(m.runner, eos_id=-1, prefill_budget=16, idle_prefill_budget=16)
    prompts = {"g0": toks(19, seed=23), "g1": toks(40, seed=24), "g2": toks(3, seed=25), "g3": toks(33, seed=26)}
    for cid, p in prompts.items():
        eng.add_request(cid, p, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
    out = {cid: [] for cid in prompts}
    for ev in eng.run_until_idle():
        if not ev.done:
            out[ev.conversation_id].append(ev.token_id)
    for cid, p in prompts.items():
        assert len(out[cid]) == 12, (cid, out[cid])
        logits = m.expect(p + out[cid])
        for i, tok in enumerate(out[cid]):
            row = logits[len(p) + i - 1]
            top = torch.topk(row, 2).values
            if float(top[0] - top[1]) > 1e-3 * float(row.abs().max()):
                assert tok == int(row.argmax()), f"{cid}: token {i} is {tok}, the oracle says {int(row.argmax())}"
    assert eng.alloc.num_free == eng.alloc.num_blocks


@pytest.mark.gpu
@pytest.mark.parametrize("cfgd", [settled(STACK), config([att(heads=4, kv_heads=2, dim=32, vdim=32, window=20, mlp=moe(experts=2, top=2)),
                                                          att(heads=4, kv_heads=2, dim=32, vdim=32, kv_from=0, mlp=moe(experts=1, top=1))])])
def test_decode_graphs_match_eager(cfgd):
    """The captured decode step replayed over several steps (with eager work between the replays) gives the eager
    step's logits."""
    m = Model(cfgd, "cuda", torch.bfloat16)
    t = toks(60, seed=27)
    eager = m.run_cut("e", t, [20, 1])
    m.runner.use_graphs = True
    m.runner.capture()
    assert m.runner.graphs
    graphed = m.run_cut("g", t, [20, 1])
    assert torch.allclose(eager, graphed, atol=1e-5, rtol=1e-5)
    m.check(graphed, m.expect(t), "graph replays")


def test_config_round_trip_and_registry(tmp_path):
    cfg = KagoraxConfig.from_dict(STACK)
    again = KagoraxConfig.from_dict(cfg.to_dict())
    assert again.layers == cfg.layers and again == cfg
    assert [cfg.kv_layer(i) for i in range(5)] == [0, 1, 1, 0, 1]
    bare = KagoraxConfig.from_dict(config([att(window=None)]))
    assert KagoraxConfig.from_dict(bare.to_dict()) == bare and set(tensor_shapes(bare)) == {
        "embed", "final.norm", "l0.norm1", "l0.mix.q", "l0.mix.q.b", "l0.mix.k", "l0.mix.k.b", "l0.mix.v", "l0.mix.v.b",
        "l0.mix.rel", "l0.mix.g", "l0.mix.o"}
    from safetensors.torch import save_file

    (tmp_path / "config.json").write_text(json.dumps(STACK))
    weights = init_weights(cfg, seed=3, rows=14)
    save_file({k: v.contiguous() for k, v in weights.items()}, str(tmp_path / "model.safetensors"))
    fam, cfg2, path = registry.resolve(str(tmp_path))
    assert fam.name == "kagorax" and cfg2.layers == cfg.layers and cfg2.width == cfg.width and path == str(tmp_path)
    w = registry.load_weights(fam, cfg2, path, device="cpu", dtype=torch.float32)
    assert w.layers[0].mlp.gate.shape == (5, 9, 40) and w.layers[0].mlp.router.shape == (6, 40)
    assert w.layers[2].mlp.sgate is None and w.layers[3].mlp is None and w.layers[2].mix.bias.shape == (24,)
    assert w.head is w.embed and w.layers[0].mix.big.shape == (4 * 10 + 2 * 16 + 4 * 6, 40)
    assert torch.equal(w.layers[0].mix.rel[:, -1], weights["l0.mix.rel"][-1].float())
    assert set(tensor_shapes(cfg)) == set(weights)
    assert registry.resolve("kagorax-tiny")[0].name == "kagorax"
    assert cfg.cache_bytes_per_token() == (2 * 16 + 3 * 16) * 2
    assert registry.cache_blocks_for_budget(cfg, cfg.cache_bytes_per_token() * 32 * 7) == 7
    bad = dict(weights)
    bad["l0.mix.q"] = bad["l0.mix.q"][:-1]
    with pytest.raises(ValueError):
        convert_kagorax(cfg, bad)
    for layers in ([att(kv_from=0)], [att(), att(kv_from=0), att(kv_from=1)], [att(), att(dim=12, kv_from=0)],
                   [att(mlp=moe(experts=2, top=3))], [att(heads=3)]):
        with pytest.raises(ValueError):
            KagoraxConfig.from_dict(config(layers))
    with pytest.raises(ValueError):
        cfg.validate(tp=2)


def test_serving_builds_the_family_by_name():
    """The serving launcher's engine builder resolves the family through the registry and generates with it."""
    from distributed_sse_for_llm_response_amd.serving.app import build_engine
    from distributed_sse_for_llm_response_amd.serving.config import ServeConfig

    eng, _ = build_engine(ServeConfig(model="kagorax-tiny", engine="cpu"))
    eng.add_request("c1", [5, 6, 7, 8, 9, 10], SamplingParams(temperature=0.0, max_tokens=4, ignore_eos=True))
    eng.add_request("c2", [11, 12], SamplingParams(temperature=0.8, max_tokens=3, ignore_eos=True))
    ev = eng.run_until_idle()
    assert sum(1 for e in ev if e.conversation_id == "c1" and not e.done) == 4
    assert sum(1 for e in ev if e.conversation_id == "c2" and not e.done) == 3
