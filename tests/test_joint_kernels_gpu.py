"""HIP kernels of the side-by-side designs against their plain PyTorch references (ops/layers_reference.py), op by op: the
embedding with a scale and position vectors, two sublayers added as they are, the attention's operands in one launch,
distance biases, kept first keys and element-wise gates in the attention kernels (row form, MFMA form, key split),
sigmoid routing with a shared expert's gate, and weights on the experts' inputs."""
import math

import pytest
import torch

from distributed_sse_for_llm_response_amd import ops
from distributed_sse_for_llm_response_amd.models.surodra import HalfRotarySpec
from distributed_sse_for_llm_response_amd.ops import layers_reference as lref

pytestmark = pytest.mark.gpu

PAGE = 32
DTYPES = [torch.float32, torch.bfloat16]


def dev():
    return torch.device("cuda")


def i32(x):
    return torch.tensor(x, dtype=torch.int32)


def c(t):
    return None if t is None else t.to(dev())


def close(a, b, tol):
    a, b = a.float().cpu(), b.float().cpu()
    err = (a - b).abs().max().item()
    ref = b.abs().max().item() + 1e-6
    assert err <= tol * ref, f"max abs err {err} vs scale {ref}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [1, 333, 1024])
def test_embed_rows_with_scale_and_positions(dtype, W):
    g = torch.Generator().manual_seed(0)
    embed, table = torch.randn(50, W, generator=g).to(dtype), torch.randn(20, W, generator=g)
    ids, pos = i32([3, 49, 0, 7, 100, 12]), i32([0, 19, 5, 40, 7, -3])   # an id and two positions out of range
    for with_table, with_xb in ((1, 1), (1, 0), (0, 1)):
        r_ref, x_ref = torch.zeros(6, W), torch.zeros(6, W, dtype=dtype)
        lref.embed_rows(ids, embed, r_ref, x_ref if with_xb else None, 2.5, pos, table if with_table else None)
        r, x = torch.zeros(6, W, device=dev()), torch.zeros(6, W, dtype=dtype, device=dev())
        ops.embed_rows(c(ids), c(embed), r, x if with_xb else None, 2.5, c(pos), c(table) if with_table else None)
        close(r, r_ref, 1e-6)
        close(x, x_ref, 1e-6 if dtype == torch.float32 else 1e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,nsum", [(1, 1), (19, 3), (256, 2), (2052, 1), (4096, 3), (9000, 1)])
def test_add_norm_rows_as_they_are(dtype, W, nsum):
    g = torch.Generator().manual_seed(1)
    y, y2, resid = (torch.randn(n, W, generator=g) for n in (5 * nsum, 5, 5))
    go = torch.randn(W, generator=g)
    for second, norm, out32 in ((1, 1, 1), (0, 1, 0), (1, 0, 1), (1, 0, 0)):
        r_ref, o_ref, f_ref = resid.clone(), torch.zeros(5, W, dtype=dtype), torch.zeros(5, W)
        args = dict(y2=y2 if second else None)
        lref.add_norm_rows(y, nsum, None, r_ref, go if norm else None, 1e-5, o_ref if norm else None,
                           f_ref if out32 else None, **args)
        r, o, f = c(resid.clone()), torch.zeros(5, W, dtype=dtype, device=dev()), torch.zeros(5, W, device=dev())
        ops.add_norm_rows(c(y), nsum, None, r, c(go) if norm else None, 1e-5, o if norm else None, f if out32 else None,
                          c(y2) if second else None)
        close(r, r_ref, 2e-6)
        close(o, o_ref, 1e-5 if dtype == torch.float32 else 1e-2)
        close(f, f_ref, 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V", [(4, 2, 64, 32), (3, 3, 10, 7), (1, 1, 1, 1), (7, 1, 130, 512)])
def test_qkv_rows(dtype, H, G, D, V):
    g = torch.Generator().manual_seed(2)
    T, N = 9, H * D + G * (D + V)
    x, b = torch.randn(T, N + 6, generator=g), torch.randn(N, generator=g)
    rows = i32([5, 64, -1, 95, 0, 1, 33, 96, 2])   # one row out of the pages, one inactive
    for bias, own in ((b, True), (None, True), (b, False)):
        caches = [torch.zeros(3, PAGE, G, D, dtype=dtype), torch.zeros(3, PAGE, G, V, dtype=dtype),
                  torch.zeros(3, G, V, PAGE, dtype=dtype)]
        q_ref, got = torch.zeros(T, H, D), [c(t.clone()) for t in caches]
        ref_args = caches if own else [None] * 3
        lref.qkv_rows(x[:, 2:], bias, H, G, D, V, 1e-5, rows, q_ref, *ref_args)
        q = torch.zeros(T, H, D, device=dev())
        ops.qkv_rows(c(x)[:, 2:], c(bias), H, G, D, V, 1e-5, c(rows), q, *(got if own else [None] * 3))
        close(q, q_ref, 1e-5)
        for a, r in zip(got, caches):
            close(a, r, 1e-5 if dtype == torch.float32 else 1e-2)
            assert bool(a.any()) == own


def _pages(lens, g):
    need = [math.ceil(n / PAGE) for n in lens]
    perm = torch.randperm(sum(need) + 3, generator=g).tolist()
    bt = torch.zeros(len(lens), max(need) + 1, dtype=torch.int32)
    k = 0
    for s, n in enumerate(need):
        bt[s, :n] = torch.tensor(perm[k:k + n], dtype=torch.int32)
        k += n
    return bt, sum(need) + 3


# (window, kept keys, distances in the table)
REACHES = [(10 ** 9, 0, 30), (37, 5, 60), (33, 40, 1), (20, 3, 5000), (64, 96, 33), (1, 1, 2)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V", [(4, 2, 64, 64), (6, 1, 40, 24), (3, 3, 128, 130)])
def test_attention_row_form_with_bias_and_kept_keys(dtype, H, G, D, V):
    g = torch.Generator().manual_seed(3)
    ctx, ql = [300, 1, 70, 33], [40, 1, 70, 1]
    bt, pages = _pages(ctx, g)
    T = sum(ql)
    q = torch.randn(T, H, D, generator=g)
    kc = torch.randn(pages, PAGE, G, D, generator=g).to(dtype)
    vc = torch.randn(pages, PAGE, G, V, generator=g).to(dtype)
    gate = torch.randn(T, H * V + 3, generator=g)[:, 1:1 + H * V]
    qs, qt = i32([0, 40, 41, 111]), 4
    ws = [s for s, n in enumerate(ql) for _ in range(math.ceil(n / qt))]
    wt = [t for n in ql for t in range(math.ceil(n / qt))]
    for window, keep, dist in REACHES:
        rel = torch.randn(H, dist, generator=g) * 2
        o_ref, o = torch.zeros(T, H, V, dtype=dtype), torch.zeros(T, H, V, dtype=dtype, device=dev())
        lref.sink_attention(q, kc, vc, bt, qs, i32(ql), i32(ctx), None, gate, o_ref, window, 0.2, rel=rel, keep_first=keep)
        ops.sink_attention(c(q), c(kc), c(vc), c(bt), c(qs), c(i32(ql)), c(i32(ctx)), c(i32(ws)), c(i32(wt)), None, c(gate),
                           o, window, 0.2, qt, rel=c(rel), keep_first=keep)
        close(o, o_ref, 1e-5 if dtype == torch.float32 else 1e-2)


def _transposed(vc):
    pages, _, G, V = vc.shape
    vt = torch.zeros(pages, G, V, PAGE, dtype=vc.dtype)
    for off in range(PAGE):
        vt[:, :, :, int(lref.vt_position(torch.tensor(off)))] = vc[:, off]
    return vt


@pytest.mark.parametrize("H,G,D,V", [(4, 2, 64, 64), (6, 1, 32, 32), (5, 5, 128, 96), (8, 2, 96, 320), (16, 1, 64, 128)])
def test_attention_mfma_form_with_bias_and_kept_keys(H, G, D, V):
    """Prompt tiles, and for decode rows the key split, against the reference on the same transposed pages."""
    g = torch.Generator().manual_seed(4)
    ctx, ql = [300, 1, 70, 45], [40, 1, 70, 2]
    bt, pages = _pages(ctx, g)
    T = sum(ql)
    q = torch.randn(T, H, D, generator=g)
    kc = torch.randn(pages, PAGE, G, D, generator=g).bfloat16()
    vc = torch.randn(pages, PAGE, G, V, generator=g).bfloat16()
    vt = _transposed(vc)
    gate = torch.randn(T, H * V + 3, generator=g)[:, 1:1 + H * V]
    qs = i32([0, 40, 41, 111])
    ws = [s for s, n in enumerate(ql) for _ in range(math.ceil(n / 16))]
    wt = [t for n in ql for t in range(math.ceil(n / 16))]
    for window, keep, dist in REACHES:
        rel = torch.randn(H, dist, generator=g) * 2
        o_ref = torch.zeros(T, H, V, dtype=torch.bfloat16)
        lref.sink_attention(q, kc, vc, bt, qs, i32(ql), i32(ctx), None, gate, o_ref, window, 0.2, vt, rel=rel, keep_first=keep)
        for split in (False, True) if V <= 128 else (False,):
            o = torch.zeros(T, H, V, dtype=torch.bfloat16, device=dev())
            ops.sink_attention(c(q), c(kc), c(vc), c(bt), c(qs), c(i32(ql)), c(i32(ctx)), c(i32(ws)), c(i32(wt)), None,
                               c(gate), o, window, 0.2, 16, c(vt), split, rel=c(rel), keep_first=keep)
            close(o, o_ref, 2e-2)


@pytest.mark.parametrize("H,G,D,V", [(4, 2, 64, 64), (6, 1, 32, 32), (5, 5, 128, 96), (8, 2, 96, 320), (16, 1, 64, 128),
                                     (40, 2, 160, 16), (2, 1, 512, 128)])
def test_attention_decode_form(H, G, D, V):
    """One row per item (also two rows of one sequence), the heads of a group side by side in up to two column tiles, with
    and without bias, kept keys, sink, cap, output rotation, per-head and per-element gates; a long walk (more than 64
    pages per wave in the widest case)."""
    g = torch.Generator().manual_seed(7)
    ctx, ql = [300, 1, 33, 45, 0, 2400], [1, 1, 1, 2, 0, 1]
    if H == 6:
        ctx[5] = 18000
    bt, pages = _pages(ctx, g)
    T = sum(ql)
    q = torch.randn(T, H, D, generator=g)
    kc = torch.randn(pages, PAGE, G, D, generator=g).bfloat16()
    vc = torch.randn(pages, PAGE, G, V, generator=g).bfloat16()
    vt = _transposed(vc)
    wide = torch.randn(T, H * V + 3, generator=g)
    sink = torch.randn(H, generator=g)
    rope = HalfRotarySpec(dims=V, base=50.0).table(310)
    qs, ws, wt = i32([0, 1, 2, 3, 5, 5]), i32([5, 0, 1, 2, 3, 3, 4]), i32([0, 0, 0, 0, 0, 1, 0])
    for window, keep, dist, gate, sk, cap, turn in (
            (10 ** 9, 0, 30, wide[:, 1:1 + H * V], None, 0.0, None), (37, 5, 60, wide[:, :H], sink, 0.0, None),
            (33, 40, 1, None, None, 3.0, None), (20, 3, 5000, wide[:, 1:1 + H * V], None, 0.0, rope), (1, 1, 2, None, sink, 0.0, None),
            (64, 0, 0, wide[:, :H], sink, 2.0, rope), (10 ** 9, 0, 0, None, None, 0.0, None)):
        rel = torch.randn(H, dist, generator=g) * 2 if dist else None
        o_ref = torch.zeros(T, H, V, dtype=torch.bfloat16)
        lref.sink_attention(q, kc, vc, bt, qs, i32(ql), i32(ctx), sk, gate, o_ref, window, 0.2, vt, cap, turn, rel, keep)
        o = torch.zeros(T, H, V, dtype=torch.bfloat16, device=dev())
        ops.sink_attention(c(q), c(kc), c(vc), c(bt), c(qs), c(i32(ql)), c(i32(ctx)), c(ws), c(wt), c(sk), c(gate), o, window,
                           0.2, 1, c(vt), False, cap, c(turn), c(rel), keep)
        close(o, o_ref, 2e-2)


@pytest.mark.parametrize("E,top", [(1, 1), (6, 2), (16, 1), (64, 8), (256, 5)])
def test_sigmoid_routing_with_a_shared_gate(E, top):
    g = torch.Generator().manual_seed(5)
    for shared in (0, 1):
        z = torch.randn(33, E + shared, generator=g) * 2
        i_ref, w_ref = torch.zeros(33, top, dtype=torch.int32), torch.zeros(33, top + shared)
        lref.moe_route(z, None, i_ref, w_ref, 1, 1, 1.5, 2)
        i, w = torch.zeros(33, top, dtype=torch.int32, device=dev()), torch.zeros(33, top + shared, device=dev())
        ops.moe_route(c(z), None, i, w, 1, 1, 1.5, 2)
        assert torch.equal(i.cpu(), i_ref)
        close(w, w_ref, 1e-6)


@pytest.mark.parametrize("M,W,E,top,shared", [(1, 1, 1, 1, 0), (16, 2048, 16, 2, 1), (64, 333, 70, 4, 1), (5, 1024, 256, 8, 0),
                                             (33, 64, 3, 3, 1)])
def test_route_rows_in_one_launch(M, W, E, top, shared):
    """The one-launch router against the reference's choice, and its work list: every (row, slot) once, under its expert,
    tiles beyond the last marked; several launches on the same scratch."""
    g = torch.Generator().manual_seed(8)
    S, tiles = top + shared, -(-M * (top + shared) // 64) + E + 2
    w = torch.randn(E + shared, W, generator=g) / math.sqrt(W) * 2
    srt, til, num = (torch.zeros(n, dtype=torch.int32, device=dev()) for n in (tiles * 64, tiles, 2))
    for _ in range(3):
        x = torch.randn(M, W, generator=g)
        i_ref, w_ref = torch.zeros(M, top, dtype=torch.int32), torch.zeros(M, S)
        z = x @ w.t()
        lref.moe_route(z, None, i_ref, w_ref, 1, 1, 1.25, 2)
        i, wt = torch.zeros(M, top, dtype=torch.int32, device=dev()), torch.zeros(M, S, device=dev())
        ops.moe_route_rows(c(x), c(w), i, wt, 1.25, srt, til, num)
        i, wt = i.cpu(), wt.cpu()
        # rows whose scores come close are decided by rounding: judge the scores, and the indices elsewhere
        close(wt, w_ref, 1e-5)
        sc = torch.sigmoid(z[:, :E]).sort(-1, descending=True).values
        clear = (sc[:, :-1] - sc[:, 1:])[:, :top].amin(-1) > 1e-5 if E > 1 else torch.ones(M, dtype=torch.bool)
        assert torch.equal(i[clear], i_ref[clear])
        n = int(num[0])
        assert int(num[1]) == 0 and bool((til[n:] == -1).all())
        seen = []
        for t in range(n):
            for v in srt[t * 64:(t + 1) * 64].tolist():
                if v >= 0:
                    seen.append(v)
                    assert int(til[t]) == (E if v % S == top else int(i[v // S, v % S]))
        assert sorted(seen) == list(range(M * S))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,W,F,Fs,E,top", [(16, 520, 136, 72, 5, 2), (32, 64, 96, 0, 4, 2), (3, 48, 24, 40, 5, 2), (19, 33, 7, 0, 4, 1), (300, 128, 72, 136, 6, 2), (200, 64, 64, 32, 3, 3)])
def test_expert_weights_on_the_input(dtype, M, W, F, Fs, E, top):
    """Register-direct and LDS-staged expert GEMMs, with and without a shared expert."""
    g = torch.Generator().manual_seed(6)

    def rnd(*s):
        return (torch.randn(*s, generator=g) / math.sqrt(s[-1])).to(dtype)

    x = torch.randn(M, W, generator=g).to(dtype)
    gate, up, down = rnd(E, F, W), rnd(E, F, W), rnd(E, W, F)
    sh = (rnd(Fs, W), rnd(Fs, W), rnd(W, Fs)) if Fs else (None, None, None)
    S = top + (1 if Fs else 0)
    idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(M)]).to(torch.int32)
    w = torch.rand(M, S, generator=g) * 1.5
    tiles = -(-M * S // 64) + E + 2
    o_ref, plain = torch.zeros(M * S, W), torch.zeros(M * S, W)
    lref.moe_grouped(x, idx, w, gate, up, down, *sh, o_ref, True)
    lref.moe_grouped(x, idx, w, gate, up, down, *sh, plain, False)
    assert float((o_ref - plain).abs().max()) > 1e-2
    for ref, inp in ((o_ref, True), (plain, False)):
        o = torch.zeros(M * S, W, device=dev())
        ops.moe_grouped(c(x), c(idx), c(w), c(gate), c(up), c(down), *(c(t) for t in sh),
                        torch.zeros(tiles * 64, dtype=torch.int32, device=dev()),
                        torch.zeros(tiles, dtype=torch.int32, device=dev()), torch.zeros(1, dtype=torch.int32, device=dev()),
                        torch.zeros(M * S, -(-max(F, Fs) // 8) * 8, dtype=dtype, device=dev()), o, inp)
        close(o, ref, 1e-5 if dtype == torch.float32 else 2e-2)
