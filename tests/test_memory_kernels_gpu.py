"""HIP kernels of the convolved-attention / matrix-memory designs against their plain PyTorch references
(ops/layers_reference.py), op by op: convolved and rotated q | k | v rows into their pages, the matrix memory's walk and its
MFMA chunk form, the work lists of table-routed experts, gelu rows, and scaled attention outputs in a wider row."""
import math

import pytest
import torch

from distributed_sse_for_llm_response_amd import ops
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


def tiles(lens, qt):
    ws, wt = [], []
    for s, n in enumerate(lens):
        k = max(1, -(-n // qt))
        ws += [s] * k
        wt += list(range(k))
    return i32(ws), i32(wt)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V", [(4, 2, 64, 32), (3, 3, 10, 0), (1, 1, 1, 1), (7, 1, 130, 0), (2, 1, 7, 5)])
@pytest.mark.parametrize("K", [0, 1, 2, 3, 4, 6])
def test_conv_qkv_rows(dtype, H, G, D, V, K):
    """Sequences that start, continue, are shorter than the taps, and one that is inactive; portions in tiles and single
    rows; tails, pages, transposed pages and queries."""
    g = torch.Generator().manual_seed(2)
    C, VW = (H + G) * D, V or D
    for lens, ctx, qt in (([9, 2, 0, 40], [9, 35, 3, 73], 4), ([9, 2, 0, 40], [9, 35, 3, 73], 16), ([1, 1, 0, 1], [1, 33, 5, 64], 1)):
        T = sum(lens)
        qs = i32([0, lens[0], lens[0] + lens[1], lens[0] + lens[1]])
        x = torch.randn(T, C + G * V + 3, generator=g)
        taps = torch.randn(C, K, generator=g) if K else None
        tail = torch.randn(5, K - 1, C, generator=g) if K > 1 else None
        rope = torch.randn(70, min(4, D // 2), 2, generator=g) if D > 1 else None   # shorter than the last position
        factor = torch.rand(60, generator=g) if V else None
        slots, pos = torch.empty(T, dtype=torch.int32), 0
        for s, n in enumerate(lens):
            slots[pos:pos + n] = 96 * s + torch.arange(ctx[s] - n, ctx[s], dtype=torch.int32)
            pos += n
        slots[-1] = 96 * 4 + 7                       # out of the pages
        if T > 3:
            slots[3] = -1
        caches = [torch.zeros(12, PAGE, G, D, dtype=dtype), torch.zeros(12, PAGE, G, VW, dtype=dtype),
                  torch.zeros(12, G, VW, PAGE, dtype=dtype)]
        got, q_ref, q = [c(t.clone()) for t in caches], torch.zeros(T, H, D), torch.zeros(T, H, D, device=dev())
        gtail = c(tail)
        meta = (qs, i32(lens), i32(ctx), i32([4, 0, 2, 1]))
        lref.conv_qkv_rows(x[:, 2:], taps, tail, *meta, H, G, D, V, rope, factor, slots, q_ref, *caches)
        work = tiles(lens, qt)
        ops.conv_qkv_rows(c(x)[:, 2:], c(taps), gtail, *map(c, meta), *map(c, work), qt, H, G, D, V, c(rope), c(factor), c(slots),
                          q, *got)
        close(q, q_ref, 1e-5)
        for a, r in zip(got, caches):
            close(a, r, 1e-5 if dtype == torch.float32 else 1e-2)
        if K > 1:
            assert torch.equal(gtail.cpu(), tail)


def memory_inputs(lens, H, D, V, seed, gate_scale=2.0, slots=6):
    g = torch.Generator().manual_seed(seed)
    T = sum(lens)
    w = 2 * H * D + 2 * H * V + 2 * H
    big = torch.randn(T, w + 4, generator=g)
    big[:, 2 * H * (D + V):w] *= gate_scale
    gb = torch.cat([torch.randn(H, generator=g) - 1.0, torch.randn(H, generator=g) + 2.0])
    state, norm = torch.randn(slots, H, D, V, generator=g), torch.randn(slots, H, D + 1, generator=g)
    return big, gb, state, norm, torch.randn(H * V, generator=g)


def memory_views(big, H, D, V):
    q, k = big[:, :H * D].unflatten(1, (H, D)), big[:, H * D:2 * H * D].unflatten(1, (H, D))
    o = 2 * H * D
    return q, k, big[:, o:o + H * V].unflatten(1, (H, V)), big[:, o + H * V:o + 2 * H * V], big[:, o + 2 * H * V:o + 2 * H * V + 2 * H]


def run_memory(fn, big, gb, state, norm, nw, meta, H, D, V, dtype, extra=(), cap=5.0):
    q, k, v, og, gates = memory_views(big, H, D, V)
    out = torch.zeros(big.shape[0], H * V + 8, dtype=dtype, device=big.device)
    fn(q, k, v, gates, gb, cap, state, norm, *meta, og, nw, 1e-5, 1e-6, D ** -0.5, 0.7, out[:, :H * V], *extra)
    assert not out[:, H * V:].any()
    return out[:, :H * V]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,V", [(2, 32, 48), (3, 10, 9), (1, 1, 1), (2, 128, 128), (1, 512, 512), (1, 270, 130), (2, 64, 500), (1, 3, 512)])
def test_matrix_memory_walk(dtype, H, D, V):
    """Sequences that start and continue, one inactive, single rows and short portions."""
    for lens, ctx in (([1, 1, 0, 1], [1, 40, 7, 2]), ([5, 3, 0, 9], [5, 50, 7, 9])):
        big, gb, state, norm, nw = memory_inputs(lens, H, D, V, 3)
        qs = i32([0, lens[0], lens[0] + lens[1], lens[0] + lens[1]])
        meta = (qs, i32(lens), i32(ctx), i32([4, 0, 2, 1]))
        gs, gn = c(state.clone()), c(norm.clone())
        want = run_memory(lref.matrix_memory, big, gb, state, norm, nw, meta, H, D, V, dtype)
        got = run_memory(ops.matrix_memory, c(big), c(gb), gs, gn, c(nw), tuple(map(c, meta)), H, D, V, dtype)
        close(got, want, 1e-4 if dtype == torch.float32 else 1e-2)
        close(gs, state, 1e-5)
        close(gn, norm, 1e-5)


@pytest.mark.parametrize("H,D,V", [(2, 32, 48), (3, 12, 9), (4, 128, 128), (2, 256, 320), (1, 96, 16), (2, 64, 34), (1, 4, 1),
                                   (1, 192, 64), (1, 160, 100), (1, 224, 512)])
@pytest.mark.parametrize("gate_scale", [0.5, 8.0])
def test_matrix_memory_chunk_form(H, D, V, gate_scale):
    """The MFMA form against the token walk's reference: lengths around the chunk, sequences that continue, rows of another
    group ahead of the call's rows, gates from gentle to saturated.  Operands are bf16-rounded projections; the states
    agree to the rounding of the keys."""
    lens, ctx = [33, 64, 1, 100, 31], [33, 164, 9, 100, 40]
    skip = 3                                       # rows of another group at the front
    big, gb, state, norm, nw = memory_inputs([skip] + lens, H, D, V, 4, gate_scale)
    # q, k, v as bf16 projections give them: the reference then differs from the kernel by its own rounding alone
    big[:, :2 * H * D + H * V] = big[:, :2 * H * D + H * V].to(torch.bfloat16).float()
    qs = [skip]
    for n in lens[:-1]:
        qs.append(qs[-1] + n)
    meta = (i32(qs), i32(lens), i32(ctx), i32([4, 0, 2, 1, 5]))
    gs, gn = c(state.clone()), c(norm.clone())
    want = run_memory(lref.matrix_memory, big, gb, state, norm, nw, meta, H, D, V, torch.bfloat16)
    T = big.shape[0]
    work = torch.zeros(ops.memory_work_floats(T, H, V, len(lens)), device=dev())
    got = run_memory(ops.matrix_memory, c(big), c(gb), gs, gn, c(nw), tuple(map(c, meta)), H, D, V, torch.bfloat16,
                     (work, skip, T - skip))
    assert not got[:skip].any()
    close(gs, state, 2e-3)
    close(gn, norm, 2e-3)
    # a row whose normaliser product all but cancels magnifies the rounding of q times its scale: judge the bulk
    err = (got[skip:].float().cpu() - want[skip:].float()).view(T - skip, H, V).pow(2).mean(-1).sqrt()
    ref = want[skip:].float().view(T - skip, H, V).pow(2).mean(-1).sqrt().clamp_min(1e-3)
    rel = (err / ref).flatten()
    assert float((rel < 3e-2).float().mean()) > 0.97 and float(rel.median()) < 1e-2, (float(rel.median()), float(rel.max()))


def test_chunk_form_in_portions_agrees_with_one_pass():
    """A sequence cut at odd places, the state carried in the slot, against one pass; then a decode row on the walk."""
    H, D, V, T = 2, 64, 64, 150
    big, gb, state, norm, nw = memory_inputs([T], H, D, V, 5)
    big = c(big)

    def go(cuts):
        s, n, outs, at = c(state.clone()), c(norm.clone()), [], 0
        for k in cuts:
            part = big[at:at + k]
            meta = tuple(map(c, (i32([0]), i32([k]), i32([at + k]), i32([2]))))
            work = torch.zeros(ops.memory_work_floats(k, H, V, 1), device=dev())
            outs.append(run_memory(ops.matrix_memory, part, c(gb), s, n, c(nw), meta, H, D, V, torch.bfloat16,
                                   (work, 0, k) if k > 1 else ()))
            at += k
        return torch.cat(outs), s, n

    a, sa, na = go([T])
    b, sb, nb = go([2, 31, 64, 1, 1, 33, 18])
    close(b, a, 3e-2)
    close(sb[2], sa[2], 5e-3)
    close(nb[2], na[2], 5e-3)


@pytest.mark.parametrize("M", [1, 5, 64, 300])
def test_moe_table_lists(M):
    """Lists of several layers from one launch: every (row, slot) once, in a tile of its expert, counts and pads right;
    the grouped experts on a ready list give what they give on a list of their own."""
    g = torch.Generator().manual_seed(6)
    vocab = 40
    specs = [(5, 2, True), (3, 3, False), (70, 1, True)]
    tables = [torch.rand(vocab, E, generator=g).argsort(-1)[:, :top].to(torch.int32).contiguous() for E, top, _ in specs]
    ids = torch.randint(-1, vocab + 1, (M,), generator=g, dtype=torch.int32)   # ids out of range read row 0
    dims = [(-(-M * (top + sh) // 64) + E + 2) for E, top, sh in specs]
    tki = [torch.zeros(M, top, dtype=torch.int32, device=dev()) for _, top, _ in specs]
    srt = [torch.full((n * 64,), -7, dtype=torch.int32, device=dev()) for n in dims]
    te = [torch.zeros(n, dtype=torch.int32, device=dev()) for n in dims]
    nt = [torch.zeros(1, dtype=torch.int32, device=dev()) for _ in dims]
    for _ in range(2):
        ops.moe_table_lists(c(ids), [c(t) for t in tables], [s[0] for s in specs], [s[2] for s in specs], tki, srt, te, nt)
    for i, (E, top, sh) in enumerate(specs):
        want = torch.zeros(M, top, dtype=torch.int32)
        lref.moe_table_lists(ids, [tables[i]], [want])
        assert torch.equal(tki[i].cpu(), want)
        S, n = top + sh, int(nt[i])
        got, exp = srt[i].cpu()[:n * 64].view(n, 64), te[i].cpu()
        assert sorted(x for x in got.flatten().tolist() if x >= 0) == list(range(M * S))
        for t in range(n):
            for x in got[t].tolist():
                if x >= 0:
                    e = int(want[x // S, x % S]) if x % S < top else E
                    assert e == int(exp[t])
        assert (exp[n:] == -1).all()
    E, top, _ = specs[0]
    W, F, Fs = 32, 16, 24
    x = torch.randn(M, W, generator=g).to(torch.bfloat16)
    ws = [torch.randn(E, F, W, generator=g), torch.randn(E, F, W, generator=g), torch.randn(E, W, F, generator=g),
          torch.randn(Fs, W, generator=g), torch.randn(Fs, W, generator=g), torch.randn(W, Fs, generator=g)]
    ws = [c((t / 4).to(torch.bfloat16)) for t in ws]
    tw = torch.full((M, top), 1.0 / top, device=dev())
    h, o1, o2 = (torch.zeros(M * 3, n, dtype=d, device=dev()) for n, d in ((24, torch.bfloat16), (W, torch.float32), (W, torch.float32)))
    ops.moe_grouped(c(x), tki[0], tw, *ws, srt[0], te[0], nt[0], h, o1, False, True)
    ops.moe_grouped(c(x), tki[0], tw, *ws, srt[0], te[0], nt[0], h, o2)
    assert torch.equal(o1, o2)
    ref = torch.zeros(M * 3, W)
    none = torch.zeros(1)
    lref.moe_grouped(x, tki[0].cpu(), tw.cpu(), *[t.cpu() for t in ws], ref)
    close(o1, ref, 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_gelu_rows(dtype):
    x = torch.linspace(-12, 12, 7 * 33).view(7, 33)
    want, got = torch.zeros(7, 30, dtype=dtype), torch.zeros(7, 30, dtype=dtype, device=dev())
    lref.act_rows(x[:, 1:31], want, 3, None, None)
    ops.act_rows(c(x)[:, 1:31], got, 3)
    close(got, want, 1e-5 if dtype == torch.float32 else 1e-2)


@pytest.mark.parametrize("wide_gate", [False, True])
@pytest.mark.parametrize("form", ["row", "row fp32", "tiles", "split", "decode", "decode in 3 parts", "decode in 16 parts"])
def test_attention_into_a_wider_row(form, wide_gate):
    """Every form of the paged attention with an output that is a column slice of a wider row, times a scale, with a
    sink."""
    g = torch.Generator().manual_seed(7)
    H, G, D, V = 6, 2, 32, 48
    dtype = torch.float32 if form == "row fp32" else torch.bfloat16
    ctx, ql = ([70, 33], [70, 9]) if form in ("row", "row fp32", "tiles") else ([300, 33], [1, 1])
    T = sum(ql)
    need = [math.ceil(n / PAGE) for n in ctx]
    perm = torch.randperm(sum(need) + 2, generator=g).tolist()
    bt = torch.zeros(2, max(need), dtype=torch.int32)
    bt[0, :need[0]], bt[1, :need[1]] = i32(perm[:need[0]]), i32(perm[need[0]:need[0] + need[1]])
    q = torch.randn(T, H, D, generator=g)
    kc, vc = (torch.randn(sum(need) + 2, PAGE, G, n, generator=g).to(dtype) for n in (D, V))
    vt = torch.zeros(sum(need) + 2, G, V, PAGE, dtype=dtype)
    for off in range(PAGE):
        vt[:, :, :, lref.vt_position(off)] = vc[:, off]
    gate, sink = torch.randn(T, H * V if wide_gate else H, generator=g), torch.randn(H, generator=g)
    meta = (i32([0, ql[0]]), i32(ql), i32(ctx))
    want = torch.zeros(T, H * V + 16, dtype=dtype)
    lref.sink_attention(q, kc, vc, bt, *meta, sink, gate, want[:, 8:8 + H * V].unflatten(1, (H, V)), 10 ** 9, 0.2, out_scale=-1.5)
    qt, args = {"row": (4, (None, False)), "row fp32": (4, (None, False)), "tiles": (16, (c(vt), False)),
                "split": (16, (c(vt), True))}.get(form, (1, (c(vt), False)))
    nparts = int(form.split()[2]) if "parts" in form else 1   # sixteen: more than the sequences have pages
    got = torch.zeros(T, H * V + 16, dtype=dtype, device=dev())
    ops.sink_attention(c(q), c(kc), c(vc), c(bt), *map(c, meta), *map(c, tiles(ql, qt)), c(sink), c(gate),
                       got[:, 8:8 + H * V].unflatten(1, (H, V)), 10 ** 9, 0.2, qt, *args, out_scale=-1.5,
                       part=torch.zeros(2 * H * nparts * (V + 2), device=dev()) if nparts > 1 else None, nparts=nparts)
    close(got, want, 1e-5 if dtype == torch.float32 else 2e-2)
    assert not got[:, :8].any() and not got[:, 8 + H * V:].any()


@pytest.mark.parametrize("H,G,D,V", [(4, 2, 32, 48), (6, 6, 64, 16), (8, 2, 128, 128), (8, 1, 96, 112), (3, 1, 64, 64), (1, 1, 128, 80)])
@pytest.mark.parametrize("window,keep,cap", [(10 ** 9, 0, 0.0), (40, 0, 0.0), (33, 5, 0.0), (70, 40, 3.0), (1, 0, 0.0)])
def test_shared_page_attention(H, G, D, V, window, keep, cap):
    """The shared-page form for prompt portions: sequences that start, continue in the middle of a page and are shorter
    than a tile, one inactive; windows, kept keys, caps, sinks and both kinds of gate."""
    g = torch.Generator().manual_seed(8)
    ctx, ql = [150, 300, 9, 2], [150, 131, 0, 2]
    T = sum(ql)
    need = [math.ceil(n / PAGE) for n in ctx]
    perm = torch.randperm(sum(need) + 2, generator=g).tolist()
    bt, k = torch.zeros(4, max(need), dtype=torch.int32), 0
    for s, n in enumerate(need):
        bt[s, :n], k = i32(perm[k:k + n]), k + n
    q = torch.randn(T, H, D, generator=g)
    kc, vc = (torch.randn(sum(need) + 2, PAGE, G, n, generator=g).to(torch.bfloat16) for n in (D, V))
    vt = torch.zeros(sum(need) + 2, G, V, PAGE, dtype=torch.bfloat16)
    for off in range(PAGE):
        vt[:, :, :, lref.vt_position(off)] = vc[:, off]
    meta = (i32([0, ql[0], 281, 281]), i32(ql), i32(ctx))
    rows = ops.sink_tile_rows(torch.bfloat16, H, G, D, V)
    assert rows in (32, 64, 128)
    for sink, cols in ((torch.randn(H, generator=g), H * V), (None, H), (torch.zeros(H), None)):
        gate = torch.randn(T, cols, generator=g) if cols else None
        want, got = torch.zeros(T, H, V, dtype=torch.bfloat16), torch.zeros(T, H, V, dtype=torch.bfloat16, device=dev())
        lref.sink_attention(q, kc, vc, bt, *meta, sink, gate, want, window, 0.2, softcap=cap, keep_first=keep, out_scale=0.6)
        ops.sink_attention(c(q), c(kc), c(vc), c(bt), *map(c, meta), *map(c, tiles(ql, rows)), c(sink), c(gate), got, window, 0.2,
                           rows, c(vt), softcap=cap, keep_first=keep, out_scale=0.6)
        close(got, want, 2e-2)
