"""The gated parallel stacks of head-mixing window attention, latent attention with sinks and window attention beside a minimal gated
recurrence (Zevilorn) against the float64 restatement in oracle/zevilorn.py: every new mechanism alone through the C ABI, then whole
models through the engine's step function -- whole prompts, token-by-token decoding, portions, mixed batches, reused pages and slots,
crafted keys far back, at page borders and at window edges, a token only the recurrent state carries, layers gone through several
times, greedy generation.  Small random configurations of their own; `be` runs each test on the CPU twin and (gpu) on the MI355X."""
import json
import math
import os
import subprocess

import numpy as np
import pytest
import torch

from oracle import zevilorn as OZ
from tests.conftest import ROOT

F32, BF16, I32 = torch.float32, torch.bfloat16, torch.int32
TOL = {F32: 3e-5, BF16: 4e-2}


def dev(be, a, dtype=F32):
    return be.t(np.asarray(a, dtype=np.float32)).to(dtype).contiguous()


def ints(be, a):
    return be.t(np.asarray(a, dtype=np.int32))


def pos_errs(got, want):
    """per position: rms of the difference (mean removed) relative to the rms of the reference"""
    d = np.asarray(got, dtype=np.float64) - want
    d = d - d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / (np.sqrt((w * w).mean(-1)) + 1e-30)


def rel_err(got, want):
    return float(pos_errs(got, want).max())


def ok(got, want, dtype):
    """float32: every position within 3e-5 of the logits' rms; bfloat16: the typical position within 2e-2, nine in ten within 4e-2"""
    e = pos_errs(got, want)
    return e.max() <= TOL[F32] if dtype is F32 else bool(np.median(e) <= 2e-2 and (e <= TOL[BF16]).mean() >= 0.9 and e.max() <= 0.12)


def close(got, want, tol):
    return np.abs(np.asarray(got, dtype=np.float64) - want).max() <= tol * (1 + np.abs(want).max())


def spans_of(be, lens):
    row0 = np.cumsum([0] + list(lens[:-1]))
    return ints(be, row0), ints(be, lens), len(lens), max(lens)


# ---- row-wise steps, router, epilogues ---------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("width", [6, 48, 1030, 2052])
@pytest.mark.parametrize("form", ["one", "two_normed", "no_experts", "embedding"])
def test_gated_residual_step(be, dtype, width, form):
    rng = np.random.default_rng(width)
    rows, eps, top, ldg, vocab = 5, 1e-3, 3, 2 * width + 8, 11
    x = rng.standard_normal((rows, width)).astype(np.float32) * 3 + 1
    y, y2 = rng.standard_normal((2, rows, width)).astype(np.float32) * np.float32(2)
    my = rng.standard_normal((rows * top, width)).astype(np.float32)
    mw = rng.uniform(0, 1, (rows, top)).astype(np.float32)
    gates = rng.standard_normal((rows, ldg)).astype(np.float32) * 2
    w_in, wy, wy2 = OZ.bf16_round(1 + 0.3 * rng.standard_normal((3, width)))
    table = OZ.bf16_round(rng.standard_normal((vocab, width)))
    ids = rng.integers(0, vocab, rows)
    x32, out = be.t(x), torch.zeros((rows, width), dtype=dtype, device=be.device)
    kw = dict(gates=be.t(gates), ldg=ldg, g1_off=4, g2_off=width + 6 if width % 4 else width + 8)
    want = x.astype(np.float64)
    t = y.astype(np.float64)
    if form == "two_normed":
        kw.update(y=be.t(y), y2=be.t(y2), wy=dev(be, wy, dtype), wy2=dev(be, wy2, dtype), ya=0.5, yb=0.25)
        t = np.array([0.5 * OZ.rms_norm(y[r].astype(np.float64), wy, eps) + 0.25 * OZ.rms_norm(y2[r].astype(np.float64), wy2, eps) for r in range(rows)])
    elif form != "embedding":
        kw.update(y=be.t(y))
    if form != "embedding":
        want = want + t * OZ.sigmoid(gates[:, 4:4 + width])
    if form in ("one", "two_normed"):
        kw.update(moe_y=be.t(my), moe_w=be.t(mw), top=top)
        g2 = kw["g2_off"]
        want = want + (my.reshape(rows, top, width) * mw[:, :, None].astype(np.float64)).sum(1) * OZ.sigmoid(gates[:, g2:g2 + width])
    if form in ("embedding", "two_normed"):
        kw.update(table=dev(be, table, dtype), ids=ints(be, ids))
        want = want + table[ids]
    be.ext.gated_residual(x32, out, rows, eps, w_in=dev(be, w_in, dtype), dtype=dtype, **kw)
    normed = np.array([OZ.rms_norm(v, w_in, eps) for v in want])
    assert close(be.n(x32), want, 3e-6)
    assert close(be.n(out.float()), normed, 3e-6 if dtype is F32 else 1e-2)
    # gathered rows, no addition
    idx = np.array([4, 1, 4], dtype=np.int32)
    out2 = torch.zeros((3, width), dtype=F32, device=be.device)
    be.ext.gated_residual(x32, out2, 3, eps, w_in=dev(be, w_in, dtype), row_idx=be.t(idx), dtype=dtype)
    assert close(be.n(out2), normed[idx], 3e-6)
    # the stream starts from the table; only the addition
    be.ext.gated_residual(x32, None, rows, eps, table=dev(be, table, dtype), ids=ints(be, ids), init=True, dtype=dtype)
    assert close(be.n(x32), table[ids].astype(np.float64), 0)


@pytest.mark.parametrize("experts,count,keep,top", [(8, 4, 2, 3), (12, 4, 3, 4), (6, 6, 2, 2), (6, 1, 1, 6), (130, 13, 4, 9), (512, 2, 1, 8), (5, 1, 1, 1)])
def test_router_among_the_best_groups(be, experts, count, keep, top):
    """the chosen experts and their scores, and the per-expert lists; includes rows where a group of two good experts beats the group
    of the single best one, and equal scores (the first of equals wins)"""
    rng = np.random.default_rng(experts)
    rows, ld, off = 9, experts + 7, 3
    z = (rng.standard_normal((rows, ld)) * 2).astype(np.float32)
    if count > 1 and experts // count > 1:
        z[0, off:off + experts] = -3.0
        z[0, off] = 4.0                                          # the best expert, alone in its group
        gs = experts // count
        for g in range(1, min(count, keep + 1)):
            z[0, off + g * gs:off + g * gs + 2] = 2.0
    z[1, off:off + experts] = 0.5                                # all equal
    ids = torch.zeros((rows, top), dtype=I32, device=be.device)
    wts = torch.zeros((rows, top), dtype=F32, device=be.device)
    lists = tuple(torch.zeros((n,), dtype=I32, device=be.device) for n in (experts, experts, rows * top))
    be.ext.moe_route_grouped(be.t(z), ld, off, ids, wts, rows, experts, top, 1.0, count, keep, groups=lists)
    gi, gw = be.n(ids), be.n(wts)
    router = {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}}
    for r in range(rows):
        s = (1.0 / (1.0 + np.exp(-z[r, off:off + experts].astype(np.float32)))).astype(np.float64)
        picks, gap = OZ.route(s, router)
        if gap > 1e-5 or r == 1:
            assert [int(e) for e in gi[r]] == [e for e, _ in picks], r
            assert close(gw[r], np.array([w for _, w in picks]), 1e-6)
    cnt, offs, lst = (be.n(t) for t in lists)
    for e in range(experts):
        assert sorted(lst[offs[e]:offs[e] + cnt[e]]) == [i for i in range(rows * top) if gi.reshape(-1)[i] == e]


@pytest.mark.parametrize("dtype,M,N,K", [(F32, 1, 9, 40), (F32, 33, 66, 50), (BF16, 3, 7, 24), (BF16, 17, 40, 64), (BF16, 130, 150, 72)])
def test_dense_linear_gelu_and_head_gate(be, dtype, M, N, K):
    rng = np.random.default_rng(M * 1000 + N * 10 + K)
    x = OZ.bf16_round(rng.standard_normal((M, K)))
    w = OZ.bf16_round(rng.standard_normal((N, K)) / math.sqrt(K) * 3)
    z = x.astype(np.float64) @ w.astype(np.float64).T
    y = torch.full((M, N), float("nan"), dtype=F32, device=be.device)
    be.ext.dense_linear(dev(be, x, dtype), dev(be, w, dtype), y, M, N, K, K, K, N, epi=be.ext.EPI_GELU_ERF)
    assert close(be.n(y), OZ.gelu(z), 3e-6)
    # two batches (heads), one gate per row and batch
    gate = rng.standard_normal((M, 5)).astype(np.float32) * 2
    y2 = torch.full((M, 2 * N), float("nan"), dtype=F32, device=be.device)
    be.ext.dense_linear(dev(be, x, dtype), dev(be, np.stack([w, -w]), dtype), y2, M, N, K, K, K, 2 * N, batch=2, sxb=0, swb=N * K, syb=N,
                        aux=be.t(gate), ldaux=5, sauxb=1, aux_off=2, epi=be.ext.EPI_MUL_SIGMOID_ROW_AUX)
    sg = OZ.sigmoid(gate)
    assert close(be.n(y2), np.concatenate([z * sg[:, 2:3], -z * sg[:, 3:4]], 1), 3e-6)


# ---- convolution, recurrence ---------------------------------------------------------------------------------------------------------


def token_steps():
    """unequal portions of two sequences in slots 0 and 2: single tokens, two tokens, spans longer than a chunk"""
    return [[(0, 2), (2, 1)], [(2, 40), (0, 1)], [(0, 1)], [(0, 5), (2, 3)], [(2, 1)], [(0, 1), (2, 1)], [(2, 150), (0, 70)], [(0, 64), (2, 1)]]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
def test_plain_convolution_over_spans_and_steps(be, dtype, taps):
    """no activation, no identity beside it; whichever step brought a token, its output is the weighted sum of the sequence's last
    inputs; stale rows of a slot's earlier user are not seen"""
    rng = np.random.default_rng(taps)
    ch, ld, off = 38, 45, 4
    cw = OZ.bf16_round(rng.standard_normal((ch, taps)))
    tail = torch.full((3, max(taps - 1, 1), ch), 7.0, dtype=F32, device=be.device)
    hist, n_tok = {0: [], 2: []}, {0: 0, 2: 0}
    for step in token_steps():
        lens = [n for _s, n in step]
        rows = sum(lens)
        f = rng.standard_normal((rows, ld)).astype(np.float32)
        seq = np.concatenate([[s] * n for s, n in step])
        pos = np.concatenate([np.arange(n_tok[s], n_tok[s] + n) for s, n in step])
        out = torch.zeros((rows, ch), dtype=F32, device=be.device)
        be.ext.conv_rows(be.t(f), ld, off, dev(be, cw, dtype), None, out, tail, spans_of(be, lens), ints(be, seq), ints(be, pos), ch, taps, residual=2)
        got, r = be.n(out), 0
        for s, n in step:
            for _ in range(n):
                hist[s] = (hist[s] + [f[r, off:off + ch].astype(np.float64)])[-taps:]
                assert close(got[r], OZ.causal_conv(hist[s], cw.astype(np.float64)), 3e-6), (step, r)
                n_tok[s] += 1
                r += 1


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("width,chunk", [(5, 64), (300, 64), (33, 7)])
def test_minimal_gated_recurrence(be, dtype, width, chunk):
    """token by token, in short spans and in the chunked form, alternating on the same slots; channels that forget at once, channels that
    keep nearly everything, candidates on both sides of zero"""
    rng = np.random.default_rng(width)
    ld = 3 * width + 5
    state = torch.full((3, width), 5.0, dtype=F32, device=be.device)
    S, n_tok = {0: np.zeros(width), 2: np.zeros(width)}, {0: 0, 2: 0}
    for step in token_steps():
        lens = [n for _s, n in step]
        rows = sum(lens)
        f = rng.standard_normal((rows, ld)).astype(np.float32) * 2
        f[:, :width] += np.linspace(-7, 7, width).astype(np.float32)
        f[0, width] = 0.0
        seq = np.concatenate([[s] * n for s, n in step])
        pos = np.concatenate([np.arange(n_tok[s], n_tok[s] + n) for s, n in step])
        out = torch.zeros((rows, width), dtype=dtype, device=be.device)
        kw = {}
        if max(lens) > chunk // 2:
            per = [-(-n // chunk) for n in lens]
            total = sum(per)
            kw = dict(chunks=(ints(be, np.cumsum([0] + per[:-1])), chunk, total),
                      scratch=torch.full((2 * total + len(lens), width), float("nan"), dtype=F32, device=be.device))
        be.ext.mingru_scan(be.t(f), ld, 0, width, 2 * width, out, state, spans_of(be, lens), ints(be, seq), ints(be, pos), width, **kw)
        got, r = be.n(out.float()), 0
        for s, n in step:
            for _ in range(n):
                row = f[r].astype(np.float64)
                z, u, g = OZ.sigmoid(row[:width]), row[width:2 * width], row[2 * width:3 * width]
                S[s] = (1 - z) * S[s] + z * np.where(u >= 0, u + 0.5, OZ.sigmoid(u))
                assert close(got[r], S[s] * g * OZ.sigmoid(g), 5e-6 if dtype is F32 else 1e-2), (step, r)
                n_tok[s] += 1
                r += 1
        assert close(be.n(state)[0], S[0], 5e-6) and close(be.n(state)[2], S[2], 5e-6)
    assert close(be.n(state)[1], np.full(width, 5.0), 0)


# ---- attention forms on random caches ---------------------------------------------------------------------------------------------------


def fill_pages(be, rng, lens, page, tail_shapes, dtype, spread):
    """a pool whose pages are dealt to the sequences in shuffled order; per shape one cache tensor and the rows in sequence order"""
    per = [-(-n // page) for n in lens]
    order = rng.permutation(sum(per) + 2)
    table = np.zeros((len(lens), max(per) + 1), dtype=np.int32)
    at = 0
    for s, p in enumerate(per):
        table[s, :p] = order[at:at + p]
        at += p
    caches, rows = [], []
    for shape in tail_shapes:
        c = (rng.standard_normal((sum(per) + 2, page) + shape) * spread).astype(np.float32)
        c = OZ.bf16_round(c) if dtype is BF16 else c
        caches.append(c)
        rows.append([np.concatenate([c[table[s, i]] for i in range(p)])[:lens[s]] for s, p in enumerate(per)])
    return table, caches, rows


@pytest.mark.parametrize("dtype,heads,kv_heads,dim,vdim,window,cap,page", [
    (F32, 6, 3, 10, 7, 13, 5.0, 8), (F32, 1, 1, 8, 8, 1, 0.0, 4), (F32, 5, 5, 16, 24, 300, 3.0, 64), (BF16, 4, 2, 24, 20, 70, 4.0, 16),
    (BF16, 6, 2, 64, 64, 40, 6.0, 16), (BF16, 16, 4, 32, 32, 1 << 30, 0.0, 32), (BF16, 12, 12, 32, 32, 90, 5.0, 64), (BF16, 20, 4, 32, 32, 50, 5.0, 16),
    (BF16, 32, 8, 128, 128, 1 << 30, 8.0, 64), (BF16, 8, 1, 64, 128, 100, 5.0, 12), (BF16, 3, 1, 128, 64, 65, 5.0, 16)])
def test_head_mixing_attention(be, dtype, heads, kv_heads, dim, vdim, window, cap, page):
    """random caches, rows at positions inside, at and past the window: the row kernel with and without split keys and, for the sizes it
    takes, the tile kernel (one row up to sixteen per tile), against the equations"""
    rng = np.random.default_rng(heads * 100 + dim)
    big = heads * dim > 1024
    lens = [9, 40 if big and be.is_emu else 150]
    table, (kc, vc), (K, V) = fill_pages(be, rng, lens, page, ((kv_heads, dim), (kv_heads, vdim)), dtype, 1.0)
    spots = [(0, 0), (0, 1), (0, 8)] + [(1, p) for p in sorted({0, 1, lens[1] // 2, lens[1] - 1, min(window, lens[1] - 1), min(window - 1, lens[1] - 1)})]
    tiles = [(0, 3, 5), (1, lens[1] - 16, 16), (1, 17, 1), (1, 0, 16), (1, 20, 2)]
    for s, p, n in tiles:
        spots += [(s, p + i) for i in range(n)]
    rows = len(spots)
    q = (rng.standard_normal((rows, heads, dim)) * 1.5 / math.sqrt(dim)).astype(np.float32)
    q = OZ.bf16_round(q) if dtype is BF16 else q
    talk = OZ.bf16_round(np.eye(heads) + rng.standard_normal((heads, heads)) * 0.5 / math.sqrt(heads) * 2)
    hpg = heads // kv_heads

    def want_row(i):
        s, p = spots[i]
        lo = max(0, p - window + 1)
        a = np.stack([K[s][lo:p + 1, h // hpg].astype(np.float64) @ q[i, h] for h in range(heads)])
        a = cap * np.tanh(a / cap) if cap else a
        sc = talk.astype(np.float64) @ a
        return np.concatenate([OZ.softmax_plus(sc[h], 0.0) @ V[s][lo:p + 1, h // hpg] for h in range(heads)])
    want = np.stack([want_row(i) for i in range(rows)])
    args = (dev(be, q, dtype), dev(be, kc, dtype), dev(be, vc, dtype), be.t(talk), torch.zeros((heads,), dtype=F32, device=be.device),
            ints(be, [s for s, _ in spots]), ints(be, [p for _, p in spots]), be.t(table), page)
    shape = (heads, kv_heads, dim, vdim, window, cap)
    tol = 1e-5 if dtype is F32 else 8e-3
    for nsplit in (1, 3):
        out = torch.zeros((rows, heads * vdim), dtype=dtype, device=be.device)
        part = dict(part_o=torch.full((rows, heads, nsplit, vdim), float("nan"), dtype=F32, device=be.device),
                    part_ml=torch.full((rows, heads, nsplit, 2), float("nan"), dtype=F32, device=be.device)) if nsplit > 1 else {}
        be.ext.talk_attn(*args, out, None, rows, *shape, nsplit=nsplit, **part)
        assert close(be.n(out.float()), want, tol), nsplit
    pick = np.array([rows - 1, 2, 5], dtype=np.int32)                       # a list of rows leaves the others alone
    for nsplit in (1, 2, 3):
        out = torch.full((rows, heads * vdim), 3.0, dtype=dtype, device=be.device)
        part = dict(part_o=torch.full((rows, heads, nsplit, vdim), float("nan"), dtype=F32, device=be.device),
                    part_ml=torch.full((rows, heads, nsplit, 2), float("nan"), dtype=F32, device=be.device)) if nsplit > 1 else {}
        be.ext.talk_attn(*args, out, be.t(pick), 3, *shape, nsplit=nsplit, **part)
        got = be.n(out.float())
        assert close(got[pick], want[pick], max(tol, 1e-2) if dtype is BF16 else tol) and (got[[i for i in range(rows) if i not in pick]] == 3.0).all(), nsplit
    if be.ext.talk_attn_tiles_supported(dtype, heads, dim, vdim):
        base = rows - sum(n for *_x, n in tiles)
        row0 = base + np.cumsum([0] + [n for *_x, n in tiles[:-1]])
        for nsplit in (1, 2, 5):
            out = torch.full((rows, heads * vdim), 3.0, dtype=dtype, device=be.device)
            part = dict(part_o=torch.full((rows, heads, nsplit, vdim), float("nan"), dtype=F32, device=be.device),
                        part_ml=torch.full((rows, heads, nsplit, 2), float("nan"), dtype=F32, device=be.device)) if nsplit > 1 else {}
            be.ext.talk_attn_tiles(*args, out, (ints(be, row0), ints(be, [n for *_x, n in tiles]), len(tiles)), *shape, nsplit=nsplit, **part)
            got = be.n(out.float())
            assert close(got[base:], want[base:], 1e-2) and (got[:base] == 3.0).all(), nsplit


@pytest.mark.parametrize("dtype,heads,R,rot,rot_dims,halves,sink", [
    (F32, 3, 20, 6, 6, True, True), (F32, 2, 40, 8, 4, True, False), (F32, 2, 24, 8, 8, False, True), (BF16, 5, 32, 8, 8, True, True),
    (BF16, 4, 128, 32, 32, True, True), (BF16, 6, 64, 16, 12, True, True), (BF16, 20, 128, 64, 64, True, True), (BF16, 4, 96, 32, 32, False, True)])
def test_latent_attention_with_sinks_and_either_rotary_layout(be, dtype, heads, R, rot, rot_dims, halves, sink):
    """the cached rows (norm, rotation) and the attention over them: row kernel and matrix-core kernels (prompt tiles, decoded rows with
    the keys split), no window"""
    rng = np.random.default_rng(heads * 100 + R)
    n, page, eps, scale, window = 70, 16, 1e-5, 0.4, 1 << 30
    rd = {"base": 500.0, "dims": rot_dims}
    freq = dev(be, OZ.frequencies(rd))
    dkv = rng.standard_normal((n, R + rot + 3)).astype(np.float32)
    w = OZ.bf16_round(1 + 0.2 * rng.standard_normal(R))
    table = rng.permutation(8)[:6].astype(np.int32).reshape(1, 6)
    cache = torch.zeros((8, page, R + rot), dtype=dtype, device=be.device)
    seq, pos, bt = ints(be, np.zeros(n)), ints(be, np.arange(n)), be.t(table)
    be.ext.latent_append(be.t(dkv), R + rot + 3, dev(be, w, dtype), eps, n, R, rot, rot_dims, freq, seq, pos, bt, page, cache, dkv_off=2, halves=halves)
    rows = be.n(cache.float())[table[0]].reshape(-1, R + rot)[:n].astype(np.float64)

    def turned(v, p):
        return OZ.turn(v.astype(np.float64), p, rd, not halves)
    want_rows = np.stack([np.concatenate([OZ.rms_norm(dkv[p, 2:2 + R].astype(np.float64), w, eps), turned(dkv[p, 2 + R:2 + R + rot], p)]) for p in range(n)])
    assert close(rows, want_rows, 1e-5 if dtype is F32 else 1e-2)
    q = OZ.bf16_round(rng.standard_normal((n, heads, rot + 4)))
    q_abs = rng.standard_normal((n, heads, R)).astype(np.float32) * np.float32(1.5 / math.sqrt(R))
    sk = rng.standard_normal(heads).astype(np.float32) * 2 if sink else None
    want = np.stack([np.stack([OZ.softmax_plus((rows[:p + 1, :R] @ q_abs[p, h].astype(np.float64) + rows[:p + 1, R:] @ turned(q[p, h, 4:], p)) * scale,
                                               float(sk[h]) if sink else None) @ rows[:p + 1, :R] for h in range(heads)]) for p in range(n)])
    qd, qa = dev(be, q, dtype), be.t(q_abs)
    common = (qd, heads * (rot + 4), rot + 4, 4, qa, cache, page, seq, pos, bt)
    var = dict(halves=halves, sink=be.t(sk) if sink else None)
    out = torch.zeros((n, heads, R), dtype=dtype, device=be.device)
    be.ext.latent_attn(*common, out, n, heads, R, rot, rot_dims, freq, scale, window, **var)
    assert close(be.n(out.float()), want, 2e-5 if dtype is F32 else 1e-2)
    if be.ext.latent_attn_tiles_supported(dtype, R, rot):
        out = torch.zeros((n, heads, R), dtype=dtype, device=be.device)
        row0 = list(range(0, n - 6, 16))
        be.ext.latent_attn_tiles(*common, out, ints(be, row0), ints(be, [min(16, n - 6 - r) for r in row0]), len(row0), 16, heads, R, rot, rot_dims,
                                 freq, scale, window, **var)
        for nsplit, rr in ((1, range(n - 6, n - 3)), (3, range(n - 3, n))):
            part = dict(part_o=torch.zeros((n, heads, nsplit, R), dtype=F32, device=be.device),
                        part_ml=torch.zeros((n, heads, nsplit, 2), dtype=F32, device=be.device)) if nsplit > 1 else {}
            be.ext.latent_attn_tiles(*common, out, ints(be, list(rr)), None, 3, 1, heads, R, rot, rot_dims, freq, scale, window, nsplit=nsplit, **part, **var)
        assert close(be.n(out.float()), want, 1.5e-2)


def test_frequency_scaling_tables():
    from exllamav2_amd.window_attn import rotary_tables
    for sc in (None, {"factor": 3.0}, {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 96}, {"factor": 1.0, "low": 1.0, "high": 1.0, "original": 50}):
        rot = {"base": 700.0, "dims": 24, "scaling": sc}
        if sc and sc.get("high") == sc.get("low") and "low" in sc:
            want = [700.0 ** (-2.0 * i / 24) for i in range(12)]
        else:
            want = OZ.frequencies(rot)
        f, amp = rotary_tables(700.0, 24, sc, "cpu")
        assert amp == 1.0 and np.allclose(f.numpy(), want, rtol=1e-6)


# ---- whole models -----------------------------------------------------------------------------------------------------------------------

CONFIGS = {
    # every mixer, with and without a feed-forward, two layers of three gone through twice; sizes differ per layer
    "mixed": lambda: OZ.small_config([
        OZ.layer(OZ.parallel_mixer(), OZ.moe_ff_spec()),
        OZ.layer(OZ.talking_mixer(), OZ.moe_ff_spec(experts=6, top=2, ff=10, count=3, keep=2)),
        OZ.layer(OZ.latent_mixer(), None),
        OZ.layer(OZ.parallel_mixer(OZ.window_spec(heads=3, kv_heads=1, dim=10, vdim=6, dims=10, window=12), width=9), OZ.moe_ff_spec(experts=4, top=1, ff=7, count=2, keep=1)),
        OZ.layer(OZ.talking_mixer(heads=3, kv_heads=3, dim=8, vdim=14, dims=4, window=5, conv=2), None)], loop=(1, 3, 2)),
    # odd sizes, one head, one tap, window 1, no scaling, no loop, every expert chosen, groups of one
    "odd": lambda: OZ.small_config([
        OZ.layer(OZ.talking_mixer(heads=1, kv_heads=1, dim=6, vdim=5, dims=6, window=1, conv=1, scaling=None), OZ.moe_ff_spec(experts=3, top=3, ff=5, count=1, keep=1)),
        OZ.layer(OZ.latent_mixer(heads=1, dim=4, rot_dim=4, vdim=1, kv_rank=11, q_rank=7), OZ.moe_ff_spec(experts=5, top=2, ff=3, count=5, keep=3)),
        OZ.layer(OZ.parallel_mixer(OZ.window_spec(heads=1, kv_heads=1, dim=4, vdim=3, dims=2, window=3, factor=1.0), width=1), None)],
        width=30, vocab=50, loop=None),
    # the loop at the end of the stack, three times; the sizes of the matrix-core kernels
    "wide": lambda: OZ.small_config([
        OZ.layer(OZ.talking_mixer(heads=6, kv_heads=2, dim=32, vdim=32, dims=16, window=33, conv=4), OZ.moe_ff_spec(experts=8, top=2, ff=16, count=2, keep=1)),
        OZ.layer(OZ.latent_mixer(heads=4, dim=16, rot_dim=8, vdim=24, kv_rank=32, q_rank=24), OZ.moe_ff_spec(experts=4, top=2, ff=16, count=2, keep=2)),
        OZ.layer(OZ.parallel_mixer(OZ.window_spec(heads=4, kv_heads=2, dim=32, vdim=32, dims=32, window=40), width=72), OZ.moe_ff_spec(ff=8))],
        width=64, vocab=70, loop=(1, 3, 3)),
}


def make_engine(be, cfg, W, dtype, max_tokens, page=4, max_seqs=4, graphs=None):
    from exllamav2_amd.config import LayeredConfig
    from exllamav2_amd.engine import Engine
    from exllamav2_amd.layered import LayeredModel
    tensors = {k: be.t(v).to(BF16) for k, v in W.items()}
    model = LayeredModel(LayeredConfig.from_dict_parallel_gated(cfg), device=be.device, dtype=dtype, ext=be.ext).load(tensors)
    return Engine(model, max_tokens=max_tokens, max_seqs=max_seqs, page_size=page, graphs=graphs)


def run_cuts(be, eng, rid, tokens, cuts):
    out, at = [], 0
    for c in cuts:
        out.append(be.n(eng.step([(rid, tokens[at:at + c], list(range(c)))])))
        at += c
    assert at == len(tokens)
    return np.concatenate(out, 0)


def clear_tokens(cfg, W, n, seed, gap=0.008):
    """n random tokens none of whose router decisions is a close call (so that bfloat16 rounding cannot pick another expert or group);
    grown token by token: a token whose routing is a close call is replaced by the next draw"""
    import copy
    rng = np.random.default_rng(seed)
    o = OZ.Oracle(cfg, W)
    toks = []
    while len(toks) < n:
        for _ in range(400):
            t = int(rng.integers(0, cfg["vocab"]))
            keep = copy.deepcopy(o.seqs.get("g"))
            gaps = []
            o.feed("g", [t], gaps=gaps)
            if gaps[0] > gap:
                toks.append(t)
                break
            if keep is None:
                o.drop("g")
            else:
                o.seqs["g"] = keep
        else:
            raise AssertionError("no token with clear routing found")
    return toks


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_whole_prompt(be, name, dtype):
    cfg = CONFIGS[name]()
    W = OZ.random_model(cfg, seed=1)
    toks = clear_tokens(cfg, W, 23, 2, gap=0.01)
    want = OZ.Oracle(cfg, W).feed("a", toks)
    eng = make_engine(be, cfg, W, dtype, 32)
    got = run_cuts(be, eng, "a", toks, [23])
    assert ok(got, want, dtype), pos_errs(got, want)


def test_residual_stream_after_every_layer_run(be):
    """the oracle's stream behind the last layer of a stack against the model's, for stacks of one layer up to all of them, gone through
    once, twice and three times"""
    cfg = CONFIGS["mixed"]()
    cfg["loop"] = {"start": 0, "stop": 5, "times": 1}
    W = OZ.random_model(cfg, seed=31)
    toks = [int(t) for t in np.random.default_rng(32).integers(0, cfg["vocab"], size=9)]
    for times in (1, 2, 3):
        for depth in range(1, 6):
            sub = dict(cfg, layers=cfg["layers"][:depth], loop={"start": 0, "stop": depth, "times": times})
            trail = []
            OZ.Oracle(sub, W).feed("a", toks, residuals=trail)
            Ws = dict(W)
            Ws["final.norm"] = np.ones(cfg["width"], dtype=np.float32)
            Ws["head"] = np.concatenate([np.eye(cfg["width"], dtype=np.float32),
                                         np.zeros((cfg["vocab"] - cfg["width"], cfg["width"]), dtype=np.float32)])      # logits = the normed stream
            eng = make_engine(be, sub, Ws, F32, 16)
            got = run_cuts(be, eng, "a", toks, [9])[:, :cfg["width"]]
            want = np.array([OZ.rms_norm(trail[t][-1], np.ones(cfg["width"]), cfg["norm"]["eps"]) for t in range(9)])
            assert close(got, want, 2e-5), (times, depth)


@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 3, 2), (2, 3, 4), (1, 2, 3), (1, 1, 2)])
def test_loops_anywhere(be, loop):
    """no loop, one pass, the whole stack, the last layer only, one layer in the middle, an empty run: whole prompt and decoding"""
    cfg = CONFIGS["mixed"]()
    cfg["layers"] = cfg["layers"][:3]
    cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]} if loop else None
    W = OZ.random_model(cfg, seed=33)
    toks = list(np.random.default_rng(34).integers(0, cfg["vocab"], size=17))
    want = OZ.Oracle(cfg, W).feed("a", toks)
    for cuts in ([17], [6, 2, 3] + [1] * 6):
        assert rel_err(run_cuts(be, make_engine(be, cfg, W, F32, 20), "a", toks, cuts), want) <= TOL[F32], cuts


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_decoding_and_portions(be, name):
    """the same positions through a whole prompt, token by token from the first token on (the convolutions' tails, every pass's keys and
    the recurrent states pass over decoded tokens), and in portions down to two tokens that end inside pages"""
    cfg = CONFIGS[name]()
    W = OZ.random_model(cfg, seed=3)
    toks = list(np.random.default_rng(4).integers(0, cfg["vocab"], size=26))
    want = OZ.Oracle(cfg, W).feed("a", toks)
    for cuts in ([1] * 26, [2, 3, 2, 5, 2, 1, 1, 4, 2, 2, 2], [9] + [1] * 17, [25, 1], [1, 25]):
        eng = make_engine(be, cfg, W, F32, 28, page=4)
        assert rel_err(run_cuts(be, eng, "a", toks, cuts), want) <= TOL[F32], cuts


def test_mixed_batches_reuse_pages_and_slots(be):
    """five unequal requests over four slots and a pool smaller than their sum: portions beside single tokens, a request left out of
    a step, finished requests' pages and slot (with its tails, every pass's keys and its recurrent state) taken by the next; every
    position equals the request alone"""
    cfg = CONFIGS["mixed"]()
    W = OZ.random_model(cfg, seed=5)
    rng = np.random.default_rng(6)
    reqs = {r: list(rng.integers(0, cfg["vocab"], size=n)) for r, n in (("a", 13), ("b", 5), ("c", 9), ("d", 2), ("e", 11))}
    oracle = OZ.Oracle(cfg, W)
    want = {r: oracle.feed(r, t) for r, t in reqs.items()}
    eng = make_engine(be, cfg, W, F32, max_tokens=32, page=4, max_seqs=4)
    plan = [[("a", 5), ("b", 2)], [("a", 1), ("b", 3), ("c", 4), ("d", 2)], [("a", 2), ("c", 1)], [("c", 2), ("e", 3), ("a", 1)],
            [("a", 4), ("e", 2), ("c", 2)], [("e", 1)], [("e", 5)]]
    at, got = {r: 0 for r in reqs}, {r: [] for r in reqs}
    for step in plan:
        entries, end = [], []
        for r, n in step:
            entries.append((r, reqs[r][at[r]:at[r] + n], list(range(n))))
            at[r] += n
            if at[r] == len(reqs[r]):
                end.append(r)
        lg = be.n(eng.step(entries, end))
        k = 0
        for r, n in step:
            got[r].append(lg[k:k + n])
            k += n
    assert all(at[r] == len(reqs[r]) for r in reqs)
    assert len(eng.pool.free_pages) == eng.pool.num_pages and len(eng.pool.free_slots) == 4
    assert sum(-(-len(t) // 4) for t in reqs.values()) > eng.pool.num_pages            # pages were used again
    for r in reqs:
        assert rel_err(np.concatenate(got[r], 0), want[r]) <= TOL[F32], r


def test_a_reused_slot_starts_from_zeros(be):
    """one slot, three requests one after the other: the second and third find the first one's tails, recurrent state and cached
    keys of every pass in their slot and pages and must not see them"""
    cfg = CONFIGS["mixed"]()
    W = OZ.random_model(cfg, seed=15)
    rng = np.random.default_rng(16)
    eng = make_engine(be, cfg, W, F32, max_tokens=16, page=4, max_seqs=1)
    for r, n, cuts in (("a", 14, [14]), ("b", 9, [1, 1, 7]), ("c", 12, [2, 10])):
        toks = list(rng.integers(0, cfg["vocab"], size=n))
        want = OZ.Oracle(cfg, W).feed(r, toks)
        assert rel_err(run_cuts(be, eng, r, toks, cuts), want) <= TOL[F32], r
        eng.finish(r)


def drive(be, eng, reqs, plan):
    """plan: steps of [(request, first, last + 1)] with the requests that end after them; returns logits per request in token order"""
    got = {r: {} for r in reqs}
    for parts, end in plan:
        lg = be.n(eng.step([(r, reqs[r][lo:hi], list(range(hi - lo))) for r, lo, hi in parts], end))
        k = 0
        for r, lo, hi in parts:
            for p in range(lo, hi):
                got[r][p] = lg[k]; k += 1
    return {r: np.stack([got[r][p] for p in range(len(reqs[r]))]) for r in reqs}


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_decode_steps_as_graphs(be, dtype):
    """decoding steps through the engine's persistent-input path (on a GPU: captured once per batch size and replayed; every replay
    is checked): two requests decode side by side, one ends, the other goes on alone, a third joins"""
    cfg = CONFIGS["mixed"]()
    W = OZ.random_model(cfg, seed=21)
    reqs = {r: clear_tokens(cfg, W, n, 22 + i, gap=0.01) for i, (r, n) in enumerate((("a", 14), ("b", 9), ("c", 8)))}
    oracle = OZ.Oracle(cfg, W)
    want = {r: oracle.feed(r, t) for r, t in reqs.items()}
    eng = make_engine(be, cfg, W, dtype, max_tokens=48, page=4, graphs=True)
    plan = [([("a", 0, 3), ("b", 0, 2)], [])] + [([("a", 3 + i, 4 + i), ("b", 2 + i, 3 + i)], []) for i in range(6)] + [([("b", 8, 9)], ["b"])]
    plan += [([("a", 9 + i, 10 + i)], []) for i in range(3)] + [([("c", 0, 4)], [])]
    plan += [([("c", 4 + i, 5 + i), ("a", 12 + i, 13 + i)], []) for i in range(2)] + [([("c", 6, 8)], ["c", "a"])]
    got = drive(be, eng, reqs, plan)
    for r in reqs:
        assert ok(got[r], want[r], dtype), (r, pos_errs(got[r], want[r]))
    eng.close()


def test_matrix_core_sizes_in_portions_and_decoding_bf16(be):
    """head sizes of the tile kernels: a prompt of many tiles that crosses page borders and passes every window, then decoding, beside a
    second request"""
    cfg = CONFIGS["wide"]()
    W = OZ.random_model(cfg, seed=41)
    reqs = {"a": clear_tokens(cfg, W, 12, 42, gap=0.006), "b": clear_tokens(cfg, W, 160, 43, gap=0.006)}
    oracle = OZ.Oracle(cfg, W)
    want = {r: oracle.feed(r, t) for r, t in reqs.items()}
    eng = make_engine(be, cfg, W, BF16, max_tokens=256, page=16, graphs=True)
    plan = [([("a", i, i + 1)], []) for i in range(5)] + [([("b", 0, 139), ("a", 5, 6)], [])]
    plan += [([("a", i, i + 1), ("b", 133 + i, 134 + i)], []) for i in range(6, 12)] + [([("b", 145, 160)], [])]
    got = drive(be, eng, reqs, plan)
    for r in reqs:
        assert ok(got[r], want[r], BF16), (r, pos_errs(got[r], want[r]))
    eng.close()


def test_head_sizes_of_a_real_model_bf16_and_f32(be):
    """sizes at which every tuned kernel path is taken (head-mixing tiles of 128 with 16 and more heads and with split keys, the matrix-core
    decode kernel, latent tiles of 128 + 64, window tiles of 128, the chunked recurrence, the vector residual step, grouped expert
    launches): a prompt in portions, then decoding, beside a second request"""
    if be.is_emu:
        pytest.skip("minutes on the CPU twin; the small configurations cover its logic")
    for dtype in (F32, BF16):
        # (bfloat16 without routers: at this depth a rounded input tips a close choice now and then, which later positions remember)
        moe = OZ.moe_ff_spec(experts=8, top=2, ff=64, count=4, keep=2) if dtype is F32 else None
        cfg = OZ.small_config([
            OZ.layer(OZ.talking_mixer(heads=16, kv_heads=4, dim=128, vdim=128, dims=128, window=1000, conv=4, softcap=20.0, base=500000.0,
                                      scaling={"factor": 8.0, "low": 1.0, "high": 4.0, "original": 2048}), moe),
            OZ.layer(OZ.latent_mixer(heads=8, dim=64, rot_dim=64, vdim=64, kv_rank=128, q_rank=96), moe),
            OZ.layer(OZ.talking_mixer(heads=24, kv_heads=8, dim=64, vdim=64, dims=32, window=90, conv=3, softcap=20.0), None),
            OZ.layer(OZ.parallel_mixer(OZ.window_spec(heads=4, kv_heads=2, dim=128, vdim=128, dims=64, window=100, base=500000.0), width=256), moe)],
            width=256, vocab=300, loop=(1, 3, 2))
        W = OZ.random_model(cfg, seed=61)
        rng = np.random.default_rng(62)
        reqs = {"a": list(rng.integers(0, 300, 420)), "b": list(rng.integers(0, 300, 20))}
        oracle = OZ.Oracle(cfg, W)
        want = {r: oracle.feed(r, t) for r, t in reqs.items()}
        plan = [([("a", 0, 70)], []), ([("a", 70, 405), ("b", 0, 9)], []), ([("a", 405, 407), ("b", 9, 10)], [])]
        plan += [([("a", 407 + i, 408 + i), ("b", 10 + i, 11 + i)], []) for i in range(10)] + [([("a", 417, 420)], [])]
        eng = make_engine(be, cfg, W, dtype, max_tokens=1024, page=64, graphs=True)
        got = drive(be, eng, reqs, plan)
        for r in reqs:
            e = pos_errs(got[r], want[r])
            assert e.max() <= TOL[F32] if dtype is F32 else (np.median(e) <= 4e-2 and e.max() <= 8e-2), (r, dtype, np.sort(e)[-20:])
        eng.close()


def crafted_model(kind, window, seed=31):
    """one layer whose attention is made so that token 0's query matches token 1's key and nothing else: queries read inputs 0-3, keys
    inputs 4-7 through the same matrix, values the other inputs; token 0 is marked in inputs 0-3, token 1 in 4-7, all other tokens
    are zero there; no rotation to speak of.  Wherever a token 1 stands in front of token 0 inside the window, however far, that key
    takes the softmax among hundreds."""
    small = dict(base=1e30, dims=2)
    if kind == "talking":
        mix = OZ.talking_mixer(heads=2, kv_heads=2, dim=8, vdim=8, window=window, conv=2, softcap=30.0, scale=1.0, scaling=None, **small)
    elif kind == "parallel":
        mix = OZ.parallel_mixer(OZ.window_spec(heads=2, kv_heads=2, dim=8, vdim=8, window=window, scale=1.0, factor=1.0, **small), width=4)
    else:
        mix = OZ.latent_mixer(heads=2, dim=8, rot_dim=2, vdim=8, kv_rank=16, q_rank=8, base=1e30, scale=1.0)
    cfg = OZ.small_config([OZ.layer(mix, OZ.moe_ff_spec(experts=4, top=1, ff=8, count=2, keep=1))], width=16, vocab=40, loop=None)
    W = OZ.random_model(cfg, seed=seed)
    rng = np.random.default_rng(seed + 1)
    E = W["embed"]
    E[:, :8] = 0.0
    mark = rng.standard_normal(4)
    mark *= 6.0 / np.linalg.norm(mark)
    E[0, :4], E[1, 4:8] = mark, mark
    W["embed"] = OZ.bf16_round(E)
    W["l0.norm1"][:] = 1.0
    M = rng.standard_normal((16, 4))
    M[[0, 1, 8, 9]] = 0.0                                         # (the turned pair of each head stays empty)
    x = "l0.mix.left" if kind == "parallel" else "l0.mix"
    if kind == "latent":
        for n in ("dq", "dkv", "uq", "uk"):
            W[f"{x}.{n}"][:] = 0.0
        W[x + ".dq"][:4, :4] = np.eye(4)
        W[x + ".uq"][2:6, :4] = W[x + ".uq"][12:16, :4] = 2.0 * np.eye(4)
        W[x + ".dkv"][:4, 4:8] = np.eye(4)
        W[x + ".dkv"][4:12, 8:16] = np.eye(8)
        W[x + ".uk"][2:6, :4] = W[x + ".uk"][10:14, :4] = np.eye(4)
        W[x + ".uv"][:, :4] = 0.0
        W[x + ".uv"] = OZ.bf16_round(W[x + ".uv"] * 4)
        W[x + ".dq.norm"][:] = 1.0; W[x + ".dkv.norm"][:] = 1.0; W[x + ".sink"][:] = 0.0
    else:
        W[x + ".q"], W[x + ".k"] = np.zeros((16, 16), dtype=np.float32), np.zeros((16, 16), dtype=np.float32)
        W[x + ".q"][:, :4], W[x + ".k"][:, 4:8] = OZ.bf16_round(M), OZ.bf16_round(M)
        W[x + ".v"][:, :8] = 0.0
        W[x + ".v"] = OZ.bf16_round(W[x + ".v"] * 4)
    if kind == "talking":
        for s in "qkv":
            W[f"{x}.{s}.b"][:] = 0.0
            W[f"{x}.{s}.conv"][:] = 0.0
            W[f"{x}.{s}.conv"][:, -1] = 1.0
    return cfg, W


@pytest.mark.parametrize("kind", ["talking", "latent", "parallel"])
@pytest.mark.parametrize("page", [4, 64])
def test_a_marked_key_far_back_and_at_page_borders(be, kind, page):
    """whole prompt, portions and decoding: the marked key sits right in front of the query, at the sequence's first token, on both
    sides of a page border and hundreds of tokens back; where it stands it decides the query's logits"""
    cfg, W = crafted_model(kind, 400)
    rng = np.random.default_rng(page)
    T = 330
    query = T - 1
    changes = 0
    for target in (0, 1, page - 1, page, 2 * page, 200, query - page, query - 1):
        toks = [int(t) for t in rng.integers(2, cfg["vocab"], size=T)]
        toks[target], toks[query] = 1, 0                      # the marked pair, nowhere else
        base = list(toks)
        base[target] = 2
        want = OZ.Oracle(cfg, W).feed("t", toks)
        other = OZ.Oracle(cfg, W).feed("t", base)[-1]
        changes += rel_err(want[-1:], other[None]) > 0.05
        plans = [[T], [target + 1, T - target - 2, 1], [T - 3, 2, 1], [T - 20] + [1] * 20]
        for cuts in plans if target in (0, 200) else plans[2:3]:
            eng = make_engine(be, cfg, W, F32, max_tokens=T + page, page=page)
            got = run_cuts(be, eng, "t", toks, [c for c in cuts if c > 0])
            assert rel_err(got[-4:], want[-4:]) <= TOL[F32], (target, cuts[:3])
    assert changes >= 7


@pytest.mark.parametrize("kind", ["talking", "parallel"])
@pytest.mark.parametrize("window", [1, 2, 16, 21, 64])
def test_a_marked_key_at_the_window_edge(be, kind, window):
    """the marked key at the last place the window reaches and one in front of it, in a prompt, at a portion's start and decoded token by
    token: inside it decides the logits, outside nothing of it is left"""
    cfg, W = crafted_model(kind, window)
    rng = np.random.default_rng(window)
    T = window + 30
    query = T - 1
    for dist in ([window - 1, window] if window > 1 else [1]):
        toks = [int(t) for t in rng.integers(2, cfg["vocab"], size=T)]
        toks[query - dist], toks[query] = 1, 0
        base = list(toks)
        base[query - dist] = 2
        want, other = OZ.Oracle(cfg, W).feed("t", toks), OZ.Oracle(cfg, W).feed("t", base)
        if kind == "talking":                                     # (beside the window attention the recurrence remembers the token either way)
            assert (rel_err(want[-1:], other[-1:]) > 0.05) == (dist < window), dist
        for cuts in ([T], [T - 1, 1], [T - dist - 1, dist + 1], [T - 25] + [1] * 25):
            eng = make_engine(be, cfg, W, F32, max_tokens=T + 8, page=8)
            assert rel_err(run_cuts(be, eng, "t", toks, [c for c in cuts if c > 0])[-3:], want[-3:]) <= TOL[F32], (dist, cuts[:3])


def test_the_state_carries_a_far_token(be):
    """a token 300 positions back reaches the last position of a layer with a window of three only through the recurrent state: changing
    it changes the logits, and portions and decoding carry it like the whole prompt does"""
    cfg = OZ.small_config([OZ.layer(OZ.parallel_mixer(OZ.window_spec(heads=2, kv_heads=1, dim=8, vdim=8, dims=4, window=3), width=24),
                                    OZ.moe_ff_spec(experts=4, top=1, ff=8, count=2, keep=1))], width=16, vocab=40, loop=None)
    W = OZ.random_model(cfg, seed=51)
    W["l0.mix.right.z.b"][:] = -7.0                                                # slow forgetting
    rng = np.random.default_rng(52)
    toks = [int(t) for t in rng.integers(0, cfg["vocab"], size=310)]
    other = list(toks)
    other[9] = (toks[9] + 1) % cfg["vocab"]
    want = OZ.Oracle(cfg, W).feed("a", toks)
    assert rel_err(OZ.Oracle(cfg, W).feed("a", other)[-1:], want[-1:]) > 1e-3
    for cuts in ([310], [100, 2, 65, 143], [290] + [1] * 20):
        eng = make_engine(be, cfg, W, F32, max_tokens=320, page=16)
        assert rel_err(run_cuts(be, eng, "a", toks, cuts)[-8:], want[-8:]) <= 2 * TOL[F32], cuts


def test_sinks_take_weight_at_the_first_tokens(be):
    """with one or two keys the sinks hold much of the softmax: the first tokens' logits differ clearly from the same model with the
    learned sinks far down, and match the equations"""
    cfg = OZ.small_config([OZ.layer(OZ.latent_mixer(), None), OZ.layer(OZ.talking_mixer(), None)], loop=None)
    W = OZ.random_model(cfg, seed=71)
    W["l0.mix.sink"][:] = 3.0
    toks = [5, 9, 2, 30, 7]
    want = OZ.Oracle(cfg, W).feed("a", toks)
    low = dict(W)
    low["l0.mix.sink"] = np.full_like(W["l0.mix.sink"], -60.0)
    assert pos_errs(OZ.Oracle(cfg, low).feed("a", toks), want)[:2].min() > 0.05
    for dtype in (F32, BF16):
        for cuts in ([5], [1] * 5, [2, 3]):
            assert ok(run_cuts(be, make_engine(be, cfg, W, dtype, 16), "a", toks, cuts), want, dtype), (dtype, cuts)


def test_long_decoding_bf16(be):
    cfg = CONFIGS["mixed"]()
    W = OZ.random_model(cfg, seed=7)
    toks = clear_tokens(cfg, W, 60, 8, gap=0.008)
    want = OZ.Oracle(cfg, W).feed("a", toks)
    eng = make_engine(be, cfg, W, BF16, 64, page=8)
    got = run_cuts(be, eng, "a", toks, [3] + [1] * 57)
    assert ok(got, want, BF16), pos_errs(got, want)


def test_greedy_generation_through_the_generator(be):
    from exllamav2_amd.engine import Generator
    cfg = CONFIGS["mixed"]()
    W = OZ.random_model(cfg, seed=9)
    rng = np.random.default_rng(10)
    prompts = [list(map(int, rng.integers(0, cfg["vocab"], size=n))) for n in (7, 3, 5, 4, 6)]
    eng = make_engine(be, cfg, W, F32, max_tokens=64, page=4, max_seqs=3)
    out = Generator(eng, chunk=3).generate(prompts, 6)
    oracle = OZ.Oracle(cfg, W)
    checked = 0
    for i, p in enumerate(prompts):
        lg = oracle.feed(i, p)[-1]
        for t in out[i]:
            top2 = np.sort(lg)[-2:]
            if top2[1] - top2[0] < 1e-3:
                break                                             # a near tie: later tokens may differ legitimately
            assert t == int(np.argmax(lg))
            checked += 1
            lg = oracle.feed(i, [t])[-1]
        assert len(out[i]) == 6
    assert checked >= 20
    assert len(eng.pool.free_pages) == eng.pool.num_pages


def test_model_directory_registry(be, tmp_path):
    """config.json + model.safetensors -> architectures.load_model picks the class by the architecture name"""
    from safetensors.torch import save_file
    from exllamav2_amd.architectures import load_model, read_config
    from exllamav2_amd.engine import Engine
    cfg = CONFIGS["odd"]()
    W = OZ.random_model(cfg, seed=11)
    save_file({k: torch.from_numpy(np.asarray(v)).to(BF16) for k, v in W.items()}, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert read_config(str(tmp_path))[0] == "Zevilorn"
    model = load_model(str(tmp_path), device=be.device, dtype=F32, ext=be.ext)
    toks = [1, 5, 9, 2, 2, 7]
    got = be.n(Engine(model, 16, page_size=4).step([("x", toks, list(range(6)))]))
    assert rel_err(got, OZ.Oracle(cfg, W).feed("x", toks)) <= TOL[F32]


def test_bad_configurations_are_refused(be):
    from exllamav2_amd.config import LayeredConfig
    cfg = CONFIGS["mixed"]()
    with pytest.raises(RuntimeError, match="loop"):
        LayeredConfig.from_dict_parallel_gated(dict(cfg, loop={"start": 1, "stop": 9, "times": 2}))
    with pytest.raises(RuntimeError, match="missing key"):
        LayeredConfig.from_dict_parallel_gated({k: v for k, v in cfg.items() if k != "norm"})
    W = OZ.random_model(cfg, seed=1)
    with pytest.raises(RuntimeError, match="unknown mixer"):
        make_engine(be, dict(cfg, layers=[dict(cfg["layers"][0], type="nonesuch")], loop=None), W, F32, 16)
    bad = dict(W)
    bad["l1.mix.talk"] = bad["l1.mix.talk"][:, :-1]
    with pytest.raises(RuntimeError, match="mixing"):
        make_engine(be, cfg, bad, F32, 16)
    bad = dict(W)
    bad["l0.rg1"] = bad["l0.rg1"][:-1]
    with pytest.raises(RuntimeError, match="gates"):
        make_engine(be, cfg, bad, F32, 16)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_command_replays_steps(tmp_path, dtype):
    """bin/trace_run in a process of its own: steps on standard input, logits files and `done` lines out"""
    if not torch.cuda.is_available():
        pytest.skip("no GPU visible")
    from safetensors.torch import save_file
    cfg = CONFIGS["mixed"]()
    W = OZ.random_model(cfg, seed=12)
    mdir = tmp_path / "model"
    mdir.mkdir()
    save_file({k: torch.from_numpy(np.asarray(v)).to(BF16) for k, v in W.items()}, str(mdir / "model.safetensors"))
    (mdir / "config.json").write_text(json.dumps(cfg))
    a, b = clear_tokens(cfg, W, 300, 13, gap=0.008), clear_tokens(cfg, W, 9, 14)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:290], "want": [0, 289]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[290:295], "want": []}, {"id": "b", "tokens": b[:8], "want": [7]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[8:], "want": [0]}, {"id": "a", "tokens": a[295:], "want": [4]}], "end": ["a", "b"]}]
    out = tmp_path / "out"
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(mdir), "--dtype", dtype, "--out", str(out), "--max-tokens", "512"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600, cwd=str(tmp_path))
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    oracle = OZ.Oracle(cfg, W)
    wa, wb = oracle.feed("a", a), oracle.feed("b", b)
    got = np.concatenate([np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(k, -1) for n, k in ((0, 2), (1, 1), (2, 2))])
    want = np.stack([wa[0], wa[289], wb[7], wb[8], wa[299]])
    e = pos_errs(got, want)
    assert (e.max() <= TOL[F32]) if dtype == "float32" else (np.median(e) <= 2e-2 and e.max() <= 6e-2), e
