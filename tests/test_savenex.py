"""The pre-norm stacks of window attention with kept first tokens and normed heads beside a delta rule with a decay per key channel
(Savenex) against the float64 restatement in oracle/savenex.py: every new mechanism alone through the C ABI, then whole models through
the engine's step function -- whole prompts, token-by-token decoding, portions, mixed batches, reused pages and slots, crafted keys far
back, at page borders, at the window's edge and at the edge of the kept tokens, a token only the recurrent state carries, layers gone
through several times, greedy generation.  Small random configurations of their own; `be` runs each test on the CPU twin and (gpu) on
the MI355X."""
import json
import math
import os
import subprocess

import numpy as np
import pytest
import torch

from oracle import savenex as OS
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


# ---- row-wise steps, router, linears -----------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("width", [6, 48, 1030, 2052])
def test_residual_step_with_a_factor_and_stream_copies(be, dtype, width):
    """x += mult (two normed results | a linear's output + weighted expert rows), then the norm, or the stream itself into a wider row"""
    rng = np.random.default_rng(width)
    rows, eps, top, mult = 5, 1e-3, 3, 0.37
    x = rng.standard_normal((rows, width)).astype(np.float32) * 3 + 1
    y, y2 = rng.standard_normal((2, rows, width)).astype(np.float32) * np.float32(2)
    my = rng.standard_normal((rows * top, width)).astype(np.float32)
    mw = rng.uniform(0, 1, (rows, top)).astype(np.float32)
    w_in, wy, wy2 = OS.bf16_round(1 + 0.3 * rng.standard_normal((3, width)))
    tol = 3e-6 if dtype is F32 else 1e-2
    for form in ("two_normed", "experts", "both", "one"):
        x32, out = be.t(x), torch.zeros((rows, width), dtype=dtype, device=be.device)
        kw, want = {}, np.zeros((rows, width))
        if form == "two_normed":
            kw.update(y=be.t(y), y2=be.t(y2), wy=dev(be, wy, dtype), wy2=dev(be, wy2, dtype), ya=0.5, yb=0.5)
            want = np.stack([0.5 * (OS.rms(y[r].astype(np.float64), eps) * wy + OS.rms(y2[r].astype(np.float64), eps) * wy2) for r in range(rows)])
        if form in ("experts", "both"):
            kw.update(moe_y=be.t(my), moe_w=be.t(mw), top=top)
            want = want + (my.reshape(rows, top, width) * mw[:, :, None].astype(np.float64)).sum(1)
        if form in ("one", "both"):
            kw.update(y=be.t(y))
            want = want + y
        want = x.astype(np.float64) + mult * want
        be.ext.gated_residual(x32, out, rows, eps, w_in=dev(be, w_in, dtype), dtype=dtype, mult=mult, **kw)
        assert close(be.n(x32), want, 3e-6), form
        assert close(be.n(out.float()), np.stack([OS.rms(v, eps) * w_in for v in want]), tol), form
        wide = torch.full((rows, 2 * width + 4), 9.0, dtype=dtype, device=be.device)
        x32 = be.t(x)
        be.ext.gated_residual(x32, wide, rows, eps, dtype=dtype, mult=mult, ldo=wide.shape[1], **kw)
        assert close(be.n(x32), want, 3e-6) and close(be.n(wide.float())[:, :width], want, tol) and (be.n(wide.float())[:, width:] == 9.0).all(), form
    # nothing to add: a copy
    wide = torch.full((rows, 2 * width), 9.0, dtype=dtype, device=be.device)
    be.ext.gated_residual(be.t(x), wide, rows, eps, dtype=dtype, ldo=2 * width)
    assert close(be.n(wide.float())[:, :width], x.astype(np.float64), tol)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("width", [10, 300])
def test_normed_embedding_and_its_copy(be, dtype, width):
    rng = np.random.default_rng(width)
    table, w = OS.bf16_round(rng.standard_normal((7, width))), OS.bf16_round(1 + 0.2 * rng.standard_normal(width))
    ids, eps = rng.integers(0, 7, 5), 1e-3
    x32 = torch.zeros((5, width), dtype=F32, device=be.device)
    both = torch.full((5, 2 * width + 2), 9.0, dtype=dtype, device=be.device)
    zero = ints(be, np.zeros(5))
    be.ext.embed_pair(dev(be, table, dtype), None, dev(be, w, dtype), ints(be, ids), None, zero, zero, spans_of(be, [5]), x32, 0, 0, 0, 1.0, 1,
                      eps, xh=both, xh_off=width)
    want = np.stack([OS.rms(table[t].astype(np.float64), eps) * w for t in ids])
    got = be.n(both.float())
    assert close(be.n(x32), want, 3e-6) and close(got[:, width:2 * width], want, 3e-6 if dtype is F32 else 1e-2)
    assert (got[:, :width] == 9.0).all() and (got[:, 2 * width:] == 9.0).all()


@pytest.mark.parametrize("experts,top,extra,gate", [(8, 3, 2, True), (5, 5, 1, True), (6, 1, 0, False), (130, 9, 3, False), (512, 8, 0, True), (1, 1, 1, True)])
def test_router_softmax_over_the_chosen(be, experts, top, extra, gate):
    """the largest logits choose, weights = softmax over them; logits far apart and all equal; the experts every token uses behind them"""
    rng = np.random.default_rng(experts)
    rows, ld, off = 9, experts + 7, 3
    z = (rng.standard_normal((rows, ld)) * 2).astype(np.float32)
    z[1, off:off + experts] = 0.5                                # all equal: the first of them
    z[2, off:off + experts] *= 60                                # nearly all the weight on one
    z[3, off:off + experts] -= 200
    per = top + extra
    ids = torch.zeros((rows, per), dtype=I32, device=be.device)
    wts = torch.zeros((rows, per), dtype=F32, device=be.device)
    lists = tuple(torch.zeros((n,), dtype=I32, device=be.device) for n in (experts + extra, experts + extra, rows * per))
    be.ext.moe_route_chosen(be.t(z), ld, off, ids, wts, rows, experts, top, extra=extra, extra_col=experts if gate else -1, groups=lists)
    gi, gw = be.n(ids), be.n(wts)
    for r in range(rows):
        picks, gap = OS.route(z[r, off:off + experts].astype(np.float64), top)
        assert [int(e) for e in gi[r, :top]] == [e for e, _ in picks], r
        assert close(gw[r, :top], np.array([w for _, w in picks]), 1e-6)
        assert list(gi[r, top:]) == [experts + i for i in range(extra)]
        assert close(gw[r, top:], np.full(extra, OS.sigmoid(z[r, off + experts]) if gate else 1.0), 1e-6) if extra else True
    cnt, offs, lst = (be.n(t) for t in lists)
    for e in range(experts + extra):
        assert sorted(lst[offs[e]:offs[e] + cnt[e]]) == [i for i in range(rows * per) if gi.reshape(-1)[i] == e]


@pytest.mark.parametrize("dtype,M,N,K,n2", [(F32, 1, 19, 40, 11), (F32, 33, 66, 50, 64), (BF16, 3, 24, 24, 16), (BF16, 3, 7, 21, 1), (BF16, 17, 300, 64, 252),
                                            (BF16, 60, 40, 32, 8), (BF16, 130, 150, 72, 100)])
def test_split_linear(be, dtype, M, N, K, n2):
    """columns in front of the split in fp32, the ones behind it in the operand dtype, both with their biases"""
    rng = np.random.default_rng(M * 1000 + N * 10 + K)
    x, w = OS.bf16_round(rng.standard_normal((M, K))), OS.bf16_round(rng.standard_normal((N, K)) / math.sqrt(K))
    b = rng.standard_normal(N).astype(np.float32)
    want = x.astype(np.float64) @ w.astype(np.float64).T + b
    y = torch.full((M, n2), float("nan"), dtype=F32, device=be.device)
    y2 = torch.full((M, N - n2), float("nan"), dtype=dtype, device=be.device)
    be.ext.dense_linear_split(dev(be, x, dtype), dev(be, w, dtype), be.t(b), y, y2, M, n2)
    assert close(be.n(y), want[:, :n2], 3e-6) and close(be.n(y2.float()), want[:, n2:], 3e-6 if dtype is F32 else 1e-2)


@pytest.mark.parametrize("dtype,M,N,K", [(F32, 1, 9, 40), (F32, 33, 66, 50), (BF16, 3, 7, 24), (BF16, 17, 40, 64), (BF16, 130, 150, 72)])
def test_decay_and_gate_epilogue(be, dtype, M, N, K):
    """exp(c_n softplus(z + b)) with one c per column: decays; with c = -1 and a negated weight the sigmoid; arguments far out"""
    rng = np.random.default_rng(M * 1000 + N * 10 + K)
    x = OS.bf16_round(rng.standard_normal((M, K)) * 4)
    w = OS.bf16_round(rng.standard_normal((N, K)) / math.sqrt(K) * 4)
    c, b = -np.exp(rng.standard_normal(N)).astype(np.float32), rng.standard_normal(N).astype(np.float32)
    c[0] = -1.0
    z = x.astype(np.float64) @ w.astype(np.float64).T + b
    y = torch.full((M, N), float("nan"), dtype=F32, device=be.device)
    be.ext.dense_linear(dev(be, x, dtype), dev(be, w, dtype), y, M, N, K, K, K, N, aux=be.t(c), ldaux=0, bias=be.t(b), epi=be.ext.EPI_EXP_SOFTPLUS)
    assert close(be.n(y), np.exp(c * OS.softplus(z)), 5e-6)
    assert close(be.n(y)[:, 0], OS.sigmoid(-z[:, 0]), 5e-6)


@pytest.mark.parametrize("M", [1, 20, 64, 150])
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_clamped_and_row_gated_feed_forward(be, dtype, M):
    """DenseGatedMLP with the clamped unit, and the silu unit whose result one number per token gates (what a shared expert is)"""
    from types import SimpleNamespace
    from exllamav2_amd.mlp import DenseGatedMLP
    rng = np.random.default_rng(M)
    width, ff = 24, 40
    bufs = lambda tag, shape, dt: torch.zeros(shape, dtype=dt, device=be.device)
    model = SimpleNamespace(ext=be.ext, width=width, dtype=dtype, device=be.device, buf=bufs)
    W = {n: OS.bf16_round(rng.standard_normal(s) * 2 / math.sqrt(s[1])) for n, s in (("gate", (ff, width)), ("up", (ff, width)), ("down", (width, ff)))}
    h = OS.bf16_round(rng.standard_normal((M, width)))
    WW = {"m." + n: v.astype(np.float64) for n, v in W.items()}
    load = lambda mlp: mlp.load(lambda n: dev(be, W[n], dtype))
    got = be.n(load(DenseGatedMLP(model, "m", 0, limit=0.8)).forward(dev(be, h, dtype), M)[0])
    assert close(got, np.stack([OS.clamped_ff(WW, "m", 0.8, r) for r in h.astype(np.float64)]), 5e-6 if dtype is F32 else 1e-2)
    gates = rng.standard_normal((M, 5)).astype(np.float32) * 2
    got = be.n(load(DenseGatedMLP(model, "m", 0)).forward(dev(be, h, dtype), M, row_gate=(be.t(gates), 5, 3))[0])
    want = np.stack([OS.expert(WW, "m", r) for r in h.astype(np.float64)]) * OS.sigmoid(gates[:, 3:4])
    assert close(got, want, 5e-6 if dtype is F32 else 1e-2)


# ---- attention ---------------------------------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,dims,page", [(4, 2, 12, 10, 8, 8), (3, 3, 7, 5, 6, 4), (6, 1, 64, 80, 64, 64), (2, 1, 33, 16, 0, 16), (1, 1, 300, 3, 200, 8)])
def test_normed_heads_after_the_rotation(be, dtype, heads, kv_heads, dim, vdim, dims, page):
    """queries (scaled) and keys turned, then divided by their root mean square per head; values as they are; rows land in their pages"""
    rng = np.random.default_rng(dim)
    rows, eps, ld = 21, 1e-2, heads * dim + kv_heads * (dim + vdim) + 9
    f = rng.standard_normal((rows, ld)).astype(np.float32)
    f[3, 2:2 + dim] = 0.01                                       # a head next to nothing: eps decides
    rot = {"base": 900.0, "dims": dims, "scaling": {"factor": 2.5}}
    freq = dev(be, OS.frequencies(rot) if dims else [0.0])
    pos = rng.permutation(60)[:rows]
    table = rng.permutation(70)[:60].astype(np.int32)[None, :]
    scale = rng.uniform(0.2, 2, heads).astype(np.float32)
    q = torch.zeros((rows, heads * dim), dtype=dtype, device=be.device)
    kc = torch.zeros((70, page, kv_heads, dim), dtype=dtype, device=be.device)
    vc = torch.zeros((70, page, kv_heads, vdim), dtype=dtype, device=be.device)
    qo, ko, vo = 2, 2 + heads * dim, 2 + (heads + kv_heads) * dim
    be.ext.kv_rot_append(be.t(f), ld, qo, ko, vo, q, be.t(scale), kc, vc, None, None, freq, 1.0, dims, freq, False, False,
                         ints(be, np.zeros(rows)), ints(be, pos), be.t(table), page, 0, rows, heads, kv_heads, dim, vdim, head_norm_eps=eps)
    turn = (lambda v, p: OS.turn(v, p, rot)) if dims else (lambda v, p: v)
    gq, gk, gv = be.n(q.float()).reshape(rows, heads, dim), be.n(kc.float()), be.n(vc.float())
    tol = 1e-5 if dtype is F32 else 1e-2
    for r in range(rows):
        p, at = int(pos[r]), (table[0, pos[r] // page], pos[r] % page)
        for h in range(heads):
            assert close(gq[r, h], OS.rms(turn(f[r, qo + h * dim:qo + (h + 1) * dim].astype(np.float64), p), eps) * scale[h], tol), (r, h)
        for g in range(kv_heads):
            assert close(gk[at][g], OS.rms(turn(f[r, ko + g * dim:ko + (g + 1) * dim].astype(np.float64), p), eps), tol), (r, g)
            assert close(gv[at][g], f[r, vo + g * vdim:vo + (g + 1) * vdim].astype(np.float64), tol), (r, g)


@pytest.mark.parametrize("dtype,heads,kv_heads,dim,vdim,window,keep,page", [
    (F32, 4, 2, 10, 7, 13, 5, 8), (F32, 1, 1, 8, 8, 1, 1, 4), (F32, 2, 2, 16, 24, 300, 40, 64), (F32, 2, 1, 6, 6, 30, 0, 8), (F32, 2, 1, 6, 6, 3, 400, 8),
    (BF16, 4, 2, 24, 20, 70, 4, 16), (BF16, 6, 2, 64, 64, 40, 6, 16), (BF16, 4, 4, 32, 32, 90, 130, 32), (BF16, 3, 1, 64, 80, 65, 7, 64),
    (BF16, 4, 2, 64, 96, 20, 64, 12), (BF16, 2, 1, 128, 128, 1 << 30, 3, 16), (BF16, 2, 1, 64, 32, 1, 2, 64), (BF16, 2, 2, 128, 96, 64, 1, 16),
    (BF16, 20, 1, 64, 64, 33, 17, 16)])
def test_window_with_kept_first_tokens(be, dtype, heads, kv_heads, dim, vdim, window, keep, page):
    """random caches; rows inside, at and past the window, at and past the kept tokens: the row kernel, and for the sizes it takes the
    tile kernel (tiles of 1 .. 64 positions that start anywhere) and the decode kernel with and without split keys"""
    rng = np.random.default_rng(heads * 100 + dim + window % 1000)
    T = 210
    pages = -(-T // page)
    table = rng.permutation(pages + 3)[:pages].astype(np.int32)[None, :]
    rnd = lambda *s: OS.bf16_round(rng.standard_normal(s)) if dtype is BF16 else rng.standard_normal(s).astype(np.float32)
    kc, vc = rnd(pages + 3, page, kv_heads, dim), rnd(pages + 3, page, kv_heads, vdim)
    K, V = (np.concatenate([c[i] for i in table[0]])[:T].astype(np.float64) for c in (kc, vc))
    pos = np.arange(T)
    q = rnd(T, heads, dim) * np.float32(1.5 / math.sqrt(dim))
    q = OS.bf16_round(q) if dtype is BF16 else q
    mask = {"size": window, "keep_first": keep}
    picked = sorted({0, 1, 2, 5, T - 1, T // 2, *[p for e in (window, keep, window + keep, page) for p in (e - 2, e - 1, e, e + 1) if 0 <= p < T],
                     *rng.integers(0, T, 12).tolist()})

    def want_row(p):
        js = OS.visible(p, mask)
        return np.concatenate([OS.softmax(K[js][:, h // (heads // kv_heads)] @ q[p, h].astype(np.float64)) @ V[js][:, h // (heads // kv_heads)]
                               for h in range(heads)])
    want = {p: want_row(p) for p in picked}
    qd = dev(be, q, dtype).view(T, heads * dim)
    vf = torch.zeros((max(vdim // 2, 1),), dtype=F32, device=be.device)
    common = (qd, dev(be, kc, dtype), dev(be, vc, dtype), None, None, None, None, 0, 0, vf, False, False, ints(be, np.zeros(T)), ints(be, pos),
              be.t(table), page, 0)
    tol = 1e-5 if dtype is F32 else 1e-2
    out = torch.zeros((T, heads * vdim), dtype=dtype, device=be.device)
    if not be.is_emu or T * heads * dim < 200000:
        be.ext.window_attn(*common, out, T, heads, kv_heads, dim, vdim, window, keep=keep)
        got = be.n(out.float())
        assert all(close(got[p], want[p], tol) for p in picked), [p for p in picked if not close(got[p], want[p], tol)]
    if not be.ext.window_attn_tiles_supported(dtype, dim, vdim):
        return
    cuts, at = [], 0
    for n in (3, 64, 1, 2, 50, 64, 64):
        n = min(n, T - at)
        if n > 0:
            cuts.append((at, n))
        at += n
    out = torch.zeros((T, heads * vdim), dtype=BF16, device=be.device)
    be.ext.window_attn_tiles(*common, out, (ints(be, [c[0] for c in cuts]), ints(be, [c[1] for c in cuts]), len(cuts)), 64, heads, kv_heads, dim, vdim,
                             window, keep=keep)
    got = be.n(out.float())
    assert all(close(got[p], want[p], tol) for p in picked), [p for p in picked if not close(got[p], want[p], tol)]
    for nsplit in (1, 3):
        out = torch.zeros((T, heads * vdim), dtype=BF16, device=be.device)
        part = dict(part_o=torch.full((T, heads, nsplit, vdim), float("nan"), dtype=F32, device=be.device),
                    part_ml=torch.full((T, heads, nsplit, 2), float("nan"), dtype=F32, device=be.device)) if nsplit > 1 else {}
        be.ext.window_attn_tiles(*common, out, (ints(be, picked), None, len(picked)), 1, heads, kv_heads, dim, vdim, window, nsplit=nsplit, keep=keep, **part)
        got = be.n(out.float())
        assert all(close(got[p], want[p], tol) for p in picked), (nsplit, [p for p in picked if not close(got[p], want[p], tol)])


def test_impossible_variants_are_refused(be):
    t = torch.zeros((4, 8), dtype=F32, device=be.device)
    i = ints(be, np.zeros(4))
    bt = ints(be, np.zeros((1, 2)))
    cache = torch.zeros((2, 4, 1, 8), dtype=F32, device=be.device)
    with pytest.raises(Exception, match="kept first tokens"):
        be.ext.window_attn(t, cache, cache, None, None, None, None, 0, 0, t, False, False, i, i, bt, 4, 0, t, 4, 1, 1, 8, 8, 5, chunk=3, keep=2)
    with pytest.raises(Exception, match="normed heads"):
        be.ext.kv_rot_append(t, 24, 0, 8, 16, t, t, cache, cache, None, None, t, 1.0, 8, t, True, False, i, i, bt, 4, 0, 1, 1, 1, 8, 8, head_norm_eps=1e-5)
    with pytest.raises(Exception, match="split"):
        be.ext.dense_linear_split(t, t, None, t, t, 4, 0)


# ---- the recurrence ------------------------------------------------------------------------------------------------------------------


def token_steps():
    """unequal portions of two sequences in slots 0 and 2: single tokens, two tokens, spans longer than a staged batch of tokens"""
    return [[(0, 2), (2, 1)], [(2, 40), (0, 1)], [(0, 1)], [(0, 5), (2, 3)], [(2, 1)], [(0, 1), (2, 1)], [(2, 70), (0, 33)], [(0, 32), (2, 1)]]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("heads,kv_heads,N,P", [(4, 2, 5, 7), (2, 2, 64, 20), (1, 1, 128, 64), (3, 1, 40, 33), (2, 1, 250, 12), (2, 1, 1, 1)])
def test_delta_rule_with_a_decay_per_channel(be, dtype, heads, kv_heads, N, P):
    """token by token and over spans, through both kernels by turns on the same slots (stale state in a slot that starts anew);
    channels that forget at once beside channels that keep everything"""
    rng = np.random.default_rng(N)
    ldf, ldc, ldd = heads + 3, 2 * kv_heads * N + heads * P + 2, heads * (N + P) + 5
    nw = OS.bf16_round(1 + 0.2 * rng.standard_normal(P))
    state = torch.full((3, heads, N, P), 5.0, dtype=F32, device=be.device)
    S, n_tok, eps = {0: np.zeros((heads, N, P)), 2: np.zeros((heads, N, P))}, {0: 0, 2: 0}, 1e-4
    for turn, step in enumerate(token_steps()):
        lens = [n for _s, n in step]
        rows = sum(lens)
        f, c = rng.standard_normal((rows, ldf)).astype(np.float32), rng.standard_normal((rows, ldc)).astype(np.float32)
        d = rng.uniform(0, 1, (rows, ldd)).astype(np.float32)
        g = d[:, 2:2 + heads * N].reshape(rows, heads, N)
        g[:, :, 0] = 1.0
        if N > 2:
            g[:, :, 1] = 1e-6
            g[:, :, 2:] = 1 - 0.05 * g[:, :, 2:]
        seq = np.concatenate([[s] * n for s, n in step])
        pos = np.concatenate([np.arange(n_tok[s], n_tok[s] + n) for s, n in step])
        out = torch.zeros((rows, heads * P), dtype=dtype, device=be.device)
        o_raw = torch.zeros((rows, heads * P), dtype=F32, device=be.device) if turn % 3 != 1 else None
        be.ext.gated_scan(be.ext.SCAN_DELTA_CHANNELS, be.t(f), ldf, 0, kv_heads * N, be.t(c), ldc, 2 * kv_heads * N, be.t(nw), out, state,
                          spans_of(be, lens), ints(be, seq), ints(be, pos), heads, kv_heads, N, P, eps, q_scale=N ** -0.5, beta_off=1,
                          qk=be.t(c), ldqk=ldc, decay=be.t(d), ld_decay=ldd, decay_off=2, ready_gate_off=2 + heads * N, o_raw=o_raw)
        got, r = be.n(out.float()), 0
        for s, n in step:
            for _ in range(n):
                cr = c[r].astype(np.float64)
                for h in range(heads):
                    j = h // (heads // kv_heads)
                    q, k = cr[j * N:(j + 1) * N], cr[(kv_heads + j) * N:(kv_heads + j + 1) * N]
                    v = cr[2 * kv_heads * N + h * P:2 * kv_heads * N + (h + 1) * P]
                    S[s][h], o = OS.delta_step(S[s][h], OS.unit(q) * N ** -0.5, OS.unit(k), v, float(OS.sigmoid(f[r, 1 + h])), g[r, h].astype(np.float64))
                    want = OS.rms(o, eps) * nw * d[r, 2 + heads * N + h * P:2 + heads * N + (h + 1) * P]
                    assert close(got[r, h * P:(h + 1) * P], want, 5e-5 if dtype is F32 else 1e-2), (turn, r, h)
                n_tok[s] += 1
                r += 1
        for s in (0, 2):
            if n_tok[s]:
                assert close(be.n(state)[s], S[s], 2e-5), (turn, s)
    assert (be.n(state)[1] == 5.0).all()


# ---- whole models -----------------------------------------------------------------------------------------------------------------------

CONFIGS = {
    # dense, sparse and no feed-forward; a shared expert in two slabs / of another width / none; two layers of four gone through twice
    "mixed": lambda: OS.small_config([
        OS.layer(None, None, OS.dense_spec()),
        OS.layer(OS.left_spec(heads=3, kv_heads=1, dim=10, vdim=6, dims=10, size=12, keep=1), OS.right_spec(heads=2, kv_heads=2, conv=4), OS.moe_spec()),
        OS.layer(OS.left_spec(heads=2, kv_heads=2, dim=8, vdim=14, dims=4, size=5, keep=7), OS.right_spec(heads=6, kv_heads=2, dim=12, vdim=5, conv=2),
                 OS.moe_spec(experts=6, top=2, ff=10, shared=13)),
        OS.layer(None, OS.right_spec(conv=1), None)], loop=(1, 3, 2)),
    # odd sizes, one head, one tap, window 1, nothing kept, every expert chosen, no shared expert, no loop, factor 1
    "odd": lambda: OS.small_config([
        OS.layer(OS.left_spec(heads=1, kv_heads=1, dim=7, vdim=5, dims=6, size=1, keep=0, factor=1.0), OS.right_spec(heads=1, kv_heads=1, dim=3, vdim=1, conv=1),
                 OS.moe_spec(experts=3, top=3, ff=5, shared=5)),
        OS.layer(OS.left_spec(heads=5, kv_heads=5, dim=4, vdim=3, dims=2, size=3, keep=2), OS.right_spec(heads=3, kv_heads=1, dim=9, vdim=6, conv=7), OS.dense_spec(ff=7, limit=0.3)),
        OS.layer(None, None, OS.moe_spec(experts=1, top=1, ff=9, shared=0))], width=30, vocab=50, mult=1.0, loop=None),
    # the whole stack three times; sizes of the matrix-core kernels
    "wide": lambda: OS.small_config([
        OS.layer(OS.left_spec(heads=6, kv_heads=2, dim=32, vdim=32, dims=16, size=33, keep=5), OS.right_spec(heads=4, kv_heads=2, dim=64, vdim=32, conv=4), OS.dense_spec(ff=72)),
        OS.layer(OS.left_spec(heads=4, kv_heads=4, dim=64, vdim=80, dims=64, size=40, keep=3), OS.right_spec(heads=2, kv_heads=2, dim=32, vdim=48, conv=3),
                 OS.moe_spec(experts=8, top=2, ff=16, shared=48))],
        width=64, vocab=70, mult=0.4, loop=(0, 2, 3)),
}


def make_engine(be, cfg, W, dtype, max_tokens, page=4, max_seqs=4, graphs=None):
    from exllamav2_amd.config import LayeredConfig
    from exllamav2_amd.engine import Engine
    from exllamav2_amd.layered import LayeredModel
    tensors = {k: be.t(v).to(BF16) for k, v in W.items()}
    model = LayeredModel(LayeredConfig.from_dict_prerms(cfg), device=be.device, dtype=dtype, ext=be.ext).load(tensors)
    return Engine(model, max_tokens=max_tokens, max_seqs=max_seqs, page_size=page, graphs=graphs)


def run_cuts(be, eng, rid, tokens, cuts):
    out, at = [], 0
    for c in cuts:
        out.append(be.n(eng.step([(rid, tokens[at:at + c], list(range(c)))])))
        at += c
    assert at == len(tokens)
    return np.concatenate(out, 0)


def clear_tokens(cfg, W, n, seed, gap=0.05):
    """n random tokens none of whose router decisions is a close call (so that bfloat16 rounding cannot pick another expert); grown token
    by token: a token whose routing is a close call is replaced by the next draw"""
    import copy
    rng = np.random.default_rng(seed)
    o = OS.Oracle(cfg, W)
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
    W = OS.random_model(cfg, seed=1)
    toks = clear_tokens(cfg, W, 23, 2)
    want = OS.Oracle(cfg, W).feed("a", toks)
    got = run_cuts(be, make_engine(be, cfg, W, dtype, 32), "a", toks, [23])
    assert ok(got, want, dtype), pos_errs(got, want)


def test_residual_stream_after_every_layer_run(be):
    """the oracle's stream behind the last layer of a stack against the model's, for stacks of one layer up to all of them, gone through
    once, twice and three times"""
    cfg = CONFIGS["mixed"]()
    cfg["loop"] = {"start": 0, "stop": 4, "times": 1}
    W = OS.random_model(cfg, seed=31)
    toks = [int(t) for t in np.random.default_rng(32).integers(0, cfg["vocab"], size=9)]
    for times in (1, 2, 3):
        for depth in range(1, 5):
            sub = dict(cfg, layers=cfg["layers"][:depth], loop={"start": 0, "stop": depth, "times": times})
            trail = []
            OS.Oracle(sub, W).feed("a", toks, residuals=trail)
            Ws = dict(W)
            Ws["final.norm"] = np.ones(cfg["width"], dtype=np.float32)
            Ws["head"] = np.concatenate([np.eye(cfg["width"], dtype=np.float32),
                                         np.zeros((cfg["vocab"] - cfg["width"], cfg["width"]), dtype=np.float32)])      # logits = the normed stream
            got = run_cuts(be, make_engine(be, sub, Ws, F32, 16), "a", toks, [9])[:, :cfg["width"]]
            want = np.array([OS.rms(trail[t][-1], cfg["norm"]["eps"]) for t in range(9)])
            assert close(got, want, 2e-5), (times, depth)


@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 3, 2), (2, 3, 4), (1, 2, 3), (1, 1, 2)])
def test_loops_anywhere(be, loop):
    """no loop, one pass, the whole stack, the last layer only, one layer in the middle, an empty run: whole prompt and decoding"""
    cfg = CONFIGS["mixed"]()
    cfg["layers"] = cfg["layers"][:3]
    cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]} if loop else None
    W = OS.random_model(cfg, seed=33)
    toks = list(np.random.default_rng(34).integers(0, cfg["vocab"], size=17))
    want = OS.Oracle(cfg, W).feed("a", toks)
    for cuts in ([17], [6, 2, 3] + [1] * 6):
        assert rel_err(run_cuts(be, make_engine(be, cfg, W, F32, 20), "a", toks, cuts), want) <= TOL[F32], cuts


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_decoding_and_portions(be, name):
    """the same positions through a whole prompt, token by token from the first token on (the convolutions' tails, every pass's keys and
    the recurrent states pass over decoded tokens), and in portions down to two tokens that end inside pages"""
    cfg = CONFIGS[name]()
    W = OS.random_model(cfg, seed=3)
    toks = list(np.random.default_rng(4).integers(0, cfg["vocab"], size=26))
    want = OS.Oracle(cfg, W).feed("a", toks)
    plans = ([1] * 26, [2, 3, 2, 5, 2, 1, 1, 4, 2, 2, 2], [9] + [1] * 17, [25, 1], [1, 25])
    for cuts in plans[1:2] + plans[3:] if be.is_emu and name == "wide" else plans:
        eng = make_engine(be, cfg, W, F32, 28, page=4)
        assert rel_err(run_cuts(be, eng, "a", toks, cuts), want) <= TOL[F32], cuts


def test_mixed_batches_reuse_pages_and_slots(be):
    """five unequal requests over four slots and a pool smaller than their sum: portions beside single tokens, a request left out of
    a step, finished requests' pages and slot (with its tails, every pass's keys and its recurrent state) taken by the next; every
    position equals the request alone"""
    cfg = CONFIGS["mixed"]()
    W = OS.random_model(cfg, seed=5)
    rng = np.random.default_rng(6)
    reqs = {r: list(rng.integers(0, cfg["vocab"], size=n)) for r, n in (("a", 13), ("b", 5), ("c", 9), ("d", 2), ("e", 11))}
    oracle = OS.Oracle(cfg, W)
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
    W = OS.random_model(cfg, seed=15)
    rng = np.random.default_rng(16)
    eng = make_engine(be, cfg, W, F32, max_tokens=16, page=4, max_seqs=1)
    for r, n, cuts in (("a", 14, [14]), ("b", 9, [1, 1, 7]), ("c", 12, [2, 10])):
        toks = list(rng.integers(0, cfg["vocab"], size=n))
        want = OS.Oracle(cfg, W).feed(r, toks)
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
    W = OS.random_model(cfg, seed=21)
    reqs = {r: clear_tokens(cfg, W, n, 22 + i) for i, (r, n) in enumerate((("a", 14), ("b", 9), ("c", 8)))}
    oracle = OS.Oracle(cfg, W)
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
    W = OS.random_model(cfg, seed=41)
    reqs = {"a": clear_tokens(cfg, W, 12, 42), "b": clear_tokens(cfg, W, 160, 43)}
    oracle = OS.Oracle(cfg, W)
    want = {r: oracle.feed(r, t) for r, t in reqs.items()}
    eng = make_engine(be, cfg, W, BF16, max_tokens=256, page=16, graphs=True)
    plan = [([("a", i, i + 1)], []) for i in range(5)] + [([("b", 0, 139), ("a", 5, 6)], [])]
    plan += [([("a", i, i + 1), ("b", 133 + i, 134 + i)], []) for i in range(6, 12)] + [([("b", 145, 160)], [])]
    got = drive(be, eng, reqs, plan)
    for r in reqs:
        assert ok(got[r], want[r], BF16), (r, pos_errs(got[r], want[r]))
    eng.close()


def test_head_sizes_of_a_real_model_bf16_and_f32(be):
    """sizes at which every tuned kernel path is taken (window tiles of 128 and split keys, full-state column scans, the vector residual step,
    grouped expert launches with a shared expert among them): a prompt in portions, then decoding, beside a second request"""
    if be.is_emu:
        pytest.skip("minutes on the CPU twin; the small configurations cover its logic")
    for dtype in (F32, BF16):
        # (bfloat16 without routers: at this depth a rounded input tips a close choice now and then, which later positions remember)
        ff = OS.moe_spec(experts=8, top=2, ff=64, shared=128) if dtype is F32 else OS.dense_spec(ff=320, limit=2.0)
        cfg = OS.small_config([
            OS.layer(OS.left_spec(heads=8, kv_heads=2, dim=128, vdim=128, dims=128, size=1000, keep=4, base=500000.0),
                     OS.right_spec(heads=4, kv_heads=2, dim=128, vdim=128, conv=4), ff),
            OS.layer(OS.left_spec(heads=4, kv_heads=4, dim=64, vdim=64, dims=32, size=90, keep=9, base=500000.0),
                     OS.right_spec(heads=4, kv_heads=4, dim=64, vdim=64, conv=4), ff)],
            width=256, vocab=300, mult=0.5, loop=(0, 2, 2))
        W = OS.random_model(cfg, seed=61, ranks=(24, 16))
        rng = np.random.default_rng(62)
        reqs = {"a": list(rng.integers(0, 300, 420)), "b": list(rng.integers(0, 300, 20))}
        oracle = OS.Oracle(cfg, W)
        want = {r: oracle.feed(r, t) for r, t in reqs.items()}
        plan = [([("a", 0, 70)], []), ([("a", 70, 405), ("b", 0, 9)], []), ([("a", 405, 407), ("b", 9, 10)], [])]
        plan += [([("a", 407 + i, 408 + i), ("b", 10 + i, 11 + i)], []) for i in range(10)] + [([("a", 417, 420)], [])]
        eng = make_engine(be, cfg, W, dtype, max_tokens=1024, page=64, graphs=True)
        got = drive(be, eng, reqs, plan)
        for r in reqs:
            e = pos_errs(got[r], want[r])
            assert e.max() <= TOL[F32] if dtype is F32 else (np.median(e) <= 3e-2 and e.max() <= 8e-2), (r, dtype, np.sort(e)[-20:])
        eng.close()


def crafted_model(window, keep, seed=31, gain=14.0):
    """one layer whose attention is made so that token 0's query matches token 1's key and nothing else: queries read inputs 0-3, keys
    inputs 4-7 through the same matrix (plus one input that keeps every head's norm from being decided by nothing), values the other
    inputs; token 0 is marked in inputs 0-3, token 1 in 4-7, all other tokens are zero there; no rotation to speak of.  Wherever a token 1
    stands in front of token 0 in sight, however far, that key takes the softmax among hundreds."""
    cfg = OS.small_config([OS.layer(OS.left_spec(heads=2, kv_heads=1, dim=10, vdim=8, dims=2, size=window, keep=keep, base=1e30, factor=1.0, scale=gain / 10),
                                    OS.right_spec(heads=1, kv_heads=1, dim=2, vdim=2, conv=1), OS.dense_spec(ff=8))], width=16, vocab=40, loop=None)
    W = OS.random_model(cfg, seed=seed)
    rng = np.random.default_rng(seed + 1)
    E = W["embed"]
    E[:, :8] = 0.0
    E[:, 8] = 1.0
    mark = rng.standard_normal(4)
    mark *= 6.0 / np.linalg.norm(mark)
    E[0, :4], E[1, 4:8] = mark, mark
    W["embed"] = OS.bf16_round(E)
    W["embed.norm"][:] = 1.0
    W["l0.norm1"][:] = 1.0
    M = rng.standard_normal((10, 4))
    M[[0, 1, 8, 9]] = 0.0                                        # (the turned pair stays empty; two values take the constant input)
    x = "l0.mix.left"
    W[x + ".q"], W[x + ".k"] = np.zeros((20, 16), dtype=np.float32), np.zeros((10, 16), dtype=np.float32)
    W[x + ".q"][:10, :4] = W[x + ".q"][10:, :4] = W[x + ".k"][:, 4:8] = OS.bf16_round(M)
    W[x + ".q"][[8, 18], 8] = 0.25
    W[x + ".k"][9, 8] = 0.25
    W[x + ".v"][:, :9] = 0.0
    W[x + ".v"] = OS.bf16_round(W[x + ".v"] * 4)
    return cfg, W


def marked(rng, cfg, T, target, query):
    """random tokens with the marked pair at two places, and the same without the key"""
    toks = [int(t) for t in rng.integers(2, cfg["vocab"], size=T)]
    toks[target], toks[query] = 1, 0
    base = list(toks)
    base[target] = 2
    return toks, base


@pytest.mark.parametrize("page", [4, 64])
def test_a_marked_key_far_back_and_at_page_borders(be, page):
    """whole prompt, portions and decoding: the marked key sits right in front of the query, at the sequence's first token, on both
    sides of a page border and hundreds of tokens back; where it stands it decides the query's logits"""
    cfg, W = crafted_model(400, 2)
    rng = np.random.default_rng(page)
    T = 330
    query = T - 1
    changes = 0
    for target in (0, 1, page - 1, page, 2 * page, 200, query - page, query - 1):
        toks, base = marked(rng, cfg, T, target, query)
        want = OS.Oracle(cfg, W).feed("t", toks)
        other = OS.Oracle(cfg, W).feed("t", base)[-1]
        changes += rel_err(want[-1:], other[None]) > 0.05
        plans = [[T], [target + 1, T - target - 2, 1], [T - 3, 2, 1], [T - 20] + [1] * 20]
        for cuts in plans if target in (0, 200) else plans[2:3]:
            eng = make_engine(be, cfg, W, F32, max_tokens=T + page, page=page)
            got = run_cuts(be, eng, "t", toks, [c for c in cuts if c > 0])
            assert rel_err(got[-4:], want[-4:]) <= TOL[F32], (target, cuts[:3])
    assert changes >= 7


@pytest.mark.parametrize("window,keep", [(1, 0), (2, 1), (16, 3), (21, 0), (64, 5), (9, 40)])
def test_a_marked_key_at_the_window_edge_and_among_the_kept(be, window, keep):
    """the marked key at the last place the window reaches, one in front of it, at the last kept token and right behind the kept ones, in a
    prompt, at a portion's start and decoded token by token: in sight it decides the logits, out of sight nothing of it is left (but for
    what the recurrence remembers)"""
    cfg, W = crafted_model(window, keep)
    W["l0.mix.right.out"][:] = 0.0                               # (the recurrence beside it is silent)
    rng = np.random.default_rng(window)
    T = window + keep + 30
    query = T - 1
    for target in sorted({query - window + 1, query - window, keep - 1, keep, 0} - {query, -1}):
        toks, base = marked(rng, cfg, T, target, query)
        want, other = OS.Oracle(cfg, W).feed("t", toks), OS.Oracle(cfg, W).feed("t", base)
        assert (rel_err(want[-1:], other[-1:]) > 0.05) == (query - target < window or target < keep), target
        for cuts in ([T], [T - 1, 1], [max(target, 1), T - max(target, 1)], [T - 25] + [1] * 25):
            for dtype in (F32, BF16) if cuts[0] != max(target, 1) else (F32,):
                eng = make_engine(be, cfg, W, dtype, max_tokens=T + 8, page=8)
                got = run_cuts(be, eng, "t", toks, [c for c in cuts if c > 0])
                assert rel_err(got[-3:], want[-3:]) <= (TOL[F32] if dtype is F32 else 5e-2), (target, cuts[:3], dtype)


@pytest.mark.parametrize("dims", [(64, 64), (64, 80)])
def test_marked_keys_through_the_matrix_core_kernels(be, dims):
    """the same at head sizes of the tile kernels in bfloat16: the last token the window shows, the one behind it, kept tokens and the first
    one behind them; prompts of several tiles and decoded tokens"""
    window, keep = 70, 6
    cfg, W = crafted_model(window, keep)
    dim, vdim = dims
    le = cfg["layers"][0]["mixer"]["left"]
    le.update(dim=dim, vdim=vdim, scale=14.0 / dim)
    rng = np.random.default_rng(dim + vdim)
    x = "l0.mix.left"
    old = {n: W[f"{x}.{n}"] for n in ("q", "k")}
    W[x + ".q"], W[x + ".k"] = np.zeros((2 * dim, 16), dtype=np.float32), np.zeros((dim, 16), dtype=np.float32)
    W[x + ".k"][:10] = old["k"]
    for h in range(2):
        W[x + ".q"][h * dim:h * dim + 10] = old["q"][h * 10:h * 10 + 10]
    W[x + ".v"] = OS.bf16_round(rng.standard_normal((vdim, 16)))
    W[x + ".v"][:, :9] = 0.0
    W[x + ".o"] = OS.bf16_round(rng.standard_normal((16, 2 * vdim)) / math.sqrt(2 * vdim))
    W["l0.mix.right.out"][:] = 0.0
    T = 190
    query = T - 1
    for target in (query - window + 1, query - window, keep - 1, keep):
        toks, base = marked(rng, cfg, T, target, query)
        want, other = OS.Oracle(cfg, W).feed("t", toks), OS.Oracle(cfg, W).feed("t", base)
        assert (rel_err(want[-1:], other[-1:]) > 0.05) == (query - target < window or target < keep), target
        for cuts in ([T], [T - 1, 1], [100, 88, 2], [T - 8] + [1] * 8):
            got = run_cuts(be, make_engine(be, cfg, W, BF16, max_tokens=T + 64, page=64), "t", toks, cuts)
            assert rel_err(got[-1:], want[-1:]) <= 4e-2, (target, cuts[:3])


def test_the_state_carries_a_far_token(be):
    """a token 300 positions back reaches the last position of a layer with a window of three only through the recurrent state: changing
    it changes the logits, and portions and decoding carry it like the whole prompt does"""
    cfg = OS.small_config([OS.layer(OS.left_spec(heads=2, kv_heads=1, dim=8, vdim=8, dims=4, size=3, keep=0),
                                    OS.right_spec(heads=2, kv_heads=1, dim=48, vdim=8), OS.dense_spec())], width=64, vocab=40, loop=None)
    W = OS.random_model(cfg, seed=51)
    W["l0.mix.right.dt_bias"][:] = -9.0                                            # slow forgetting ..
    W["l0.mix.right.b"] = OS.bf16_round(W["l0.mix.right.b"] * 0.1)
    rng = np.random.default_rng(52)
    toks = [int(t) for t in rng.integers(0, 4, size=310)]                          # .. and few keys that would write over the first ones
    toks[9] = 30
    other = list(toks)
    other[9] = 31
    want = OS.Oracle(cfg, W).feed("a", toks)
    assert rel_err(OS.Oracle(cfg, W).feed("a", other)[-1:], want[-1:]) > 1e-3
    for cuts in ([310], [100, 2, 65, 143], [290] + [1] * 20):
        eng = make_engine(be, cfg, W, F32, max_tokens=320, page=16)
        assert rel_err(run_cuts(be, eng, "a", toks, cuts)[-8:], want[-8:]) <= 2 * TOL[F32], cuts


def test_long_decoding_bf16(be):
    cfg = CONFIGS["mixed"]()
    W = OS.random_model(cfg, seed=7)
    toks = clear_tokens(cfg, W, 60, 8)
    want = OS.Oracle(cfg, W).feed("a", toks)
    eng = make_engine(be, cfg, W, BF16, 64, page=8)
    got = run_cuts(be, eng, "a", toks, [3] + [1] * 57)
    assert ok(got, want, BF16), pos_errs(got, want)


def test_greedy_generation_through_the_generator(be):
    from exllamav2_amd.engine import Generator
    cfg = CONFIGS["mixed"]()
    W = OS.random_model(cfg, seed=9)
    rng = np.random.default_rng(10)
    prompts = [list(map(int, rng.integers(0, cfg["vocab"], size=n))) for n in (7, 3, 5, 4, 6)]
    eng = make_engine(be, cfg, W, F32, max_tokens=64, page=4, max_seqs=3)
    out = Generator(eng, chunk=3).generate(prompts, 6)
    oracle = OS.Oracle(cfg, W)
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
    W = OS.random_model(cfg, seed=11)
    save_file({k: torch.from_numpy(np.asarray(v)).to(BF16) for k, v in W.items()}, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert read_config(str(tmp_path))[0] == "Savenex"
    model = load_model(str(tmp_path), device=be.device, dtype=F32, ext=be.ext)
    toks = [1, 5, 9, 2, 2, 7]
    got = be.n(Engine(model, 16, page_size=4).step([("x", toks, list(range(6)))]))
    assert rel_err(got, OS.Oracle(cfg, W).feed("x", toks)) <= TOL[F32]


def test_a_delta_rule_with_a_linear_of_its_own(be):
    """the mixer outside a joined layer: its own linear brings everything, the result is the same"""
    from exllamav2_amd.linear_attn import GatedDeltaRule
    cfg = CONFIGS["mixed"]()
    W = OS.random_model(cfg, seed=17)
    eng = make_engine(be, cfg, W, F32, 16)
    model, r = eng.model, cfg["layers"][0]["mixer"]["right"]
    alone = GatedDeltaRule(model, "x", (0, "right"), heads=r["heads"], kv_heads=r["kv_heads"], dim=r["dim"], vdim=r["vdim"], taps=r["conv"],
                           channel_decay=True).load(lambda n, optional=False: dev(be, W["l0.mix.right." + n]))
    h = np.random.default_rng(18).standard_normal((6, cfg["width"])).astype(np.float32)
    from exllamav2_amd.layered import StepBatch
    slot = eng.pool.open()
    eng.pool.extend(slot, 6)
    batch = StepBatch(ints(be, np.zeros(6)), ints(be, np.full(6, slot)), ints(be, np.arange(6)), eng.pool.device_table(), ints(be, [0]), 6, 1,
                      spans_dev=spans_of(be, [6]))
    got = be.n(alone.forward(be.t(h), 6, batch, eng.cache))
    W64 = {k: np.asarray(v, dtype=np.float64) for k, v in W.items()}
    mem = {"hq": [], "hk": [], "hv": [], "S": np.zeros((r["heads"], r["dim"], r["vdim"]))}
    want = np.stack([OS.delta_token(W64, "l0.mix.right", r, row.astype(np.float64), mem, cfg["norm"]["eps"]) for row in h])
    assert close(got, want, 3e-5)


def test_bad_configurations_are_refused(be):
    from exllamav2_amd.config import LayeredConfig
    cfg = CONFIGS["mixed"]()
    with pytest.raises(RuntimeError, match="loop"):
        LayeredConfig.from_dict_prerms(dict(cfg, loop={"start": 1, "stop": 9, "times": 2}))
    with pytest.raises(RuntimeError, match="missing key"):
        LayeredConfig.from_dict_prerms({k: v for k, v in cfg.items() if k != "norm"})
    W = OS.random_model(cfg, seed=1)
    with pytest.raises(RuntimeError, match="unknown mixer"):
        make_engine(be, dict(cfg, layers=[dict(cfg["layers"][0], type="nonesuch")], loop=None), W, F32, 16)
    for name, cut, text in (("l0.mix.right.a2", np.s_[:, :-1], "mixer's sizes"), ("loop.in", np.s_[:, :-1], "loop.in"), ("l1.mix.left.out", np.s_[:-1], "model width"),
                            ("l1.mlp.router.b", np.s_[:-1], "biases"), ("l1.mlp.shared.gate", np.s_[:-1], "shared expert")):
        bad = dict(W)
        bad[name] = bad[name][cut]
        with pytest.raises(RuntimeError, match=text):
            make_engine(be, cfg, bad, F32, 16)
    bad = dict(W)
    del bad["l0.mix.right.g2"]
    with pytest.raises(RuntimeError, match="no tensor"):
        make_engine(be, cfg, bad, F32, 16)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_command_replays_steps(tmp_path, dtype):
    """bin/trace_run in a process of its own: steps on standard input, logits files and `done` lines out"""
    if not torch.cuda.is_available():
        pytest.skip("no GPU visible")
    from safetensors.torch import save_file
    cfg = CONFIGS["mixed"]()
    W = OS.random_model(cfg, seed=12)
    mdir = tmp_path / "model"
    mdir.mkdir()
    save_file({k: torch.from_numpy(np.asarray(v)).to(BF16) for k, v in W.items()}, str(mdir / "model.safetensors"))
    (mdir / "config.json").write_text(json.dumps(cfg))
    a, b = clear_tokens(cfg, W, 300, 13), clear_tokens(cfg, W, 9, 14)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:290], "want": [0, 289]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[290:295], "want": []}, {"id": "b", "tokens": b[:8], "want": [7]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[8:], "want": [0]}, {"id": "a", "tokens": a[295:], "want": [4]}], "end": ["a", "b"]}]
    out = tmp_path / "out"
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(mdir), "--dtype", dtype, "--out", str(out), "--max-tokens", "512"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600, cwd=str(tmp_path))
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    oracle = OS.Oracle(cfg, W)
    wa, wb = oracle.feed("a", a), oracle.feed("b", b)
    got = np.concatenate([np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(k, -1) for n, k in ((0, 2), (1, 1), (2, 2))])
    want = np.stack([wa[0], wa[289], wb[7], wb[8], wa[299]])
    e = pos_errs(got, want)
    assert (e.max() <= TOL[F32]) if dtype == "float32" else (np.median(e) <= 2e-2 and e.max() <= 6e-2), e
