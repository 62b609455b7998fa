"""Plain float64 restatement of the Savenex layer stack (pre-norm layers of softmax attention with a sliding window and kept first tokens
beside a delta rule whose decay is per key channel; a run of layers that is gone through several times behind a linear of the stream
and the embedding; clamped dense and chosen-softmax sparse feed-forwards) -- TEST INFRASTRUCTURE ONLY.

One function per mechanism, token by token, written from the equations; nothing is shared with the product path (no pages, no
slots, no batching: a sequence's memory is python lists and per-layer-run arrays).

Notation: W x with W stored [out, in]; p = a token's position (from 0); n(v) = v / sqrt(mean(v^2) + eps); sg = sigmoid; m = residual factor.
    stack:      x0 = n(embed[t]) w_e;  x = x0;  layers in order, the layers start .. stop - 1 gone through `times` times in a row (same
                weights, memory of their own for every pass); in front of EVERY pass  x <- W_in [x; x0]
    layer:      x <- x + m mixer(n(x) w1);  x <- x + m ff(n(x) w2)  (a layer may lack the second)
    mixer:      (n(left(h)) w_l + n(right(h)) w_r) / 2
      left      q, k, v = W h;  the first `dims` values of every q / k head turned in pairs (i, i + dims / 2) by p base^(-2i / dims) / factor;
                q <- n(q), k <- n(k) per head;  s_j = (q . k_j) scale over the j <= p with p - j < size or j < keep_first;  softmax;  W_o heads
      right     q, k, v = silu(conv(W h)) per channel (causal, `conv` taps);  q, k per head / sqrt(sum(.^2) + 1e-6), q also / sqrt(dim);
                beta = sg(W_b h);  g = exp(-exp(A) softplus(W_a2 W_a1 h + b)) per head and key channel;
                S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q;  W_o concat(n(o) w * sg(W_g2 W_g1 h))
    dense:      a = min(W_gate h, L), u = clamp(W_up h, -L, L);  W_down (a sg(1.702 a) (u + 1))
    moe:        z = W_router h + b;  the `top` largest z choose, weights = softmax over the chosen z;  sum_e w_e E_e(h) + sg(W_sg h) E_shared(h),
                E(h) = W_down (silu(W_gate h) * W_up h)
    logits:     head (n(x) w_final)
"""
from __future__ import annotations

import math

import numpy as np


def sigmoid(z):
    z = np.asarray(z, dtype=np.float64)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def rms(v, eps):
    return v / math.sqrt(float((v * v).mean()) + eps)


def unit(v):
    return v / math.sqrt(float((v * v).sum()) + 1e-6)


def softmax(s):
    e = np.exp(s - s.max())
    return e / e.sum()


def frequencies(rot):
    factor = (rot.get("scaling") or {}).get("factor", 1.0)
    return [rot["base"] ** (-2.0 * i / rot["dims"]) / factor for i in range(rot["dims"] // 2)]


def turn(vec, pos, rot):
    out, half = vec.copy(), rot["dims"] // 2
    for i, f in enumerate(frequencies(rot)):
        c, s = math.cos(pos * f), math.sin(pos * f)
        out[i], out[i + half] = vec[i] * c - vec[i + half] * s, vec[i + half] * c + vec[i] * s
    return out


def causal_conv(history, taps_w):
    """history: the inputs up to and including the current token, newest last; the last column weighs the current token"""
    taps = taps_w.shape[1]
    acc = np.zeros(taps_w.shape[0])
    for back in range(min(taps, len(history))):
        acc = acc + taps_w[:, taps - 1 - back] * history[-1 - back]
    return acc


def visible(pos, mask):
    """positions of the keys that position `pos` sees"""
    return [j for j in range(pos + 1) if pos - j < mask["size"] or j < mask["keep_first"]]


def attention_token(W, key, m, h, pos, mem, eps):
    """mem["kv"]: list of (keys, values) of the sequence's tokens"""
    H, G, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = [rms(turn(v, pos, m["rot"]), eps) for v in (W[key + ".q"] @ h).reshape(H, dim)]
    k = np.stack([rms(turn(v, pos, m["rot"]), eps) for v in (W[key + ".k"] @ h).reshape(G, dim)])
    mem["kv"].append((k, (W[key + ".v"] @ h).reshape(G, vd)))
    js = visible(pos, m["mask"])
    K = np.stack([mem["kv"][j][0] for j in js])
    V = np.stack([mem["kv"][j][1] for j in js])
    heads = [softmax(K[:, i // (H // G)] @ q[i] * m["scale"]) @ V[:, i // (H // G)] for i in range(H)]
    return W[key + ".o"] @ np.concatenate(heads)


def channel_decay(z, a_log, heads, dim):
    """z [heads * dim] in front of the softplus, a_log [heads]"""
    return np.exp(-np.exp(a_log)[:, None] * softplus(z).reshape(heads, dim))


def delta_step(S, q, k, v, beta, g):
    """one head, one token: (new state [dim, vdim], read-out [vdim])"""
    S = g[:, None] * S
    u = beta * (v - S.T @ k)
    S = S + np.outer(k, u)
    return S, S.T @ q


def delta_token(W, key, m, h, mem, eps):
    """mem: {"hq" / "hk" / "hv": lists of the last convolution inputs, "S": [heads, dim, vdim]}"""
    H, G, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = {}
    for s in "qkv":
        mem["h" + s] = (mem["h" + s] + [W[f"{key}.{s}"] @ h])[-m["conv"]:]
        conv[s] = silu(causal_conv(mem["h" + s], W[f"{key}.{s}.conv"]))
    q, k, v = conv["q"].reshape(G, dim), conv["k"].reshape(G, dim), conv["v"].reshape(H, vd)
    beta = sigmoid(W[key + ".b"] @ h)
    g = channel_decay(W[key + ".a2"] @ (W[key + ".a1"] @ h) + W[key + ".dt_bias"], W[key + ".A_log"], H, dim)
    gate = sigmoid(W[key + ".g2"] @ (W[key + ".g1"] @ h)).reshape(H, vd)
    out = []
    for i in range(H):
        j = i // (H // G)
        mem["S"][i], o = delta_step(mem["S"][i], unit(q[j]) * dim ** -0.5, unit(k[j]), v[i], beta[i], g[i])
        out.append(rms(o, eps) * W[key + ".norm"] * gate[i])
    return W[key + ".o"] @ np.concatenate(out)


def mixer_token(W, key, m, h, pos, mem, eps):
    left = attention_token(W, key + ".left", m["left"], h, pos, mem, eps)
    right = delta_token(W, key + ".right", m["right"], h, mem, eps)
    return 0.5 * (rms(left, eps) * W[key + ".left.out"] + rms(right, eps) * W[key + ".right.out"])


def clamped_ff(W, key, limit, h):
    a = np.minimum(W[key + ".gate"] @ h, limit)
    u = np.clip(W[key + ".up"] @ h, -limit, limit)
    return W[key + ".down"] @ (a * sigmoid(1.702 * a) * (u + 1.0))


def expert(W, key, h):
    return W[key + ".down"] @ (silu(W[key + ".gate"] @ h) * (W[key + ".up"] @ h))


def route(z, top):
    """([(expert, weight)] of one token, the distance of the closest choice)"""
    order = sorted(range(len(z)), key=lambda e: (-z[e], e))
    gap = float(z[order[top - 1]] - z[order[top]]) if top < len(order) else math.inf
    w = softmax(np.array([z[e] for e in order[:top]]))
    return list(zip(order[:top], w)), gap


def moe_ff(W, key, ms, h):
    picks, gap = route(W[key + ".router"] @ h + W[key + ".router.b"], ms["router"]["top"])
    y = sum(w * expert(W, f"{key}.e{e}", h) for e, w in picks)
    if ms.get("shared"):
        y = y + float(sigmoid(W[key + ".shared.sg"] @ h)[0]) * expert(W, key + ".shared", h)
    return y, gap


def layer_runs(cfg):
    """[(layer, a pass starts in front of it)] in the order they are gone through"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return [(i, False) for i in range(a)] + [(i, i == a) for _ in range(loop["times"]) for i in range(a, b)] + [(i, False) for i in range(b, n)]


class Oracle:
    """feed(seq, tokens) -> logits [len(tokens), vocab] of the sequence's next tokens; state is kept per sequence name"""

    def __init__(self, cfg: dict, weights: dict):
        self.cfg = cfg
        self.W = {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}
        self.runs = layer_runs(cfg)
        self.seqs = {}

    def _new(self):
        mem = []
        for i, _start in self.runs:
            r = self.cfg["layers"][i]["mixer"]["right"]
            mem.append({"kv": [], "hq": [], "hk": [], "hv": [], "S": np.zeros((r["heads"], r["dim"], r["vdim"]))})
        return {"n": 0, "mem": mem}

    def feed(self, seq, tokens, residuals=None, gaps=None):
        """residuals (a list): takes the stream after every layer run per token; gaps (a list): takes every token's smallest router gap"""
        cfg, W, eps, m = self.cfg, self.W, self.cfg["norm"]["eps"], self.cfg["residual_mult"]
        if seq not in self.seqs:
            self.seqs[seq] = self._new()
        st, out = self.seqs[seq], []
        for t in tokens:
            x0 = rms(W["embed"][int(t)], eps) * W["embed.norm"]
            x, trail, gap = x0.copy(), [], math.inf
            for (i, pass_starts), mem in zip(self.runs, st["mem"]):
                spec, key = cfg["layers"][i], f"l{i}"
                if pass_starts:
                    x = W["loop.in"] @ np.concatenate([x, x0])
                x = x + m * mixer_token(W, key + ".mix", spec["mixer"], rms(x, eps) * W[key + ".norm1"], st["n"], mem, eps)
                ms = spec.get("mlp")
                if ms is not None:
                    h = rms(x, eps) * W[key + ".norm2"]
                    if ms["kind"] == "dense":
                        y = clamped_ff(W, key + ".mlp", ms["limit"], h)
                    else:
                        y, gp = moe_ff(W, key + ".mlp", ms, h)
                        gap = min(gap, gp)
                    x = x + m * y
                trail.append(x.copy())
            if residuals is not None:
                residuals.append(np.stack(trail))
            if gaps is not None:
                gaps.append(gap)
            out.append(W["head"] @ (rms(x, eps) * W["final.norm"]))
            st["n"] += 1
        return np.stack(out)

    def drop(self, seq):
        self.seqs.pop(seq, None)


# ---- small random models for the tests ---------------------------------------------------------------------------------------


def bf16_round(a):
    u = np.asarray(a, dtype=np.float32).view(np.uint32)
    return (((u + 0x7fff + ((u >> 16) & 1)) & 0xffff0000).astype(np.uint32)).view(np.float32)


def left_spec(heads=4, kv_heads=2, dim=12, vdim=10, dims=8, size=9, keep=3, base=1000.0, factor=3.0, scale=None):
    return {"dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"keep_first": keep, "size": size},
            "rot": {"base": base, "dims": dims, "scaling": {"factor": factor}}, "scale": scale or dim ** -0.5, "vdim": vdim}


def right_spec(heads=4, kv_heads=2, dim=8, vdim=14, conv=3):
    return {"conv": conv, "dim": dim, "heads": heads, "kv_heads": kv_heads, "vdim": vdim}


def dense_spec(ff=24, limit=1.5):
    return {"ff": ff, "kind": "dense", "limit": limit}


def moe_spec(experts=8, top=3, ff=12, shared=24):
    return {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": experts, "top": top}, "shared": {"ff": shared} if shared else None}


def layer(left=None, right=None, ff=None):
    return {"type": "parallel", "mixer": {"left": left or left_spec(), "right": right or right_spec()}, "mlp": ff}


def small_config(layers, width=32, vocab=61, eps=1e-5, mult=0.6, loop=(0, 2, 2)):
    return {"architecture": "Savenex", "layers": layers, "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]} if loop else None,
            "norm": {"eps": eps}, "residual_mult": mult, "vocab": vocab, "width": width}


def random_model(cfg: dict, seed: int = 0, ranks=(5, 3)) -> dict:
    """name -> float32 array (bfloat16-representable values), shapes from the configuration; ranks = inner sizes of the low-rank pairs
    (decay, output gate)"""
    rng = np.random.default_rng(seed)
    Wd, out = cfg["width"], {}

    def mat(name, o, i, gain=1.0):
        out[name] = bf16_round(rng.standard_normal((o, i)) * gain / math.sqrt(i))

    def vec(name, n, centre=0.0, spread=0.1):
        out[name] = bf16_round(centre + rng.standard_normal(n) * spread)

    out["embed"] = bf16_round(rng.standard_normal((cfg["vocab"], Wd)))
    vec("embed.norm", Wd, 1.0, 0.2)
    if cfg.get("loop"):
        mat("loop.in", Wd, 2 * Wd, 1.3)
    for i, spec in enumerate(cfg["layers"]):
        k, m = f"l{i}", spec["mixer"]
        vec(k + ".norm1", Wd, 1.0)
        x, a = k + ".mix.left", m["left"]
        H, G, dim, vd = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
        mat(x + ".q", H * dim, Wd); mat(x + ".k", G * dim, Wd); mat(x + ".v", G * vd, Wd); mat(x + ".o", Wd, H * vd)
        vec(x + ".out", Wd, 1.0, 0.2)
        x, r = k + ".mix.right", m["right"]
        H, G, dim, vd = r["heads"], r["kv_heads"], r["dim"], r["vdim"]
        for s, n in (("q", G * dim), ("k", G * dim), ("v", H * vd)):
            mat(f"{x}.{s}", n, Wd, 1.5)
            taps = rng.standard_normal((n, r["conv"])) * 0.5
            taps[:, -1] += 0.8
            out[f"{x}.{s}.conv"] = bf16_round(taps)
        mat(x + ".b", H, Wd, 2.0); vec(x + ".A_log", H, -0.5, 0.7); vec(x + ".norm", vd, 1.0, 0.2)
        mat(x + ".a1", ranks[0], Wd); mat(x + ".a2", H * dim, ranks[0], 1.5); vec(x + ".dt_bias", H * dim, -2.0, 1.0)
        mat(x + ".g1", ranks[1], Wd, 1.5); mat(x + ".g2", H * vd, ranks[1], 1.5); mat(x + ".o", Wd, H * vd)
        vec(x + ".out", Wd, 1.0, 0.2)
        ms = spec.get("mlp")
        if ms is None:
            continue
        vec(k + ".norm2", Wd, 1.0)
        f = k + ".mlp"

        def gated(name, ff):
            mat(name + ".gate", ff, Wd, 1.5); mat(name + ".up", ff, Wd, 1.5); mat(name + ".down", Wd, ff, 1.5)
        if ms["kind"] == "dense":
            gated(f, ms["ff"])
        else:
            mat(f + ".router", ms["router"]["experts"], Wd, 2.0); vec(f + ".router.b", ms["router"]["experts"], 0.0, 0.7)
            for e in range(ms["router"]["experts"]):
                gated(f"{f}.e{e}", ms["expert"]["ff"])
            if ms.get("shared"):
                gated(f + ".shared", ms["shared"]["ff"])
                mat(f + ".shared.sg", 1, Wd, 1.5)
    vec("final.norm", Wd, 1.0)
    mat("head", cfg["vocab"], Wd)
    return out
