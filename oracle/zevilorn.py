"""Plain float64 restatement of the Zevilorn layer stack (one norm per layer, mixer and sparse feed-forward side by side behind gates of
their own, a run of layers that is gone through several times; head-mixing window attention with a short convolution, latent
attention with a sink per head, window attention beside a minimal gated recurrence) -- TEST INFRASTRUCTURE ONLY.

One function per mechanism, token by token, written from the equations; nothing is shared with the product path (no pages, no
slots, no batching: a sequence's memory is python lists and per-layer-run arrays).

Notation: W x with W stored [out, in]; p = a token's position (from 0); n(v) = v / sqrt(mean(v^2) + eps); sg = sigmoid.
    stack:      x = embed[t] =: e;  layers in order, the layers start .. stop - 1 gone through `times` times in a row (same weights,
                memory of their own for every pass); in front of every pass but the first  x <- x + e
    layer:      h = n(x) w;  x <- x + mixer(h) * sg(W_rg1 h + b1) + ff(h) * sg(W_rg2 h + b2)        (both read the same h)
    attention:  q, k, v = conv(W h + b) per channel (causal, `conv` taps, no activation);  the first `dims` values of every q / k head
                turned in pairs (2i, 2i + 1);  a_g = c tanh(q_g . k scale / c);  s_h = sum_g T[h, g] a_g over ALL heads;
                weights exp(s_j) / (1 + sum exp(s)) over 0 <= p - j < window;  W_o heads + b_o
    latent:     q = W_uq (n(W_dq h) w_q), per head [dim | rot_dim];  W_dkv h = [c' | k'];  c = n(c') w_kv;  k_r = turned k' (pairs
                (i, i + dims / 2));  s_j = (q_u . W_uk c_j + turned q_r . k_r,j) scale;  weights exp(s_j) / (exp(sink_h) + sum exp(s));
                head output sum_j w_j W_uv c_j * sg(W_g h)_h;  W_o heads
    parallel:   (n(left(h)) w_l + n(right(h)) w_r) / 2
      left      window attention with plain softmax, angles p f_i / factor, pairs (2i, 2i + 1), heads times sg(W_g h)_h
      right     z = sg(W_z h + b_z);  u = W_x h + b_x;  c = u + 1/2 where u >= 0, sg(u) elsewhere;  S <- (1 - z) S + z c;
                W_o (S silu(W_g h))
    moe:        s = sg(W_router h);  the experts stand in `count` equal groups, a group scores the sum of its two largest s, the best
                `keep` groups stay;  the `top` largest s among them choose;  y = sum_e s_e W_down gelu(W_up h), gelu(z) = z Phi(z)
    logits:     head (n(x) w_final)
"""
from __future__ import annotations

import math

import numpy as np


def sigmoid(z):
    z = np.asarray(z, dtype=np.float64)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def gelu(z):
    return np.array([0.5 * v * (1.0 + math.erf(v / math.sqrt(2.0))) for v in np.ravel(z)]).reshape(np.shape(z))


def rms_norm(v, w, eps):
    return v / math.sqrt(float((v * v).mean()) + eps) * w


def frequencies(rot):
    """turns per token (in radians) of every pair, after the configured frequency scaling"""
    f = [rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f
    if "original" not in sc:
        return [v / sc["factor"] for v in f]
    out = []
    for v in f:
        wave = 2.0 * math.pi / v
        if wave < sc["original"] / sc["high"]:
            out.append(v)
        elif wave > sc["original"] / sc["low"]:
            out.append(v / sc["factor"])
        else:
            s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
            out.append((1.0 - s) * v / sc["factor"] + s * v)
    return out


def turn(vec, pos, rot, neighbours):
    """pair i is (2i, 2i + 1) when `neighbours`, else (i, i + dims / 2)"""
    out, half = vec.copy(), rot["dims"] // 2
    for i, f in enumerate(frequencies(rot)):
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + half)
        c, s = math.cos(pos * f), math.sin(pos * f)
        out[a], out[b] = vec[a] * c - vec[b] * s, vec[b] * c + vec[a] * s
    return out


def causal_conv(history, taps_w):
    """history: the inputs up to and including the current token, newest last; taps_w [channels, taps], the last column weighs the
    current token"""
    taps = taps_w.shape[1]
    acc = np.zeros(taps_w.shape[0])
    for j in range(taps):
        back = taps - 1 - j
        if back < len(history):
            acc = acc + taps_w[:, j] * history[len(history) - 1 - back]
    return acc


def softmax_plus(s, extra):
    """exp(s_j) / (exp(extra) + sum exp(s)); extra None: nothing is added to the denominator"""
    m = s.max() if extra is None else max(float(s.max()), extra)
    e = np.exp(s - m)
    return e / (e.sum() + (0.0 if extra is None else math.exp(extra - m)))


def seen(pos, m):
    size = (m.get("mask") or {}).get("size")
    return max(0, pos - size + 1) if size else 0


def talking_attention_token(W, key, m, h, pos, mem):
    """mem: {"kv": list of (keys, values), "hq" / "hk" / "hv": the last projected values}"""
    H, G, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = {}
    for s in "qkv":
        mem["h" + s] = (mem["h" + s] + [W[f"{key}.{s}"] @ h + W[f"{key}.{s}.b"]])[-m["conv"]:]
        conv[s] = causal_conv(mem["h" + s], W[f"{key}.{s}.conv"])
    q = [turn(v, pos, m["rot"], True) for v in conv["q"].reshape(H, dim)]
    k = np.stack([turn(v, pos, m["rot"], True) for v in conv["k"].reshape(G, dim)])
    mem["kv"].append((k, conv["v"].reshape(G, vd)))
    lo = seen(pos, m)
    K = np.stack([kv[0] for kv in mem["kv"][lo:]])
    V = np.stack([kv[1] for kv in mem["kv"][lo:]])
    cap = m["softcap"]
    a = np.stack([cap * np.tanh(K[:, i // (H // G)] @ q[i] * m["scale"] / cap) for i in range(H)])
    s = W[key + ".talk"] @ a
    heads = [softmax_plus(s[i], 0.0) @ V[:, i // (H // G)] for i in range(H)]
    return W[key + ".o"] @ np.concatenate(heads) + W[key + ".o.b"]


def latent_attention_token(W, key, m, h, pos, mem, eps):
    """mem: {"kv": list of (latent, turned shared key part)}"""
    H, dim, rd, vd, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (W[key + ".uq"] @ rms_norm(W[key + ".dq"] @ h, W[key + ".dq.norm"], eps)).reshape(H, dim + rd)
    dkv = W[key + ".dkv"] @ h
    mem["kv"].append((rms_norm(dkv[:R], W[key + ".dkv.norm"], eps), turn(dkv[R:], pos, m["rot"], False)))
    C = np.stack([c for c, _ in mem["kv"]])
    Kr = np.stack([k for _, k in mem["kv"]])
    gate = sigmoid(W[key + ".g"] @ h)
    heads = []
    for i in range(H):
        Ku = C @ W[key + ".uk"][i * dim:(i + 1) * dim].T
        V = C @ W[key + ".uv"][i * vd:(i + 1) * vd].T
        s = (Ku @ q[i, :dim] + Kr @ turn(q[i, dim:], pos, m["rot"], False)) * m["scale"]
        heads.append(softmax_plus(s, float(W[key + ".sink"][i])) @ V * gate[i])
    return W[key + ".o"] @ np.concatenate(heads)


def gated_window_attention_token(W, key, m, h, pos, kv):
    H, G, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = [turn(v, pos, m["rot"], True) for v in (W[key + ".q"] @ h).reshape(H, dim)]
    k = np.stack([turn(v, pos, m["rot"], True) for v in (W[key + ".k"] @ h).reshape(G, dim)])
    kv.append((k, (W[key + ".v"] @ h).reshape(G, vd)))
    lo = seen(pos, m)
    K, V = np.stack([x[0] for x in kv[lo:]]), np.stack([x[1] for x in kv[lo:]])
    gate = sigmoid(W[key + ".g"] @ h)
    heads = []
    for i in range(H):
        g = i // (H // G)
        heads.append(softmax_plus(K[:, g] @ q[i] * m["scale"], None) @ V[:, g] * gate[i])
    return W[key + ".o"] @ np.concatenate(heads)


def mingru_token(W, key, h, mem):
    """mem: {"S": [width]}"""
    z = sigmoid(W[key + ".z"] @ h + W[key + ".z.b"])
    u = W[key + ".x"] @ h + W[key + ".x.b"]
    mem["S"] = (1.0 - z) * mem["S"] + z * np.where(u >= 0, u + 0.5, sigmoid(u))
    g = W[key + ".g"] @ h
    return W[key + ".o"] @ (mem["S"] * g * sigmoid(g))


def parallel_token(W, key, m, h, pos, mem, eps):
    left = gated_window_attention_token(W, key + ".left", m["left"], h, pos, mem["kv"])
    right = mingru_token(W, key + ".right", h, mem)
    return 0.5 * (rms_norm(left, W[key + ".left.out"], eps) + rms_norm(right, W[key + ".right.out"], eps))


def allowed_experts(s, router):
    """indices of the experts whose group is kept"""
    n, gr = router["experts"], router.get("groups")
    if not gr:
        return list(range(n)), math.inf
    size = n // gr["count"]
    score = np.array([np.sort(s[g * size:(g + 1) * size])[::-1][:2].sum() for g in range(gr["count"])])
    order = np.argsort(-score, kind="stable")
    gap = float(score[order[gr["keep"] - 1]] - score[order[gr["keep"]]]) if gr["keep"] < gr["count"] else math.inf
    kept = sorted(order[:gr["keep"]])
    return [g * size + i for g in kept for i in range(size)], gap


def route(s, router):
    """([(expert, weight)] of one token, the smallest distance of a choice)"""
    ok, gap = allowed_experts(s, router)
    order = sorted(ok, key=lambda e: (-s[e], e))
    top = router["top"]
    if top < len(order):
        gap = min(gap, float(s[order[top - 1]] - s[order[top]]))
    return [(int(e), float(s[e])) for e in order[:top]], gap


def moe_ff(W, key, ms, h):
    picks, gap = route(sigmoid(W[key + ".router"] @ h), ms["router"])
    y = np.zeros(W[key + ".e0.down"].shape[0])
    for e, w in picks:
        y += w * (W[f"{key}.e{e}.down"] @ gelu(W[f"{key}.e{e}.up"] @ h))
    return y, gap


def layer_runs(cfg):
    """[(layer, pass, the embedding is added in front)] in the order they are gone through"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, 0, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, 0, False) for i in range(a)]
    for p in range(loop["times"]):
        runs += [(i, p, p > 0 and i == a) for i in range(a, b)]
    return runs + [(i, 0, False) for i in range(b, n)]


class Oracle:
    """feed(seq, tokens) -> logits [len(tokens), vocab] of the sequence's next tokens; state is kept per sequence name"""

    def __init__(self, cfg: dict, weights: dict):
        self.cfg = cfg
        self.W = {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}
        self.runs = layer_runs(cfg)
        self.seqs = {}

    def _new(self):
        mem = []
        for i, _p, _e in self.runs:
            spec = self.cfg["layers"][i]
            st = {"kv": []}
            if spec["type"] == "attention":
                st.update(hq=[], hk=[], hv=[])
            elif spec["type"] == "parallel":
                st.update(S=np.zeros(spec["mixer"]["right"]["width"]))
            mem.append(st)
        return {"n": 0, "mem": mem}

    def feed(self, seq, tokens, residuals=None, gaps=None):
        """residuals (a list): takes the stream after every layer run per token; gaps (a list): takes every token's smallest router gap"""
        cfg, W, eps = self.cfg, self.W, self.cfg["norm"]["eps"]
        st = self.seqs.setdefault(seq, None) or self._new()
        self.seqs[seq] = st
        out = []
        for t in tokens:
            pos = st["n"]
            e = W["embed"][int(t)]
            x = e.copy()
            trail, gap = [], math.inf
            for (i, _pass, add_e), mem in zip(self.runs, st["mem"]):
                spec, key = cfg["layers"][i], f"l{i}"
                m = spec["mixer"]
                if add_e:
                    x = x + e
                h = rms_norm(x, W[key + ".norm1"], eps)
                if spec["type"] == "attention":
                    y = talking_attention_token(W, key + ".mix", m, h, pos, mem)
                elif spec["type"] == "latent_attention":
                    y = latent_attention_token(W, key + ".mix", m, h, pos, mem, eps)
                else:
                    y = parallel_token(W, key + ".mix", m, h, pos, mem, eps)
                x = x + y * sigmoid(W[key + ".rg1"] @ h + W[key + ".rg1.b"])
                if spec.get("mlp") is not None:
                    f, g = moe_ff(W, key + ".mlp", spec["mlp"], h)
                    gap = min(gap, g)
                    x = x + f * sigmoid(W[key + ".rg2"] @ h + W[key + ".rg2.b"])
                trail.append(x.copy())
            if residuals is not None:
                residuals.append(np.stack(trail))
            if gaps is not None:
                gaps.append(gap)
            out.append(W["head"] @ rms_norm(x, W["final.norm"], eps))
            st["n"] += 1
        return np.stack(out)

    def drop(self, seq):
        self.seqs.pop(seq, None)


# ---- small random models for the tests ---------------------------------------------------------------------------------------


def bf16_round(a):
    u = np.asarray(a, dtype=np.float32).view(np.uint32)
    return (((u + 0x7fff + ((u >> 16) & 1)) & 0xffff0000).astype(np.uint32)).view(np.float32)


def talking_mixer(heads=4, kv_heads=2, dim=12, vdim=10, dims=8, window=9, conv=4, softcap=6.0, base=1000.0, scale=None, scaling="wave"):
    sc = {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 96} if scaling == "wave" else scaling
    return {"type": "attention", "mixer": {"conv": conv, "dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"size": window},
                                           "rot": {"base": base, "dims": dims, "scaling": sc}, "scale": scale or dim ** -0.5,
                                           "softcap": softcap, "vdim": vdim}}


def latent_mixer(heads=3, dim=10, rot_dim=8, vdim=14, kv_rank=24, q_rank=20, base=2000.0, scale=None):
    return {"type": "latent_attention", "mixer": {"dim": dim, "heads": heads, "kv_rank": kv_rank, "q_rank": q_rank,
                                                  "rot": {"base": base, "dims": rot_dim}, "rot_dim": rot_dim,
                                                  "scale": scale or (dim + rot_dim) ** -0.5, "vdim": vdim}}


def window_spec(heads=4, kv_heads=2, dim=8, vdim=12, dims=6, window=7, base=800.0, factor=3.0, scale=None):
    return {"dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"size": window},
            "rot": {"base": base, "dims": dims, "scaling": {"factor": factor}}, "scale": scale or dim ** -0.5, "vdim": vdim}


def parallel_mixer(left=None, width=28):
    return {"type": "parallel", "mixer": {"left": left or window_spec(), "right": {"width": width}}}


def moe_ff_spec(experts=8, top=3, ff=12, count=4, keep=2):
    return {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": experts, "groups": {"count": count, "keep": keep}, "top": top}}


def layer(mix, ff=None):
    return dict(mix, mlp=ff)


def small_config(layers, width=32, vocab=61, eps=1e-5, loop=(0, 2, 2)):
    return {"architecture": "Zevilorn", "layers": layers, "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]} if loop else None,
            "norm": {"eps": eps}, "vocab": vocab, "width": width}


def random_model(cfg: dict, seed: int = 0) -> dict:
    """name -> float32 array (bfloat16-representable values), shapes from the configuration"""
    rng = np.random.default_rng(seed)
    Wd, out = cfg["width"], {}

    def mat(name, o, i, gain=1.0):
        out[name] = bf16_round(rng.standard_normal((o, i)) * gain / math.sqrt(i))

    def vec(name, n, centre=0.0, spread=0.1):
        out[name] = bf16_round(centre + rng.standard_normal(n) * spread)

    out["embed"] = bf16_round(rng.standard_normal((cfg["vocab"], Wd)))
    for i, spec in enumerate(cfg["layers"]):
        k, m = f"l{i}", spec["mixer"]
        x = k + ".mix"
        vec(k + ".norm1", Wd, 1.0)
        mat(k + ".rg1", Wd, Wd); vec(k + ".rg1.b", Wd, 0.5, 0.5)
        if spec["type"] == "attention":
            H, G, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for s, n in (("q", H * dim), ("k", G * dim), ("v", G * vd)):
                mat(f"{x}.{s}", n, Wd, 1.0 if s == "v" else 2.0); vec(f"{x}.{s}.b", n, 0.0, 0.3)
                taps = rng.standard_normal((n, m["conv"])) * 0.5
                taps[:, -1] += 0.8
                out[f"{x}.{s}.conv"] = bf16_round(taps)
            out[x + ".talk"] = bf16_round(np.eye(H) + rng.standard_normal((H, H)) * 0.4)
            mat(x + ".o", Wd, H * vd, 1.5); vec(x + ".o.b", Wd, 0.0, 0.3)
        elif spec["type"] == "latent_attention":
            H, dim, rd, vd, R, Q = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
            mat(x + ".dq", Q, Wd); vec(x + ".dq.norm", Q, 1.0); mat(x + ".uq", H * (dim + rd), Q, 2.0)
            mat(x + ".dkv", R + rd, Wd, 1.5); vec(x + ".dkv.norm", R, 1.0)
            mat(x + ".uk", H * dim, R, 1.5); mat(x + ".uv", H * vd, R)
            vec(x + ".sink", H, 0.5, 1.0); mat(x + ".g", H, Wd, 2.0); mat(x + ".o", Wd, H * vd, 1.5)
        else:
            le, r = m["left"], m["right"]["width"]
            H, G, dim, vd = le["heads"], le["kv_heads"], le["dim"], le["vdim"]
            mat(x + ".left.q", H * dim, Wd, 2.0); mat(x + ".left.k", G * dim, Wd, 2.0); mat(x + ".left.v", G * vd, Wd)
            mat(x + ".left.g", H, Wd, 2.0); mat(x + ".left.o", Wd, H * vd)
            mat(x + ".right.z", r, Wd, 2.0); vec(x + ".right.z.b", r, -1.5, 1.0); mat(x + ".right.x", r, Wd, 2.0)
            vec(x + ".right.x.b", r, 0.0, 0.5); mat(x + ".right.g", r, Wd, 2.0); mat(x + ".right.o", Wd, r)
            vec(x + ".left.out", Wd, 1.0, 0.2); vec(x + ".right.out", Wd, 1.0, 0.2)
        ms = spec.get("mlp")
        if ms is not None:
            mat(k + ".rg2", Wd, Wd); vec(k + ".rg2.b", Wd, 0.5, 0.5)
            mat(k + ".mlp.router", ms["router"]["experts"], Wd, 2.0)
            for e in range(ms["router"]["experts"]):
                mat(f"{k}.mlp.e{e}.up", ms["expert"]["ff"], Wd, 1.5); mat(f"{k}.mlp.e{e}.down", Wd, ms["expert"]["ff"], 2.0)
    vec("final.norm", Wd, 1.0)
    mat("head", cfg["vocab"], Wd)
    return out
