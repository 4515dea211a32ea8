"""Plain per-sequence model of the Lefuvik design in double precision: one function per mechanism,
written from the equations below, sharing no code with the package.

Notation: U(u) = u / sqrt(mean(u^2) + eps); N_w(u) = U(u) (1 + w); sp(z) = log(1 + e^z); rows of a
matrix argument are tokens 0, 1, 2, ... of one sequence.

    x = N_embed(embed[token])
    layer i:   x <- x + a1 * mixer(N_1(x));   x <- x + a2 * ff(N_2(x))        a1, a2 one number per coordinate
               x <- x + U(P (gelu(G x) * e_i)) * w                           e_i = slice i of the token's side row
    logits = cap tanh(embed N_final(x) / cap)
"""
from __future__ import annotations

import math

import torch

D64 = torch.float64


def unit(u, eps):
    return u / torch.sqrt((u * u).mean(-1, keepdim=True) + eps)


def norm_one_plus(u, w, eps):
    return unit(u, eps) * (1.0 + w)


def gelu(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def rotate(x, dims, base, interleaved):
    """x [T, heads, d]: the first ``dims`` coordinates of every head turn by position * base^(-2i/dims)."""
    out, p = x.clone(), torch.arange(x.shape[0], dtype=D64)
    for i in range(dims // 2):
        a = (p * base ** (-2.0 * i / dims))[:, None]
        iu, iv = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
        u, v = x[:, :, iu], x[:, :, iv]
        out[:, :, iu] = u * torch.cos(a) - v * torch.sin(a)
        out[:, :, iv] = v * torch.cos(a) + u * torch.sin(a)
    return out


def distance_bucket(n, B, D):
    """Bucket of distance n among B: the first B/2 exact, the rest evenly spaced in log n up to D."""
    h = B // 2
    if n < h:
        return n
    return min(B - 1, h + math.floor(math.log(n / h) / math.log(D / h) * (B - h) + 1e-12))


def visible(i, j, size, keep):
    return j <= i and (size <= 0 or i - j < size or j < keep)


def softmax_rows(q, k, v, scale, size, keep=0, rel=None, bias_max=0):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]: softmax over the visible keys of
    q . k * scale + rel[bucket(i - j), h]."""
    T, H, _ = q.shape
    G, V = k.shape[1], v.shape[2]
    o = torch.zeros((T, H, V), dtype=D64)
    if rel is not None:
        per = torch.stack([rel[distance_bucket(n, rel.shape[0], bias_max)] for n in range(T)])      # [T, H]
    for i in range(T):
        js = [j for j in range(i + 1) if visible(i, j, size, keep)]
        for h in range(H):
            g = h // (H // G)
            s = (k[js, g] @ q[i, h]) * scale
            if rel is not None:
                s = s + per[[i - j for j in js], h]
            o[i, h] = torch.softmax(s, 0) @ v[js, g]
    return o


def biased_attention(h, t, m, eps):
    """Grouped-query attention without rotation: unit-RMS heads (weighted q and k, plain v), a learned
    distance bias, a sliding window and the first tokens kept visible."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit((h @ t["q"].T).view(T, H, D), eps) * t["q.norm"]
    k = unit((h @ t["k"].T).view(T, G, D), eps) * t["k.norm"]
    v = unit((h @ t["v"].T).view(T, G, V), eps)
    mask = m.get("mask") or {}
    o = softmax_rows(q, k, v, m["scale"], mask.get("size", 0), mask.get("keep_first", 0), t["rel"], m["bias_max"])
    return o.reshape(T, H * V) @ t["o"].T


def causal_filter(u, c, bias):
    T, C = u.shape
    K = c.shape[1]
    y = bias.repeat(T, 1)
    for tt in range(T):
        for j in range(K):
            if tt - (K - 1) + j >= 0:
                y[tt] = y[tt] + u[tt - (K - 1) + j] * c[:, j]
    return y


def gated_linear_recurrence(u, ra, ra_b, ri, ri_b, lam):
    """S_t = a S_(t-1) + sqrt(1 - a^2) i u with a = exp(-8 r sp(lam)); r, i sigmoids of block-diagonal products."""
    T, C = u.shape
    nb, w = ra.shape[0], ra.shape[1]
    ub = u.view(T, nb, w)
    r = torch.sigmoid(torch.einsum("boi,tbi->tbo", ra, ub) + ra_b).reshape(T, C)
    i = torch.sigmoid(torch.einsum("boi,tbi->tbo", ri, ub) + ri_b).reshape(T, C)
    a = torch.exp(-8.0 * r * softplus(lam))
    S, out = torch.zeros(C, dtype=D64), torch.zeros((T, C), dtype=D64)
    for tt in range(T):
        S = a[tt] * S + torch.sqrt(1 - a[tt] ** 2) * i[tt] * u[tt]
        out[tt] = S
    return out


def recurrent_block(h, t, m):
    y = gelu(h @ t["y"].T + t["y.b"])
    u = causal_filter(h @ t["x"].T + t["x.b"], t["conv"], t["conv.b"])
    S = gated_linear_recurrence(u, t["ra"], t["ra.b"], t["ri"], t["ri.b"], t["lam"])
    return (S * y) @ t["o"].T


def sub(t, p):
    return {k[len(p):]: v for k, v in t.items() if k.startswith(p)}


def parallel(h, t, m, eps):
    return (m["left_scale"] * biased_attention(h, sub(t, "left."), m["left"], eps)
            + m["right_scale"] * recurrent_block(h, sub(t, "right."), m["right"]))


def retention(h, t, m, eps):
    """S_t = decay S_(t-1) + k v^T, o = S^T q per head; unit RMS per head, a SiLU gate."""
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q, k, v = (h @ t["q"].T).view(T, H, D), (h @ t["k"].T).view(T, H, D), (h @ t["v"].T).view(T, H, V)
    if m.get("rot"):
        q = rotate(q, m["rot"]["dims"], m["rot"]["base"], False)
        k = rotate(k, m["rot"]["dims"], m["rot"]["base"], False)
    k = k * D ** -0.5
    o = torch.zeros((T, H, V), dtype=D64)
    for hh in range(H):
        S = torch.zeros((D, V), dtype=D64)
        for tt in range(T):
            S = m["decay"][hh] * S + torch.outer(k[tt, hh], v[tt, hh])
            o[tt, hh] = S.T @ q[tt, hh]
    return (unit(o, eps).reshape(T, H * V) * silu(h @ t["g"].T)) @ t["o"].T


def latent_attention(h, t, m, eps, shared):
    """``shared``: list of (latent, rotated key part) per layer so far; appended to."""
    T = h.shape[0]
    H, D, Dr, V, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = unit(h @ t["dq"].T, eps) * t["dq.norm"]
    q = (cq @ t["uq"].T).view(T, H, D + Dr)
    qn, qr = q[..., :D], q[..., D:]
    rot = m.get("rot")
    if rot:
        qr = rotate(qr, rot["dims"], rot["base"], True)
    if "kv_from" in m and m["kv_from"] is not None:
        c, kr = shared[m["kv_from"]]
    else:
        d = h @ t["dkv"].T
        c, kr = unit(d[:, :R], eps) * t["dkv.norm"], d[:, R:][:, None, :]
        if rot:
            kr = rotate(kr, rot["dims"], rot["base"], True)
    shared.append((c, kr))
    kn, v = (c @ t["uk"].T).view(T, H, D), (c @ t["uv"].T).view(T, H, V)
    k = torch.cat([kn, kr.expand(T, H, Dr)], -1)
    o = softmax_rows(torch.cat([qn, qr], -1), k, v, m["scale"], (m.get("mask") or {}).get("size", 0))
    return o.reshape(T, H * V) @ t["o"].T


def xielu(z, p, q):
    return torch.where(z > 0, softplus(p) * z * z + 0.5 * z, (0.5 + softplus(q)) * (torch.expm1(z) - z) + 0.5 * z)


def dense(h, t):
    return xielu(h @ t["up"].T, t["act"][0], t["act"][1]) @ t["down"].T


def route(z, corr, top, groups):
    """Scores softmax(z); the ``top`` largest score + corr inside the best groups: list of expert ids and scores."""
    E = z.shape[0]
    s = torch.softmax(z, 0)
    choice = s + corr
    cand = list(range(E))
    if groups:
        n = E // groups["count"]
        best = sorted(range(groups["count"]), key=lambda g: (-float(choice[g * n:(g + 1) * n].max()), g))[:groups["keep"]]
        cand = [e for e in cand if e // n in best]
    ids = sorted(cand, key=lambda e: (-float(choice[e]), e))[:top]
    return ids, [s[e] for e in ids]


def mixture(h, t, f):
    out = torch.zeros_like(h)
    z = h @ t["router"].T
    for tt in range(h.shape[0]):
        ids, ws = route(z[tt], t["correction"], f["router"]["top"], f["router"].get("groups"))
        for e, wgt in zip(ids, ws):
            out[tt] = out[tt] + wgt * (t[f"e{e}.down"] @ torch.clamp(t[f"e{e}.up"] @ h[tt], min=0) ** 2)
    return out


def side_input(x, rows, t, eps):
    """rows [T, dim]: this layer's slice of the tokens' side table."""
    g = gelu(x @ t["gate"].T) * rows
    return unit(g @ t["proj"].T, eps) * t["norm"]


def forward(cfg, w, tokens):
    """-> (logits [T, vocab], the stream after every layer)."""
    w = {k: v.to(D64) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    ids = torch.tensor(tokens)
    x = norm_one_plus(w["embed"][ids], w["embed.norm"], eps)
    shared, trail = [], []
    for i, l in enumerate(cfg["layers"]):
        t = sub(w, f"l{i}.")
        h, mt, m = norm_one_plus(x, t["norm1"], eps), sub(t, "mix."), l["mixer"]
        n_before = len(shared)
        if l["type"] == "parallel":
            y = parallel(h, mt, m, eps)
        elif l["type"] == "retention":
            y = retention(h, mt, m, eps)
        else:
            y = latent_attention(h, mt, m, eps, shared)
        if len(shared) == n_before:
            shared.append(None)
        x = x + y * t["ls1"]
        f = l.get("mlp")
        if f is not None:
            h2 = norm_one_plus(x, t["norm2"], eps)
            y = dense(h2, sub(t, "mlp.")) if f["kind"] == "dense" else mixture(h2, sub(t, "mlp."), f)
            x = x + y * t["ls2"]
        if cfg.get("token_side"):
            d = cfg["token_side"]["dim"]
            x = x + side_input(x, w["side.embed"][ids][:, i * d:(i + 1) * d], sub(t, "side."), eps)
        trail.append(x)
    logits = norm_one_plus(x, w["final.norm"], eps) @ w["embed"].T
    cap = cfg.get("logit_softcap")
    return (cap * torch.tanh(logits / cap) if cap else logits), trail


# ------------------------------------------------------------------ small random models
def random_model(cfg, seed=0, std=None, dtype=torch.bfloat16, buckets=8):
    """Random weights (representable in ``dtype``) under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    W, w = cfg["width"], {}

    def r(name, shape, s, mean=0.0):
        w[name] = (mean + torch.randn(shape, generator=g, dtype=D64) * s).to(dtype).to(D64)

    lin = lambda name, o, i: r(name, (o, i), std or i ** -0.5)
    r("embed", (cfg["vocab"], W), 1.0), r("embed.norm", (W,), 0.3), r("final.norm", (W,), 0.3)
    if cfg.get("token_side"):
        r("side.embed", (cfg["vocab"], len(cfg["layers"]) * cfg["token_side"]["dim"]), 1.0)
    for i, l in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", l["mixer"], l.get("mlp")
        q = p + "mix."
        r(p + "norm1", (W,), 0.3), r(p + "ls1", (W,), 0.3, 0.7)
        if l["type"] == "parallel":
            a, b, q1, q2 = m["left"], m["right"], q + "left.", q + "right."
            lin(q1 + "q", a["heads"] * a["dim"], W), lin(q1 + "k", a["kv_heads"] * a["dim"], W)
            lin(q1 + "v", a["kv_heads"] * a["vdim"], W), lin(q1 + "o", W, a["heads"] * a["vdim"])
            r(q1 + "q.norm", (a["dim"],), 0.3, 1.0), r(q1 + "k.norm", (a["dim"],), 0.3, 1.0)
            r(q1 + "rel", (buckets, a["heads"]), 1.0)
            C, nb = b["width"], b["blocks"]
            for n in "yx":
                lin(q2 + n, C, W), r(q2 + n + ".b", (C,), 0.3)
            r(q2 + "conv", (C, b["conv"]), 0.5), r(q2 + "conv.b", (C,), 0.2)
            for n in ("ra", "ri"):
                r(q2 + n, (nb, C // nb, C // nb), (C // nb) ** -0.5), r(q2 + n + ".b", (nb, C // nb), 0.5)
            r(q2 + "lam", (C,), 1.5, -4.0), lin(q2 + "o", W, C)
        elif l["type"] == "retention":
            for n, d in (("q", "dim"), ("k", "dim"), ("v", "vdim"), ("g", "vdim")):
                lin(q + n, m["heads"] * m[d], W)
            lin(q + "o", W, m["heads"] * m["vdim"])
        else:
            lin(q + "dq", m["q_rank"], W), r(q + "dq.norm", (m["q_rank"],), 0.3, 1.0)
            lin(q + "uq", m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"])
            if m.get("kv_from") is None:
                lin(q + "dkv", m["kv_rank"] + m["rot_dim"], W), r(q + "dkv.norm", (m["kv_rank"],), 0.3, 1.0)
            lin(q + "uk", m["heads"] * m["dim"], m["kv_rank"]), lin(q + "uv", m["heads"] * m["vdim"], m["kv_rank"])
            lin(q + "o", W, m["heads"] * m["vdim"])
        if f is not None:
            r(p + "norm2", (W,), 0.3), r(p + "ls2", (W,), 0.3, 0.7)
            if f["kind"] == "dense":
                lin(p + "mlp.up", f["ff"], W), lin(p + "mlp.down", W, f["ff"]), r(p + "mlp.act", (2,), 0.7)
            else:
                E = f["router"]["experts"]
                r(p + "mlp.router", (E, W), 2.0 * W ** -0.5), r(p + "mlp.correction", (E,), 0.2)
                for e in range(E):
                    lin(p + f"mlp.e{e}.up", f["expert"]["ff"], W), lin(p + f"mlp.e{e}.down", W, f["expert"]["ff"])
        if cfg.get("token_side"):
            d = cfg["token_side"]["dim"]
            lin(p + "side.gate", d, W), lin(p + "side.proj", W, d), r(p + "side.norm", (W,), 0.2, 0.5)
    return w


def make_config(pattern=("parallel:dense", "retention:moe", "latent:moe", "parallel:none", "shared:moe"), vocab=61, width=40, heads=4,
                kv_heads=2, dim=12, vdim=8, window=21, keep=6, bias_max=30, rwidth=36, blocks=3, conv=4, left=0.7, right=1.2,
                rheads=3, rdim=10, rvdim=14, rrot=6, lheads=2, ldim=9, lvdim=11, kv_rank=20, q_rank=26, rot_dim=8, lwindow=18,
                ff=52, experts=6, top=2, eff=24, groups=3, keep_groups=2, side=5, cap=12.0, eps=1e-5):
    """A small configuration: ``pattern`` lists mixer:feed-forward ("shared" is latent attention on the
    last "latent" layer's cache)."""
    layers, last = [], None
    for i, item in enumerate(pattern):
        kind, f = item.split(":")
        if kind == "parallel":
            mask = {"size": window, "keep_first": keep}
            m = {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 1.3 * dim ** -0.5,
                          "bias_max": bias_max, "mask": mask},
                 "right": {"width": rwidth, "blocks": blocks, "conv": conv}, "left_scale": left, "right_scale": right}
        elif kind == "retention":
            m = {"heads": rheads, "dim": rdim, "vdim": rvdim, "decay": [1 - 2.0 ** (-2 - 2 * h) for h in range(rheads)],
                 "rot": {"dims": rrot, "base": 700.0}}
        else:
            m = {"heads": lheads, "dim": ldim, "vdim": lvdim, "kv_rank": kv_rank, "q_rank": q_rank, "rot_dim": rot_dim,
                 "scale": 1.1 * (ldim + rot_dim) ** -0.5, "rot": {"dims": rot_dim, "base": 300.0}, "mask": {"size": lwindow}}
            if kind == "shared":
                m["kv_from"] = last
                m["mask"] = {"size": lwindow + 7}
            else:
                last = i
        mlp = None
        if f == "dense":
            mlp = {"kind": "dense", "ff": ff}
        elif f == "moe":
            mlp = {"kind": "moe", "expert": {"ff": eff}, "router": {"experts": experts, "top": top}}
            if groups > 1:
                mlp["router"]["groups"] = {"count": groups, "keep": keep_groups}
        layers.append({"type": {"latent": "latent_attention", "shared": "latent_attention"}.get(kind, kind), "mixer": m, "mlp": mlp})
    cfg = {"architecture": "Lefuvik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers, "logit_softcap": cap}
    if side:
        cfg["token_side"] = {"dim": side}
    return cfg
