"""Plain per-sequence model of the Vagelix design in double precision: one function per mechanism,
written from the equations below, sharing no code with the package.

Notation: U(u) = u / sqrt(mean(u^2) + eps); sp(z) = log(1 + e^z); s(z) = 1 / (1 + e^-z); rows of a
matrix argument are tokens 0, 1, 2, ... of one sequence.

    x = U(embed[token]) * w_e
    layer i:   x <- x + U(mixer(x)) * w1;   x <- x + U(ff(x)) * w2          (no ff: the first half only)
    logits = embed (U(x) * w_f)

A layer may name an earlier layer whose weights it uses; its cache and state are its own, which for a
whole sequence means nothing more than running that layer's equations again.
"""
from __future__ import annotations

import math

import torch

D64 = torch.float64


def unit(u, eps):
    return u / torch.sqrt((u * u).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def rotate(x, dims, base):
    """x [T, heads, d]: coordinates (i, i + dims/2) of every head turn by position * base^(-2i/dims)."""
    out, p = x.clone(), torch.arange(x.shape[0], dtype=D64)
    for i in range(dims // 2):
        a = (p * base ** (-2.0 * i / dims))[:, None]
        u, v = x[:, :, i], x[:, :, i + dims // 2]
        out[:, :, i] = u * torch.cos(a) - v * torch.sin(a)
        out[:, :, i + dims // 2] = v * torch.cos(a) + u * torch.sin(a)
    return out


def visible(i, j, chunk):
    return j <= i and (chunk <= 0 or i // chunk == j // chunk)


def softmax_rows(q, k, v, scale, chunk=0, one_more=False):
    """q [T, H, D], k [T, Gk, D], v [T, Gv, V] -> [T, H, V]; query head h on key head h / (H / Gk) and
    value head h / (H / Gv).  ``one_more``: the denominator holds one more term exp(0)."""
    T, H, _ = q.shape
    Gk, Gv, V = k.shape[1], v.shape[1], v.shape[2]
    o = torch.zeros((T, H, V), dtype=D64)
    for i in range(T):
        js = [j for j in range(i + 1) if visible(i, j, chunk)]
        lo, hi = js[0], js[-1] + 1
        for h in range(H):
            sc = (k[lo:hi, h // (H // Gk)] @ q[i, h]) * scale
            top = max(float(sc.max()), 0.0)
            e = torch.exp(sc - top)
            o[i, h] = (e / (e.sum() + (math.exp(-top) if one_more else 0.0))) @ v[lo:hi, h // (H // Gv)]
    return o


def chunk_attention(h, t, m, eps):
    """Grouped-query attention inside blocks of positions: biased projections, the raw keys as values,
    one RMS norm over all query (key) heads together, a partial rotation, one more softmax term and one
    gate per head."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = h @ t["q"].T + t["q.b"], h @ t["k"].T + t["k.b"]
    v = k.view(T, G, V)
    q = (unit(q, eps) * t["q.norm"]).view(T, H, D)
    k = (unit(k, eps) * t["k.norm"]).view(T, G, D)
    if m.get("rot"):
        q, k = rotate(q, m["rot"]["dims"], m["rot"]["base"]), rotate(k, m["rot"]["dims"], m["rot"]["base"])
    o = softmax_rows(q, k, v, m["scale"], (m.get("mask") or {}).get("size", 0), True)
    o = o * sigmoid(h @ t["g"].T)[:, :, None]
    return o.reshape(T, H * V) @ t["o"].T


def causal_filter(u, c, bias=None):
    """y_t = sum_j c[:, j] u_(t - K + 1 + j) (+ bias), zeros before the start."""
    T, C = u.shape
    K = c.shape[1]
    y = torch.zeros((T, C), dtype=D64) if bias is None else bias.repeat(T, 1)
    for tt in range(T):
        for j in range(K):
            if tt - (K - 1) + j >= 0:
                y[tt] = y[tt] + u[tt - (K - 1) + j] * c[:, j]
    return y


def delta_memory(q, k, v, beta, g):
    """q, k, g [T, H, D], v [T, H, V], beta [T, H]: per head S [D, V] decays row by row, the value read at k
    is moved towards v by beta, and q reads the new S."""
    T, H, D = q.shape
    V = v.shape[2]
    S, o = torch.zeros((H, D, V), dtype=D64), torch.zeros((T, H, V), dtype=D64)
    for tt in range(T):
        S = S * g[tt][:, :, None]
        u = beta[tt][:, None] * (v[tt] - torch.einsum("hdv,hd->hv", S, k[tt]))
        S = S + k[tt][:, :, None] * u[:, None, :]
        o[tt] = torch.einsum("hdv,hd->hv", S, q[tt])
    return o


def channel_decay(z, A_log, dt_bias):
    """z [T, H * D], A_log [H]: exp(-e^A sp(z + b)) as [T, H, D]."""
    H = A_log.numel()
    return torch.exp(-torch.exp(A_log)[:, None] * softplus(z + dt_bias).view(z.shape[0], H, -1))


def delta_branch(h, t, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    f = lambda n: silu(causal_filter(h @ t[n].T, t[n + ".conv"]))
    length = lambda u: u / torch.sqrt((u * u).sum(-1, keepdim=True) + 1e-6)
    q, k = length(f("q").view(T, G, D)) * D ** -0.5, length(f("k").view(T, G, D))
    q, k = q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1)
    g = channel_decay(h @ t["a1"].T @ t["a2"].T, t["A_log"].reshape(-1), t["dt_bias"].reshape(-1))
    o = delta_memory(q, k, f("v").view(T, H, V), sigmoid(h @ t["b"].T), g)
    o = (unit(o, eps) * t["norm"]).reshape(T, H * V) * sigmoid(h @ t["g1"].T @ t["g2"].T)
    return o @ t["o"].T


def parallel(h, t, m, eps):
    part = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p)}
    a = chunk_attention(h, part("left."), m["left"], eps)
    b = delta_branch(h, part("right."), m["right"], eps)
    return 0.5 * (unit(a, eps) * t["left.out"] + unit(b, eps) * t["right.out"])


def group_norm(y, parts, w, eps):
    T, C = y.shape
    return unit(y.view(T, parts, C // parts), eps).reshape(T, C) * w


def step_memory(x, B, C, dt, A_log, D_skip):
    """x [T, H, V], B, C [T, G, N], dt [T, H]: S [N, V] per head decays by exp(-e^A dt) and takes dt B x^T."""
    T, H, V = x.shape
    r = H // B.shape[1]
    S, y = torch.zeros((H, B.shape[2], V), dtype=D64), torch.zeros((T, H, V), dtype=D64)
    for tt in range(T):
        b, c = B[tt].repeat_interleave(r, 0), C[tt].repeat_interleave(r, 0)
        S = torch.exp(-torch.exp(A_log) * dt[tt])[:, None, None] * S + dt[tt][:, None, None] * b[:, :, None] * x[tt][:, None, :]
        y[tt] = torch.einsum("hnv,hn->hv", S, c) + D_skip[:, None] * x[tt]
    return y


def state_space(h, t, m, eps):
    T = h.shape[0]
    H, V, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    I = H * V
    p = h @ t["in"].T
    z, xbc, dt = p[:, :I], p[:, I:2 * I + 2 * G * N], p[:, 2 * I + 2 * G * N:]
    xbc = silu(causal_filter(xbc, t["conv"], t["conv.b"]))
    y = step_memory(xbc[:, :I].reshape(T, H, V), xbc[:, I:I + G * N].reshape(T, G, N), xbc[:, I + G * N:].reshape(T, G, N),
                    softplus(dt + t["dt_bias"].reshape(-1)), t["A_log"].reshape(-1), t["D"].reshape(-1))
    return group_norm(y.reshape(T, I) * silu(z), m["norm_groups"], t["norm"], eps) @ t["o"].T


def query_temperature(T, coef, every):
    return torch.tensor([1.0 + coef * math.log(math.floor((p + 1) / every) + 1) for p in range(T)], dtype=D64)


def diff_attention(h, t, m, eps):
    """Two causal softmax maps per head over the same values, the second taken off with one learned factor."""
    T = h.shape[0]
    H, G, D, V, d0 = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["diff"]
    q = unit((h @ t["q"].T).view(T, H, 2, D), eps) * t["q.norm"]
    k = unit((h @ t["k"].T).view(T, G, 2, D), eps) * t["k.norm"]
    v = (h @ t["v"].T).view(T, G, V)
    if m.get("q_temp"):
        q = q * query_temperature(T, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None, None]
    a1, a2 = (softmax_rows(q[:, :, i], k[:, :, i], v, m["scale"]) for i in (0, 1))
    lam = torch.exp((t["lq1"] * t["lk1"]).sum()) - torch.exp((t["lq2"] * t["lk2"]).sum()) + d0
    return (unit(a1 - lam * a2, eps) * (1 - d0)).reshape(T, H * V) @ t["o"].T


def dense(h, t):
    return (silu(h @ t["gate"].T) * (h @ t["up"].T)) @ t["down"].T


MIXERS = {"parallel": parallel, "mamba2": state_space, "attention": diff_attention}


def forward(cfg, w, toks):
    """Logits [T, vocab] and the stream after every layer."""
    w = {k: v.to(D64) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = unit(w["embed"][torch.as_tensor(list(toks))], eps) * w["embed.norm"]
    trail = []
    for i, l in enumerate(cfg["layers"]):
        p = f"l{source(cfg, i)}."
        part = lambda q: {k[len(p + q):]: v for k, v in w.items() if k.startswith(p + q)}
        x = x + unit(MIXERS[l["type"]](x, part("mix."), l["mixer"], eps), eps) * w[p + "norm1"]
        if l.get("mlp") is not None:
            x = x + unit(dense(x, part("mlp.")), eps) * w[p + "norm2"]
        trail.append(x)
    return (unit(x, eps) * w["final.norm"]) @ w["embed"].T, trail


def source(cfg, i):
    """The layer whose weights layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def greedy(cfg, w, prompt, n):
    toks, out = list(prompt), []
    for _ in range(n):
        out.append(int(forward(cfg, w, toks)[0][-1].argmax()))
        toks.append(out[-1])
    return out


# ------------------------------------------------------------------ small random models
def parallel_spec(H=4, G=2, D=12, chunk=24, rot=8, base=50.0, rH=4, rG=2, rD=10, rV=14, conv=3, scale=None):
    return {"left": {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": 1.5 * D ** -0.5 if scale is None else scale,
                     "rot": {"dims": rot, "base": base}, "mask": {"size": chunk}},
            "right": {"heads": rH, "kv_heads": rG, "dim": rD, "vdim": rV, "conv": conv}}


def mamba_spec(H=6, V=9, N=11, G=3, conv=4, parts=2):
    return {"heads": H, "vdim": V, "state": N, "groups": G, "conv": conv, "norm_groups": parts}


def diff_spec(H=4, G=2, D=9, V=13, diff=0.35, coef=0.4, every=16, scale=None):
    return {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": 1.3 * D ** -0.5 if scale is None else scale, "diff": diff,
            "q_temp": {"coef": coef, "every": every}}


def make_config(vocab=61, width=40, ff=56, layers=None, eps=1e-5):
    ff_ = {"kind": "dense", "ff": ff}
    if layers is None:
        layers = [{"type": "attention", "mixer": diff_spec(), "mlp": ff_},
                  {"type": "parallel", "mixer": parallel_spec(), "mlp": ff_},
                  {"type": "mamba2", "mixer": mamba_spec(), "mlp": None},
                  {"type": "parallel", "mixer": parallel_spec(), "mlp": ff_, "weights_of": 1},
                  {"type": "mamba2", "mixer": mamba_spec(5, 8, 7, 1, 2, 4), "mlp": ff_}]
    return {"architecture": "Vagelix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def random_model(cfg, seed, rank=7, grank=5):
    g = torch.Generator().manual_seed(seed)
    W, out = cfg["width"], {}
    r = lambda *s: torch.randn(s, generator=g)

    def lin(name, n, k, gain=1.0):
        out[name] = (gain * k ** -0.5 * r(n, k)).bfloat16()

    def near(name, n, mean=1.0, s=0.3):
        out[name] = (mean + s * r(n)).bfloat16()
    out["embed"] = r(cfg["vocab"], W).bfloat16()
    near("embed.norm", W), near("final.norm", W)
    for i, l in enumerate(cfg["layers"]):
        if l.get("weights_of") is not None:
            continue
        p, q, m = f"l{i}.", f"l{i}.mix.", l["mixer"]
        near(p + "norm1", W, 0.6)
        if l["type"] == "parallel":
            a, b, x, y = m["left"], m["right"], q + "left.", q + "right."
            for n, hh in (("q", a["heads"]), ("k", a["kv_heads"])):
                lin(x + n, hh * a["dim"], W), near(x + n + ".b", hh * a["dim"], 0.0, 0.5), near(x + n + ".norm", hh * a["dim"])
            lin(x + "g", a["heads"], W), lin(x + "o", W, a["heads"] * a["vdim"])
            for n, c in (("q", b["kv_heads"] * b["dim"]), ("k", b["kv_heads"] * b["dim"]), ("v", b["heads"] * b["vdim"])):
                lin(y + n, c, W), near(y + n + ".conv", c * b["conv"], 0.0, 0.6)
                out[y + n + ".conv"] = out[y + n + ".conv"].view(c, b["conv"])
            lin(y + "b", b["heads"], W), near(y + "A_log", b["heads"], -0.5, 1.0), near(y + "norm", b["vdim"])
            lin(y + "a1", rank, W), lin(y + "a2", b["heads"] * b["dim"], rank), near(y + "dt_bias", b["heads"] * b["dim"], -3.0, 1.5)
            lin(y + "g1", grank, W), lin(y + "g2", b["heads"] * b["vdim"], grank), lin(y + "o", W, b["heads"] * b["vdim"])
            near(q + "left.out", W, 0.8), near(q + "right.out", W, 0.8)
        elif l["type"] == "mamba2":
            I, gn = m["heads"] * m["vdim"], m["groups"] * m["state"]
            lin(q + "in", 2 * I + 2 * gn + m["heads"], W)
            out[q + "conv"], out[q + "conv.b"] = (0.6 * r(I + 2 * gn, m["conv"])).bfloat16(), (0.2 * r(I + 2 * gn)).bfloat16()
            near(q + "dt_bias", m["heads"], -2.0, 1.5), near(q + "A_log", m["heads"], -0.5, 1.0), near(q + "D", m["heads"])
            near(q + "norm", I), lin(q + "o", W, I)
        else:
            lin(q + "q", 2 * m["heads"] * m["dim"], W), lin(q + "k", 2 * m["kv_heads"] * m["dim"], W)
            lin(q + "v", m["kv_heads"] * m["vdim"], W), lin(q + "o", W, m["heads"] * m["vdim"])
            near(q + "q.norm", m["dim"]), near(q + "k.norm", m["dim"])
            for n in ("lq1", "lk1", "lq2", "lk2"):
                near(q + n, m["dim"], 0.0, 0.3)
        if l.get("mlp") is not None:
            near(p + "norm2", W, 0.6)
            lin(p + "mlp.gate", l["mlp"]["ff"], W), lin(p + "mlp.up", l["mlp"]["ff"], W), lin(p + "mlp.down", W, l["mlp"]["ff"])
    return out
