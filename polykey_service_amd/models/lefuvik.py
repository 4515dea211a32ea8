"""Lefuvik decoder: one fp32 residual stream that starts from the normed embedding, pre-norm sublayers
with a learned scale per output coordinate, and a per-layer input from the token's own side table.
Mixers are distance-biased attention beside a gated linear recurrence, retention, or windowed latent
attention (optionally on an earlier layer's cache); feed-forwards are dense xIELU or a group-routed
mixture of squared-ReLU experts.

Per layer, for the step's tokens (x: fp32 stream [T, W]; a = the model's dtype, bf16 or fp32; norms,
the stream, rotations, scores, softmax, routers, decays, gates of the recurrence and recurrent states
are fp32):

    h   = N1(x) -> a                                                                  HIP  hyper.hip
    parallel:   q | k | v | y | u = h @ [Wq; Wk; Wv; Wy; Wx]^T   (both branches, one product)  hipBLASLt / decode GEMM
                left  q, k unit RMS per head times a weight, v unit RMS ; k, v -> paged caches  HIP  masked_attention.hip
                      softmax over the window and the first tokens of q . k * scale + bias[h, distance]
                right u = filter(u + b) + b' ; r, i = sigmoid(block-diagonal u) ; a = exp(lam r)  HIP  short_conv.hip, lru.hip
                      S <- a S + sqrt(1 - a^2) i u ; S * gelu(y + b)         (state [C] fp32 per slot)
                o = [left_scale * left | right_scale * right] -> one output projection
    retention:  q | k | v | g = h @ [...]^T ; q, k turned by the position, k / sqrt(D)
                S <- decay_h S + k v^T ; o = S^T q          (state [H, D, V] fp32 per slot)  HIP  lightning.hip
                o = unit_rms_per_head(o) * silu(g)                                     HIP  head_norm_gate
    latent:     as models/nopunex.py WindowLatentAttention, without a sink
    y   = o @ Wo^T
    x  <- x + s1 * y ;  h2 = N2(x)                                     (one kernel)    HIP  hyper.hip
    dense:      f = xielu(h2 @ Wup^T) @ Wdown^T                                        HIP  group_moe.hip
    moe:        z = Wr h2 (fp32) ; s = softmax(z) ; experts by s + correction inside the best groups
                f = sum_e s_e down_e(max(up_e h2, 0)^2)
    x  <- x + s2 * f ;  x -> a                                         (one kernel)
    e   = gelu(x @ Wg^T) * side[token, layer] ;  y = e @ Wp^T                          HIP  group_moe.hip
    x  <- x + unit_rms(y) * w ;  the next layer's h                    (one kernel)    HIP  hyper.hip

and logits = cap tanh(embed @ N_final(x) / cap), N_w(u) = u / sqrt(mean(u^2) + eps) * (1 + w).  Tensor
parallelism is not implemented for this family.
"""
from __future__ import annotations

from typing import List, Optional

import torch
from torch import nn

from ..ops import gemm
from ..ops import hyper as hyper_ops
from ..ops import lightning as lightning_ops
from ..ops import lru as lru_ops
from ..ops import masked_attention as ma_ops
from ..ops import moe as moe_ops
from ..ops import short_conv as conv_ops
from ..parallel.state import ParallelState
from .bibezen import _f32
from .config import GroupedMoESpec, LefuvikConfig, XieluFFSpec
from .kivezen import _p, _packed, _project, tanh_cap
from .nopunex import WindowLatentAttention, _pad_rows
from .weights import SafetensorsIndex, random_full


class BiasedRecurrentMixer(nn.Module):
    """Distance-biased attention (left) beside a gated linear recurrence (right): one input and one
    output projection over both branches."""

    def __init__(self, spec, width: int):
        super().__init__()
        self.spec, self.width = spec, width
        self.w_in = self.w_in_p = None          # [H*D | G*D | G*V | C | C (+ padding), W]: q, k, v, y, u rows
        self.q_norm = self.k_norm = None        # [D] fp32
        self.bias = None                        # [H, distances] fp32
        self.y_b = self.x_b = self.conv_b = None    # [C] fp32
        self.taps = None                        # [C, K] fp32
        self.ra = self.ri = None                # [blocks, C / blocks, C / blocks]
        self.ra_b = self.ri_b = self.lam = None     # [C] fp32; lam = -8 softplus(stored)
        self.w_o = self.w_o_p = None            # [W, H*V | C]

    def pack(self) -> None:
        self.w_in_p, self.w_o_p = _packed(self.w_in), _packed(self.w_o)

    def set(self, get, dtype, device) -> None:
        s, r, W = self.spec.left, self.spec.right, self.width
        H, G, D, V, C, w = s.heads, s.kv_heads, s.dim, s.vdim, r.width, r.width // r.blocks
        a, b = (lambda n: get("left." + n)), (lambda n: get("right." + n))
        assert a("q").shape == (H * D, W) and a("k").shape == (G * D, W) and a("v").shape == (G * V, W)
        assert a("o").shape == (W, H * V) and b("y").shape == b("x").shape == (C, W) and b("o").shape == (W, C)
        assert b("conv").shape == (C, r.conv) and b("ra").shape == b("ri").shape == (r.blocks, w, w) and a("rel").shape[1] == H
        to = lambda t: _p(t.to(device=device, dtype=dtype))
        f32 = lambda t, n: _f32(t.reshape(n), device)
        self.w_in = to(_pad_rows(torch.cat([a("q"), a("k"), a("v"), b("y"), b("x")], 0)))
        self.q_norm, self.k_norm = f32(a("q.norm"), D), f32(a("k.norm"), D)
        self.bias = _p(ma_ops.distance_bias(a("rel").cpu(), s.bias_max).to(device))
        self.y_b, self.x_b, self.conv_b = f32(b("y.b"), C), f32(b("x.b"), C), f32(b("conv.b"), C)
        self.taps = _f32(b("conv"), device)
        self.ra, self.ri = to(b("ra")), to(b("ri"))
        self.ra_b, self.ri_b = f32(b("ra.b"), C), f32(b("ri.b"), C)
        self.lam = _f32(-8.0 * torch.nn.functional.softplus(b("lam").double().reshape(C)), device)
        self.w_o = to(torch.cat([a("o"), b("o")], 1))

    def forward(self, h, positions, md, cache: dict, eps: float):
        p, s, C = self.spec, self.spec.left, self.spec.right.width
        H, G, D, V = s.heads, s.kv_heads, s.dim, s.vdim
        n, nl = (H + G) * D + G * V, H * V
        o = torch.empty((h.shape[0], nl + C), dtype=h.dtype, device=h.device)
        proj = _project(h, self.w_in, self.w_in_p)
        q = ma_ops.rotate_cache(proj[:, :n], positions, md.slot_mapping, None, True, cache["k"], cache["v"], H, G, G, D, V,
                                q_norm=self.q_norm, k_norm=self.k_norm, eps=eps, v_unit=True)
        ma_ops.masked_attention(q, cache["k"], cache["v"], V, md.block_tables, md.cu_q, md.context_lens, md.num_seqs, s.scale,
                                window=s.window, num_decode=md.num_decode, keep=s.keep, bias=self.bias, post=p.left_scale,
                                out=o[:, :nl])
        u = conv_ops.causal_conv(proj[:, n + C:n + 2 * C], self.taps, self.conv_b, cache.get("conv"), md.cu_q, md.num_seqs,
                                 positions, md.state_slots, md.token_seq, in_bias=self.x_b, num_decode=md.num_decode)
        lru_ops.gated_lru(u, proj[:, n:n + C], self.y_b, self.ra, self.ri, self.ra_b, self.ri_b, self.lam, cache["lru"], md.cu_q,
                          md.num_seqs, positions, md.state_slots, md.num_decode, p.right_scale, o[:, nl:])
        return _project(o, self.w_o, self.w_o_p, partial=True)

    def state(self, slots: int, device) -> dict:
        r = self.spec.right
        out = {"lru": torch.zeros((slots, r.width), dtype=torch.float32, device=device)}
        if r.conv > 1:
            out["conv"] = torch.zeros((slots, r.conv - 1, r.width), dtype=torch.float32, device=device)
        return out

    def state_floats(self) -> int:
        return self.spec.right.width * self.spec.right.conv


class RetentionMixer(nn.Module):
    """Weights of one retention mixer."""

    def __init__(self, spec, width: int):
        super().__init__()
        self.spec, self.width = spec, width
        self.w_in = self.w_in_p = None      # [H*D | H*D | H*V | H*V (+ padding), W]: q, k, v, gate rows
        self.w_o = self.w_o_p = None        # [W, H*V]
        self.decay = None                   # [H] fp32
        self.table = None                   # [positions, pairs, 2] fp32; None: no rotation

    def pack(self) -> None:
        self.w_in_p, self.w_o_p = _packed(self.w_in), _packed(self.w_o)

    def set(self, get, dtype, device) -> None:
        s, W = self.spec, self.width
        H, D, V = s.heads, s.dim, s.vdim
        assert get("q").shape == get("k").shape == (H * D, W) and get("v").shape == get("g").shape == (H * V, W)
        assert get("o").shape == (W, H * V)
        self.w_in = _p(_pad_rows(torch.cat([get(n) for n in "qkvg"], 0)).to(device=device, dtype=dtype))
        self.w_o = _p(get("o").to(device=device, dtype=dtype))
        self.decay = _p(torch.tensor(s.decay, dtype=torch.float64).float().to(device))

    def forward(self, h, positions, md, cache: dict, eps: float):
        s = self.spec
        H, D, V = s.heads, s.dim, s.vdim
        n = H * (2 * D + V)
        proj = _project(h, self.w_in, self.w_in_p)
        o = lightning_ops.retention(proj[:, :n], cache["ret"], self.decay, self.table, D ** -0.5, md.cu_q, md.num_seqs, positions,
                                    md.state_slots, H, D, V)
        a = ma_ops.head_norm_gate(o, H, V, eps, proj[:, n:n + H * V], ma_ops.GATE_SILU, h.dtype)
        return _project(a, self.w_o, self.w_o_p, partial=True)

    def state(self, slots: int, device) -> dict:
        s = self.spec
        return {"ret": torch.zeros((slots, s.heads, s.dim, s.vdim), dtype=torch.float32, device=device)}

    def state_floats(self) -> int:
        return self.spec.heads * self.spec.dim * self.spec.vdim


class XieluFF(nn.Module):
    def __init__(self, spec: XieluFFSpec):
        super().__init__()
        self.spec = spec
        self.up = self.down = self.up_p = self.down_p = None
        self.p = self.q = 0.0    # softplus(first), 1/2 + softplus(second) of the layer's two numbers

    def set(self, up, down, act, dtype, device) -> None:
        assert up.shape == (self.spec.ff, down.shape[0]) and down.shape[1] == self.spec.ff and act.numel() == 2
        self.up, self.down = _p(up.to(device=device, dtype=dtype)), _p(down.to(device=device, dtype=dtype))
        sp = torch.nn.functional.softplus(act.double().reshape(2))
        self.p, self.q = float(sp[0]), 0.5 + float(sp[1])

    def pack(self) -> None:
        self.up_p, self.down_p = _packed(self.up), _packed(self.down)

    def forward(self, h, h32):
        a = moe_ops.activate(_project(h, self.up, self.up_p, partial=True), moe_ops.ACT_XIELU, self.p, self.q, h.dtype)
        return _project(a, self.down, self.down_p, partial=True)


class GroupedMoE(nn.Module):
    """fp32 router with a choice correction and expert groups, squared-ReLU experts."""

    def __init__(self, spec: GroupedMoESpec):
        super().__init__()
        self.spec = spec
        self.router = self.correction = None     # [E, W], [E] fp32
        self.up = self.down = self.up_p = self.down_p = None   # [E, F, W], [E, W, F]
        self.mfma = False

    def set(self, router, correction, ups, downs, dtype, device) -> None:
        s = self.spec
        E, (F_, W) = len(ups), ups[0].shape
        assert router.shape == (E, W) and downs[0].shape == (W, F_) and (E, F_) == (s.experts, s.ff)
        to = lambda ts: _p(torch.stack(ts).to(device=device, dtype=dtype))
        self.router, self.up, self.down = _f32(router, device), to(ups), to(downs)
        self.correction = _f32(correction.reshape(E), device) if correction is not None else None
        self.mfma = moe_ops.mfma_experts_ok(E, F_, W, dtype, torch.device(device))

    def pack(self) -> None:
        if self.mfma and self.up_p is None:
            for n in ("up", "down"):
                E, N, K = getattr(self, n).shape
                setattr(self, n + "_p", gemm.pack_weight(getattr(self, n).view(E * N, K)).view(E, N, K))

    def forward(self, h, h32) -> hyper_ops.ExpertSum:
        s = self.spec
        ids, wts = moe_ops.route_group_topk(moe_ops.router_logits(h32, self.router), self.correction, s.top, s.groups, s.keep)
        y, inv = moe_ops.relu2_experts(h, ids, self.up, self.down, self.up_p, self.down_p, self.mfma)
        return hyper_ops.ExpertSum(y, inv, wts, s.top)


class SideInput(nn.Module):
    """One layer's token input: gate and output projection around the token's side row."""

    def __init__(self):
        super().__init__()
        self.gate = self.proj = self.gate_p = self.proj_p = None   # [dim, W], [W, dim]
        self.norm_w = None                                         # [W] fp32
        self.off = 0

    def set(self, gate, proj, norm_w, off: int, dtype, device) -> None:
        assert gate.shape == proj.shape[::-1] and norm_w.numel() == gate.shape[1]
        self.gate, self.proj = _p(gate.to(device=device, dtype=dtype)), _p(proj.to(device=device, dtype=dtype))
        self.norm_w, self.off = _f32(norm_w.reshape(-1), device), off

    def pack(self) -> None:
        self.gate_p, self.proj_p = _packed(self.gate), _packed(self.proj)

    def forward(self, x, table, ids):
        g = moe_ops.activate(_project(x, self.gate, self.gate_p, partial=True), moe_ops.ACT_GELU, dtype=x.dtype,
                             rows=(table, ids, self.off))
        return _project(g, self.proj, self.proj_p, partial=True)


_MIXERS = {"parallel": BiasedRecurrentMixer, "retention": RetentionMixer, "latent_attention": WindowLatentAttention}


class LefuvikLayer(nn.Module):
    def __init__(self, spec, width: int, side: bool):
        super().__init__()
        self.kind = spec.type
        self.mix = _MIXERS[spec.type](spec.mixer, width)
        self.mlp = None
        if spec.mlp is not None:
            self.mlp = XieluFF(spec.mlp) if isinstance(spec.mlp, XieluFFSpec) else GroupedMoE(spec.mlp)
        self.side = SideInput() if side else None
        self.norm1 = self.norm2 = None      # [W] fp32, 1 + the stored weight
        self.scale1 = self.scale2 = None    # [W] fp32


class LefuvikForCausalLM(nn.Module):
    # engine hooks (engine/model_runner.py): this family owns its cache and state layouts
    supports_graphs = True

    def __init__(self, cfg: LefuvikConfig, st: ParallelState, dtype: torch.dtype, device: torch.device):
        super().__init__()
        if st.tp_size > 1 or getattr(st, "ep_size", 1) > 1:
            raise ValueError("Lefuvik runs on one GPU (no TP / EP sharding for this family)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Lefuvik runs in bfloat16 or float32, not {dtype}")
        self.cfg, self.st, self.dtype, self.device = cfg, st, dtype, device
        self.needs_state = cfg.needs_state
        self.layers = nn.ModuleList(LefuvikLayer(l, cfg.hidden_size, cfg.side_dim > 0) for l in cfg.layers)
        self.embed = self.embed_norm = self.final_norm = self.side_embed = None
        self.one = self.unit_mix = None     # the plain residual's stream coefficients [1], [1, 1]
        self._max_pos = 0

    # ------------------------------------------------------------------ weights
    def _norm(self, get, name: str) -> nn.Parameter:
        w = get(name)
        assert w.numel() == self.cfg.hidden_size, name
        return _f32(1.0 + w.double().reshape(-1), self.device)

    def _set_layer(self, i: int, get, has) -> None:
        cfg, L, spec = self.cfg, self.layers[i], self.cfg.layers[i]
        p, dev, dt, W = f"l{i}.", self.device, self.dtype, self.cfg.hidden_size
        m = lambda n: get(p + "mix." + n)
        if L.kind == "latent_attention":
            own = spec.mixer.kv_from < 0
            L.mix.set(m("dq"), m("dq.norm"), m("uq"), m("dkv") if own else None, m("dkv.norm") if own else None, m("uk"), m("uv"),
                      None, m("o"), dt, dev)
        else:
            L.mix.set(m, dt, dev)
        L.norm1, L.scale1 = self._norm(get, p + "norm1"), _f32(get(p + "ls1").reshape(W), dev)
        f = spec.mlp
        if f is not None:
            L.norm2, L.scale2 = self._norm(get, p + "norm2"), _f32(get(p + "ls2").reshape(W), dev)
            if isinstance(f, XieluFFSpec):
                L.mlp.set(get(p + "mlp.up"), get(p + "mlp.down"), get(p + "mlp.act"), dt, dev)
            else:
                part = lambda n: [get(p + f"mlp.e{e}.{n}") for e in range(f.experts)]
                corr = get(p + "mlp.correction") if has(p + "mlp.correction") else None
                L.mlp.set(get(p + "mlp.router"), corr, part("up"), part("down"), dt, dev)
        if L.side is not None:
            L.side.set(get(p + "side.gate"), get(p + "side.proj"), get(p + "side.norm"), i * cfg.side_dim, dt, dev)

    def load_hf(self, path: str) -> "LefuvikForCausalLM":
        """Load a checkpoint folder (safetensors; tensors under the design's own names)."""
        idx = SafetensorsIndex(path)
        return self._load(idx.get, idx.has)

    def load_state(self, tensors: dict) -> "LefuvikForCausalLM":
        """The same from a dict name -> tensor (tests)."""
        return self._load(tensors.__getitem__, tensors.__contains__)

    def _load(self, get, has) -> "LefuvikForCausalLM":
        cfg, dev = self.cfg, self.device
        self.embed = _p(get("embed").to(device=dev, dtype=self.dtype))
        assert self.embed.shape == (cfg.vocab_size, cfg.hidden_size)
        self.embed_norm, self.final_norm = self._norm(get, "embed.norm"), self._norm(get, "final.norm")
        if cfg.side_dim:
            self.side_embed = _p(get("side.embed").to(device=dev, dtype=self.dtype))
            assert self.side_embed.shape == (cfg.vocab_size, cfg.side_dim * len(cfg.layers))
        self.one = _p(torch.ones(1, dtype=torch.float32, device=dev))
        self.unit_mix = _p(torch.ones((1, 1), dtype=torch.float32, device=dev))
        for i in range(len(self.layers)):
            self._set_layer(i, get, has)
        if self._max_pos:
            self._build_tables()
        return self

    def random_state(self, seed: int = 0) -> dict:
        """Random bf16-representable tensors under the checkpoint names (norm weights near 0, output
        scales near 1/2, decays spread over fast and slow channels)."""
        cfg, W, D = self.cfg, self.cfg.hidden_size, self.cfg.side_dim
        r = lambda name, shape, s: random_full(name, shape, s, seed, self.device, torch.bfloat16)
        out = {"embed": r("embed", (cfg.vocab_size, W), W ** -0.5)}

        def t(name, shape, s, mean=0.0):
            out[name] = r(name, shape, s) if mean == 0.0 else (mean + r(name, shape, s)).bfloat16()

        def lin(name, n, k):
            t(name, (n, k), k ** -0.5)
        t("embed.norm", (W,), 0.1), t("final.norm", (W,), 0.1)
        if D:
            t("side.embed", (cfg.vocab_size, D * len(cfg.layers)), 1.0)
        for i, l in enumerate(cfg.layers):
            p, q, m, f = f"l{i}.", f"l{i}.mix.", l.mixer, l.mlp
            t(p + "norm1", (W,), 0.1), t(p + "ls1", (W,), 0.1, 0.5)
            if l.type == "parallel":
                a, b, x, y = m.left, m.right, q + "left.", q + "right."
                lin(x + "q", a.heads * a.dim, W), lin(x + "k", a.kv_heads * a.dim, W), lin(x + "v", a.kv_heads * a.vdim, W)
                t(x + "q.norm", (a.dim,), 0.1, 1.0), t(x + "k.norm", (a.dim,), 0.1, 1.0)
                t(x + "rel", (cfg.buckets, a.heads), 0.5), lin(x + "o", W, a.heads * a.vdim)
                C, w = b.width, b.width // b.blocks
                lin(y + "y", C, W), lin(y + "x", C, W), t(y + "y.b", (C,), 0.1), t(y + "x.b", (C,), 0.1)
                t(y + "conv", (C, b.conv), 0.5), t(y + "conv.b", (C,), 0.1), lin(y + "o", W, C)
                for n in ("ra", "ri"):
                    t(y + n, (b.blocks, w, w), w ** -0.5), t(y + n + ".b", (b.blocks, w), 0.1)
                t(y + "lam", (C,), 1.5, -4.0)
            elif l.type == "retention":
                for n, d in (("q", m.dim), ("k", m.dim), ("v", m.vdim), ("g", m.vdim)):
                    lin(q + n, m.heads * d, W)
                lin(q + "o", W, m.heads * m.vdim)
            else:
                lin(q + "dq", m.q_rank, W), t(q + "dq.norm", (m.q_rank,), 0.1, 1.0)
                lin(q + "uq", m.heads * (m.dim + m.rot_dim), m.q_rank)
                if m.kv_from < 0:
                    lin(q + "dkv", m.kv_rank + m.rot_dim, W), t(q + "dkv.norm", (m.kv_rank,), 0.1, 1.0)
                lin(q + "uk", m.heads * m.dim, m.kv_rank), lin(q + "uv", m.heads * m.vdim, m.kv_rank)
                lin(q + "o", W, m.heads * m.vdim)
            if f is not None:
                t(p + "norm2", (W,), 0.1), t(p + "ls2", (W,), 0.1, 0.5)
                if isinstance(f, XieluFFSpec):
                    lin(p + "mlp.up", f.ff, W), lin(p + "mlp.down", W, f.ff), t(p + "mlp.act", (2,), 0.5)
                else:
                    t(p + "mlp.router", (f.experts, W), 0.5), t(p + "mlp.correction", (f.experts,), 0.05)
                    for e in range(f.experts):
                        lin(p + f"mlp.e{e}.up", f.ff, W), lin(p + f"mlp.e{e}.down", W, f.ff)
            if D:
                lin(p + "side.gate", D, W), lin(p + "side.proj", W, D), t(p + "side.norm", (W,), 0.1, 0.5)
        return out

    def init_random(self, seed: int = 0) -> "LefuvikForCausalLM":
        return self.load_state(self.random_state(seed))

    def pack_decode_weights(self) -> None:
        """Block-packed copies of the projections and expert weights for the decode GEMM (engine hook)."""
        for L in self.layers:
            for m in (L.mix, L.mlp, L.side):
                if m is not None:
                    m.pack()

    def to(self, device, *a, **k):  # keeps the fp32 tensors fp32 (no dtype argument)
        super().to(device)
        self.device = torch.device(device)
        if self._max_pos:
            self._build_tables()
        return self

    # ------------------------------------------------------- rotations, cache and state
    def reserve_positions(self, max_pos: int) -> None:
        """Build the rotation tables for positions below ``max_pos`` (engine hook: max_model_len)."""
        if max_pos > self._max_pos:
            self._max_pos = max_pos
            if self.embed is not None:
                self._build_tables()

    def _build_tables(self) -> None:
        made = {}
        for L in self.layers:
            rot = getattr(L.mix.spec, "rot", None)
            if rot is None:
                continue
            key = (rot.dims, rot.base)
            if key not in made:
                made[key] = ma_ops.table_for(rot, self._max_pos, self.device)
            L.mix.table = made[key]

    def cache_bytes_per_block(self, block_size: int) -> int:
        esz = 2 if self.dtype == torch.bfloat16 else 4
        return max(self.cfg.kv_bytes_per_token(esz) * block_size, 1)

    def state_bytes_per_slot(self) -> int:
        return 4 * sum(L.mix.state_floats() for L in self.layers if L.kind != "latent_attention")

    def alloc_cache(self, num_blocks: int, block_size: int, num_slots: int) -> list:
        """Per layer: a dict with the mixer's state tensors ([slots, ...] fp32) and, for a parallel mixer, the
        paged ``k`` / ``v`` [blocks, G, block_size, D | V]; for latent attention a tuple of one paged cache
        [blocks, 1, block_size, R + Dr], the very one of layer ``kv_from`` where that is set."""
        out, dev = [], self.device
        page = lambda heads, w: torch.zeros((num_blocks, heads, block_size, w), dtype=self.dtype, device=dev)
        for L, l in zip(self.layers, self.cfg.layers):
            m = l.mixer
            if l.type == "latent_attention":
                out.append(out[m.kv_from] if m.kv_from >= 0 else (page(1, m.kv_rank + m.rot_dim),))
                continue
            c = L.mix.state(max(num_slots, 1), dev)
            if l.type == "parallel":
                c["k"], c["v"] = page(m.left.kv_heads, m.left.dim), page(m.left.kv_heads, m.left.vdim)
            out.append(c)
        return out

    def activation_bytes_per_token(self) -> int:
        W, widest = self.cfg.hidden_size, 0
        for l in self.cfg.layers:
            m, f = l.mixer, l.mlp
            if l.type == "parallel":
                a, b = m.left, m.right
                n = 2 * ((a.heads + a.kv_heads) * a.dim + (a.kv_heads + a.heads) * a.vdim) + 8 * b.width
            elif l.type == "retention":
                n = 2 * m.heads * (2 * m.dim + 4 * m.vdim)
            else:
                n = 2 * m.q_rank + m.kv_rank + m.rot_dim + m.heads * (m.dim + m.rot_dim) + 4 * m.heads * (
                    m.kv_rank + m.rot_dim) + 2 * m.heads * m.vdim
            if isinstance(f, XieluFFSpec):
                n = max(n, 2 * f.ff)
            elif f is not None:
                n = max(n, f.top * (2 * f.ff + 2 * W) + f.experts)
            widest = max(widest, n)
        return 4 * W * 6 + 4 * widest + 4 * self.cfg.side_dim

    # ------------------------------------------------------------------ forward
    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, md, caches: list, trail: Optional[List] = None) -> torch.Tensor:
        """The fp32 stream [T, 1, W] after the last layer, for the step described by ``md``
        (ops/attention.py AttnMetadata: the whole-batch fields).  ``trail``: a list that receives a copy
        of the stream after every layer (diagnostics)."""
        cfg, eps, dt = self.cfg, self.cfg.rms_eps, self.dtype
        if positions.numel() and self._max_pos == 0:
            raise RuntimeError("Lefuvik: reserve_positions(max_model_len) has not been called")
        close = (self.unit_mix, self.one)

        def step(y, open_, **kw):
            return hyper_ops.hyper_step(x, y, close if y is not None else None, open_, eps, dt, **kw)
        x = hyper_ops.embed_norm_rows(self.embed, input_ids, self.embed_norm, eps)
        h, _ = step(None, (self.one, self.layers[0].norm1))
        for i, L in enumerate(self.layers):
            nxt = (self.one, self.layers[i + 1].norm1) if i + 1 < len(self.layers) else None
            y, scale = L.mix(h, positions, md, caches[i], eps), L.scale1
            if L.mlp is not None:
                h, h32 = step(y, (self.one, L.norm2), y_scale=scale, want_f32=isinstance(L.mlp, GroupedMoE))
                y, scale = L.mlp(h, h32), L.scale2
            if L.side is not None:
                xa, _ = step(y, (self.one, None), y_scale=scale)
                h, _ = step(L.side(xa, self.side_embed, input_ids), nxt, post_w=L.side.norm_w)
            else:
                h, _ = step(y, nxt, y_scale=scale)
            if trail is not None:
                trail.append(x[:, 0].clone())
        return x

    def compute_logits(self, rows: torch.Tensor) -> torch.Tensor:
        """fp32 logits of stream rows [n, 1, W]: the final norm, the embedding table, the cap."""
        act, _ = hyper_ops.hyper_step(rows.contiguous(), None, None, (self.one, self.final_norm), self.cfg.rms_eps, self.dtype)
        return tanh_cap(gemm.linear(act, self.embed).float(), self.cfg.logit_softcap)
