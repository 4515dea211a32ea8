"""Vagelix decoder: one fp32 residual stream that starts from the normed embedding; sublayers read the
stream itself and only their outputs are normed.  Mixers are chunked attention beside a gated delta rule
with per-channel decays, state-space duality, or causal differential attention; feed-forwards are
SiLU-gated dense ones.  A layer may use another one's weights with a cache / state of its own.

Per layer, for the step's tokens (x: fp32 stream [T, W]; a = the model's dtype, bf16 or fp32; norms,
the stream, rotations, query temperatures, scores, softmax, step sizes, decays, unit vectors and
recurrent states are fp32):

    h   = x -> a
    parallel:   q | k | q' | k' | v' | low | g | b = h @ [...]^T   (both branches, one product)  hipBLASLt / decode GEMM
                left  v = k + bias -> cache ; all q heads (all k heads) together set to unit RMS times a
                      weight, turned by the position ; k -> cache                      HIP  row_norm.hip
                      softmax with one exp(0) more over the keys of the token's chunk, times sigmoid(g)
                                                                                       HIP  masked_attention.hip
                right z | y = low @ blockdiag(Wa2, Wg2)^T
                      q', k', v' = silu(filter(.)), q', k' unit ; decay = exp(-exp(A) softplus(z + bias))  HIP  delta.hip
                      S <- decay S (rows) ; u = beta (v - S^T k) ; S += k u^T ; o = S^T q  (state [H, D, V] fp32 per slot)
                      o = unit_rms_per_head(o) w sigmoid(y)                            HIP  head_norm_gate
                m_l, m_r = left @ Wo^T, right @ Wo'^T
                x <- x + unit_rms((unit_rms(m_l) wl + unit_rms(m_r) wr) / 2) w1 ; h   (one kernel)  HIP  hyper.hip
    mamba2:     z | x | B | C | dt = h @ Win^T ; x, B, C = silu(filter(.) + bias)      HIP  short_conv.hip
                S <- exp(-exp(A) d) S + d B x^T ; y = S^T C + D x, d = softplus(dt + bias)  (state [H, N, V] fp32)  HIP  lightning.hip
                o = unit_rms_per_part(y silu(z)) w                                     HIP  row_norm.hip
    attention:  as models/nopunex.py DiffAttention: normed heads, a query temperature, no rotation, no gate
    x   <- x + unit_rms(o @ Wo^T) w1 ; h                                 (one kernel)  HIP  hyper.hip
    f   = (silu(h @ Wgate^T) * (h @ Wup^T)) @ Wdown^T
    x   <- x + unit_rms(f) w2 ; the next layer's h                       (one kernel)

and logits = embed @ (unit_rms(x) w).  Tensor parallelism is not implemented for this family.
"""
from __future__ import annotations

from typing import List, Optional

import torch
from torch import nn

from ..ops import delta as delta_ops
from ..ops import gemm
from ..ops import hyper as hyper_ops
from ..ops import lightning as lightning_ops
from ..ops import masked_attention as ma_ops
from ..ops import short_conv as conv_ops
from ..parallel.state import ParallelState
from .bibezen import _f32
from .config import VagelixConfig
from .kivezen import _p, _packed, _project
from .nopunex import DiffAttention, GatedFF, _pad_rows
from .weights import SafetensorsIndex, random_full


def _stack_rows(parts: list) -> tuple:
    """The parts' rows under each other, each part from a multiple of 8 rows on (16-byte column slices of the
    product), and the parts' first rows."""
    rows, at = [], []
    for w in parts:
        at.append(sum(r.shape[0] for r in rows))
        rows += [w, w.new_zeros((-w.shape[0] % 8, w.shape[1]))]
    return torch.cat(rows, 0), at


class ChunkDeltaMixer(nn.Module):
    """Chunked attention on its own keys (left) beside a gated delta rule with per-channel decays (right): one
    input projection over both branches, one output projection each."""

    def __init__(self, spec, width: int):
        super().__init__()
        self.spec, self.width = spec, width
        self.w_in = self.w_in_p = None      # rows: left q, k | right q, k, v | low ranks (decay, gate) | left g | right b
        self.at = ()                        # the first rows of these parts
        self.qk_b = self.q_norm = self.k_norm = self.sink = None    # [(H + G) D], [H D], [G D], [H] fp32
        self.table = None                   # [positions, pairs, 2] fp32; None: no rotation
        self.taps = None                    # [2 G' D' + H' V', K] fp32
        self.low = self.low_p = None        # [H' D' | H' V', ranks]: block diagonal
        self.a_log = self.dt_bias = self.norm_w = None              # [H'], [H' D'], [V'] fp32
        self.w_l = self.w_r = self.w_l_p = self.w_r_p = None        # [W, H D], [W, H' V']
        self.out_l = self.out_r = None      # [W] fp32: weights of the branches' output norms

    def pack(self) -> None:
        self.w_in_p, self.low_p, self.w_l_p, self.w_r_p = (_packed(w) for w in (self.w_in, self.low, self.w_l, self.w_r))

    def set(self, get, dtype, device) -> None:
        s, r, W = self.spec.left, self.spec.right, self.width
        H, G, D = s.heads, s.kv_heads, s.dim
        RH, RG, RD, RV, K = r.heads, r.kv_heads, r.dim, r.vdim, r.conv
        a, b = (lambda n: get("left." + n)), (lambda n: get("right." + n))
        assert a("q").shape == (H * D, W) and a("k").shape == (G * D, W) and a("g").shape == (H, W) and a("o").shape == (W, H * D)
        assert b("q").shape == (RG * RD, W) == b("k").shape and b("v").shape == (RH * RV, W) and b("b").shape == (RH, W)
        assert b("q.conv").shape == (RG * RD, K) == b("k.conv").shape and b("v.conv").shape == (RH * RV, K) and b("o").shape == (W, RH * RV)
        ra, rg = b("a1").shape[0], b("g1").shape[0]
        assert b("a1").shape == (ra, W) and b("a2").shape == (RH * RD, ra) and b("g1").shape == (rg, W) and b("g2").shape == (RH * RV, rg)
        to = lambda t: _p(t.to(device=device, dtype=dtype))
        f32 = lambda t, n: _f32(t.reshape(n), device)
        w, self.at = _stack_rows([torch.cat([a("q"), a("k")], 0), torch.cat([b("q"), b("k"), b("v")], 0),
                                  torch.cat([b("a1"), b("g1")], 0), a("g"), b("b")])
        self.w_in = to(_pad_rows(w))
        self.qk_b = f32(torch.cat([a("q.b").reshape(-1), a("k.b").reshape(-1)]), (H + G) * D)
        self.q_norm, self.k_norm = f32(a("q.norm"), H * D), f32(a("k.norm"), G * D)
        # ``sink`` terms exp(0) in the denominator are one sink logit ln(sink) per head
        self.sink = _f32(torch.full((H,), s.sink).log(), device) if s.sink > 0 else None
        self.taps = _f32(torch.cat([b("q.conv"), b("k.conv"), b("v.conv")], 0), device)
        low = b("a2").new_zeros((RH * (RD + RV), ra + rg))
        low[:RH * RD, :ra], low[RH * RD:, ra:] = b("a2"), b("g2")
        self.low = to(_pad_rows(low))
        self.a_log, self.dt_bias, self.norm_w = f32(b("A_log"), RH), f32(b("dt_bias"), RH * RD), f32(b("norm"), RV)
        self.w_l, self.w_r = to(a("o")), to(b("o"))
        self.out_l, self.out_r = f32(get("left.out"), W), f32(get("right.out"), W)
        self.ranks = ra + rg

    def forward(self, h, positions, md, cache: dict, eps: float) -> tuple:
        s, r = self.spec.left, self.spec.right
        H, G, D = s.heads, s.kv_heads, s.dim
        RH, RG, RD, RV = r.heads, r.kv_heads, r.dim, r.vdim
        proj = _project(h, self.w_in, self.w_in_p)
        qk, dl, lo, gt, bt = (proj[:, i:i + n] for i, n in zip(self.at, ((H + G) * D, 2 * RG * RD + RH * RV, self.ranks, H, RH)))
        q = ma_ops.row_norm_cache(qk, self.qk_b, self.q_norm, self.k_norm, eps, positions, md.slot_mapping, self.table,
                                  s.rot is None or s.rot.halves, cache["k"], cache["v"], H, G, D)
        a = ma_ops.masked_attention(q, cache["k"], cache["v"], D, md.block_tables, md.cu_q, md.context_lens, md.num_seqs, s.scale,
                                    chunk=s.chunk, sink=self.sink, fine=True, head_gate=gt, out_dtype=h.dtype,
                                    num_decode=md.num_decode).view(-1, H * D)
        z = _project(lo, self.low, self.low_p)
        qkv, gates = delta_ops.conv_unit(dl, self.taps, cache["conv"], md.cu_q, md.num_seqs, positions, md.state_slots, md.token_seq,
                                         RG, RD, RH, RV, num_decode=md.num_decode,
                                         decay=(z[:, :RH * RD], self.a_log, self.dt_bias))
        o = delta_ops.delta_rule(qkv, bt, None, None, cache["delta"], md.cu_q, md.num_seqs, positions, md.state_slots, RG, RD, RH,
                                 RV, gates=gates)
        b = ma_ops.head_norm_gate(o, RH, RV, eps, z[:, RH * RD:RH * (RD + RV)], ma_ops.GATE_SIGMOID, h.dtype, weight=self.norm_w)
        return _project(a, self.w_l, self.w_l_p, partial=True), _project(b, self.w_r, self.w_r_p, partial=True)

    def close(self, x, y: tuple, norm_w, eps: float, dtype):
        return hyper_ops.pair_step(x, y[0], y[1], self.out_l, self.out_r, self.spec.left_scale, self.spec.right_scale, norm_w, eps,
                                   dtype)

    def state(self, slots: int, device) -> dict:
        r = self.spec.right
        z = lambda *s: torch.zeros((slots,) + s, dtype=torch.float32, device=device)
        return {"delta": z(r.heads, r.dim, r.vdim), "conv": z(max(r.conv - 1, 1), 2 * r.kv_heads * r.dim + r.heads * r.vdim)}

    def state_floats(self) -> int:
        r = self.spec.right
        return r.heads * r.dim * r.vdim + max(r.conv - 1, 1) * (2 * r.kv_heads * r.dim + r.heads * r.vdim)


class StepScanMixer(nn.Module):
    """Weights of one state-space-duality mixer."""

    def __init__(self, spec, width: int):
        super().__init__()
        self.spec, self.width = spec, width
        self.w_in = self.w_in_p = None      # [inner z | inner x | G*N B | G*N C | H dt (+ padding), W]
        self.taps = self.conv_b = None      # [inner + 2 G N, K], [inner + 2 G N] fp32
        self.dt_bias = self.a_log = self.skip = self.norm_w = None   # [H], [H], [H], [inner] fp32
        self.w_o = self.w_o_p = None        # [W, inner]

    def pack(self) -> None:
        self.w_in_p, self.w_o_p = _packed(self.w_in), _packed(self.w_o)

    def set(self, get, dtype, device) -> None:
        s, W = self.spec, self.width
        I, C = s.inner, s.inner + 2 * s.groups * s.state
        assert get("in").shape == (I + C + s.heads, W) and get("conv").shape == (C, s.conv) and get("o").shape == (W, I)
        self.w_in = _p(_pad_rows(get("in")).to(device=device, dtype=dtype))
        self.w_o = _p(get("o").to(device=device, dtype=dtype))
        self.taps, self.conv_b = _f32(get("conv"), device), _f32(get("conv.b").reshape(C), device)
        self.dt_bias, self.a_log, self.skip = (_f32(get(n).reshape(s.heads), device) for n in ("dt_bias", "A_log", "D"))
        self.norm_w = _f32(get("norm").reshape(I), device)

    def forward(self, h, positions, md, cache: dict, eps: float):
        s = self.spec
        I, C = s.inner, s.inner + 2 * s.groups * s.state
        proj = _project(h, self.w_in, self.w_in_p)
        xbc = conv_ops.causal_conv(proj[:, I:I + C], self.taps, self.conv_b, cache.get("conv"), md.cu_q, md.num_seqs, positions,
                                   md.state_slots, md.token_seq, act=conv_ops.ACT_SILU, num_decode=md.num_decode)
        y = lightning_ops.step_scan(xbc, proj[:, I + C:I + C + s.heads], self.dt_bias, self.a_log, self.skip, cache["scan"], md.cu_q,
                                    md.num_seqs, positions, md.state_slots, s.heads, s.state, s.vdim, s.groups)
        o = lightning_ops.gated_group_norm(y, proj[:, :I], self.norm_w, s.norm_groups, eps, h.dtype)
        return _project(o, self.w_o, self.w_o_p, partial=True)

    def state(self, slots: int, device) -> dict:
        s = self.spec
        out = {"scan": torch.zeros((slots, s.heads, s.state, s.vdim), dtype=torch.float32, device=device)}
        if s.conv > 1:
            out["conv"] = torch.zeros((slots, s.conv - 1, s.inner + 2 * s.groups * s.state), dtype=torch.float32, device=device)
        return out

    def state_floats(self) -> int:
        s = self.spec
        return s.heads * s.state * s.vdim + (s.conv - 1) * (s.inner + 2 * s.groups * s.state)


_MIXERS = {"parallel": ChunkDeltaMixer, "mamba2": StepScanMixer, "attention": DiffAttention}


class VagelixLayer(nn.Module):
    def __init__(self, spec, width: int):
        super().__init__()
        self.kind = spec.type
        self.mix = _MIXERS[spec.type](spec.mixer, width)
        self.mlp = GatedFF(spec.mlp) if spec.mlp is not None else None
        self.norm1 = self.norm2 = None      # [W] fp32: weights of the norms behind the sublayers


class VagelixForCausalLM(nn.Module):
    # engine hooks (engine/model_runner.py): this family owns its cache and state layouts
    supports_graphs = True

    def __init__(self, cfg: VagelixConfig, st: ParallelState, dtype: torch.dtype, device: torch.device):
        super().__init__()
        if st.tp_size > 1 or getattr(st, "ep_size", 1) > 1:
            raise ValueError("Vagelix runs on one GPU (no TP / EP sharding for this family)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Vagelix runs in bfloat16 or float32, not {dtype}")
        self.cfg, self.st, self.dtype, self.device = cfg, st, dtype, device
        self.needs_state = cfg.needs_state
        own = [VagelixLayer(l, cfg.hidden_size) if l.weights_of < 0 else None for l in cfg.layers]
        # one entry per layer run; a layer on another one's weights is that very module
        self.layers = nn.ModuleList(own[l.weights_of] if l.weights_of >= 0 else own[i] for i, l in enumerate(cfg.layers))
        self.embed = self.embed_norm = self.final_norm = None
        self.one = self.unit_mix = None     # the plain residual's stream coefficients [1], [1, 1]
        self._max_pos = 0

    # ------------------------------------------------------------------ weights
    def _norm(self, get, name: str) -> nn.Parameter:
        w = get(name)
        assert w.numel() == self.cfg.hidden_size, name
        return _f32(w.reshape(-1), self.device)

    def _set_layer(self, i: int, get) -> None:
        L, spec, W = self.layers[i], self.cfg.layers[i], self.cfg.hidden_size
        p, dev, dt = f"l{i}.", self.device, self.dtype
        m = lambda n: get(p + "mix." + n)
        if L.kind == "attention":
            L.mix.set(m("q"), m("k"), m("v"), None, m("o"), m("lq1"), m("lk1"), m("lq2"), m("lk2"), dt, dev, m("q.norm"), m("k.norm"))
        else:
            L.mix.set(m, dt, dev)
        L.norm1 = self._norm(get, p + "norm1")
        if spec.mlp is not None:
            L.norm2 = self._norm(get, p + "norm2")
            gate, up, down = get(p + "mlp.gate"), get(p + "mlp.up"), get(p + "mlp.down")
            assert gate.shape == (spec.mlp.ff, W) == up.shape and down.shape == (W, spec.mlp.ff)
            L.mlp.set(gate, up, down, dt, dev)

    def load_hf(self, path: str) -> "VagelixForCausalLM":
        """Load a checkpoint folder (safetensors; tensors under the design's own names)."""
        return self._load(SafetensorsIndex(path).get)

    def load_state(self, tensors: dict) -> "VagelixForCausalLM":
        """The same from a dict name -> tensor (tests)."""
        return self._load(tensors.__getitem__)

    def _load(self, get) -> "VagelixForCausalLM":
        cfg, dev = self.cfg, self.device
        self.embed = _p(get("embed").to(device=dev, dtype=self.dtype))
        assert self.embed.shape == (cfg.vocab_size, cfg.hidden_size)
        self.embed_norm, self.final_norm = self._norm(get, "embed.norm"), self._norm(get, "final.norm")
        self.one = _p(torch.ones(1, dtype=torch.float32, device=dev))
        self.unit_mix = _p(torch.ones((1, 1), dtype=torch.float32, device=dev))
        for i, l in enumerate(cfg.layers):
            if l.weights_of < 0:
                self._set_layer(i, get)
        if self._max_pos:
            self._build_tables()
        return self

    def random_state(self, seed: int = 0) -> dict:
        """Random bf16-representable tensors under the checkpoint names (norm weights near 1, decays spread
        over fast and slow channels)."""
        cfg, W = self.cfg, self.cfg.hidden_size
        r = lambda name, shape, s: random_full(name, shape, s, seed, self.device, torch.bfloat16)
        out = {"embed": r("embed", (cfg.vocab_size, W), W ** -0.5)}

        def t(name, shape, s, mean=0.0):
            out[name] = r(name, shape, s) if mean == 0.0 else (mean + r(name, shape, s)).bfloat16()

        def lin(name, n, k):
            t(name, (n, k), k ** -0.5)
        t("embed.norm", (W,), 0.1, 1.0), t("final.norm", (W,), 0.1, 1.0)
        for i, l in enumerate(cfg.layers):
            if l.weights_of >= 0:
                continue
            p, q, m, f = f"l{i}.", f"l{i}.mix.", l.mixer, l.mlp
            t(p + "norm1", (W,), 0.1, 0.5)
            if l.type == "parallel":
                a, b, x, y = m.left, m.right, q + "left.", q + "right."
                for n, rows in (("q", a.heads * a.dim), ("k", a.kv_heads * a.dim)):
                    lin(x + n, rows, W), t(x + n + ".b", (rows,), 0.1), t(x + n + ".norm", (rows,), 0.1, 1.0)
                lin(x + "g", a.heads, W), lin(x + "o", W, a.heads * a.dim)
                for n, rows in (("q", b.kv_heads * b.dim), ("k", b.kv_heads * b.dim), ("v", b.heads * b.vdim)):
                    lin(y + n, rows, W), t(y + n + ".conv", (rows, b.conv), 0.5)
                ra, rg = b.decay_rank or b.dim, b.gate_rank or b.dim
                lin(y + "b", b.heads, W), lin(y + "a1", ra, W), lin(y + "a2", b.heads * b.dim, ra)
                lin(y + "g1", rg, W), lin(y + "g2", b.heads * b.vdim, rg), lin(y + "o", W, b.heads * b.vdim)
                t(y + "A_log", (b.heads,), 0.5), t(y + "dt_bias", (b.heads * b.dim,), 1.5, -4.0), t(y + "norm", (b.vdim,), 0.1, 1.0)
                t(q + "left.out", (W,), 0.1, 1.0), t(q + "right.out", (W,), 0.1, 1.0)
            elif l.type == "mamba2":
                C = m.inner + 2 * m.groups * m.state
                lin(q + "in", m.inner + C + m.heads, W), lin(q + "o", W, m.inner)
                t(q + "conv", (C, m.conv), 0.5), t(q + "conv.b", (C,), 0.1), t(q + "norm", (m.inner,), 0.1, 1.0)
                t(q + "dt_bias", (m.heads,), 1.0, -3.0), t(q + "A_log", (m.heads,), 0.5, 1.0), t(q + "D", (m.heads,), 0.1, 1.0)
            else:
                lin(q + "q", 2 * m.heads * m.dim, W), lin(q + "k", 2 * m.kv_heads * m.dim, W)
                lin(q + "v", m.kv_heads * m.vdim, W), lin(q + "o", W, m.heads * m.vdim)
                t(q + "q.norm", (m.dim,), 0.1, 1.0), t(q + "k.norm", (m.dim,), 0.1, 1.0)
                for n in ("lq1", "lk1", "lq2", "lk2"):
                    t(q + n, (m.dim,), 0.1)
            if f is not None:
                t(p + "norm2", (W,), 0.1, 0.5)
                lin(p + "mlp.gate", f.ff, W), lin(p + "mlp.up", f.ff, W), lin(p + "mlp.down", W, f.ff)
        return out

    def init_random(self, seed: int = 0) -> "VagelixForCausalLM":
        return self.load_state(self.random_state(seed))

    def _own_layers(self):
        return (L for L, l in zip(self.layers, self.cfg.layers) if l.weights_of < 0)

    def pack_decode_weights(self) -> None:
        """Block-packed copies of the projections for the decode GEMM (engine hook)."""
        for L in self._own_layers():
            L.mix.pack()
            if L.mlp is not None:
                L.mlp.pack()

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
        for L in self._own_layers():
            rot = L.mix.spec.left.rot if L.kind == "parallel" else None
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
        return 4 * sum(L.mix.state_floats() for L in self.layers if L.kind != "attention")

    def alloc_cache(self, num_blocks: int, block_size: int, num_slots: int) -> list:
        """Per layer run, also where the weights are another layer's: a dict with the mixer's state tensors
        ([slots, ...] fp32) and, for a parallel mixer, the paged ``k`` / ``v`` [blocks, G, block_size, D];
        for attention the paged (k, v) [blocks, 2G, block_size, D], [blocks, G, block_size, V]."""
        out, dev = [], self.device
        page = lambda heads, w: torch.zeros((num_blocks, heads, block_size, w), dtype=self.dtype, device=dev)
        for L, l in zip(self.layers, self.cfg.layers):
            m = l.mixer
            if l.type == "attention":
                out.append((page(2 * m.kv_heads, m.dim), page(m.kv_heads, m.vdim)))
                continue
            c = L.mix.state(max(num_slots, 1), dev)
            if l.type == "parallel":
                c["k"], c["v"] = page(m.left.kv_heads, m.left.dim), page(m.left.kv_heads, m.left.dim)
            out.append(c)
        return out

    def activation_bytes_per_token(self) -> int:
        W, widest = self.cfg.hidden_size, 0
        for l in self.cfg.layers:
            m = l.mixer
            if l.type == "parallel":
                a, b = m.left, m.right
                n = (3 * a.heads + a.kv_heads) * a.dim + 2 * W + 4 * b.kv_heads * b.dim + b.heads * (3 * b.dim + 6 * b.vdim)
            elif l.type == "mamba2":
                n = 5 * m.inner + 4 * m.groups * m.state + W
            else:
                n = 4 * m.heads * m.dim + 2 * m.kv_heads * m.dim + m.kv_heads * m.vdim + 4 * m.heads * m.vdim
            widest = max(widest, n, 3 * l.mlp.ff if l.mlp is not None else 0)
        return 4 * W * 6 + 4 * widest

    # ------------------------------------------------------------------ forward
    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, md, caches: list, trail: Optional[List] = None) -> torch.Tensor:
        """The fp32 stream [T, 1, W] after the last layer, for the step described by ``md``
        (ops/attention.py AttnMetadata: the whole-batch fields).  ``trail``: a list that receives a copy
        of the stream after every layer (diagnostics)."""
        eps, dt = self.cfg.rms_eps, self.dtype
        if positions.numel() and self._max_pos == 0:
            raise RuntimeError("Vagelix: reserve_positions(max_model_len) has not been called")
        close, copy = (self.unit_mix, self.one), (self.one, None)
        x = hyper_ops.embed_norm_rows(self.embed, input_ids, self.embed_norm, eps)
        h, _ = hyper_ops.hyper_step(x, None, None, copy, eps, dt)
        for L, cache in zip(self.layers, caches):
            y = L.mix(h, positions, md, cache, eps)
            if isinstance(y, tuple):
                h = L.mix.close(x, y, L.norm1, eps, dt)
            else:
                h, _ = hyper_ops.hyper_step(x, y, close, copy, eps, dt, post_w=L.norm1)
            if L.mlp is not None:
                h, _ = hyper_ops.hyper_step(x, L.mlp(h), close, copy, eps, dt, post_w=L.norm2)
            if trail is not None:
                trail.append(x[:, 0].clone())
        return x

    def compute_logits(self, rows: torch.Tensor) -> torch.Tensor:
        """fp32 logits of stream rows [n, 1, W]: the final norm, then the embedding table."""
        act, _ = hyper_ops.hyper_step(rows.contiguous(), None, None, (self.one, self.final_norm), self.cfg.rms_eps, self.dtype)
        return gemm.linear(act, self.embed).float()
