"""Real-gated linear recurrence: one fp32 number of state per channel, block-diagonal gates, a GELU
branch on the output (csrc/mixers/lru.hip; PyTorch on CPU).

    r = sigmoid(R_b u_b + rb),  i = sigmoid(I_b u_b + ib)        u split into equal parts u_b
    a = exp(lam * r);  S <- a S + sqrt(1 - a^2) i u;  out = S * gelu_tanh(y + yb) * post

``state`` [slots, C] fp32 per sequence; a portion's first token reads it unless it is position 0 (a
new sequence starts from zeros), the slot then takes the state after the portion's last token.  The
gate products accumulate and stay in fp32, as do decays and the recurrence.
"""
from __future__ import annotations

from typing import Optional

import torch

from . import native

RUN = 32  # tokens per run of the prompt scan (csrc/mixers/lru.hip kRun)


def gated_lru(u: torch.Tensor, y: torch.Tensor, y_bias: torch.Tensor, ra: torch.Tensor, ri: torch.Tensor, ra_b: torch.Tensor,
              ri_b: torch.Tensor, lam: torch.Tensor, state: torch.Tensor, cu_q: torch.Tensor, n_seqs: int,
              positions: torch.Tensor, slots: torch.Tensor, num_decode: int = 0, post: float = 1.0,
              out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """u, y [T, C] (each may be a column slice), ra / ri [blocks, C / blocks, C / blocks] ([out, in]) in u's
    dtype, y_bias, ra_b, ri_b, lam [C] fp32 (lam negative).  The first ``num_decode`` sequences hold one
    token each (all of them: one fused kernel).  ``out``: write there (may be a column slice)."""
    T, C = u.shape
    nb, w = ra.shape[0], ra.shape[1]
    if out is None:
        out = torch.empty((T, C), dtype=u.dtype, device=u.device)
    assert ra.shape == ri.shape == (nb, w, w) and nb * w == C and y.shape == (T, C) == out.shape
    if not u.is_cuda:
        f = u.float()
        ub = f.view(T, nb, w).transpose(0, 1)
        r = torch.sigmoid(torch.bmm(ub, ra.float().transpose(1, 2)).transpose(0, 1).reshape(T, C) + ra_b)
        i = torch.sigmoid(torch.bmm(ub, ri.float().transpose(1, 2)).transpose(0, 1).reshape(T, C) + ri_b)
        la = lam * r
        a, b = torch.exp(la), torch.sqrt(-torch.expm1(2 * la)) * i * f
        g = torch.nn.functional.gelu(y.float() + y_bias, approximate="tanh") * post
        for s in range(n_seqs):
            lo, hi, slot = int(cu_q[s]), int(cu_q[s + 1]), int(slots[s])
            if hi <= lo:
                continue
            S = state[slot].clone() if (slot >= 0 and int(positions[lo]) > 0) else torch.zeros(C)
            for t in range(lo, hi):
                S = a[t] * S + b[t]
                out[t] = (S * g[t]).to(out.dtype)
            if slot >= 0:
                state[slot] = S
        return out
    for t in (u, y, out):
        assert t.stride(1) == 1 and t.dtype == u.dtype
    for t in (ra, ri):
        assert t.is_contiguous() and t.dtype == u.dtype
    for t in (y_bias, ra_b, ri_b, lam):
        assert t.dtype == torch.float32 and t.numel() == C and t.is_contiguous()
    assert state.dtype == torch.float32 and state.is_contiguous() and state.shape[1] == C
    single = num_decode >= n_seqs
    ab = ends = starts = None
    if not single:
        runs = T // RUN + n_seqs
        ab = torch.empty((T, C, 2), dtype=torch.float32, device=u.device)
        ends = torch.empty((runs, C, 2), dtype=torch.float32, device=u.device)
        starts = torch.empty((runs, C), dtype=torch.float32, device=u.device)
    native.call("pkm_gated_lru", out.data_ptr(), out.stride(0), u.data_ptr(), u.stride(0), y.data_ptr(), y.stride(0),
                y_bias.data_ptr(), ra.data_ptr(), ri.data_ptr(), ra_b.data_ptr(), ri_b.data_ptr(), lam.data_ptr(),
                state.data_ptr(), cu_q.data_ptr(), positions.data_ptr(), slots.data_ptr(), n_seqs, T, C, nb, float(post),
                int(single), native.ptr(ab), native.ptr(ends), native.ptr(starts), native.dt_code(u.dtype),
                native.stream_ptr())
    return out
