"""Lightning attention: linear attention with one constant decay per head (or one per step and head) and an
fp32 state per (sequence, head) carried from step to step (csrc/mixers/lightning.hip; PyTorch on CPU).

    S_t = decay_h * S_{t-1} + k_t v_t^T        o_t = S_t^T q_t        q, k, v = silu(projections)

The state of one layer run is ``[slots, H, D, V]`` fp32; a sequence's slot is read by the first
token of its portion (zeros at position 0, whatever an earlier owner left there) and takes the
state after the portion's last token.
"""
from __future__ import annotations

from typing import Optional

import torch

from . import native
from .masked_attention import turn


def lightning_attention(qkv: torch.Tensor, state: torch.Tensor, decay: torch.Tensor, cu_q: torch.Tensor,
                        n_seqs: int, positions: torch.Tensor, slots: torch.Tensor, H: int, D: int, V: int,
                        num_decode: int = 0) -> torch.Tensor:
    """qkv [T, H*D | H*D | H*V] pre-activation projections (may be a column slice), heads side by
    side.  Returns o [T, H * V] fp32.  Sequences without a slot (slot < 0) start from zeros and
    leave nothing.  The first ``num_decode`` sequences hold one token each."""
    T = qkv.shape[0]
    out = torch.empty((T, H * V), dtype=torch.float32, device=qkv.device)
    if not qkv.is_cuda:
        f = torch.nn.functional.silu(qkv.float())
        q, k, v = f[:, :H * D].view(T, H, D), f[:, H * D:2 * H * D].view(T, H, D), f[:, 2 * H * D:].view(T, H, V)
        o3 = out.view(T, H, V)
        for s in range(n_seqs):
            a, b, slot = int(cu_q[s]), int(cu_q[s + 1]), int(slots[s])
            if b <= a:
                continue
            S = state[slot].clone() if (slot >= 0 and int(positions[a]) > 0) else torch.zeros((H, D, V))
            for t in range(a, b):
                S = decay[:, None, None] * S + k[t, :, :, None] * v[t, :, None, :]
                o3[t] = torch.einsum("hdv,hd->hv", S, q[t])
            if slot >= 0:
                state[slot] = S
        return out
    assert qkv.stride(1) == 1 and state.is_contiguous() and state.dtype == torch.float32 and decay.dtype == torch.float32
    assert state.shape[1:] == (H, D, V) and qkv.shape[1] == H * (2 * D + V)
    native.call("pkm_lightning_attention", out.data_ptr(), qkv.data_ptr(), qkv.stride(0), state.data_ptr(),
                decay.data_ptr(), cu_q.data_ptr(), positions.data_ptr(), slots.data_ptr(), n_seqs, T, H, D, V,
                int(num_decode), native.dt_code(qkv.dtype), native.stream_ptr())
    return out


def retention(qkv: torch.Tensor, state: torch.Tensor, decay: torch.Tensor, table: Optional[torch.Tensor], k_scale: float,
              cu_q: torch.Tensor, n_seqs: int, positions: torch.Tensor, slots: torch.Tensor, H: int, D: int,
              V: int) -> torch.Tensor:
    """The same recurrence on plain projections: q and k turn by the token's position (``table``
    [positions, pairs, 2] fp32 (cos, sin), pair i = (i, i + pairs); None: not) and k is multiplied by
    ``k_scale``, both in fp32.  qkv [T, H*D | H*D | H*V] (may be a column slice) -> o [T, H * V] fp32."""
    T = qkv.shape[0]
    out = torch.empty((T, H * V), dtype=torch.float32, device=qkv.device)
    if not qkv.is_cuda:
        f = qkv.float()
        q, k, v = f[:, :H * D].view(T, H, D), f[:, H * D:2 * H * D].view(T, H, D), f[:, 2 * H * D:].view(T, H, V)
        if table is not None:
            cs = table[positions.long()]
            q, k = turn(q, cs), turn(k, cs)
        k = k * k_scale
        o3 = out.view(T, H, V)
        for s in range(n_seqs):
            a, b, slot = int(cu_q[s]), int(cu_q[s + 1]), int(slots[s])
            if b <= a:
                continue
            S = state[slot].clone() if (slot >= 0 and int(positions[a]) > 0) else torch.zeros((H, D, V))
            for t in range(a, b):
                S = decay[:, None, None] * S + k[t, :, :, None] * v[t, :, None, :]
                o3[t] = torch.einsum("hdv,hd->hv", S, q[t])
            if slot >= 0:
                state[slot] = S
        return out
    assert qkv.stride(1) == 1 and state.is_contiguous() and state.dtype == torch.float32 and decay.dtype == torch.float32
    assert state.shape[1:] == (H, D, V) and qkv.shape[1] == H * (2 * D + V) and decay.numel() == H
    assert table is None or (table.dtype == torch.float32 and table.is_contiguous() and 2 * table.shape[1] <= D)
    native.call("pkm_retention", out.data_ptr(), qkv.data_ptr(), qkv.stride(0), state.data_ptr(), decay.data_ptr(),
                native.ptr(table), table.shape[1] if table is not None else 0, table.shape[0] if table is not None else 0,
                float(k_scale), cu_q.data_ptr(), positions.data_ptr(), slots.data_ptr(), n_seqs, T, H, D, V,
                native.dt_code(qkv.dtype), native.stream_ptr())
    return out


def step_scan(xbc: torch.Tensor, dt: torch.Tensor, dt_bias: torch.Tensor, a_log: torch.Tensor, skip: torch.Tensor,
              state: torch.Tensor, cu_q: torch.Tensor, n_seqs: int, positions: torch.Tensor, slots: torch.Tensor, H: int, N: int,
              V: int, G: int) -> torch.Tensor:
    """The recurrence with a step size per (token, head) (state-space duality): d = softplus(dt + dt_bias_h),

        S <- exp(-exp(a_log_h) d) S + d B x^T        y = S^T C + skip_h x        S [N, V] fp32 per head

    xbc [T, H*V x | G*N B | G*N C] (may be a column slice), head h on B / C group h // (H / G); ``dt``
    [T, H] pre-activations of the same element type (may be a column slice); dt_bias, a_log, skip [H] fp32;
    ``state`` [slots, H, N, V] fp32.  Returns y [T, H * V] fp32."""
    T = xbc.shape[0]
    out = torch.empty((T, H * V), dtype=torch.float32, device=xbc.device)
    assert xbc.shape[1] == H * V + 2 * G * N and dt.shape == (T, H) and H % G == 0
    if not xbc.is_cuda:
        f = xbc.float()
        x, r = f[:, :H * V].view(T, H, V), H // G
        b = f[:, H * V:H * V + G * N].view(T, G, N).repeat_interleave(r, 1)
        c = f[:, H * V + G * N:].view(T, G, N).repeat_interleave(r, 1)
        d = torch.nn.functional.softplus(dt.float() + dt_bias)
        dec = torch.exp(-torch.exp(a_log) * d)
        o3 = out.view(T, H, V)
        for s in range(n_seqs):
            a, e, slot = int(cu_q[s]), int(cu_q[s + 1]), int(slots[s])
            if e <= a:
                continue
            S = state[slot].clone() if (slot >= 0 and int(positions[a]) > 0) else torch.zeros((H, N, V))
            for t in range(a, e):
                S = dec[t, :, None, None] * S + b[t, :, :, None] * (d[t, :, None] * x[t])[:, None, :]
                o3[t] = torch.einsum("hnv,hn->hv", S, c[t]) + skip[:, None] * x[t]
            if slot >= 0:
                state[slot] = S
        return out
    assert xbc.stride(1) == 1 and dt.stride(1) == 1 and dt.dtype == xbc.dtype
    assert state.is_contiguous() and state.dtype == torch.float32 and state.shape[1:] == (H, N, V)
    for w in (dt_bias, a_log, skip):
        assert w.dtype == torch.float32 and w.numel() == H
    native.call("pkm_step_scan", out.data_ptr(), xbc.data_ptr(), xbc.stride(0), dt.data_ptr(), dt.stride(0), G, dt_bias.data_ptr(),
                a_log.data_ptr(), skip.data_ptr(), state.data_ptr(), cu_q.data_ptr(), positions.data_ptr(), slots.data_ptr(),
                n_seqs, T, H, N, V, native.dt_code(xbc.dtype), native.stream_ptr())
    return out


def gated_group_norm(y: torch.Tensor, z: torch.Tensor, w: torch.Tensor, parts: int, eps: float, dtype: torch.dtype) -> torch.Tensor:
    """u = y * silu(z); each of ``parts`` equal parts of u over its own root mean square, times w [N]: y [T, N]
    fp32, z [T, N] (may be a column slice) -> [T, N] in ``dtype``."""
    T, N = y.shape
    out = torch.empty((T, N), dtype=dtype, device=y.device)
    assert N % parts == 0 and w.numel() == N and z.shape == (T, N)
    if not y.is_cuda:
        u = (y * torch.nn.functional.silu(z.float())).view(T, parts, N // parts)
        out.copy_((u / torch.sqrt((u * u).mean(-1, keepdim=True) + eps)).view(T, N) * w)
        return out
    assert y.dtype == torch.float32 and y.is_contiguous() and w.dtype == torch.float32 and z.stride(1) == 1
    native.call("pkm_gated_group_norm", out.data_ptr(), y.data_ptr(), z.data_ptr(), z.stride(0), w.data_ptr(), T, N, parts,
                float(eps), native.dt_code(z.dtype), native.dt_code(dtype), native.stream_ptr())
    return out


def gated_rms_norm(o: torch.Tensor, w: torch.Tensor, g: torch.Tensor, eps: float, dtype: torch.dtype) -> torch.Tensor:
    """o [T, N] fp32 -> o / sqrt(mean(o^2) + eps) * w * sigmoid(g) in ``dtype``; g [T, N] may be a
    column slice of a wider projection output."""
    T, N = o.shape
    out = torch.empty((T, N), dtype=dtype, device=o.device)
    if not o.is_cuda:
        z = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps) * w
        out.copy_(z * torch.sigmoid(g.float()))
        return out
    assert o.dtype == torch.float32 and o.is_contiguous() and w.dtype == torch.float32 and g.stride(1) == 1
    native.call("pkm_gated_rms_norm", out.data_ptr(), o.data_ptr(), w.data_ptr(), g.data_ptr(), g.stride(0), T, N,
                float(eps), native.dt_code(g.dtype), native.dt_code(dtype), native.stream_ptr())
    return out
