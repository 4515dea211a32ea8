"""Lefuvik through the framework (checkpoint loader, scheduler, block manager and state slots,
model runner, kernels) against the plain per-sequence model of tests/oracle_lefuvik.py.

Every test builds its own small configuration and random weights, writes them as a checkpoint
folder and loads that through the engine, or drives one op or mixer with hand-made inputs over a
hand-made paged cache and hand-made state slots.  The same tests run on the CPU (the ops' PyTorch
compositions) and, marked gpu, on the HIP kernels."""
import os
import random
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
import oracle_lefuvik as O  # noqa: E402
from engine_replay import (BS, Feed, checkpoint, close, cut, engine, full, i32, interleave, rand_tokens, rel, replay,  # noqa: E402
                           rows_of)

from polykey_service_amd.engine import EngineConfig, LLMEngine, SamplingParams  # noqa: E402
from polykey_service_amd.models.config import LefuvikConfig  # noqa: E402
from polykey_service_amd.parallel.state import ParallelState  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
D64 = torch.float64
PORTIONS = [3, 1, 1, 30, 2, 40, 1, 1, 1, 17]      # 97 tokens over shuffled pages


def logits_of(cfg, w, toks):
    return O.forward(cfg, w, toks)[0]


@pytest.fixture
def small(tmp_path):
    cfg = O.make_config()
    w = O.random_model(cfg, seed=3)
    return cfg, w, checkpoint(tmp_path, cfg, w)


def _mixer(kind, m, W, dev, seed, n, others=(), **kw):
    """The framework's mixer module of the last of the layers (``others`` + this one) with the oracle's
    random weights, its cache filled with what an earlier owner left, and the weights."""
    from polykey_service_amd.models import lefuvik as L
    from polykey_service_amd.ops import masked_attention as ma
    ls = [{"type": k, "mixer": mm, "mlp": None} for k, mm in list(others) + [(kind, m)]]
    cfg = {"vocab": 4, "width": W, "norm": {"eps": 1e-5}, "layers": ls}
    p = f"l{len(ls) - 1}.mix."
    w = {k[len(p):]: v for k, v in O.random_model(cfg, seed, **kw).items() if k.startswith(p)}
    spec = LefuvikConfig.from_json(cfg).layers[-1].mixer
    mod = L._MIXERS[kind](spec, W)
    nb = (n + BS - 1) // BS + 3
    if kind == "latent_attention":
        g = lambda k: w.get(k)
        mod.set(g("dq"), g("dq.norm"), g("uq"), g("dkv"), g("dkv.norm"), g("uk"), g("uv"), None, g("o"), torch.float32, dev)
        cache = (torch.full((nb, 1, BS, spec.kv_rank + spec.rot_dim), 3.0, device=dev),)
    else:
        mod.set(w.__getitem__, torch.float32, dev)
        cache = mod.state(3, dev)
        for t in cache.values():
            t.fill_(5.0)
        if kind == "parallel":
            for name, wd in (("k", spec.left.dim), ("v", spec.left.vdim)):
                cache[name] = torch.full((nb, spec.left.kv_heads, BS, wd), 3.0, device=dev)
    rot = getattr(spec, "rot", None)
    if rot is not None:
        mod.table = ma.table_for(rot, n + 3, dev)
    return mod, cache, w


def _feed(mod, cache, h, portions, pages, dev):
    return torch.cat([full(mod(h[sl].to(dev), pos, md, cache, 1e-5)) for sl, pos, md in Feed(dev, pages).portions(portions)])


# ------------------------------------------------------------------ single mechanisms
@pytest.mark.parametrize("B,D", [(8, 30), (16, 128), (32, 1024), (6, 7), (10, 1000), (2, 50), (7, 90)])
def test_distance_buckets(B, D):
    """The table by distance equals the rule, also where the logarithm's ratio is a whole number."""
    from polykey_service_amd.ops import masked_attention as ma
    rel_ = torch.arange(B).float()[:, None] * torch.tensor([1.0, -2.0])
    t = ma.distance_bias(rel_, D)
    for n in list(range(0, 2 * D + 5)):
        b = float(t[0, min(n, t.shape[1] - 1)])
        assert b == O.distance_bucket(n, B, D), n
        assert float(t[1, min(n, t.shape[1] - 1)]) == -2 * b
    if (B, D) == (16, 128):     # 8 * 16^(k / 8): a bucket starts exactly at 16, 32, 64
        assert [int(t[0, n]) for n in (7, 8, 15, 16, 31, 32, 63, 64)] == [7, 8, 9, 10, 11, 12, 13, 14]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,V,window,keep,B,bmax,C,blocks,K", [
    (4, 2, 16, 8, 24, 5, 8, 30, 24, 3, 3), (3, 3, 8, 20, 40, 33, 16, 128, 34, 1, 4), (6, 1, 6, 34, 7, 1, 4, 9, 40, 40, 1),
    (2, 2, 36, 4, 0, 0, 12, 60, 64, 1, 2), (1, 1, 70, 12, 33, 64, 6, 50, 70, 2, 6), (2, 1, 5, 3, 1, 0, 2, 5, 66, 2, 5)])
def test_parallel_mixer(device, H, G, D, V, window, keep, B, bmax, C, blocks, K):
    dev, W, n = torch.device(device), 30, sum(PORTIONS)
    m = {"left": {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": 1.4 * D ** -0.5, "bias_max": bmax,
                  "mask": {"size": window, "keep_first": keep}},
         "right": {"width": C, "blocks": blocks, "conv": K}, "left_scale": 0.6, "right_scale": 1.3}
    mod, cache, w = _mixer("parallel", m, W, dev, 13, n, buckets=B)
    h = torch.randn((n, W), generator=torch.Generator().manual_seed(3))
    want = O.parallel(h.double(), w, m, 1e-5)
    close(_feed(mod, cache, h, PORTIONS, [5, 0, 3, 1], dev), want, 5e-4)


def _probe(dev, window, keep, key, qpos, decoded, bias=None, H=4, G=2, D=8, V=4, strong=6.0):
    """Keys and values written by hand; key ``key`` points along the query, the others are small.
    Returns (the framework's output at ``qpos``, the plain rule's) [H, V] and the key's values [G, V]."""
    from polykey_service_amd.ops import masked_attention as ma
    n = qpos + 1
    g = torch.Generator().manual_seed(5)
    k, v = 0.05 * torch.randn((n, G, D), generator=g), torch.randn((n, G, V), generator=g)
    q = 0.05 * torch.randn((n, H, D), generator=g)
    k[key, :, 0], q[qpos, :, 0] = strong, strong
    pages = [3, 0, 5, 1, 2, 4][: (n + BS - 1) // BS + 1]
    kc, vc = torch.zeros((6, G, BS, D), device=dev), torch.zeros((6, G, BS, V), device=dev)
    table = None if bias is None else ma.distance_bias(bias[0], bias[1]).to(dev)
    sizes = [qpos, 1] if decoded else [max(qpos - 6, 1), n - max(qpos - 6, 1)]
    out = None
    for sl, pos, md in Feed(dev, pages).portions([c for c in sizes if c > 0]):
        at = md.slot_mapping.long()
        kc[at // BS, :, at % BS], vc[at // BS, :, at % BS] = k[sl].to(dev), v[sl].to(dev)
        out = ma.masked_attention(q[sl].contiguous().to(dev), kc, vc, V, md.block_tables, md.cu_q, md.context_lens, 1, 1.0,
                                  window=window, keep=keep, bias=table, post=0.5, num_decode=md.num_decode)
    want = O.softmax_rows(q.double(), k.double(), v.double(), 1.0, window, keep, None if bias is None else bias[0].double(),
                          None if bias is None else bias[1])
    return out[-1].view(H, V).cpu(), 0.5 * want[qpos], 0.5 * v[key].float()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("key,seen", [(100, True), (61, True), (60, False), (59, False), (0, True), (1, True), (8, True), (9, False),
                                      (10, False), (31, False), (32, False), (63, True), (64, True), (96, True)])
def test_window_edge_and_the_kept_first_tokens(device, decoded, key, seen):
    """Window 40, the first 9 kept, query at 100: keys 61..100 and 0..8 are seen."""
    got, want, val = _probe(torch.device(device), 40, 9, key, 100, decoded)
    close(got, want, 1e-4)
    if seen:
        close(got, val.repeat_interleave(2, 0), 1e-2)
    else:
        assert float((got - val.repeat_interleave(2, 0)).abs().max()) > 0.1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("key,qpos", [(0, 0), (0, 1), (31, 32), (32, 32), (32, 33), (33, 95), (34, 95), (63, 127), (64, 127)])
def test_first_tokens_page_borders_and_more_kept_than_there_are(device, key, qpos):
    """Keeping 34 tokens while the sequence holds fewer, as many or more; kept keys across a page border."""
    for decoded in ([False] if qpos == 0 else [False, True]):
        got, want, _ = _probe(torch.device(device), 16, 34, key, qpos, decoded)
        close(got, want, 1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("bucket", [0, 3, 4, 5, 7])
def test_distance_bias_picks_its_keys(device, decoded, bucket):
    """One bucket of eight far above the others: the softmax goes to that distance's keys (kept tokens by
    their true distance); the bias differs by head."""
    rel_ = torch.zeros((8, 4))
    rel_[bucket, :3] = torch.tensor([20.0, 9.0, 14.0])
    got, want, _ = _probe(torch.device(device), 50, 4, 95, 100, decoded, bias=(rel_, 40), strong=0.1)
    close(got, want, 1e-4)
    assert float((got[3] - got[2]).abs().max()) > 0.05


@pytest.mark.parametrize("device", DEVICES)
def test_unit_value_heads_and_head_norms_without_a_rotation(device):
    from polykey_service_amd.ops import masked_attention as ma
    dev = torch.device(device)
    T, QH, KH, D, V = 7, 3, 1, 12, 5
    g = torch.Generator().manual_seed(7)
    n = (QH + KH) * D + KH * V
    proj = torch.randn((T, n + 2), generator=g)
    qn, kn = torch.randn(D, generator=g), torch.randn(D, generator=g)
    kc, vc = torch.zeros((2, KH, BS, D), device=dev), torch.zeros((2, KH, BS, V), device=dev)
    pos = torch.arange(20, 20 + T, dtype=torch.int32)
    q = ma.rotate_cache(proj.to(dev)[:, :n], pos.to(dev), pos.to(dev), None, True, kc, vc, QH, KH, KH, D, V,
                        q_norm=qn.to(dev), k_norm=kn.to(dev), eps=1e-3, v_unit=True)
    f = proj.double()
    close(q, O.unit(f[:, :QH * D].view(T, QH, D), 1e-3) * qn, 1e-4)
    close(kc[0, 0, 20:20 + T], O.unit(f[:, QH * D:(QH + KH) * D], 1e-3) * kn, 1e-4)
    close(vc[0, 0, 20:20 + T], O.unit(f[:, (QH + KH) * D:n], 1e-3), 1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,V,rot", [(3, 12, 12, 12), (1, 40, 9, 8), (2, 64, 70, 0), (5, 7, 3, 2), (2, 130, 20, 130), (1, 300, 18, 256)])
def test_retention_mixer(device, H, D, V, rot):
    dev, W, n = torch.device(device), 28, sum(PORTIONS)
    m = {"heads": H, "dim": D, "vdim": V, "decay": [1 - 2.0 ** (-1 - 3 * h) for h in range(H)]}
    if rot:
        m["rot"] = {"dims": rot, "base": 90.0}
    mod, cache, w = _mixer("retention", m, W, dev, 11, n)
    h = torch.randn((n, W), generator=torch.Generator().manual_seed(1))
    close(_feed(mod, cache, h, PORTIONS, [4, 0, 2, 1], dev), O.retention(h.double(), w, m, 1e-5), 5e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_retention_keeps_a_far_token_with_slow_decay_and_loses_it_with_fast(device):
    """Value written at position 0 along key channel 0 of both heads, read at the end."""
    from polykey_service_amd.ops import lightning as lt
    dev, n, H, D, V = torch.device(device), 300, 2, 8, 6
    qkv = torch.zeros((n, H * (2 * D + V)))
    for h in range(H):
        qkv[n - 1, h * D] = qkv[0, H * D + h * D] = 1.0
        qkv[0, 2 * H * D + h * V:2 * H * D + (h + 1) * V] = torch.arange(1, V + 1).float()
    decay = torch.tensor([0.9995, 0.9])
    state = torch.full((2, H, D, V), 9.0, device=dev)
    o = torch.cat([lt.retention(qkv[sl].to(dev), state, decay.to(dev), None, 0.25, md.cu_q, 1, pos, md.state_slots, H, D, V)
                   for sl, pos, md in Feed(dev, [0] * 10).portions([100, 1, 1, 198])])
    close(o[-1].view(H, V), 0.25 * torch.arange(1, V + 1) * decay.double()[:, None] ** (n - 1), 1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("C,blocks", [(24, 3), (130, 1), (40, 40), (64, 1), (192, 2)])
@pytest.mark.parametrize("sizes", [[97], [2] * 10 + [33, 32, 1, 1, 10], [31, 32, 33, 1], [1, 96]])
def test_gated_recurrence_in_portions_with_a_dirty_slot(device, C, blocks, sizes):
    from polykey_service_amd.ops import lru
    dev, n, w = torch.device(device), sum(sizes), C // blocks
    g = torch.Generator().manual_seed(C + len(sizes))
    r = lambda *s: torch.randn(s, generator=g)
    u, y, yb = r(n, C), r(n, C + 5), r(C)
    ra, ri, rab, rib, lam = r(blocks, w, w) * w ** -0.5, r(blocks, w, w) * w ** -0.5, r(C), r(C), 1.5 * r(C) - 4.0
    d = lambda t: t.double()
    want = O.gated_linear_recurrence(d(u), d(ra), d(rab).view(blocks, w), d(ri), d(rib).view(blocks, w), d(lam)) * O.gelu(d(y[:, 2:2 + C]) + d(yb))
    state = torch.full((3, C), 7.0, device=dev)
    to = lambda t: t.to(dev)
    lam8 = to((-8 * torch.nn.functional.softplus(d(lam))).float())
    got = [lru.gated_lru(to(u[sl]), to(y[sl])[:, 2:2 + C], to(yb), to(ra), to(ri), to(rab), to(rib), lam8, state, md.cu_q, 1, pos,
                         md.state_slots, md.num_decode, 1.5) for sl, pos, md in Feed(dev, [0] * 9).portions(sizes)]
    close(torch.cat(got), 1.5 * want, 3e-4)
    assert float((state[0] - 7).abs().max()) == 0 and float((state[2] - 7).abs().max()) == 0   # other slots untouched


@pytest.mark.parametrize("device", DEVICES)
def test_gated_recurrence_remembers_far_tokens(device):
    """Closed gates (r = 0 nearly): an input of position 0 stays for hundreds of tokens; an open decay
    gate with a large lam drops it at once."""
    from polykey_service_amd.ops import lru
    dev, n, C = torch.device(device), 400, 2
    u = torch.zeros((n, C))
    u[0] = 100.0
    zero, z1 = torch.zeros((1, C, C), device=dev), torch.zeros(C, device=dev)
    ra_b = torch.tensor([-14.0, 14.0], device=dev)
    lam8 = torch.tensor([-8.0, -8.0], device=dev)
    state = torch.full((2, C), 3.0, device=dev)
    y = torch.full((n, C), 2.0, device=dev)
    o = torch.cat([lru.gated_lru(u[sl].to(dev), y[sl], z1, zero, zero, ra_b, z1, lam8, state, md.cu_q, 1, pos, md.state_slots,
                                 md.num_decode) for sl, pos, md in Feed(dev, [0] * 13).portions([150, 1, 1, 248])]).cpu().double()
    la = -8 * torch.sigmoid(ra_b.cpu().double())
    first = torch.sqrt(1 - torch.exp(2 * la)) * 50.0
    close(o[-1] / O.gelu(torch.tensor(2.0, dtype=D64)), first * torch.exp(la * (n - 1)), 1e-4)
    assert float(o[-1, 0]) > 0.1 and float(o[-1, 1]) == 0.0


@pytest.mark.gpu
@pytest.mark.parametrize("K,act,residual,bias,in_bias", [(2, 1, False, True, False), (3, 0, True, False, True), (4, 0, False, True, True)])
def test_filter_over_runs_of_tokens_in_a_batch(K, act, residual, bias, in_bias):
    """bf16 rows long enough for the run form: several sequences, some short, one continuing from its slot."""
    from polykey_service_amd.ops import short_conv as sc
    dev, C = torch.device("cuda"), 72
    lens, starts = [3, 90, 1, 2, 41, 8, 16], [0, 5, 40, 0, 0, 7, 0]
    g = torch.Generator().manual_seed(K)
    T = sum(lens)
    x, taps = torch.randn((T, C + 8), generator=g).bfloat16(), torch.randn((C, K), generator=g)
    b, ib = (torch.randn(C, generator=g) if bias else None), (torch.randn(C, generator=g) if in_bias else None)
    state = torch.randn((9, K - 1, C), generator=g)
    slots = [4, 2, 7, 0, -1, 5, 3]
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lens)])
    want, new = [], state.clone()
    for i, n in enumerate(lens):
        past = state[slots[i]].double() if starts[i] and slots[i] >= 0 else torch.zeros((K - 1, C), dtype=D64)
        xin = torch.cat([past, x[cu[i]:cu[i + 1], :C].double() + (ib.double() if in_bias else 0)])
        y = sum(xin[j:j + n] * taps.double()[:, j] for j in range(K)) + (b.double() if bias else 0)
        y = O.silu(y) if act else y
        want.append(y + (xin[K - 1:] if residual else 0))
        if slots[i] >= 0:
            new[slots[i]] = xin[-(K - 1):].float()
    to = lambda t: None if t is None else t.to(dev)
    st = to(state)
    got = sc.causal_conv(to(x)[:, :C], to(taps), to(b), st, i32(cu, dev), len(lens), to(pos.int()), i32(slots, dev),
                         i32(sum([[i] * n for i, n in enumerate(lens)], []), dev), act=act, residual=residual, in_bias=to(ib))
    close(got, torch.cat(want), 2e-2)
    close(st, new, 1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,Dr,V,R,Q,window", [(2, 9, 8, 11, 20, 26, 18), (3, 16, 4, 5, 40, 7, 33), (1, 5, 12, 30, 12, 30, 0)])
def test_latent_mixer_and_one_on_its_cache(device, H, D, Dr, V, R, Q, window):
    dev, W, n = torch.device(device), 30, sum(PORTIONS)
    m = {"heads": H, "dim": D, "vdim": V, "kv_rank": R, "q_rank": Q, "rot_dim": Dr, "scale": 0.4, "rot": {"dims": Dr, "base": 50.0},
         "mask": {"size": window}}
    m2 = dict(m, heads=H + 1, vdim=V + 2, kv_from=0, scale=0.5, mask={"size": max(window - 5, 0)})
    a, cache, wa = _mixer("latent_attention", m, W, dev, 21, n)
    b, _, wb = _mixer("latent_attention", m2, W, dev, 22, n, others=[("latent_attention", m)])
    g = torch.Generator().manual_seed(3)
    h, h2 = torch.randn((n, W), generator=g), torch.randn((n, W), generator=g)
    shared = []
    want = O.latent_attention(h.double(), wa, m, 1e-5, shared)
    want2 = O.latent_attention(h2.double(), wb, m2, 1e-5, shared)
    got, got2 = [], []
    for sl, pos, md in Feed(dev, [5, 0, 3, 1]).portions(PORTIONS):
        got.append(full(a(h[sl].to(dev), pos, md, cache, 1e-5)))
        got2.append(full(b(h2[sl].to(dev), pos, md, cache, 1e-5)))
    close(torch.cat(got), want, 5e-4)
    close(torch.cat(got2), want2, 5e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,top,groups,keep", [(6, 2, 3, 1), (16, 3, 4, 2), (5, 5, 1, 1), (100, 8, 5, 3), (8, 1, 8, 2)])
def test_group_limited_routing(device, E, top, groups, keep):
    """Choices by score + correction inside the best groups (also negative ones), weights by the score."""
    from polykey_service_amd.ops import moe
    g = torch.Generator().manual_seed(E)
    z, corr = 2 * torch.randn((40, E), generator=g), torch.randn(E, generator=g) - 0.8
    dev = torch.device(device)
    ids, wts = moe.route_group_topk(z.to(dev), corr.to(dev), top, groups, keep)
    changed = 0
    for t in range(40):
        want, ws = O.route(z[t].double(), corr.double(), top, {"count": groups, "keep": keep} if groups > 1 else None)
        assert ids[t].cpu().tolist() == want
        close(wts[t], torch.stack(ws), 1e-5)
        changed += want != O.route(z[t].double(), 0 * corr.double(), top, None)[0]
    assert changed or (E == top and groups == 1)


@pytest.mark.parametrize("device", DEVICES)
def test_router_ties_go_to_the_lower_expert_and_group(device):
    from polykey_service_amd.ops import moe
    dev = torch.device(device)
    z = torch.tensor([[1.0, 3.0, 3.0, 1.0, 3.0, 3.0], [2.0] * 6], device=dev)
    ids, wts = moe.route_group_topk(z, None, 2, 3, 2)
    assert ids.cpu().tolist() == [[1, 2], [0, 1]]
    close(wts[1], torch.full((2,), 1 / 6), 1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,top,F_,groups,keep,W", [(6, 2, 24, 3, 2, 32), (16, 3, 8, 1, 1, 30), (4, 1, 40, 2, 1, 36), (70, 4, 12, 7, 3, 20)])
def test_mixture_block(device, E, top, F_, groups, keep, W):
    from polykey_service_amd.models import lefuvik as L
    from polykey_service_amd.models.config import GroupedMoESpec
    dev, T = torch.device(device), 50
    f = {"kind": "moe", "router": {"experts": E, "top": top}, "expert": {"ff": F_}}
    if groups > 1:
        f["router"]["groups"] = {"count": groups, "keep": keep}
    cfg = {"vocab": 4, "width": W, "layers": [{"type": "retention", "mixer": {"heads": 1, "dim": 2, "vdim": 2}, "mlp": f}]}
    w = {k[len("l0.mlp."):]: v for k, v in O.random_model(cfg, 21).items() if k.startswith("l0.mlp.")}
    mod = L.GroupedMoE(GroupedMoESpec(E, top, F_, groups, keep))
    part = lambda n: [w[f"e{e}.{n}"] for e in range(E)]
    mod.set(w["router"], w["correction"], part("up"), part("down"), torch.float32, dev)
    h = torch.randn((T, W), generator=torch.Generator().manual_seed(4))
    close(mod(h.to(dev), h.to(dev)).total(), O.mixture(h.double(), w, f), 3e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("N", [40, 37])
def test_activations(device, N):
    from polykey_service_amd.ops import moe
    dev = torch.device(device)
    x = torch.cat([3 * torch.randn((20, N)), 1e-3 * torch.randn((9, N)), torch.zeros((1, N))])
    table, ids = torch.randn((5, N + 11)), torch.randint(0, 5, (30,)).int()
    d = x.double()
    close(moe.activate(x.clone().to(dev), moe.ACT_RELU2), torch.clamp(d, min=0) ** 2, 1e-5)
    close(moe.activate(x.clone().to(dev), moe.ACT_XIELU, 0.8, 1.7),
          torch.where(d > 0, 0.8 * d * d, 1.7 * (torch.expm1(d) - d)) + 0.5 * d, 1e-5)
    close(moe.activate(x.clone().to(dev), moe.ACT_GELU, rows=(table.to(dev), ids.to(dev), 7)),
          O.gelu(d) * table[ids.long(), 7:7 + N].double(), 1e-5)


@pytest.mark.parametrize("device", DEVICES)
def test_xielu_feed_forward(device):
    from polykey_service_amd.models import lefuvik as L
    from polykey_service_amd.models.config import XieluFFSpec
    dev, W, F_ = torch.device(device), 24, 40
    g = torch.Generator().manual_seed(6)
    t = {"up": torch.randn((F_, W), generator=g), "down": torch.randn((W, F_), generator=g), "act": torch.tensor([-0.7, 1.3])}
    mod = L.XieluFF(XieluFFSpec(F_))
    mod.set(t["up"], t["down"], t["act"], torch.float32, dev)
    h = 0.3 * torch.randn((30, W), generator=g)
    close(full(mod(h.to(dev), None)), O.dense(h.double(), {k: v.double() for k, v in t.items()}), 3e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W,T", [(40, 9), (42, 5), (2048, 3), (64, 1100), (33, 2)])
def test_stream_step_with_scales_norms_and_a_raw_copy(device, W, T):
    from polykey_service_amd.ops import hyper as hy
    dev = torch.device(device)
    g = torch.Generator().manual_seed(W)
    r = lambda *s: torch.randn(s, generator=g)
    table, ids, ew = r(11, W), torch.randint(0, 11, (T,), generator=g).int(), r(W)
    x = hy.embed_norm_rows(table.to(dev), ids.to(dev), ew.to(dev), 1e-4)
    x0 = O.unit(table[ids.long()].double(), 1e-4) * ew.double()
    close(x[:, 0], x0, 1e-4)
    one, mix = torch.ones(1, device=dev), torch.ones((1, 1), device=dev)
    y, s, nw, pw = r(T, W), r(W), r(W), r(W)
    act, z = hy.hyper_step(x, y.to(dev), (mix, one), (one, None), 1e-4, torch.float32, y_scale=s.to(dev))
    x1 = x0 + y.double() * s.double()
    close(x[:, 0], x1, 1e-4)
    assert z is None and torch.equal(act, x[:, 0])
    act, z = hy.hyper_step(x, y.to(dev), (mix, one), (one, nw.to(dev)), 1e-4, torch.float32, want_f32=True, post_w=pw.to(dev))
    x2 = x1 + O.unit(y.double(), 1e-4) * pw.double()
    close(x[:, 0], x2, 1e-4)
    close(act, O.unit(x2, 1e-4) * nw.double(), 2e-4)
    assert torch.equal(act, z)
    top, rows = 2, 3 * T
    yr, inv, wts = r(rows, W), torch.randint(0, rows, (T * 2,), generator=g).int(), torch.rand((T, 2), generator=g)
    hy.hyper_step(x, hy.ExpertSum(yr.to(dev), inv.to(dev), wts.to(dev), top), (mix, one), None, 1e-4, y_scale=s.to(dev))
    f = (yr[inv.long()].view(T, 2, W).double() * wts[..., None].double()).sum(1)
    close(x[:, 0], x2 + f * s.double(), 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_side_input(device):
    from polykey_service_amd.models import lefuvik as L
    dev, W, d, T = torch.device(device), 24, 6, 13
    g = torch.Generator().manual_seed(6)
    t = {"gate": torch.randn((d, W), generator=g), "proj": torch.randn((W, d), generator=g), "norm": torch.randn(W, generator=g)}
    table, ids, x = torch.randn((9, 3 * d), generator=g), torch.randint(0, 9, (T,), generator=g).int(), torch.randn((T, W), generator=g)
    mod = L.SideInput()
    mod.set(t["gate"], t["proj"], t["norm"], 2 * d, torch.float32, dev)
    y = full(mod(x.to(dev), table.to(dev), ids.to(dev))).double()
    close(O.unit(y, 1e-5) * t["norm"], O.side_input(x.double(), table[ids.long(), 2 * d:].double(), {k: v.double() for k, v in t.items()}, 1e-5))


def test_configuration_is_checked():
    bad = [("rot", dict(rot_dim=7)), ("groups", dict(experts=7)), ("top", dict(top=5)), ("heads", dict(heads=3)),
           ("blocks", dict(blocks=5)), ("kv_from", dict(pattern=("retention:none", "shared:none")))]
    for _, kw in bad:
        cfg = O.make_config(**kw)
        if "pattern" in kw:
            cfg["layers"][1]["mixer"]["kv_from"] = 0
        with pytest.raises(ValueError):
            LefuvikConfig.from_json(cfg)
    c = LefuvikConfig.from_json(O.make_config())
    assert c.layers[4].mixer.kv_from == 2 and c.side_dim == 5 and c.needs_state
    assert not LefuvikConfig.from_json(O.make_config(pattern=("latent:moe",))).needs_state


# ------------------------------------------------------------------ the whole model through the engine
@pytest.mark.parametrize("device", DEVICES)
def test_prompt_logits_and_layer_streams_match_the_plain_model(device, small):
    from types import SimpleNamespace
    cfg, w, path = small
    eng = engine(path, device)
    assert eng.model.embed.device.type == device
    toks = rand_tokens(100, cfg["vocab"], 1)
    want, layers = O.forward(cfg, w, toks)
    got = replay(eng, [[("a", toks, list(range(100)), True)]])
    close(rows_of(got, "a", 100), want, 5e-4)
    dev = torch.device(device)
    md = SimpleNamespace(slot_mapping=i32(list(range(100)), dev), block_tables=i32([[0, 1, 2, 3]], dev), cu_q=i32([0, 100], dev),
                         context_lens=i32([100], dev), num_seqs=1, state_slots=i32([0], dev), token_seq=i32([0] * 100, dev),
                         num_decode=0)
    trail = []
    eng.model(i32(toks, dev), i32(list(range(100)), dev), md, eng.model.alloc_cache(4, BS, 1), trail=trail)
    for x, y in zip(trail, layers):
        close(x, y, 5e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_decoding_equals_prefill(device, small):
    cfg, w, path = small
    toks = rand_tokens(90, cfg["vocab"], 3)
    got = replay(engine(path, device), [[s] for s in cut("a", toks, [50])])
    close(rows_of(got, "a", 90), logits_of(cfg, w, toks), 5e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("sizes", [[2, 2, 2, 3, 40, 2, 17], [33, 31, 1, 1, 2], [7] * 14, [1, 1, 1, 2, 64]])
def test_portions_of_any_size(device, small, sizes):
    cfg, w, path = small
    toks = rand_tokens(100, cfg["vocab"], 4)
    got = replay(engine(path, device), [[s] for s in cut("a", toks, sizes)])
    close(rows_of(got, "a", 100), logits_of(cfg, w, toks), 5e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_mixed_batches_and_reused_pages_and_slots(device, small):
    """Four live requests of unequal lengths, portions beside decoded tokens, a pool that only
    holds them because finished requests give their pages and state slots back."""
    cfg, w, path = small
    eng = engine(path, device, pool_tokens=384, max_seqs=4, budget=384)
    lens = {"a": 120, "b": 37, "c": 64, "d": 90, "e": 70, "f": 33}
    toks = {k: rand_tokens(n, cfg["vocab"], 10 + i) for i, (k, n) in enumerate(lens.items())}
    plans = {"a": cut("a", toks["a"], [40, 30, 2, 2, 30]), "b": cut("b", toks["b"], [30]), "c": cut("c", toks["c"], [2, 50]),
             "d": cut("d", toks["d"], [64, 20]), "e": cut("e", toks["e"], [33, 33]), "f": cut("f", toks["f"], [31])}
    got = replay(eng, interleave(plans, waiting=["e", "f"]))
    for rid, n in lens.items():
        close(rows_of(got, rid, n), logits_of(cfg, w, toks[rid]), 5e-4)
    assert eng.scheduler.bm.num_free_state_slots == 4


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_past_windows_and_pages(device, tmp_path):
    """One-token steps across several windows and pages, with other sizes: one key / value head, one
    block of gates, a single tap, no side input, no cap, every expert used, no expert groups."""
    cfg = O.make_config(pattern=("latent:moe", "parallel:dense", "shared:none", "retention:none"), vocab=50, heads=3, kv_heads=1, dim=6,
                        vdim=10, window=13, keep=1, bias_max=11, rwidth=20, blocks=1, conv=1, rheads=1, rdim=16, rvdim=6, rrot=16,
                        experts=3, top=3, groups=1, side=0, cap=0.0, lwindow=5)
    w = O.random_model(cfg, seed=8, buckets=6)
    toks = rand_tokens(150, cfg["vocab"], 5)
    got = replay(engine(checkpoint(tmp_path, cfg, w), device), [[s] for s in cut("a", toks, [3])])
    close(rows_of(got, "a", 150), logits_of(cfg, w, toks), 5e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [
    dict(pattern=("retention:none", "parallel:dense"), heads=2, kv_heads=2, dim=16, vdim=16, window=32, keep=32, side=1),
    dict(pattern=("parallel:moe",), heads=6, kv_heads=3, dim=10, vdim=5, window=20, keep=0, conv=2, blocks=36, top=1, groups=6,
         keep_groups=1),
    dict(pattern=("latent:dense", "latent:moe", "shared:dense", "shared:moe"), lheads=3, rot_dim=2, kv_rank=7, lwindow=64, experts=9,
         top=4, groups=3, keep_groups=2),
    dict(pattern=("parallel:none", "parallel:moe"), heads=3, kv_heads=1, dim=20, vdim=24, window=64, keep=70, bias_max=200, side=0)])
def test_other_sizes(device, tmp_path, kw):
    cfg = O.make_config(**kw)
    w = O.random_model(cfg, seed=9, buckets=14)
    toks = rand_tokens(120, cfg["vocab"], 6)
    got = replay(engine(checkpoint(tmp_path, cfg, w), device), [[s] for s in cut("a", toks, [31, 2, 70])])
    close(rows_of(got, "a", 120), logits_of(cfg, w, toks), 5e-4)


def _drawn_config(seed):
    r = random.Random(seed)
    kv, ffs = r.choice([1, 2, 3]), ["dense", "moe", "none"]
    pattern = [f"{r.choice(['parallel', 'retention', 'latent'])}:{r.choice(ffs)}" for _ in range(r.randint(2, 3))]
    pattern += ["parallel:moe"] if r.random() < 0.5 else ["latent:none", "retention:dense", "shared:moe"]
    groups = r.choice([1, 2, 3])
    keep_groups, per = r.randint(1, groups), r.randint(1, 4)
    blocks = r.choice([1, 2, 5])
    rdim = r.choice([4, 10, 18])
    return O.make_config(pattern=tuple(pattern), vocab=r.randint(40, 90), width=r.choice([24, 36, 50]), heads=kv * r.choice([1, 2]),
                         kv_heads=kv, dim=r.choice([4, 7, 16]), vdim=r.choice([3, 8, 12]), window=r.choice([9, 33, 70]),
                         keep=r.choice([0, 1, 4, 33]), bias_max=r.choice([12, 64, 100]), rwidth=blocks * r.choice([4, 9]),
                         blocks=blocks, conv=r.randint(1, 5), rheads=r.randint(1, 3), rdim=rdim, rvdim=r.choice([5, 12]),
                         rrot=r.choice([2, rdim]), lheads=r.randint(1, 3), ldim=r.choice([5, 8]), lvdim=r.choice([4, 13]),
                         kv_rank=r.choice([9, 24]), q_rank=r.choice([11, 30]), rot_dim=r.choice([2, 6]), lwindow=r.choice([3, 34, 60]),
                         ff=r.choice([20, 44]), experts=groups * per, top=r.randint(1, keep_groups * per), eff=r.choice([8, 20]),
                         groups=groups, keep_groups=keep_groups, side=r.choice([1, 3, 8]), cap=r.choice([0.0, 8.0]),
                         eps=r.choice([1e-6, 1e-3]))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6])
def test_drawn_configurations_in_mixed_steps(device, tmp_path, seed):
    """Layer orders and sizes drawn at random, three unequal requests in steps drawn at random (a
    request may sit out a step), against the plain model."""
    cfg = _drawn_config(seed)
    w = O.random_model(cfg, seed=seed, buckets=2 * (seed + 1))
    r = random.Random(100 + seed)
    lens = {"a": r.randint(80, 160), "b": r.randint(2, 60), "c": r.randint(40, 120)}
    toks = {k: rand_tokens(n, cfg["vocab"], seed * 7 + i) for i, (k, n) in enumerate(lens.items())}
    plans = {k: cut(k, toks[k], [r.choice([2, 3, 17, 33, 64]) for _ in range(r.randint(1, 5))]) for k in lens}
    got = replay(engine(checkpoint(tmp_path, cfg, w), device), interleave(plans, skip=r))
    for rid, n in lens.items():
        assert float(rel(rows_of(got, rid, n), logits_of(cfg, w, toks[rid])).max()) < 1e-3, (rid, cfg["layers"])


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_engine(device, small):
    """add_request / step with the scheduler's own batching: two prompts generated together equal
    the plain model's argmax continuation (steps whose top two logits nearly tie are skipped)."""
    cfg, w, path = small
    eng = engine(path, device, graphs=device == "cuda")
    prompts = [rand_tokens(45, cfg["vocab"], 20), rand_tokens(9, cfg["vocab"], 21)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    for p, out in zip(prompts, outs):
        assert len(out) == 12
        lg = logits_of(cfg, w, list(p) + list(out))
        for i, tok in enumerate(out):
            row = lg[len(p) - 1 + i]
            top = torch.topk(row, 2).values
            if float(top[0] - top[1]) > 1e-2:
                assert int(row.argmax()) == tok


@pytest.mark.parametrize("device", DEVICES)
def test_preset_with_random_weights_generates(device):
    """The registry's small preset with seeded random weights (no checkpoint folder) through
    add_request / step; the same seed gives the same tokens again."""
    outs = []
    for _ in range(2):
        cfg = EngineConfig(model="tiny-lefuvik", dtype="float32", block_size=BS, max_num_seqs=2, max_num_batched_tokens=64,
                           max_model_len=128, num_kv_blocks=8, watermark=0.0, hip_graphs=False, device=device, seed=5)
        eng = LLMEngine(cfg, ParallelState(device=torch.device(device)))
        outs.append(eng.generate([list(range(3, 40)), [7, 8, 9]], SamplingParams(max_tokens=6, temperature=0.0, ignore_eos=True)))
    assert outs[0] == outs[1] and all(len(o) == 6 for o in outs[0])
    n = sum(t.numel() for t in eng.model.random_state(0).values())
    got = eng.mcfg.num_params()
    assert abs(n - got) / n < 0.01


@pytest.mark.gpu
def test_bfloat16_stays_near_the_plain_model(small):
    """The serving precision: bf16 projections and caches, fp32 stream / norms / scores / states.
    The kernels are also held against the ops' PyTorch compositions rounding at the same places."""
    cfg, w, path = small
    toks = rand_tokens(100, cfg["vocab"], 7)
    want = logits_of(cfg, w, toks).float()
    steps = [[s] for s in cut("a", toks, [60, 20])]
    got = rows_of(replay(engine(path, "cuda", dtype="bfloat16", graphs=True), steps), "a", 100)
    ref = rows_of(replay(engine(path, "cpu", dtype="bfloat16"), steps), "a", 100)
    assert float(rel(got, want).mean()) < 0.1 and float(rel(got, want).median()) < 0.08
    assert float(rel(got, ref).mean()) < 0.03


@pytest.mark.gpu
def test_aligned_sizes_in_mixed_batches_with_decode_graphs(tmp_path):
    """A bf16 model at sizes the decode GEMM, the grouped expert GEMMs, the matrix-core attention and
    the matrix-core gates tile: unequal live requests, prompt portions beside decoded tokens, decode
    graphs; against the ops' compositions at the same precision and the plain model."""
    cfg = O.make_config(pattern=("parallel:moe", "latent:moe", "retention:dense", "shared:moe", "parallel:dense"), vocab=120, width=256,
                        heads=4, kv_heads=2, dim=64, vdim=128, window=100, keep=40, bias_max=128, rwidth=256, blocks=2, conv=4,
                        rheads=4, rdim=64, rvdim=64, rrot=64, lheads=4, ldim=64, lvdim=64, kv_rank=128, q_rank=256, rot_dim=32,
                        lwindow=90, ff=512, experts=8, top=2, eff=256, groups=4, keep_groups=2, side=256)
    w = O.random_model(cfg, seed=12, buckets=16)
    path = checkpoint(tmp_path, cfg, w)
    lens = {"a": 300, "b": 170, "c": 230, "d": 40}
    toks = {k: rand_tokens(n, cfg["vocab"], 30 + i) for i, (k, n) in enumerate(lens.items())}
    plans = {"a": cut("a", toks["a"], [200, 60]), "b": cut("b", toks["b"], [2, 150]), "c": cut("c", toks["c"], [64, 64, 90]),
             "d": cut("d", toks["d"], [33])}
    steps = interleave(plans)
    got = replay(engine(path, "cuda", dtype="bfloat16", pool_tokens=1024, budget=1024, graphs=True), steps)
    ref = replay(engine(path, "cpu", dtype="bfloat16", pool_tokens=1024, budget=1024), steps)
    for rid, n in lens.items():
        g, r = rows_of(got, rid, n), rows_of(ref, rid, n)
        assert float(rel(g, r).mean()) < 0.03, rid
        if n < 200:
            assert float(rel(g, logits_of(cfg, w, toks[rid])).median()) < 0.1, rid


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,V,window,keep", [(4, 2, 64, 64, 100, 40), (8, 2, 128, 128, 70, 1), (2, 2, 64, 128, 33, 64),
                                                 (16, 4, 128, 128, 200, 33), (6, 3, 128, 64, 50, 0), (4, 1, 128, 128, 0, 0)])
def test_matrix_core_attention_with_kept_keys_and_bias_matches_the_fma_tiles(H, G, D, V, window, keep):
    """bf16 at the matrix-core kernel's sizes, prompt portions and decoded tokens (cut into runs and
    merged), against the FMA kernel on the same caches and against the plain rule."""
    from polykey_service_amd.ops import masked_attention as ma
    from polykey_service_amd.ops import native
    dev, n, bf = torch.device("cuda"), 300, torch.bfloat16
    g = torch.Generator().manual_seed(H * 100 + D)
    q = torch.randn((n, H, D), generator=g).to(bf)
    k, v = (0.5 * torch.randn((n, G, D), generator=g)).to(bf), torch.randn((n, G, V), generator=g).to(bf)
    rel_ = torch.randn((16, H), generator=g)
    bias = ma.distance_bias(rel_, 150).to(dev)
    outs = {}
    for mfma in (1, 0):
        native.mixers().pkm_set_masked_mfma(mfma)
        try:
            kc, vc = torch.zeros((12, G, BS, D), device=dev, dtype=bf), torch.zeros((12, G, BS, V), device=dev, dtype=bf)
            out = torch.zeros((n, H * V + 8), device=dev)
            for sl, pos, md in Feed(dev, [7, 2, 11, 0, 5, 9, 3, 1, 10, 4, 6, 8]).portions([150, 1, 1, 40, 2, 1, 1, 1, 103]):
                at = md.slot_mapping.long()
                kc[at // BS, :, at % BS], vc[at // BS, :, at % BS] = k[sl].to(dev), v[sl].to(dev)
                ma.masked_attention(q[sl].contiguous().to(dev), kc, vc, V, md.block_tables, md.cu_q, md.context_lens, 1, D ** -0.5,
                                    window=window, keep=keep, bias=bias, post=0.75, num_decode=md.num_decode, out=out[sl, :H * V])
            outs[mfma] = out[:, :H * V].cpu().view(n, H, V)
        finally:
            native.mixers().pkm_set_masked_mfma(1)
    close(outs[1], outs[0], 3e-4)
    pos = torch.arange(n)
    back = pos[:, None] - pos[None, :]
    seen = (back >= 0) & ((back < window) | (pos[None, :] < keep) | torch.tensor(window == 0))
    per = torch.stack([rel_[O.distance_bucket(i, 16, 150)] for i in range(n)]).double()
    sc = torch.einsum("ihd,jhd->hij", q.double(), k.double().repeat_interleave(H // G, 1)) * D ** -0.5
    sc = (sc + per.t()[:, back.clamp(min=0)]).masked_fill(~seen, float("-inf"))
    want = 0.75 * torch.einsum("hij,jhv->ihv", torch.softmax(sc, -1), v.double().repeat_interleave(H // G, 1))
    close(outs[0], want, 3e-4)


@pytest.mark.gpu
@pytest.mark.parametrize("C,blocks,T", [(256, 2, 40), (512, 8, 300), (192, 1, 700)])
def test_matrix_core_gates_match_the_fma_tiles(C, blocks, T):
    from polykey_service_amd.ops import lru, native
    dev, w, bf = torch.device("cuda"), C // blocks, torch.bfloat16
    g = torch.Generator(device=dev).manual_seed(C)
    r = lambda *s: torch.randn(s, generator=g, device=dev)
    u, y = r(T, C).to(bf), r(T, C).to(bf)
    ra, ri = (r(blocks, w, w) * w ** -0.5).to(bf), (r(blocks, w, w) * w ** -0.5).to(bf)
    args = (r(C), ra, ri, r(C), r(C), -8 * torch.nn.functional.softplus(r(C) - 4))
    cut_at = [0, T // 3, T // 3 + 1, T]
    outs = {}
    for mfma in (1, 0):
        native.mixers().pkm_set_lru_mfma(mfma)
        try:
            state = torch.full((4, C), 2.0, device=dev)
            pos = torch.cat([torch.arange(a, b) for a, b in zip([0, 50, 9], [T // 3, 51, 9 + T - T // 3 - 1])]).int().to(dev)
            outs[mfma] = (lru.gated_lru(u, y, *args, state, i32(cut_at, dev), 3, pos, i32([2, 0, 3], dev)), state)
            one = torch.arange(3, dtype=torch.int32, device=dev)
            outs[mfma] += (lru.gated_lru(u[:3], y[:3], *args, state, i32([0, 1, 2, 3], dev), 3, one, i32([1, -1, 3], dev), 3),)
        finally:
            native.mixers().pkm_set_lru_mfma(1)
    for a, b in zip(outs[1], outs[0]):
        close(a, b, 1e-2)
