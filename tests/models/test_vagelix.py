"""Vagelix through the framework (checkpoint loader, scheduler, block manager and state slots,
model runner, kernels) against the plain per-sequence model of tests/oracle_vagelix.py.

Every test builds its own small configuration and random weights, writes them as a checkpoint
folder and loads that through the engine, or drives one op or mixer with hand-made inputs over a
hand-made paged cache and hand-made state slots.  The same tests run on the CPU (the ops' PyTorch
compositions) and, marked gpu, on the HIP kernels."""
import copy
import math
import os
import random
import sys
from types import SimpleNamespace

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
import oracle_vagelix as O  # noqa: E402
from engine_replay import (BS, Feed, checkpoint, close, cut, engine, full, i32, interleave, rand_tokens, rel, replay,  # noqa: E402
                           rows_of)

from polykey_service_amd.engine import EngineConfig, LLMEngine, SamplingParams  # noqa: E402
from polykey_service_amd.models.config import VagelixConfig  # noqa: E402
from polykey_service_amd.parallel.state import ParallelState  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
D64 = torch.float64
PORTIONS = [3, 1, 1, 30, 2, 40, 1, 1, 1, 17]      # 97 tokens over shuffled pages
FF = {"kind": "dense", "ff": 44}


def logits_of(cfg, w, toks):
    return O.forward(cfg, w, toks)[0]


@pytest.fixture
def small(tmp_path):
    cfg = O.make_config()
    w = O.random_model(cfg, seed=3)
    return cfg, w, checkpoint(tmp_path, cfg, w)


def _mixer(kind, m, W, dev, seed, n, **kw):
    """The framework's mixer module with the oracle's random weights, its cache filled with what an earlier
    owner left, and the weights."""
    from polykey_service_amd.models import vagelix as L
    from polykey_service_amd.ops import masked_attention as ma
    cfg = {"vocab": 4, "width": W, "norm": {"eps": 1e-5}, "layers": [{"type": kind, "mixer": m, "mlp": None}]}
    w = {k[len("l0.mix."):]: v.double() for k, v in O.random_model(cfg, seed, **kw).items() if k.startswith("l0.mix.")}
    spec = VagelixConfig.from_json(cfg).layers[0].mixer
    mod = L._MIXERS[kind](spec, W)
    nb = (n + BS - 1) // BS + 3
    page = lambda heads, wd: torch.full((nb, heads, BS, wd), 3.0, device=dev)
    if kind == "attention":
        g = lambda k: w.get(k)
        mod.set(g("q"), g("k"), g("v"), None, g("o"), g("lq1"), g("lk1"), g("lq2"), g("lk2"), torch.float32, dev, g("q.norm"), g("k.norm"))
        return mod, (page(2 * spec.kv_heads, spec.dim), page(spec.kv_heads, spec.vdim)), w
    mod.set(w.__getitem__, torch.float32, dev)
    cache = mod.state(3, dev)
    for t in cache.values():
        t.fill_(5.0)
    if kind == "parallel":
        cache["k"], cache["v"] = (page(spec.left.kv_heads, spec.left.dim) for _ in range(2))
        if spec.left.rot is not None:
            mod.table = ma.table_for(spec.left.rot, n + 3, dev)
    return mod, cache, w


def _feed(mod, cache, h, portions, pages, dev):
    return torch.cat([full(mod(h[sl].to(dev), pos, md, cache, 1e-5)) for sl, pos, md in Feed(dev, pages).portions(portions)])


# ------------------------------------------------------------------ single mechanisms
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("left,right,ranks", [
    (dict(H=4, G=2, D=16, chunk=24, rot=10, base=90.0), dict(rH=4, rG=2, rD=10, rV=14, conv=3), (7, 5)),
    (dict(H=3, G=3, D=7, chunk=33, rot=2), dict(rH=3, rG=3, rD=20, rV=3, conv=4), (3, 11)),
    (dict(H=6, G=1, D=36, chunk=7, rot=36), dict(rH=2, rG=1, rD=33, rV=70, conv=2), (16, 16)),
    (dict(H=1, G=1, D=70, chunk=1, rot=0), dict(rH=1, rG=1, rD=130, rV=8, conv=1), (1, 1)),
    (dict(H=2, G=2, D=8, chunk=500, rot=8), dict(rH=6, rG=2, rD=8, rV=16, conv=6), (9, 2))])
def test_parallel_mixer(device, left, right, ranks):
    """Both branches over shuffled pages in portions and decoded tokens, and the averaged, normed sum."""
    dev, W, n = torch.device(device), 30, sum(PORTIONS)
    m = O.parallel_spec(**left, **right)
    mod, cache, w = _mixer("parallel", m, W, dev, 13, n, rank=ranks[0], grank=ranks[1])
    g = torch.Generator().manual_seed(3)
    h, x = torch.randn((n, W), generator=g), torch.randn((n, W), generator=g)
    nw = torch.randn(W, generator=g)
    part = lambda p: {k[len(p):]: v for k, v in w.items() if k.startswith(p)}
    a = O.chunk_attention(h.double(), part("left."), m["left"], 1e-5)
    b = O.delta_branch(h.double(), part("right."), m["right"], 1e-5)
    got_a, got_b, got_x, got_h = [], [], [], []
    for sl, pos, md in Feed(dev, [5, 0, 3, 1]).portions(PORTIONS):
        y = mod(h[sl].to(dev), pos, md, cache, 1e-5)
        got_a.append(full(y[0])), got_b.append(full(y[1]))
        xs = x[sl].clone().to(dev)[:, None]
        got_h.append(mod.close(xs, y, nw.to(dev), 1e-5, torch.float32).cpu())
        got_x.append(xs[:, 0].cpu())
    close(torch.cat(got_a), a, 5e-4)
    close(torch.cat(got_b), b, 5e-4)
    want = x + O.unit(O.parallel(h.double(), w, m, 1e-5), 1e-5) * nw.double()
    close(torch.cat(got_x), want, 1e-3)
    assert torch.equal(torch.cat(got_x), torch.cat(got_h))


def _probe(dev, chunk, key, qpos, decoded, H=4, G=2, D=8, strong=6.0, gate=None, sink=True):
    """Keys and values written by hand; key ``key`` points along the query, the others are small.
    Returns (the framework's output at ``qpos``, the plain rule's) [H, D] and the key's values [G, D]."""
    from polykey_service_amd.ops import masked_attention as ma
    n = qpos + 1
    g = torch.Generator().manual_seed(5)
    k, v = 0.05 * torch.randn((n, G, D), generator=g), torch.randn((n, G, D), generator=g)
    q = 0.05 * torch.randn((n, H, D), generator=g)
    k[key, :, 0], q[qpos, :, 0] = strong, strong
    pages = [3, 0, 5, 1, 2, 4][: (n + BS - 1) // BS + 1]
    kc, vc = torch.zeros((6, G, BS, D), device=dev), torch.zeros((6, G, BS, D), device=dev)
    gt = None if gate is None else torch.tensor(gate).repeat(n, 1)
    sizes = [qpos, 1] if decoded else [max(qpos - 6, 1), n - max(qpos - 6, 1)]
    out = None
    for sl, pos, md in Feed(dev, pages).portions([c for c in sizes if c > 0]):
        at = md.slot_mapping.long()
        kc[at // BS, :, at % BS], vc[at // BS, :, at % BS] = k[sl].to(dev), v[sl].to(dev)
        out = ma.masked_attention(q[sl].contiguous().to(dev), kc, vc, D, md.block_tables, md.cu_q, md.context_lens, 1, 1.0,
                                  chunk=chunk, sink=torch.zeros(H, device=dev) if sink else None, num_decode=md.num_decode,
                                  head_gate=None if gt is None else gt[sl].to(dev))
    want = O.softmax_rows(q.double(), k.double(), v.double(), 1.0, chunk, sink)[qpos]
    if gate is not None:
        want = want * O.sigmoid(torch.tensor(gate).double())[:, None]
    return out[-1].view(H, D).cpu(), want, v[key].float()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("key,qpos,seen", [(80, 100, True), (79, 100, False), (100, 100, True), (0, 100, False), (80, 119, True),
                                           (79, 119, False), (119, 120, False), (120, 120, True), (95, 100, True), (96, 100, True),
                                           (40, 79, True), (39, 79, False), (63, 64, True), (0, 39, True), (0, 40, False)])
def test_a_query_sees_its_chunk_only(device, decoded, key, qpos, seen):
    """Chunks of 40 positions counted from 0; page borders lie inside them."""
    got, want, val = _probe(torch.device(device), 40, key, qpos, decoded)
    close(got, want, 1e-4)
    if seen:
        close(got, val.repeat_interleave(2, 0), 1e-2)
    else:
        assert float((got - val.repeat_interleave(2, 0)).abs().max()) > 0.1


@pytest.mark.parametrize("device", DEVICES)
def test_one_more_softmax_term_and_head_gates(device):
    """Small scores: n keys share n / (n + 1) of the weight, which halves the first token's output and a
    chunk's first; heads are scaled by their own gates, also shut and open ones."""
    dev = torch.device(device)
    for qpos in (0, 24, 25, 47):
        gate = [-30.0, 0.0, 2.0, 30.0]
        for decoded in ([False] if qpos == 0 else [False, True]):
            got, want, val = _probe(dev, 24, qpos, qpos, decoded, strong=0.0, gate=gate)
            close(got, want, 1e-5)
            none, _, _ = _probe(dev, 24, qpos, qpos, decoded, strong=0.0, gate=gate, sink=False)
            n = qpos % 24 + 1
            close(got, none * n / (n + 1), 5e-3)
            assert float(got[0].abs().max()) == 0 or float(got[0].abs().max()) < 1e-9
            assert float((none[3] - got[3]).abs().max()) > 0.01


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("QH,KH,D,rot,halves", [(3, 1, 12, 4, True), (4, 2, 16, 16, True), (2, 2, 5, 4, False), (16, 4, 64, 24, True),
                                                (1, 1, 8, 0, True), (3, 3, 24, 6, False)])
def test_norm_over_all_heads_with_keys_as_values(device, dtype, QH, KH, D, rot, halves):
    """Heads of very unequal size: a norm per head, a norm before the bias or values behind the norm would
    all show.  The projection is a column slice at an odd place, one token caches nothing."""
    from polykey_service_amd.models.config import RotarySpec
    from polykey_service_amd.ops import masked_attention as ma
    dev, T, n = torch.device(device), 9, (QH + KH) * D
    g = torch.Generator().manual_seed(D)
    size = torch.exp(torch.linspace(-2, 2, QH + KH)).repeat_interleave(D)
    off = 8 if D % 8 == 0 else 3
    proj = torch.zeros((T, n + 16))
    proj[:, off:off + n] = torch.randn((T, n), generator=g) * size
    proj = proj.to(dtype)
    b, qw, kw = torch.randn(n, generator=g), torch.randn(QH * D, generator=g), torch.randn(KH * D, generator=g)
    table = ma.table_for(RotarySpec(rot, 30.0, None, halves), 40, dev) if rot else None
    kc, vc = torch.full((2, KH, BS, D), 7.0, device=dev, dtype=dtype), torch.full((2, KH, BS, D), 7.0, device=dev, dtype=dtype)
    pos = torch.arange(25, 25 + T, dtype=torch.int32)
    slots = pos.clone()
    slots[4] = -1
    q = ma.row_norm_cache(proj.to(dev)[:, off:off + n], b.to(dev), qw.to(dev), kw.to(dev), 1e-3, pos.to(dev), slots.to(dev), table, halves,
                          kc, vc, QH, KH, D)
    f = proj[:, off:off + n].double() + b.double()
    tol = 1e-4 if dtype == torch.float32 else 1e-2
    qq, kk = (O.unit(f[:, :QH * D], 1e-3) * qw).view(T, QH, D), (O.unit(f[:, QH * D:], 1e-3) * kw).view(T, KH, D)
    if rot and halves:
        pad = torch.zeros((25, 1, 1), dtype=D64)
        turn = lambda x: O.rotate(torch.cat([pad.expand(25, x.shape[1], D), x]), rot, 30.0)[25:]
        qq, kk = turn(qq), turn(kk)
    elif rot:
        order = list(range(0, rot, 2)) + list(range(1, rot, 2)) + list(range(rot, D))
        back = [order.index(i) for i in range(D)]
        turn = lambda x: O.rotate(torch.cat([torch.zeros((25, x.shape[1], D), dtype=D64), x[:, :, order]]), rot, 30.0)[25:][:, :, back]
        qq, kk = turn(qq), turn(kk)
    close(q, qq, tol)
    for i in range(T):
        p = 25 + i
        if i == 4:
            assert float((kc[p // BS, :, p % BS] - 7).abs().max()) == 0 == float((vc[p // BS, :, p % BS] - 7).abs().max())
        else:
            close(kc[p // BS, :, p % BS], kk[i], tol)
            close(vc[p // BS, :, p % BS], f[i, QH * D:].view(KH, D), tol)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("D,rots", [(10, (6, 4)), (64, (32, 16)), (16, (16, 6)), (8, (0, 0))])
def test_query_temperature_steps_at_its_multiples(device, D, rots):
    """1 + coef ln(floor((p + 1) / every) + 1): positions around the steps, keys untouched; with and without
    head norms and a rotation, at sizes of the scalar and of the 16-byte form."""
    from polykey_service_amd.models.config import RotarySpec
    from polykey_service_amd.ops import masked_attention as ma
    dev, T = torch.device(device), 70
    g = torch.Generator().manual_seed(2)
    row = torch.randn(3 * D, generator=g)
    proj = row.repeat(T, 1)
    qn, kn = torch.randn(D, generator=g), torch.randn(D, generator=g)
    pos = torch.arange(T, dtype=torch.int32)
    for norms, rot in ((True, 0), (False, 0), (True, rots[0]), (False, rots[1])):
        kc, vc = torch.zeros((3, 1, BS, D), device=dev), torch.zeros((3, 1, BS, D), device=dev)
        table = ma.table_for(RotarySpec(rot, 30.0, None, True), T, dev) if rot else None
        kw = dict(q_norm=qn.to(dev), k_norm=kn.to(dev), eps=1e-4) if norms else {}
        args = (proj.to(dev), pos.to(dev), pos.to(dev), table, True, kc, vc, 1, 1, 1, D, D)
        plain, k0 = ma.rotate_cache(*args, **kw).cpu(), kc.clone()
        got = ma.rotate_cache(*args, **kw, temp=(0.7, 16)).cpu()
        f = O.query_temperature(T, 0.7, 16)
        close(got, plain * f.float()[:, None, None], 1e-5)
        assert torch.equal(kc, k0)
        q, k = row[:D].double().repeat(T, 1)[:, None], row[D:2 * D].double().repeat(T, 1)[:, None]
        if norms:
            q, k = O.unit(q, 1e-4) * qn, O.unit(k, 1e-4) * kn
        close(plain, O.rotate(q, rot, 30.0), 1e-4)
        at = pos.long()
        close(kc[at // BS, :, at % BS], O.rotate(k, rot, 30.0), 1e-4)
        close(vc[at // BS, 0, at % BS], row[2 * D:].repeat(T, 1), 1e-6)
        for p, want in ((0, 0), (14, 0), (15, 1), (30, 1), (31, 2), (62, 3), (63, 4)):
            assert abs(float(f[p]) - (1 + 0.7 * math.log(want + 1))) < 1e-12


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,V,every", [(4, 2, 9, 13, 16), (3, 3, 16, 4, 1), (6, 1, 6, 34, 7), (2, 2, 36, 36, 1000), (1, 1, 70, 12, 40)])
def test_differential_attention_mixer(device, H, G, D, V, every):
    dev, W, n = torch.device(device), 30, sum(PORTIONS)
    m = O.diff_spec(H, G, D, V, 0.3, 0.5, every)
    mod, cache, w = _mixer("attention", m, W, dev, 17, n)
    h = torch.randn((n, W), generator=torch.Generator().manual_seed(4))
    close(_feed(mod, cache, h, PORTIONS, [5, 0, 3, 1], dev), O.diff_attention(h.double(), w, m, 1e-5), 1e-3)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("key", [0, 1, 31, 32, 63, 64, 230, 299])
def test_differential_attention_reaches_far_keys(device, decoded, key):
    """One key of 300 far above the rest in the first map, its neighbour in the second: the output is the
    difference of their values at any distance and across page borders."""
    dev, n, W = torch.device(device), 300, 20
    m = O.diff_spec(2, 1, 8, 6, 0.25, 0.2, 50, scale=1.0)
    mod, cache, w = _mixer("attention", m, W, dev, 19, n)
    g = torch.Generator().manual_seed(6)
    h = 0.1 * torch.randn((n, W), generator=g)
    # rows of q / k weights: the first map answers coordinate 0, the second coordinate 1
    wq, wk = 0.02 * torch.randn((2 * 2 * 8, W), generator=g), 0.02 * torch.randn((2 * 8, W), generator=g)
    for head in range(2):
        wq[head * 16, 2], wq[head * 16 + 8, 2] = 5.0, 5.0
    wk[0, 0], wk[8, 1] = 5.0, 5.0
    w = dict(w, q=wq.double(), k=wk.double(), **{"q.norm": torch.full((8,), 2.0, dtype=D64), "k.norm": torch.full((8,), 2.0, dtype=D64)})
    other = key + 1 if key + 1 < n else key - 1
    h[:, :3] = 0.0
    h[key, 0], h[other, 1], h[n - 1, 2] = 3.0, 3.0, 3.0
    gt = lambda k: w[k]
    mod.set(gt("q"), gt("k"), gt("v"), None, gt("o"), gt("lq1"), gt("lk1"), gt("lq2"), gt("lk2"), torch.float32, dev, gt("q.norm"), gt("k.norm"))
    pages = [4, 0, 7, 1, 9, 2, 3, 6, 5, 8]
    got = _feed(mod, cache, h, [250, 49, 1] if decoded else [200, 100], pages, dev)[-1]
    want = O.diff_attention(h.double(), w, m, 1e-5)
    close(got, want[-1], 2e-3)
    far = h.clone()
    far[key, 3:] += 1.0     # another value at that key changes the output
    assert float((O.diff_attention(far.double(), w, m, 1e-5)[-1] - want[-1]).abs().max()) > 0.05


@pytest.mark.parametrize("device", DEVICES)
def test_channel_decays_keep_and_drop_their_rows(device):
    """A value written at position 0 along two key channels, one that never decays and one that forgets at
    once; read back 250 tokens later, over a dirty slot, with other sequences' slots untouched."""
    from polykey_service_amd.ops import delta as dl
    dev, n, D, V = torch.device(device), 252, 6, 5
    qkv = torch.zeros((n, 2 * D + V))
    qkv[0, D:2 * D] = torch.tensor([0.6, 0.8, 0, 0, 0, 0])
    qkv[0, 2 * D:] = torch.arange(1, V + 1).float()
    qkv[n - 2, 0] = qkv[n - 1, 1] = 1.0
    gates = torch.ones((n, 1, D))
    gates[:, :, 1] = 0.5
    gates[:, :, 0] = 0.9999
    beta = torch.full((n, 1), 30.0)
    state = torch.full((3, 1, D, V), 9.0, device=dev)
    o = torch.cat([dl.delta_rule(qkv[sl].to(dev), beta[sl].to(dev), None, None, state, md.cu_q, 1, pos, md.state_slots, 1, D, 1, V,
                                 gates=gates[sl].to(dev)) for sl, pos, md in Feed(dev, [0] * 9).portions([100, 1, 1, 150])]).cpu()
    close(o[n - 2, 0], 0.6 * 0.9999 ** (n - 2) * torch.arange(1, V + 1), 1e-4)
    assert float(o[n - 1].abs().max()) < 1e-20
    assert float((state[0] - 9).abs().max()) == 0 == float((state[2] - 9).abs().max())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("G,D,H,V,K", [(2, 10, 4, 7, 4), (1, 70, 3, 130, 2), (3, 5, 3, 5, 1), (1, 8, 1, 8, 7)])
def test_filters_unit_vectors_and_decays_in_a_batch(device, G, D, H, V, K):
    """Several sequences in a step (portions shorter than the filter, one without a slot), then steps in
    which all hold one token; states and decays against the plain rules."""
    from polykey_service_amd.ops import delta as dl
    dev, C = torch.device(device), 2 * G * D + H * V
    g = torch.Generator().manual_seed(K + D)
    taps, a_log, bias = torch.randn((C, K), generator=g), torch.randn(H, generator=g), torch.randn(H * D, generator=g)
    state = torch.full((5, max(K - 1, 1), C), 4.0, device=dev)
    slots, seqs = [3, 0, -1, 4], [[], [], [], []]
    to = lambda t: t.to(dev)
    for lens in ([5, 1, 2, 9], [2, 3, 1, 1], [1, 1, 1, 1], [1, 1, 1, 1], [4, 1, 1, 2]):
        starts = [sum(x.shape[0] for x, _ in s) for s in seqs]
        starts[2] = 0       # no slot: every portion of that sequence stands alone
        x, z = torch.randn((sum(lens), C + 3), generator=g), torch.randn((sum(lens), H * D + 2), generator=g)
        cu = [0]
        for n in lens:
            cu.append(cu[-1] + n)
        pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lens)]).int()
        nd = 4 if max(lens) == 1 else 0
        out, gates = dl.conv_unit(to(x)[:, :C], to(taps), state, i32(cu, dev), 4, to(pos), i32(slots, dev),
                                  i32(sum([[i] * n for i, n in enumerate(lens)], []), dev), G, D, H, V, num_decode=nd,
                                  decay=(to(z)[:, :H * D], to(a_log), to(bias)))
        for i, n in enumerate(lens):
            seqs[i] = (seqs[i] if i != 2 else []) + [(x[cu[i]:cu[i + 1], :C].double(), None)]
            whole = torch.cat([s for s, _ in seqs[i]])
            y = O.silu(O.causal_filter(whole, taps.double()))[-n:]
            qk = y[:, :2 * G * D].view(n, 2 * G, D)
            qk = qk / torch.sqrt((qk * qk).sum(-1, keepdim=True) + 1e-6)
            qk[:, :G] /= D ** 0.5
            close(out[cu[i]:cu[i + 1]], torch.cat([qk.reshape(n, -1), y[:, 2 * G * D:]], 1), 1e-4)
            if slots[i] >= 0 and K > 1:
                last = torch.cat([torch.zeros((K - 1, C), dtype=D64), whole])[-(K - 1):]
                close(state[slots[i]], last, 1e-6)
        close(gates, O.channel_decay(z[:, :H * D].double(), a_log.double(), bias.double()), 1e-4)
    assert float((state[1] - 4).abs().max()) == 0 == float((state[2] - 4).abs().max())


@pytest.mark.gpu
@pytest.mark.parametrize("G,D,H,V,K", [(2, 64, 4, 128, 4), (1, 8, 3, 16, 2), (3, 128, 3, 24, 3), (1, 512, 1, 8, 4)])
def test_filters_over_runs_of_tokens_in_a_batch(G, D, H, V, K):
    """bf16 rows long enough for the run form: several sequences, some short, two continuing from their slots,
    one without a slot."""
    from polykey_service_amd.ops import delta as dl
    dev, C = torch.device("cuda"), 2 * G * D + H * V
    lens, starts, slots = [3, 70, 1, 2, 41, 8, 16], [0, 5, 40, 0, 0, 7, 0], [4, 2, 7, 0, -1, 5, 3]
    g = torch.Generator().manual_seed(K + D)
    T = sum(lens)
    x, z = torch.randn((T, C + 8), generator=g).bfloat16(), torch.randn((T, H * D + 8), generator=g).bfloat16()
    taps, a_log, bias = torch.randn((C, K), generator=g), torch.randn(H, generator=g), torch.randn(H * D, generator=g) - 3
    state = torch.randn((9, K - 1, C), generator=g)
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lens)]).int()
    to = lambda t: t.to(dev)
    st = to(state)
    out, gates = dl.conv_unit(to(x)[:, :C], to(taps), st, i32(cu, dev), len(lens), to(pos), i32(slots, dev),
                              i32(sum([[i] * n for i, n in enumerate(lens)], []), dev), G, D, H, V,
                              decay=(to(z)[:, 8:8 + H * D], to(a_log), to(bias)))
    new = state.clone()
    for i, n in enumerate(lens):
        past = state[slots[i]].double() if starts[i] and slots[i] >= 0 else torch.zeros((K - 1, C), dtype=D64)
        xin = torch.cat([past, x[cu[i]:cu[i + 1], :C].double()])
        y = O.silu(O.causal_filter(xin, taps.double())[K - 1:])
        qk = y[:, :2 * G * D].view(n, 2 * G, D)
        qk = qk / torch.sqrt((qk * qk).sum(-1, keepdim=True) + 1e-6)
        qk[:, :G] /= D ** 0.5
        close(out[cu[i]:cu[i + 1]], torch.cat([qk.reshape(n, -1), y[:, 2 * G * D:]], 1), 1e-4)
        if slots[i] >= 0:
            new[slots[i]] = xin[-(K - 1):].float()
    close(st, new, 1e-6)
    close(gates, O.channel_decay(z[:, 8:8 + H * D].double(), a_log.double(), bias.double()), 1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,V", [(4, 64), (6, 8), (2, 512), (3, 24), (5, 7), (2, 128)])
def test_head_norms_with_every_gate(device, H, V):
    """One row or the difference of two per head, shared / own / no weights, the three kinds of gates, strided
    output; sizes of the scalar and of the 16-byte form."""
    from polykey_service_amd.ops import masked_attention as ma
    dev, T = torch.device(device), 5
    g = torch.Generator().manual_seed(V)
    r = lambda *s: torch.randn(s, generator=g)
    a, a2, gate = r(T, H, V), r(T, 2 * H, V), r(T, H * V + 8)
    for kind, act in ((ma.GATE_SIGMOID, O.sigmoid), (ma.GATE_SILU, O.silu), (ma.GATE_NONE, None)):
        for w in (None, r(V), r(H * V)):
            for pair in (0, 1, H):
                u = a.double()
                if pair:
                    p5 = a2.double().view(T, H // pair, 2, pair, V)
                    u = (p5[:, :, 0] - 0.3 * p5[:, :, 1]).reshape(T, H, V)
                want = O.unit(u, 1e-3) * 0.7
                if w is not None:
                    want = want * (w.view(H, V) if w.numel() == H * V else w).double()
                want = want.reshape(T, H * V)
                if act is not None:
                    want = want * act(gate[:, 8:].double())
                out = torch.zeros((T, H * V + 16), device=dev)
                ma.head_norm_gate((a2 if pair else a).to(dev), H, V, 1e-3, gate.to(dev)[:, 8:] if act is not None else None, kind,
                                  torch.float32, weight=None if w is None else w.to(dev), post=0.7, pair_group=pair, coef=0.3,
                                  out=out[:, 8:8 + H * V])
                close(out[:, 8:8 + H * V], want, 1e-4)
                assert float(out[:, :8].abs().max()) == 0 == float(out[:, 8 + H * V:].abs().max())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,V,N,G,K,parts", [(6, 9, 11, 3, 4, 2), (4, 12, 24, 1, 2, 1), (2, 70, 130, 2, 3, 4), (3, 5, 7, 3, 1, 3),
                                             (1, 34, 300, 1, 5, 17), (8, 4, 64, 4, 4, 8)])
def test_state_space_mixer(device, H, V, N, G, K, parts):
    dev, W, n = torch.device(device), 28, sum(PORTIONS)
    m = O.mamba_spec(H, V, N, G, K, parts)
    mod, cache, w = _mixer("mamba2", m, W, dev, 11, n)
    h = torch.randn((n, W), generator=torch.Generator().manual_seed(1))
    close(_feed(mod, cache, h, PORTIONS, [4, 0, 2, 1], dev), O.state_space(h.double(), w, m, 1e-5), 1e-3)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("N", [8, 300])
def test_step_recurrence_remembers_and_forgets_by_its_step_size(device, N):
    """Head 0 takes tiny steps (position 0 is still there 300 tokens later), head 1 large ones (only the
    current token is left); the skip adds the input itself; a large pre-activation is not clamped."""
    from polykey_service_amd.ops import lightning as lt
    dev, n, H, V = torch.device(device), 302, 2, 3
    xbc = torch.zeros((n, H * V + 2 * N))
    xbc[0, :H * V] = 1.0
    xbc[-1, :H * V] = 10.0
    xbc[0, H * V] = 1e3                       # B of the first token, along state row 0
    xbc[-1, H * V + 1] = 1.0                  # B of the last one, along row 1
    xbc[-1, H * V + N:H * V + N + 2] = 1.0    # C reads both
    dt = torch.tensor([[0.0, 0.0]]).repeat(n, 1)
    dt_bias, a_log, skip = torch.tensor([-12.0, 25.0]), torch.tensor([0.5, 0.1]), torch.tensor([0.25, -2.0])
    state = torch.full((2, H, N, V), 9.0, device=dev)
    to = lambda t: t.to(dev)
    o = torch.cat([lt.step_scan(to(xbc[sl]), to(dt[sl]), to(dt_bias), to(a_log), to(skip), state, md.cu_q, 1, pos, md.state_slots, H, N,
                                V, 1) for sl, pos, md in Feed(dev, [0] * 10).portions([120, 1, 1, 180])]).cpu().double()[-1].view(H, V)
    d = O.softplus(dt_bias.double())
    kept = torch.exp(-torch.exp(a_log.double()) * d * (n - 1)) * d * 1e3
    close(o, (kept + 10 * d + 10 * skip.double())[:, None].expand(H, V), 1e-4)
    assert float(kept[0]) > 1e-3 and float(kept[1]) < 1e-30


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("N,parts", [(48, 2), (30, 3), (21, 7), (2048, 1), (4096, 8), (17, 1)])
def test_gate_before_the_norm_in_parts(device, N, parts):
    """Parts of very unequal size: one norm over the whole row, or the gate behind the norm, would show."""
    from polykey_service_amd.ops import lightning as lt
    dev, T = torch.device(device), 6
    g = torch.Generator().manual_seed(N)
    y = torch.randn((T, N), generator=g) * torch.exp(torch.linspace(-2, 2, parts)).repeat_interleave(N // parts)
    z, w = torch.randn((T, N + 8), generator=g), torch.randn(N, generator=g)
    for dt, tol in ((torch.float32, 1e-4), (torch.bfloat16, 1e-2)):
        zz = z.to(dt)
        got = lt.gated_group_norm(y.to(dev), zz.to(dev)[:, :N], w.to(dev), parts, 1e-3, dt)
        close(got, O.group_norm(y.double() * O.silu(zz[:, :N].double()), parts, w.double(), 1e-3), tol)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W,T", [(40, 9), (42, 5), (33, 2), (2048, 3), (2048, 1030), (4100, 2), (4097, 2)])
def test_two_branch_stream_step(device, W, T):
    from polykey_service_amd.ops import hyper as hy
    dev = torch.device(device)
    g = torch.Generator().manual_seed(W)
    r = lambda *s: torch.randn(s, generator=g)
    x, ya, yb, wa, wb, pw = r(T, 1, W), 3 * r(T, W), 0.1 * r(T, W), r(W), r(W), r(W)
    for dt in (torch.float32, torch.bfloat16):
        a, b, xs = ya.to(dt), yb.to(dt), x.clone().to(dev)
        act = hy.pair_step(xs, a.to(dev), b.to(dev), wa.to(dev), wb.to(dev), 0.5, 0.3, pw.to(dev), 1e-3, dt)
        y = 0.5 * O.unit(a.double(), 1e-3) * wa + 0.3 * O.unit(b.double(), 1e-3) * wb
        close(xs[:, 0], x[:, 0] + O.unit(y, 1e-3) * pw, 1e-4)
        close(act, xs[:, 0].to(dt), 1e-6)


@pytest.mark.gpu
@pytest.mark.parametrize("W", [64, 66])
def test_two_branch_stream_step_sums_split_k_slabs(W):
    from polykey_service_amd.ops import gemm
    from polykey_service_amd.ops import hyper as hy
    dev, T = torch.device("cuda"), 5
    g = torch.Generator().manual_seed(W)
    r = lambda *s: torch.randn(s, generator=g).to(dev)
    x, sa, sb, wa, wb, pw = r(T, 1, W), r(4, T, W), r(2, T, W), r(W), r(W), r(W)
    x1, x2 = x.clone(), x.clone()
    a1 = hy.pair_step(x1, gemm.Partial(sa.flatten(), 4, T, W), gemm.Partial(sb.flatten(), 2, T, W), wa, wb, 0.5, 0.5, pw, 1e-5, torch.bfloat16)
    a2 = hy.pair_step(x2, sa.sum(0), gemm.Partial(sb.sum(0).flatten(), 1, T, W), wa, wb, 0.5, 0.5, pw, 1e-5, torch.bfloat16)
    close(x1, x2, 1e-5)
    close(a1, a2, 1e-2)
    x3, x4, h = x.clone(), x.clone(), sb[0].to(torch.bfloat16)     # one branch in slabs, the other as bf16 rows
    hy.pair_step(x3, gemm.Partial(sa.flatten(), 4, T, W), h, wa, wb, 0.5, 0.5, pw, 1e-5, torch.bfloat16)
    hy.pair_step(x4, h, gemm.Partial(sa.flatten(), 4, T, W), wb, wa, 0.5, 0.5, pw, 1e-5, torch.bfloat16)
    close(x3, x4, 1e-5)
    y = 0.5 * O.unit(sa.sum(0).double(), 1e-5) * wa + 0.5 * O.unit(h.double(), 1e-5) * wb
    close(x3[:, 0], x[:, 0] + O.unit(y, 1e-5) * pw, 1e-4)


def test_configuration_is_checked():
    def broken(i, change):
        cfg = copy.deepcopy(O.make_config())
        change(cfg["layers"][i])
        return cfg
    at = lambda *path: (lambda key, v: (lambda l: __import__("functools").reduce(lambda d, k: d[k], path, l).__setitem__(key, v)))
    for cfg in (broken(0, at("mixer")("heads", 3)), broken(0, at("mixer", "q_temp")("every", 2.5)), broken(1, at("mixer", "left")("vdim", 5)),
                broken(1, at("mixer", "left", "rot")("dims", 14)), broken(1, at("mixer", "right")("heads", 3)),
                broken(2, at("mixer")("groups", 4)), broken(2, at("mixer")("norm_groups", 4)), broken(3, at()("weights_of", 2)),
                broken(3, at()("weights_of", 3)), broken(3, at()("weights_of", 9)), broken(0, at()("type", "mamba1")),
                broken(0, at("mlp")("kind", "moe"))):
        with pytest.raises(ValueError):
            VagelixConfig.from_json(cfg)
    c = VagelixConfig.from_json(O.make_config())
    assert [l.weights_of for l in c.layers] == [-1, -1, -1, 1, -1] and c.layers[2].mlp is None and c.needs_state
    m = O.make_config(layers=[{"type": "attention", "mixer": O.diff_spec(), "mlp": None}] * 2)
    assert not VagelixConfig.from_json(m).needs_state
    chain = O.make_config()
    chain["layers"].append(dict(chain["layers"][3], weights_of=3))
    assert VagelixConfig.from_json(chain).layers[5].weights_of == 1


# ------------------------------------------------------------------ the whole model through the engine
@pytest.mark.parametrize("device", DEVICES)
def test_prompt_logits_and_layer_streams_match_the_plain_model(device, small):
    cfg, w, path = small
    eng = engine(path, device)
    assert eng.model.embed.device.type == device
    toks = rand_tokens(100, cfg["vocab"], 1)
    want, layers = O.forward(cfg, w, toks)
    got = replay(eng, [[("a", toks, list(range(100)), True)]])
    close(rows_of(got, "a", 100), want, 1e-3)
    dev = torch.device(device)
    md = SimpleNamespace(slot_mapping=i32(list(range(100)), dev), block_tables=i32([[0, 1, 2, 3]], dev), cu_q=i32([0, 100], dev),
                         context_lens=i32([100], dev), num_seqs=1, state_slots=i32([0], dev), token_seq=i32([0] * 100, dev),
                         num_decode=0)
    trail = []
    eng.model(i32(toks, dev), i32(list(range(100)), dev), md, eng.model.alloc_cache(4, BS, 1), trail=trail)
    assert len(trail) == len(layers)
    for x, y in zip(trail, layers):
        close(x, y, 1e-3)


def test_a_layer_on_another_ones_weights_has_its_own_cache(small):
    cfg, w, path = small
    eng = engine(path, "cpu")
    L, c = eng.model.layers, eng.runner.kv_caches
    assert L[3] is L[1] and L[4] is not L[2] and len(L) == 5 == len(c)
    for name in c[1]:
        assert c[1][name].data_ptr() != c[3][name].data_ptr()
    own = [l for l in cfg["layers"] if l["type"] == "parallel"]
    assert eng.model.state_bytes_per_slot() == 4 * sum(t[0].numel() for x in c if isinstance(x, dict) for n, t in x.items() if n not in "kv")
    assert eng.model.cache_bytes_per_block(BS) == 4 * BS * (len(own) * 2 * 2 * 12 + 2 * (2 * 9 + 13))


@pytest.mark.parametrize("device", DEVICES)
def test_decoding_equals_prefill(device, small):
    cfg, w, path = small
    toks = rand_tokens(90, cfg["vocab"], 3)
    got = replay(engine(path, device), [[s] for s in cut("a", toks, [50])])
    close(rows_of(got, "a", 90), logits_of(cfg, w, toks), 1e-3)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("sizes", [[2, 2, 2, 3, 40, 2, 17], [33, 31, 1, 1, 2], [7] * 14, [1, 1, 1, 2, 64]])
def test_portions_of_any_size(device, small, sizes):
    cfg, w, path = small
    toks = rand_tokens(100, cfg["vocab"], 4)
    got = replay(engine(path, device), [[s] for s in cut("a", toks, sizes)])
    close(rows_of(got, "a", 100), logits_of(cfg, w, toks), 1e-3)


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
        close(rows_of(got, rid, n), logits_of(cfg, w, toks[rid]), 1e-3)
    assert eng.scheduler.bm.num_free_state_slots == 4


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_past_chunks_and_pages(device, tmp_path):
    """One-token steps across several chunks, temperature steps and pages, with other sizes: one key /
    value head, one group, a single tap, an untouched half of the heads' coordinates."""
    cfg = O.make_config(vocab=50, width=36, layers=[
        {"type": "mamba2", "mixer": O.mamba_spec(3, 10, 16, 1, 1, 1), "mlp": None},
        {"type": "parallel", "mixer": O.parallel_spec(3, 1, 16, 13, 4, 1e3, 2, 1, 12, 7, 1), "mlp": FF},
        {"type": "attention", "mixer": O.diff_spec(3, 1, 6, 10, 0.8, 0.6, 5), "mlp": None}])
    w = O.random_model(cfg, seed=8, rank=2, grank=9)
    toks = rand_tokens(150, cfg["vocab"], 5)
    got = replay(engine(checkpoint(tmp_path, cfg, w), device), [[s] for s in cut("a", toks, [3])])
    close(rows_of(got, "a", 150), logits_of(cfg, w, toks), 1e-3)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("layers", [
    [{"type": "attention", "mixer": O.diff_spec(2, 2, 16, 16, 0.5, 0.1, 32), "mlp": None},
     {"type": "attention", "mixer": O.diff_spec(2, 2, 16, 16, 0.5, 0.1, 32), "mlp": None, "weights_of": 0}],
    [{"type": "parallel", "mixer": O.parallel_spec(6, 3, 10, 20, 2, 1e5, 3, 3, 16, 16, 2), "mlp": FF},
     {"type": "mamba2", "mixer": O.mamba_spec(4, 16, 8, 4, 5, 1), "mlp": FF},
     {"type": "mamba2", "mixer": O.mamba_spec(4, 16, 8, 4, 5, 1), "mlp": FF, "weights_of": 1},
     {"type": "parallel", "mixer": O.parallel_spec(6, 3, 10, 20, 2, 1e5, 3, 3, 16, 16, 2), "mlp": FF, "weights_of": 0}],
    [{"type": "parallel", "mixer": O.parallel_spec(2, 2, 32, 64, 32, 10.0, 8, 2, 4, 24, 5), "mlp": None}],
    [{"type": "mamba2", "mixer": O.mamba_spec(1, 64, 4, 1, 2, 1), "mlp": FF},
     {"type": "attention", "mixer": O.diff_spec(8, 2, 4, 32, 0.05, 1.5, 1), "mlp": FF}]])
def test_other_sizes_and_orders(device, tmp_path, layers):
    cfg = O.make_config(vocab=83, width=52, layers=layers, eps=1e-4)
    w = O.random_model(cfg, seed=9, rank=12, grank=3)
    toks = rand_tokens(120, cfg["vocab"], 6)
    got = replay(engine(checkpoint(tmp_path, cfg, w), device), [[s] for s in cut("a", toks, [31, 2, 70])])
    close(rows_of(got, "a", 120), logits_of(cfg, w, toks), 1e-3)


def _drawn_config(seed):
    r = random.Random(seed)

    def mixer(kind):
        kv = r.choice([1, 2, 3])
        if kind == "parallel":
            D, rkv = r.choice([6, 10, 16]), r.choice([1, 2])
            return O.parallel_spec(kv * r.choice([1, 2]), kv, D, r.choice([5, 9, 32, 70]), r.choice([2, 4, D]), r.choice([20.0, 1e4]),
                                   rkv * r.choice([1, 3]), rkv, r.choice([4, 18]), r.choice([5, 12]), r.randint(1, 5))
        if kind == "mamba2":
            return O.mamba_spec(kv * r.choice([1, 2]), r.choice([6, 12]), r.choice([5, 16, 20]), kv, r.randint(1, 5), r.choice([1, 2, 3]))
        return O.diff_spec(kv * r.choice([1, 2]), kv, r.choice([4, 7, 16]), r.choice([3, 8, 12]), r.choice([0.1, 0.7]), r.choice([0.1, 0.9]),
                           r.choice([3, 10, 64]))
    kinds = r.sample(["parallel", "mamba2", "attention"], 3) + [r.choice(["parallel", "mamba2", "attention"])]
    layers = [{"type": k, "mixer": mixer(k), "mlp": r.choice([None, {"kind": "dense", "ff": r.choice([20, 44])}])} for k in kinds]
    j = r.randrange(len(layers))
    layers.insert(r.randint(j + 1, len(layers)), dict(layers[j], weights_of=j))
    return O.make_config(vocab=r.randint(40, 90), width=r.choice([24, 36, 50]), layers=layers, eps=r.choice([1e-6, 1e-3]))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6, 7, 8])
def test_drawn_configurations_in_mixed_steps(device, tmp_path, seed):
    """Layer orders and sizes drawn at random, three unequal requests in steps drawn at random (a
    request may sit out a step), against the plain model."""
    cfg = _drawn_config(seed)
    w = O.random_model(cfg, seed=seed, rank=seed, grank=9 - seed)
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
        cfg = EngineConfig(model="tiny-vagelix", dtype="float32", block_size=BS, max_num_seqs=2, max_num_batched_tokens=64,
                           max_model_len=128, num_kv_blocks=8, watermark=0.0, hip_graphs=False, device=device, seed=5)
        eng = LLMEngine(cfg, ParallelState(device=torch.device(device)))
        outs.append(eng.generate([list(range(3, 40)), [7, 8, 9]], SamplingParams(max_tokens=6, temperature=0.0, ignore_eos=True)))
    assert outs[0] == outs[1] and all(len(o) == 6 for o in outs[0])
    assert eng.mcfg.num_params() == sum(t.numel() for t in eng.model.random_state(0).values())


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


def _aligned_config():
    return O.make_config(vocab=120, width=256, ff=512, layers=[
        {"type": "parallel", "mixer": O.parallel_spec(4, 2, 64, 72, 32, 1e4, 4, 2, 64, 128, 4), "mlp": {"kind": "dense", "ff": 512}},
        {"type": "mamba2", "mixer": O.mamba_spec(8, 64, 64, 2, 4, 2), "mlp": {"kind": "dense", "ff": 512}},
        {"type": "attention", "mixer": O.diff_spec(4, 2, 64, 128, 0.4, 0.3, 64), "mlp": {"kind": "dense", "ff": 512}},
        {"type": "parallel", "mixer": O.parallel_spec(4, 2, 64, 72, 32, 1e4, 4, 2, 64, 128, 4), "mlp": {"kind": "dense", "ff": 512},
         "weights_of": 0}])


@pytest.mark.gpu
def test_aligned_sizes_in_mixed_batches_with_decode_graphs(tmp_path):
    """A bf16 model at sizes the decode GEMM, the matrix-core attention and the vectorised kernels take:
    unequal live requests, prompt portions beside decoded tokens, decode graphs; against the ops'
    compositions at the same precision and the plain model."""
    cfg = _aligned_config()
    w = O.random_model(cfg, seed=12, rank=128, grank=128)
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
def test_decode_graph_replays_equal_eager_steps(tmp_path):
    """The same decode steps replayed from graphs (a padded bucket, state slots that change owners between
    replays) and run eagerly."""
    cfg = _aligned_config()
    path = checkpoint(tmp_path, cfg, O.random_model(cfg, seed=14, rank=128, grank=128))
    toks = {k: rand_tokens(60, cfg["vocab"], 50 + i) for i, k in enumerate("abcde")}
    steps = interleave({k: cut(k, v, [30]) for k, v in toks.items()}, waiting=["d", "e"])
    runs = [replay(engine(path, "cuda", dtype="bfloat16", pool_tokens=512, graphs=gr), steps) for gr in (True, False)]
    for k in toks:
        assert float(rel(rows_of(runs[0], k, 60), rows_of(runs[1], k, 60)).max()) < 1e-2, k


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,chunk", [(4, 2, 64, 100), (8, 2, 128, 33), (16, 4, 128, 512), (2, 2, 64, 1)])
def test_matrix_core_attention_in_chunks_with_gates_matches_the_fma_tiles(H, G, D, chunk):
    """bf16 at the matrix-core kernel's sizes, prompt portions and decoded tokens (cut into runs and
    merged), against the FMA kernel on the same caches and against the plain rule."""
    from polykey_service_amd.ops import masked_attention as ma
    from polykey_service_amd.ops import native
    dev, n, bf = torch.device("cuda"), 300, torch.bfloat16
    g = torch.Generator().manual_seed(H * 100 + D)
    q = torch.randn((n, H, D), generator=g).to(bf)
    k, v = (0.5 * torch.randn((n, G, D), generator=g)).to(bf), torch.randn((n, G, D), generator=g).to(bf)
    gate = torch.randn((n, H + 3), generator=g).to(bf)
    sink = torch.zeros(H, device=dev)
    outs = {}
    for mfma in (1, 0):
        native.mixers().pkm_set_masked_mfma(mfma)
        try:
            kc, vc = torch.zeros((12, G, BS, D), device=dev, dtype=bf), torch.zeros((12, G, BS, D), device=dev, dtype=bf)
            got = []
            for sl, pos, md in Feed(dev, [7, 2, 11, 0, 5, 9, 3, 1, 10, 4, 6, 8]).portions([150, 1, 1, 40, 2, 1, 1, 1, 103]):
                at = md.slot_mapping.long()
                kc[at // BS, :, at % BS], vc[at // BS, :, at % BS] = k[sl].to(dev), v[sl].to(dev)
                got.append(ma.masked_attention(q[sl].contiguous().to(dev), kc, vc, D, md.block_tables, md.cu_q, md.context_lens, 1,
                                               D ** -0.5, chunk=chunk, sink=sink, fine=True, head_gate=gate.to(dev)[sl, 1:1 + H],
                                               num_decode=md.num_decode))
            outs[mfma] = torch.cat(got).cpu()
        finally:
            native.mixers().pkm_set_masked_mfma(1)
    close(outs[1], outs[0], 3e-4)
    want = O.softmax_rows(q.double(), k.double(), v.double(), D ** -0.5, chunk, True)
    close(outs[0], want * O.sigmoid(gate[:, 1:1 + H].double())[..., None], 3e-4)
