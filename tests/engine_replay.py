"""Helpers of the model-family tests: checkpoint folders from dicts of tensors, engines over them,
token schedules replayed through the engine's steps, and one sequence fed to a single mixer in
portions over hand-made pages and a hand-made state slot."""
import json
import random
from types import SimpleNamespace

import torch

from polykey_service_amd.engine import EngineConfig, LLMEngine
from polykey_service_amd.parallel.state import ParallelState

BS = 32


def checkpoint(tmp_path, cfg, w, name="m"):
    from safetensors.torch import save_file
    d = tmp_path / name
    d.mkdir()
    (d / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in w.items()}, str(d / "model.safetensors"))
    return str(d)


def engine(path, device, dtype="float32", pool_tokens=512, max_seqs=4, budget=512, graphs=False, max_len=None):
    cfg = EngineConfig(model_path=path, dtype=dtype, block_size=BS, max_num_seqs=max_seqs, max_num_batched_tokens=budget,
                       max_model_len=max_len or pool_tokens, num_kv_blocks=pool_tokens // BS, watermark=0.0,
                       hip_graphs=graphs, device=device, graph_batch_sizes=(1, 2, 4))
    return LLMEngine(cfg, ParallelState(device=torch.device(device)))


def replay(eng, steps):
    """steps: list of lists of (id, tokens, want, end?) -> {id: {position: logits row}}."""
    got, at = {}, {}
    for step in steps:
        ends = [e[0] for e in step if len(e) > 3 and e[3]]
        lg = eng.replay_step([(e[0], e[1], e[2]) for e in step], ends)
        r = 0
        for e in step:
            base = at.get(e[0], 0)
            for wpos in e[2]:
                got.setdefault(e[0], {})[base + wpos] = lg[r]
                r += 1
            at[e[0]] = base + len(e[1])
            if e[0] in ends:
                at.pop(e[0])
    return got


def cut(rid, toks, sizes, end=True):
    """The request in portions of the given sizes (the rest one token at a time), all places wanted."""
    out, i = [], 0
    sizes = list(sizes)
    while i < len(toks):
        n = min(sizes.pop(0) if sizes else 1, len(toks) - i)
        out.append((rid, toks[i:i + n], list(range(n)), end and i + n == len(toks)))
        i += n
    return out


def interleave(plans, waiting=(), skip=None):
    """Steps that advance every live plan by one portion; a finished request makes room for a waiting
    one.  ``skip`` (a random.Random): a request may sit out a step."""
    plans, live, waiting, steps = {k: list(v) for k, v in plans.items()}, [], list(waiting), []
    live = [k for k in plans if k not in waiting]
    while live:
        step = []
        for rid in list(live):
            if skip is not None and skip.random() < 0.15 and len(live) > 1:
                continue
            step.append(plans[rid].pop(0))
            if not plans[rid]:
                live.remove(rid)
                if waiting:
                    live.append(waiting.pop(0))
        if step:
            steps.append(step)
    return steps


def close(a, b, tol=3e-4):
    torch.testing.assert_close(a.float().cpu(), b.float().cpu(), rtol=tol, atol=tol)


def rel(a, b):
    """Per row: root mean square of the difference over that of b."""
    a, b = a.double().cpu(), b.double().cpu()
    return (a - b).pow(2).mean(-1).sqrt() / b.pow(2).mean(-1).sqrt()


def rand_tokens(n, vocab, seed):
    return random.Random(seed).choices(range(vocab), k=n)


def rows_of(got, rid, n):
    return torch.stack([got[rid][i] for i in range(n)])


def i32(v, dev):
    return torch.tensor(v, dtype=torch.int32, device=dev)


class Feed:
    """One sequence fed in portions: pages, slot and step metadata by hand."""

    def __init__(self, dev, pages, slot=1):
        self.dev, self.pages, self.slot, self.at = dev, pages, slot, 0

    def step(self, c):
        dev, at = self.dev, self.at
        pos = torch.arange(at, at + c, dtype=torch.int32, device=dev)
        md = SimpleNamespace(slot_mapping=i32([self.pages[p // BS] * BS + p % BS for p in range(at, at + c)], dev),
                             block_tables=i32([self.pages], dev), cu_q=i32([0, c], dev), context_lens=i32([at + c], dev),
                             num_seqs=1, state_slots=i32([self.slot], dev), token_seq=i32([0] * c, dev),
                             num_decode=1 if (c == 1 and at) else 0)
        self.at += c
        return pos, md

    def portions(self, sizes):
        """(slice of the sequence, positions, metadata) per portion."""
        for c in sizes:
            pos, md = self.step(c)
            yield slice(self.at - c, self.at), pos, md


def full(y):
    """A projection's result: a tensor, or the decode GEMM's unreduced slabs."""
    return (y if isinstance(y, torch.Tensor) else y.view().sum(0)).float().cpu()
