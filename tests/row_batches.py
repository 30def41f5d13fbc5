"""Ragged batches of rows over a paged cache in random page order, for tests of single kernels."""
import random

import torch

from nanovllm_amd.context import RowGroup

BF16, F32 = torch.bfloat16, torch.float32
BLOCK = 256


def tol(dtype, bf16, f32):
    return bf16 if dtype is BF16 else f32


def close(got, want, tol, what=""):
    got, want = got.double().cpu(), want.double().cpu()
    assert torch.isfinite(got).all(), what
    err = float((got - want).abs().max() / want.abs().max().clamp_min(1e-6))
    assert err <= tol, f"{what}: {err:.3g} > {tol:.3g}"


class Batch:
    """Sequences of given lengths of which the last ``count`` tokens are this step's rows."""

    def __init__(self, dev, spans, single=False, pad=0, seed=0, extra_slots=2):
        rng = random.Random(seed)
        self.spans, self.single, self.pad = spans, single, pad
        need = [-(-n // BLOCK) for n, _ in spans]
        self.num_blocks = sum(need) + 3
        ids = list(range(self.num_blocks))
        rng.shuffle(ids)
        self.tables, at = [], 0
        for n in need:
            self.tables.append(ids[at: at + n])
            at += n
        self.state_slots = rng.sample(range(len(spans) + extra_slots), len(spans))
        self.num_state_slots = len(spans) + extra_slots
        i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=dev)
        width = max(need)
        rows = sum(c for _, c in spans) + pad
        slots, pos = [], []
        for (n, c), t in zip(spans, self.tables):
            slots += [t[p // BLOCK] * BLOCK + p % BLOCK for p in range(n - c, n)]
            pos += range(n - c, n)
        self.positions = torch.tensor(pos + [0] * pad, dtype=torch.int64, device=dev)
        table = [t + [-1] * (width - len(t)) for t in self.tables] + [[0] * width] * pad
        seqs = len(spans) + pad
        self.group = RowGroup(0, rows, seqs, i32([n for n, _ in spans] + [0] * pad), i32(slots + [-1] * pad), i32(table),
                              i32(self.state_slots + [-1] * pad))
        if single:
            assert all(c == 1 for _, c in spans)
        else:
            assert pad == 0
            cu = [0]
            for _, c in spans:
                cu.append(cu[-1] + c)
            self.group.cu, self.group.token_seq = i32(cu), i32([i for i, (_, c) in enumerate(spans) for _ in range(c)])
            self.group.max_q = max(c for _, c in spans)
            self.group.spans = [(n - c, c) for n, c in spans]

    def rows(self, full):
        """This step's rows of per-sequence tensors ``[n, ...]``, packed; zero rows for the padding."""
        out = torch.cat([x[n - c: n] for x, (n, c) in zip(full, self.spans)])
        return torch.cat([out, torch.zeros((self.pad,) + out.shape[1:], dtype=out.dtype)]) if self.pad else out

    def fill(self, cache, full, upto_start=True):
        """Writes rows of every sequence into the paged cache (those before this step's, or all)."""
        for x, (n, c), t in zip(full, self.spans, self.tables):
            for p in range(n - c if upto_start else n):
                cache[t[p // BLOCK], p % BLOCK] = x[p].to(cache.dtype)

    def gather(self, cache):
        return torch.cat([torch.stack([cache[t[p // BLOCK], p % BLOCK] for p in range(n - c, n)]) for (n, c), t in zip(self.spans, self.tables)])


PORTIONS = [(300, 300), (2, 2), (257, 3), (600, 90), (40, 2), (130, 65), (1, 1), (70, 69)]
SINGLES = [(300, 1), (2, 1), (257, 1), (1, 1), (600, 1), (33, 1), (256, 1)]


def batches(dev):
    return [Batch(dev, PORTIONS, seed=1), Batch(dev, SINGLES, single=True, pad=2, seed=2)]


def rand(g, *shape, dtype):
    return torch.randn(*shape, generator=g).to(dtype)
