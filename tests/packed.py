"""Steps over a paged cache put together by hand, for tests that call an attention kernel alone."""

from __future__ import annotations

import torch

DEV = "cuda:0"


def _i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


class PackedStep:
    """Rows of keys in a paged cache with shuffled pages, and the packed queries of a step over them: row ``r`` has
    ``lengths[r]`` keys, of which the last ``lengths[r] - starts[r]`` places are this step's queries. Pages that a window
    has passed and that hold no kept key are given back (the table says -1 and the page holds NaN)."""

    def __init__(self, lengths, starts, window, kept, seed):
        from types import SimpleNamespace

        self.lengths, self.starts, self.window, self.kept = lengths, starts, window, kept
        gen = torch.Generator().manual_seed(seed)
        self.gen = gen
        n_pages = sum(-(-n // 16) for n in lengths) + 3
        order = torch.randperm(n_pages, generator=gen).tolist()
        self.n_pages = n_pages
        table = torch.full((len(lengths), max(-(-n // 16) for n in lengths) + 1), -1, dtype=torch.int32)
        for r, n in enumerate(lengths):
            for p in range(-(-n // 16)):
                table[r, p] = order.pop()
        self.full_table = table.clone()
        if window is not None:
            for r, s in enumerate(starts):
                for p in range(max(0, s + 1 - window) // 16):
                    if p * 16 >= kept:
                        table[r, p] = -1
        token_row, kv_lo, kv_hi, cu_q, rows, first = [], [], [], [0], [], []
        for r, (n, s) in enumerate(zip(lengths, starts)):
            for b in range(0, n - s, 32):
                rows.append(r)
                first.append(len(token_row) + b)
            for p in range(s, n):
                token_row.append(r)
                kv_hi.append(p + 1)
                kv_lo.append(0 if window is None else max(0, p + 1 - window))
            cu_q.append(len(token_row))
        self.n = len(token_row)
        self.token_row, self.kv_hi, self.cu_q = _i32(token_row), _i32(kv_hi), _i32(cu_q)
        self.kv_lo = _i32(kv_lo) if window is not None else None
        self.table = table.to(DEV)
        from kestrel_amd.engine.batch import Workspace

        # (with a workspace at hand a decode step of few rows deals a row's keys out over several workgroups)
        self.batch = SimpleNamespace(decode_only=all(n - s == 1 for n, s in zip(lengths, starts)),
                                     query_blocks={32: (_i32(rows), _i32(first))}, cu_q=self.cu_q,
                                     workspace=Workspace(torch.device(DEV)))

    def pages(self, per_row, transposed=False):
        """``per_row[r]`` ``[length, heads, channels]`` into pages ``[pages, heads, 16, channels]`` (or ``[pages, heads, channels, 16]``);
        pages given back hold NaN."""
        heads, channels = per_row[0].shape[1:]
        out = torch.full((self.n_pages, heads, 16, channels), float("nan"), dtype=per_row[0].dtype)
        for r, rows in enumerate(per_row):
            for p in range(-(-rows.shape[0] // 16)):
                if self.table[r, p] >= 0:
                    part = rows[p * 16:(p + 1) * 16]
                    out[self.full_table[r, p], :, :part.shape[0]] = part.transpose(0, 1)
        return (out.transpose(2, 3) if transposed else out).contiguous().to(DEV)


# (lengths of the rows, where their queries of this step start)
CUTS = {"mixed": ([70, 133, 9, 2, 101, 64, 300], [0, 100, 7, 0, 100, 63, 267]), "decode": ([70, 133, 9, 1, 300], [69, 132, 8, 0, 299])}
