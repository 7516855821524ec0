"""One step's batch as the kernels read it: prompt portions first, then the single tokens, one upload for all index arrays."""
from __future__ import annotations

import dataclasses
from typing import List, Sequence as Seq

import numpy as np
import torch

from .cache import Sequence


@dataclasses.dataclass
class Entry:
    seq: Sequence
    tokens: Seq[int]
    want: Seq[int]            # places among `tokens` whose logits are asked for


@dataclasses.dataclass
class DeviceBatch:
    n_prompt: int             # tokens of portions (they come first)
    n_decode: int             # single tokens behind them
    n_entries: int            # portions
    max_context: int          # upper bound of the longest sequence's length after the step
    tokens: torch.Tensor      # [T]
    pos: torch.Tensor         # [T] position of each token; < 0: an empty place
    kv_slot: torch.Tensor     # [T] page * 64 + offset
    state_slot: torch.Tensor  # [n_decode]
    rows: torch.Tensor        # wanted tokens
    entry: torch.Tensor       # [n_entries, 4] first token, tokens, position, block table row
    attn_tiles: torch.Tensor  # [., 2] portion, first row
    segments: torch.Tensor    # [., 8]
    block_table: torch.Tensor # [n_entries + n_decode, pages]
    portions: torch.Tensor = None      # [n_entries, 8] first token, tokens, state slot, starts from zero, first chunk, chunks, position, 0
    chunks: torch.Tensor = None        # [.] portion of every chunk
    context_pages: torch.Tensor = None # pages of the portions' contexts, one portion behind the other
    context_table: torch.Tensor = None # [n_entries, pages] place of a portion's page among those of its expansion
    segment_len: int = 64
    multi_segment: bool = False
    expansions: tuple = ()             # (first context page, pages, first tile, tiles) of portions whose contexts are expanded at once


class BatchBuilder:
    """Lays a step out in one pinned int32 buffer and uploads it."""

    def __init__(self, model, device):
        self.page, self.attn_rows, self.device = model.page_size, model.attn_rows, device
        self.linear_wgs = model.linear_workgroups()
        self.min_segments = model.min_segments
        self.chunk, self.expand = model.chunk_rows, model.expand_pages

    def _segment_len(self, portions: List[Entry]) -> int:
        """Tokens per segment of a recurrent layer: enough segments for two workgroups per CU, none below 256 tokens, at most 32
        per portion (every segment starts from the sum of those before it); none when the longest portion makes fewer than
        min_segments (a first pass over the segments costs as much as it saves)."""
        total, longest = sum(len(e.tokens) for e in portions), max(len(e.tokens) for e in portions)
        want = max(1, 512 // max(self.linear_wgs, 1))
        n = max(256, -(-total // want), -(-longest // 32))
        if longest < n * self.min_segments:
            n = longest
        return -(-n // 64) * 64

    def build(self, entries: List[Entry]):
        """-> (DeviceBatch, [(entry index, place)] of the rows in order).  Pages must have been reserved."""
        order = sorted(range(len(entries)), key=lambda i: len(entries[i].tokens) == 1)       # stable: portions first
        portions = [entries[i] for i in order if len(entries[i].tokens) > 1]
        single = [entries[i] for i in order if len(entries[i].tokens) == 1]
        n_prompt, n_decode = sum(len(e.tokens) for e in portions), len(single)
        T, N = n_prompt + n_decode, len(entries)
        width = max([e.seq.pages for e in entries] + [1])
        tokens, pos, slot = (np.zeros((T,), np.int32) for _ in range(3))
        table = np.zeros((N, width), np.int32)
        ent, tiles, segs, rows, wanted = [], [], [], [], []
        ports, chunks, context, groups = [], [], [], []
        context_table = np.zeros((len(portions) if self.expand else 0, width), np.int32)
        seg_len, multi, at = 64, False, 0
        if portions:
            seg_len = self._segment_len(portions)
        for k, i in enumerate(order):
            e, n = entries[i], len(entries[i].tokens)
            p0 = e.seq.length
            tokens[at:at + n] = e.tokens
            pos[at:at + n] = np.arange(p0, p0 + n)
            if e.seq.pages:
                p = pos[at:at + n]
                slot[at:at + n] = e.seq.table[p // self.page] * self.page + p % self.page
                table[k, :e.seq.pages] = np.maximum(e.seq.table[:e.seq.pages], 0)
            if n > 1:
                ent.append((at, n, p0, k))
                here = [(k, r) for r in range(0, n, self.attn_rows)]
                if self.expand:
                    if not groups or groups[-1][1] + e.seq.pages > self.expand:
                        groups.append([len(context), 0, len(tiles), 0])
                    context_table[k, :e.seq.pages] = groups[-1][1] + np.arange(e.seq.pages)
                    context += table[k, :e.seq.pages].tolist()
                    groups[-1][1] += e.seq.pages
                    groups[-1][3] += len(here)
                tiles += here
                if self.chunk:
                    nc = -(-n // self.chunk)
                    ports.append((at, n, e.seq.slot, int(p0 == 0), len(chunks), nc, p0, 0))
                    chunks += [len(ports) - 1] * nc
                ns = -(-n // seg_len)
                multi |= ns > 1
                ck = (ports[-1][4], seg_len // self.chunk) if self.chunk else (0, 0)
                segs += [(at + s * seg_len, min(seg_len, n - s * seg_len), e.seq.slot, int(p0 == 0), s, ns, ck[0] + s * ck[1], 0)
                         for s in range(ns)]
            for w in e.want:
                rows.append(at + w)
                wanted.append((i, w))
            at += n
        parts = [tokens, pos, slot, np.array([e.seq.slot for e in single], np.int32), np.array(rows, np.int32),
                 np.array(ent, np.int32).reshape(-1, 4), np.array(tiles, np.int32).reshape(-1, 2),
                 np.array(segs, np.int32).reshape(-1, 8), table, np.array(ports, np.int32).reshape(-1, 8), np.array(chunks, np.int32),
                 np.array(context, np.int32), context_table]
        d = self._upload(parts)
        longest = max(e.seq.length + len(e.tokens) for e in entries)
        return DeviceBatch(n_prompt, n_decode, len(portions), longest, *d, segment_len=seg_len, multi_segment=multi,
                           expansions=tuple(map(tuple, groups))), wanted

    def _upload(self, parts):
        sizes = [p.size for p in parts]
        host = torch.empty((sum(sizes),), dtype=torch.int32, pin_memory=self.device.type == "cuda")
        np.concatenate([p.reshape(-1) for p in parts], out=host.numpy())
        dev = host.to(self.device, non_blocking=True)
        out, at = [], 0
        for p, n in zip(parts, sizes):
            out.append(dev[at:at + n].view(p.shape))
            at += n
        return out


class DecodeSlots:
    """A batch of single tokens at fixed addresses, for a captured step: `places` sequences, block tables of `width` pages."""

    def __init__(self, builder: BatchBuilder, places: int, width: int):
        self.places, self.width, self.page = places, width, builder.page
        n = places * (5 + width)
        self.host = torch.zeros((n,), dtype=torch.int32, pin_memory=True)
        self.dev = torch.zeros((n,), dtype=torch.int32, device=builder.device)
        v = lambda t: [t[i * places:(i + 1) * places] for i in range(5)] + [t[5 * places:].reshape(places, width)]      # noqa: E731
        self._np = v(self.host.numpy())
        tokens, pos, slot, state, rows, table = v(self.dev)
        none = torch.zeros((0, 8), dtype=torch.int32, device=builder.device)
        self.batch = DeviceBatch(0, places, 0, width * self.page, tokens, pos, slot, state, rows, none[:, :4], none[:, :2], none, table)
        self._copied = torch.cuda.Event()
        self.fill([])

    def fill(self, entries: List[Entry]) -> None:
        self._copied.synchronize()           # the previous upload may still read the host buffer
        tokens, pos, slot, state, rows, table = self._np
        n = len(entries)
        pos[:] = -1
        slot[:] = -1
        tokens[:] = 0
        state[:] = 0
        rows[:] = np.arange(self.places)
        for i, e in enumerate(entries):
            p = e.seq.length
            tokens[i], pos[i], state[i] = e.tokens[0], p, e.seq.slot
            if e.seq.pages:
                slot[i] = e.seq.table[p // self.page] * self.page + p % self.page
                first = e.seq.released
                table[i, first:e.seq.pages] = e.seq.table[first:e.seq.pages]
        self.dev.copy_(self.host, non_blocking=True)
        self._copied.record()
