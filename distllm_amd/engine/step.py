"""Ragged step batches: what a model that runs them gets for one step.

A step holds, for each of its sequences, the next tokens of that
sequence — a portion of a prompt or one decoded token — and where its
cache pages are. Rows (tokens) of all sequences are packed without
padding between them. Sequences with few new tokens come first ("folded"
rows, attended one by one against the paged cache); longer portions
follow and are attended by the packed flash kernel. The row count is
rounded up so that products see few distinct shapes; padding rows have
ctx 0 and touch nothing.

Models with a recurrent state also get each sequence's state slot and
where its rows are: the rows of a sequence are consecutive and in order.
A sequence that starts in the step (ctx 1) starts from a zero state,
whatever its slot holds.
"""

from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np
import torch

from .. import ops


def row_bucket(n: int) -> int:
    """Rows a step of n tokens runs with: powers of two, then multiples
    of 256 (which also lets the large MFMA GEMMs compete)."""
    b = 8
    while b < n and b < 256:
        b <<= 1
    return b if n <= b else (n + 255) // 256 * 256


@dataclass
class Expansion:
    """Visible cached tokens of the expanded portions for one window."""

    key_seq: torch.Tensor    # [Tk] block-table row of each packed key
    key_pos: torch.Tensor    # [Tk] its position
    cu_q: torch.Tensor       # [P + 1]
    cu_k: torch.Tensor       # [P + 1]
    block_map: tuple[torch.Tensor, torch.Tensor]


@dataclass
class PromptBlocks:
    """Query blocks of the expanded portions for attention over paged keys
    and values: blocks[i] = (portion, block of QBLK queries)."""

    portions: torch.Tensor   # [P, 4] table row, first row, first pos, rows
    blocks: torch.Tensor     # [N, 2]

    QBLK = 128


@dataclass
class Segments:
    """Rows of each block-table row, and its state slot. Segments of more
    than SHORT rows are also described in chunks of CHUNK rows, for
    kernels that work chunk by chunk, and in pieces for kernels that run
    parts of a segment side by side."""

    row0: torch.Tensor       # [S] int32
    rows: torch.Tensor       # [S] int32
    slot: torch.Tensor       # [S] int32
    longest: int
    longs: torch.Tensor | None = None   # [P, 2] segment, its first chunk
    chunks: torch.Tensor | None = None  # [N, 2] segment, chunk in it
    sizes: list[int] = field(default_factory=list)  # rows, on the host
    _lists: dict = field(default_factory=dict)

    SHORT = 16
    CHUNK = 32
    PIECE = 256      # rows of a piece, at least
    PIECE_WGS = 512

    @classmethod
    def build(cls, row0, rows, slots, device) -> "Segments":
        def up(a, *shape):
            return torch.from_numpy(
                np.array(a, np.int32).reshape(*shape)).to(device)

        seg = cls(up(row0, -1), up(rows, -1), up(slots, -1),
                  max(rows, default=0), sizes=list(rows))
        seg.longs, seg.chunks = seg.chunk_lists(cls.CHUNK)
        return seg

    def chunk_lists(self, size: int) -> tuple:
        """(longs, chunks) in chunks of `size` rows; None where no segment
        is long."""
        if size not in self._lists:
            longs, chunks = [], []
            for i, n in enumerate(self.sizes):
                if n > self.SHORT:
                    longs.append((i, len(chunks)))
                    chunks += [(i, c) for c in range(-(-n // size))]
            self._lists[size] = (None, None) if not longs else tuple(
                torch.tensor(a, dtype=torch.int32).to(self.row0.device)
                for a in (longs, chunks))
        return self._lists[size]

    def pieces(self, heads: int) -> tuple:
        """Long segments cut into pieces of about equal size that can run
        side by side, as many as fill the GPU with a workgroup per piece
        and head: (longs [L, 2]: segment, its first piece; pieces [P, 5]:
        segment, first row, rows, number, pieces of the segment; whether
        there are several of any). None, None, False without a long
        segment."""
        key = ("pieces", heads)
        if key not in self._lists:
            total = sum(n for n in self.sizes if n > self.SHORT)
            most = max(self.PIECE, -(-total * heads // self.PIECE_WGS))
            longs, pieces, several = [], [], False
            for i, n in enumerate(self.sizes):
                if n <= self.SHORT:
                    continue
                each = -(-n // -(-n // most))
                each = -(-each // self.CHUNK) * self.CHUNK
                count = -(-n // each)
                longs.append((i, len(pieces)))
                pieces += [(i, p * each, min(each, n - p * each), p, count)
                           for p in range(count)]
                several |= count > 1
            self._lists[key] = (None, None, False) if not longs else (
                *(torch.tensor(a, dtype=torch.int32).to(self.row0.device)
                  for a in (longs, pieces)), several)
        return self._lists[key]


@dataclass
class StepBatch:
    tokens: torch.Tensor       # [M] int64
    ctx: torch.Tensor          # [M] int32, position + 1; 0 = padding
    row_seq: torch.Tensor      # [M] int32, block-table row
    block_table: torch.Tensor  # [S, max_blocks] int32
    n_folded: int              # leading rows attended one by one
    # rows of each entry, in the order in which entries were given
    rows: list[np.ndarray] = field(default_factory=list)
    # expanded portions: (block-table row, first position, new tokens)
    portions: list[tuple[int, int, int]] = field(default_factory=list)
    segments: Segments | None = None  # with state slots
    _expansions: dict[int, Expansion] = field(default_factory=dict)
    _prompts: dict[int, PromptBlocks] = field(default_factory=dict)
    _rotations: dict = field(default_factory=dict)

    def rotation(self, key, freq: torch.Tensor, mult: float):
        """cos and sin of every row's position, [M, pairs, 2] fp32; layers
        with the same rotation (`key`) share them."""
        if key not in self._rotations:
            self._rotations[key] = ops.rotation_table(self.ctx, freq, mult)
        return self._rotations[key]

    @classmethod
    def decode(cls, tokens, block_table, ctx, slots=None) -> "StepBatch":
        """One token per sequence, everything already on the device."""
        n = tokens.shape[0]
        each = torch.arange(n, dtype=torch.int32, device=tokens.device)
        seg = None
        if slots is not None:
            seg = Segments(each, torch.ones_like(each), slots.int(), 1)
        return cls(tokens=tokens.long(), ctx=ctx.int(), row_seq=each,
                   block_table=block_table.int(), n_folded=n, segments=seg)

    @classmethod
    def build(cls, entries, blk: int, device,
              expand_min: int = 32, slots=None) -> "StepBatch":
        """entries: (new tokens, tokens already cached, cache blocks).
        Portions of at least expand_min tokens are expanded. slots: the
        entries' state slots, for models that have a state."""
        order = sorted(range(len(entries)),
                       key=lambda i: len(entries[i][0]) >= expand_min)
        total = sum(len(t) for t, _, _ in entries)
        n_folded = sum(len(t) for t, _, _ in entries
                       if len(t) < expand_min)
        M = row_bucket(total)
        tokens = np.zeros(M, np.int64)
        ctx = np.zeros(M, np.int32)
        row_seq = np.zeros(M, np.int32)
        width = max(1, max((len(b) for _, _, b in entries), default=1))
        table = np.zeros((max(1, len(entries)), width), np.int32)
        rows: list = [None] * len(entries)
        portions = []
        at = 0
        for i in order:
            toks, start, blocks = entries[i]
            n = len(toks)
            if start + n > len(blocks) * blk:
                raise ValueError("step entry exceeds its cache blocks")
            table[i, : len(blocks)] = blocks
            tokens[at: at + n] = toks
            ctx[at: at + n] = np.arange(start + 1, start + n + 1)
            row_seq[at: at + n] = i
            rows[i] = np.arange(at, at + n)
            if n >= expand_min:
                portions.append((i, start, n))
            at += n

        def up(a):
            return torch.from_numpy(a).to(device)

        seg = None
        if slots is not None:
            seg = Segments.build([r[0] if len(r) else 0 for r in rows],
                                 [len(r) for r in rows], slots, device)

        return cls(tokens=up(tokens), ctx=up(ctx), row_seq=up(row_seq),
                   block_table=up(table),
                   n_folded=n_folded if portions else M, rows=rows,
                   portions=portions, segments=seg)

    def prompt_blocks(self, chunk: int) -> PromptBlocks:
        """Query blocks of the expanded portions, those that see most keys
        (in chunks of `chunk` positions) first: they would otherwise be
        the tail of the launch."""
        p = self._prompts.get(chunk)
        if p is not None:
            return p
        dev, Q = self.tokens.device, PromptBlocks.QBLK
        meta, blocks, keys = [], [], []
        at = self.n_folded
        for i, (s, start, n) in enumerate(self.portions):
            meta.append((s, at, start, n))
            at += n
            for b in range((n + Q - 1) // Q):
                blocks.append((i, b))
                first = start + b * Q
                keys.append(min(first + Q, start + n)
                            - first // chunk * chunk)
        order = np.argsort(-np.array(keys), kind="stable")
        p = PromptBlocks(
            torch.tensor(meta, dtype=torch.int32).to(dev),
            torch.from_numpy(np.array(blocks, np.int32)[order]).to(dev))
        self._prompts[chunk] = p
        return p

    def expansion(self, window: int) -> Expansion:
        """Key map of the expanded portions under a window: each
        portion's own tokens and the window - 1 cached before them."""
        e = self._expansions.get(window)
        if e is not None:
            return e
        dev = self.tokens.device
        seqs, poss, nq, nk = [], [], [0], [0]
        for s, start, n in self.portions:
            lo = max(0, start - (window - 1))
            poss.append(np.arange(lo, start + n, dtype=np.int32))
            seqs.append(np.full(start + n - lo, s, np.int32))
            nq.append(n)
            nk.append(start + n - lo)
        cu_q = torch.from_numpy(np.cumsum(nq).astype(np.int32))
        cu_k = torch.from_numpy(np.cumsum(nk).astype(np.int32))
        b_seq, b_qb = ops.varlen_block_map(cu_q)
        # workgroups with the most keys start first: they would otherwise
        # be the tail of the launch
        start = torch.tensor([s for _, s, _ in self.portions])
        last = start[b_seq.long()] + (b_qb + 1) * 128
        order = torch.argsort(last.clamp(max=window + 127),
                              descending=True, stable=True)
        b_seq, b_qb = b_seq[order], b_qb[order]
        # packed keys get the same rounding as rows: few product shapes
        T = row_bucket(int(cu_k[-1]))
        key_seq = np.zeros(T, np.int32)
        key_pos = np.zeros(T, np.int32)
        key_seq[: cu_k[-1]] = np.concatenate(seqs)
        key_pos[: cu_k[-1]] = np.concatenate(poss)
        e = Expansion(torch.from_numpy(key_seq).to(dev),
                      torch.from_numpy(key_pos).to(dev), cu_q.to(dev),
                      cu_k.to(dev), (b_seq.to(dev), b_qb.to(dev)))
        self._expansions[window] = e
        return e
