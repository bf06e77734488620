"""Host-side construction of a step's index tensors (numpy only, no device needed)."""
from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np

from zipage_amd.sight import first_seen

from .sequence import Portion, Sequence

HEADER_ROWS = 5   # query row, position, flat K/V slot, context length, token-log column


def query_slot_mapping(seq: Sequence, block_size: int, query_cache_len: int, is_prefill=False,
                       cu_len=0, seqlen_q=0) -> list[tuple[int, int, int]]:
    """(row of q, query row, ring slot) triples for the tokens that fall into the last
    `query_cache_len` positions of a page (zipage/engine/model_runner.py:319-350)."""
    BS, W = block_size, query_cache_len
    if seq.query_id == -1:
        return []
    if is_prefill:
        pages = -(-seqlen_q // BS)
        if pages == 0:
            return []
        tail = seqlen_q - (pages - 1) * BS
        if tail <= BS - W:
            return []
        first = pages * BS - W
        return [(cu_len + pos, seq.query_id, i) for i, pos in enumerate(range(first, seqlen_q))]
    if seq.last_block_num_tokens > BS - W:
        return [(cu_len, seq.query_id, seq.last_block_num_tokens - (BS - W) - 1)]
    return []


def packed_words(batch: int, table_width: int) -> int:
    return batch * (HEADER_ROWS + table_width + 3)


def pack_decode(seqs: list[Sequence], padded: int, block_size: int, query_cache_len: int,
                table_width: int, scratch_row: int) -> np.ndarray:
    """All int32 inputs of one decode step in one buffer: the header rows (each `padded` long),
    then the block tables (padded x table_width, -1 filled) and the query triples (padded x 3).

    For the live entries this is zipage/engine/model_runner.py:633-675: position = len - 1,
    slot = last page * BS + tokens in the last page - 1, context = (pages - 1) * BS + tokens in
    the last page.  Entries past len(seqs) are inert: scratch row, slot -1, context 0, triple
    row -1, so a padded batch can replay a graph captured for a larger one.
    """
    BS, W, TW = block_size, query_cache_len, table_width
    B = len(seqs)
    n = np.fromiter((s.num_tokens for s in seqs), np.int64, B)
    npg = np.fromiter((len(s.block_table) for s in seqs), np.int64, B)
    last = np.fromiter((s.block_table[-1] for s in seqs), np.int64, B)
    rows = np.fromiter((s.query_id for s in seqs), np.int64, B)
    done = np.fromiter((s.num_completion_tokens for s in seqs), np.int64, B)
    tail = n - ((n + BS - 1) // BS - 1) * BS
    out = np.empty(packed_words(padded, TW), dtype=np.int32)
    head = out[:HEADER_ROWS * padded].reshape(HEADER_ROWS, padded)
    head[0].fill(scratch_row)
    head[1].fill(0)
    head[2].fill(-1)
    head[3].fill(0)
    head[4].fill(0)
    head[0, :B], head[1, :B] = rows, n - 1
    head[2, :B] = last * BS + tail - 1
    head[3, :B] = (npg - 1) * BS + tail
    head[4, :B] = done
    tab = out[HEADER_ROWS * padded:HEADER_ROWS * padded + padded * TW].reshape(padded, TW)
    tab.fill(-1)
    for i, s in enumerate(seqs):
        tab[i, :len(s.block_table)] = s.block_table
    tri = out[HEADER_ROWS * padded + padded * TW:].reshape(padded, 3)
    tri.fill(-1)
    hit = tail > BS - W
    tri[:B, 0] = np.where(hit, np.arange(B), -1)
    tri[:B, 1] = rows
    tri[:B, 2] = np.where(hit, tail - (BS - W) - 1, -1)
    return out


def unpack_views(buf, padded: int, table_width: int):
    """Views of a packed buffer (numpy array or torch tensor): header, tables, triples."""
    h = HEADER_ROWS * padded
    t = h + padded * table_width
    return (buf[:h].reshape(HEADER_ROWS, padded), buf[h:t].reshape(padded, table_width),
            buf[t:t + 3 * padded].reshape(padded, 3))


def encode_compress_tables(seqs: list[Sequence]) -> list[list[int]]:
    """Block tables as the compression kernels read them: last page as -id-2, -1 padding
    (zipage/engine/model_runner.py:437-463)."""
    width = max(len(s.block_table) for s in seqs)
    return [s.block_table[:-1] + [-s.block_table[-1] - 2] + [-1] * (width - len(s.block_table))
            for s in seqs]


# ---------------------------------------------------------------- steps of portions
RUN_TILE = 128    # queries per entry of a run plan


@dataclass
class Runs:
    """The multi-token portions of a step as the run attention reads them, for one kind of sight."""
    tiles: np.ndarray             # (T, 4): first query row, queries, first key row, rel. position
    key_slots: np.ndarray | None  # cache rows to gather as keys; None: the step's own tokens


@dataclass
class PortionPlan:
    ids: np.ndarray               # token ids; 0 where the id is still on the device
    rows: np.ndarray              # query row whose last sampled token is the id, or -1
    positions: np.ndarray
    slots: np.ndarray
    context_lens: np.ndarray      # of the tokens attended one by one; they come first
    table_rows: np.ndarray
    tables: np.ndarray            # (sequences, width), -1 where nothing is held
    first_row: list[int]          # token row where each portion starts, in the order given
    segments: np.ndarray          # (4, portions): token row, tokens, query row, position of the first
    short: int                    # so many of them, which come first, are attended one by one
    runs: dict = field(default_factory=dict)


def plan_runs(portions: list[Portion], block_size: int, sight) -> Runs:
    """Key rows and query tiles of `portions`, whose tokens follow one another in the query rows.  A
    run's keys start with the first its first token sees."""
    tiles, slots, q, k = [], [], 0, 0
    own = True
    for p in portions:
        k_first = first_seen(p.start, sight)
        own &= k_first == p.start
        for off in range(0, p.count, RUN_TILE):
            tiles.append((q + off, min(RUN_TILE, p.count - off), k, p.start - k_first + off))
        t = np.arange(k_first, p.start + p.count)
        table = np.asarray(p.seq.block_table, dtype=np.int64)
        slots.append(table[t // block_size] * block_size + t % block_size)
        q += p.count
        k += len(t)
    return Runs(np.asarray(tiles, dtype=np.int32),
                None if own else np.concatenate(slots).astype(np.int32))


def plan_portions(portions: list[Portion], block_size: int, sights, run_min: int | None) -> PortionPlan:
    """All inputs of a step that holds portions of any length.  Portions shorter than `run_min`
    (None: all) are attended token by token and come first."""
    short = [i for i, p in enumerate(portions) if run_min is None or p.count < run_min]
    long = [i for i, p in enumerate(portions) if not (run_min is None or p.count < run_min)]
    first_row = [0] * len(portions)
    ids, rows, pos, slots, ctx, trows = [], [], [], [], [], []
    width = max(len(p.seq.block_table) for p in portions)
    tables = np.full((len(portions), width), -1, dtype=np.int32)
    n = 0
    for i in short + long:
        p = portions[i]
        first_row[i] = n
        n += p.count
        tables[i, :len(p.seq.block_table)] = p.seq.block_table
        known = p.seq.token_ids[p.start:p.start + p.count]
        missing = p.count - len(known)      # a sampled token that never came to the host
        assert missing == 0 or p.count == 1
        ids.extend(known + [0] * missing)
        rows.extend([-1] * len(known) + [p.seq.query_id] * missing)
        t = np.arange(p.start, p.start + p.count)
        pos.append(t)
        slots.append(tables[i][t // block_size].astype(np.int64) * block_size + t % block_size)
    for i in short:
        p = portions[i]
        ctx.append(np.arange(p.start + 1, p.start + p.count + 1))
        trows.append(np.full(p.count, i))
    cat = lambda a: np.concatenate(a).astype(np.int32) if a else np.zeros(0, np.int32)
    segments = np.array([[first_row[i], portions[i].count, portions[i].seq.query_id, portions[i].start]
                         for i in short + long], np.int32).T
    plan = PortionPlan(np.asarray(ids, np.int32), np.asarray(rows, np.int32), cat(pos), cat(slots),
                       cat(ctx), cat(trows), tables, first_row, segments, len(short))
    if long:
        for w in sights:
            plan.runs[w] = plan_runs([portions[i] for i in long], block_size, w)
    return plan
