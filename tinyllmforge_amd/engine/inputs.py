"""Integer inputs of the hot path, built on the host from the scheduler's sequences.

Pure functions (numpy in, numpy out) so that slot mapping and block indexing can be checked
bit-exactly without a GPU.  They restate the reference's list-building loops
(tinyvllm/engine/model_runner.py:155-159, 164-205, 210-228) with vectorised index arithmetic.
"""
from __future__ import annotations

import numpy as np


def block_tables_array(seqs, pad: int = -1, width: int | None = None) -> np.ndarray:
    """int32 ``[len(seqs), width]``; rows padded with ``pad`` (reference pads with -1 to the batch max)."""
    w = max(len(s.block_table) for s in seqs)
    if width is not None:
        assert width >= w
        w = width
    out = np.full((len(seqs), w), pad, dtype=np.int32)
    for i, s in enumerate(seqs):
        out[i, :len(s.block_table)] = s.block_table
    return out


def prefill_inputs(seqs, block_size: int) -> dict:
    """Inputs of one prefill step (model_runner.py:164-205).

    input_ids / positions cover the uncached tail of every prompt; the slot of token ``t`` of a
    sequence is ``block_table[t // block_size] * block_size + t % block_size`` for every token
    from the first uncached *block* on; ``block_tables`` is only built when some sequence has
    a cached prefix (then the attention reads K/V of every sequence from the paged cache).
    """
    ids, pos, slots = [], [], []
    cu_q, cu_k = [0], [0]
    max_q = max_k = 0
    for s in seqs:
        n, c = len(s), s.num_cached_tokens
        ids.append(np.asarray(s.token_ids[c:n], dtype=np.int64))
        pos.append(np.arange(c, n, dtype=np.int64))
        cu_q.append(cu_q[-1] + (n - c))
        cu_k.append(cu_k[-1] + n)
        max_q, max_k = max(max_q, n - c), max(max_k, n)
        if not s.block_table:
            continue                                # warm-up sequences have no blocks
        t = np.arange(s.num_cached_blocks * block_size, n, dtype=np.int64)
        table = np.asarray(s.block_table, dtype=np.int64)
        slots.append(table[t // block_size] * block_size + t % block_size)
    cat = lambda xs, dt: np.concatenate(xs).astype(dt) if xs else np.zeros(0, dtype=dt)
    out = dict(
        input_ids=cat(ids, np.int64), positions=cat(pos, np.int64), slot_mapping=cat(slots, np.int32),
        cu_seqlens_q=np.asarray(cu_q, dtype=np.int32), cu_seqlens_k=np.asarray(cu_k, dtype=np.int32),
        max_seqlen_q=max_q, max_seqlen_k=max_k, block_tables=None,
    )
    if cu_k[-1] > cu_q[-1]:
        out["block_tables"] = block_tables_array(seqs)
    return out


def decode_inputs(seqs, block_size: int, position_quirk: bool = True) -> dict:
    """Inputs of one decode step (model_runner.py:210-228).

    The fed token is the last one (index ``len - 1``); its K/V go to slot
    ``block_table[-1] * block_size + last_block_num_tokens - 1``; ``context_lens = len``.
    The reference feeds ``positions = len(seq)`` (one past the token's index, model_runner.py:219);
    ``position_quirk=False`` gives ``len - 1`` instead.
    """
    n = np.asarray([len(s) for s in seqs], dtype=np.int64)
    last_blk = np.asarray([s.block_table[-1] for s in seqs], dtype=np.int64)
    nblocks = -(-n // block_size)
    last_cnt = n - (nblocks - 1) * block_size
    return dict(
        input_ids=np.asarray([s.last_token for s in seqs], dtype=np.int64),
        positions=(n if position_quirk else n - 1).astype(np.int64),
        slot_mapping=(last_blk * block_size + last_cnt - 1).astype(np.int32),
        context_lens=n.astype(np.int32),
        block_tables=block_tables_array(seqs),
    )


CHUNK = 16    # tokens per chunk of the recurrent layers' prompt kernels


def portion_kind(tokens: int, long_portion: int | None) -> int:
    """Order of a step's sequences: single tokens, short portions, long portions (all portions without ``long_portion``)."""
    return 0 if tokens == 1 else 1 if long_portion is not None and tokens < long_portion else 2


def portion_inputs(seqs, block_size: int, long_portion: int | None = None, windows=()) -> dict:
    """Inputs of a step in which sequence ``s`` brings its tokens ``num_computed .. num_computed + num_scheduled - 1``,
    sequences with one token first (no counterpart in the reference).  Besides the usual arrays: per sequence the tokens
    before the step and the state slot, per row its sequence, and the portions of more than one token cut into chunks of
    at most ``CHUNK`` that do not cross a sequence (rows counted from the first portion's first row).  A design with
    ``long_portion`` gets its portions of at least that many tokens last and, per attention window, the dense rows their
    keys take (from the first key the portion's first token sees to its last token)."""
    n = np.asarray([s.num_scheduled for s in seqs], dtype=np.int64)
    single = int((n == 1).sum())
    kinds = [portion_kind(int(x), long_portion) for x in n]
    assert kinds == sorted(kinds)
    short = kinds.count(1)
    start = np.asarray([s.num_computed for s in seqs], dtype=np.int64)
    ids = np.concatenate([np.asarray(s.token_ids[s.num_computed:s.num_computed + s.num_scheduled], dtype=np.int64) for s in seqs])
    cu = np.concatenate([[0], np.cumsum(n)])
    row_seq = np.repeat(np.arange(len(seqs)), n)
    pos = np.arange(cu[-1]) - cu[row_seq] + start[row_seq]
    tables = block_tables_array(seqs)
    slots = tables[row_seq, pos // block_size].astype(np.int64) * block_size + pos % block_size
    far = slice(single + short, None)
    keys = np.stack([np.minimum(start[far], w - 1) + n[far] for w in windows]) if windows else np.zeros((0, len(n[far])), np.int64)
    kv_offsets = np.concatenate([np.zeros((len(keys), 1), np.int64), np.cumsum(keys, axis=1)], axis=1)
    chunks = -(-n[single:] // CHUNK)
    cu_chunks = np.concatenate([[0], np.cumsum(chunks)])
    chunk_seq = np.repeat(np.arange(len(chunks)), chunks)
    within = (np.arange(cu_chunks[-1]) - cu_chunks[chunk_seq]) * CHUNK
    return dict(
        input_ids=ids, positions=pos.astype(np.int64), slot_mapping=slots.astype(np.int32),
        cu_seqlens_q=cu.astype(np.int32), block_tables=tables, seq_starts=start.astype(np.int32),
        state_slots=np.asarray([s.state_slot for s in seqs], dtype=np.int32), row_seq=row_seq.astype(np.int32),
        chunk_rows=(cu[single:-1][chunk_seq] - single + within).astype(np.int32),
        chunk_lens=np.minimum(CHUNK, n[single:][chunk_seq] - within).astype(np.int32),
        cu_chunks=cu_chunks.astype(np.int32), num_single=single, max_portion=int(n.max()),
        num_short=short, num_short_rows=int(cu[single + short]), max_short=int(n[single:single + short].max(initial=0)),
        kv_offsets=kv_offsets.astype(np.int32), kv_rows=tuple(kv_offsets[:, -1].tolist()),
        max_kv_rows=tuple(keys.max(axis=1, initial=0).tolist()),
    )
