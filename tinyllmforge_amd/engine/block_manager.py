"""KV-cache block allocator with hash-chained prefix caching
(reference: tinyvllm/engine/block_manager.py:8-139).

The order in which block ids are handed out is part of the contract ("bit-exact block
indexing"): the free list is FIFO (take from the left, return to the right), full blocks are
keyed by xxh64 over the previous block's hash and the block's token ids, and hash entries
outlive deallocation so that a freed block can be revived by a later prefix hit.
"""
from __future__ import annotations

from collections import deque

import numpy as np
import xxhash

from .sequence import Sequence


class Block:
    __slots__ = ("block_id", "ref_count", "hash", "token_ids")

    def __init__(self, block_id: int):
        self.block_id = block_id
        self.ref_count = 0
        self.hash = -1
        self.token_ids: list[int] = []

    def update(self, h: int, token_ids: list[int]):
        self.hash = h
        self.token_ids = token_ids

    def reset(self):
        self.ref_count = 1
        self.hash = -1
        self.token_ids = []


class BlockManager:
    def __init__(self, num_blocks: int, block_size: int):
        assert num_blocks > 0
        self.block_size = block_size
        self.blocks = [Block(i) for i in range(num_blocks)]
        self.hash_to_block_id: dict[int, int] = {}
        self.free_block_ids: deque[int] = deque(range(num_blocks))
        self.used_block_ids: set[int] = set()
        # full blocks whose last tokens are not on the host yet (a decode step running ahead of the token
        # read-back): (sequence, block index, block id, id of the block before it), sealed by seal_known()
        self.unsealed: deque[tuple[Sequence, int, int, int]] = deque()

    @staticmethod
    def compute_hash(token_ids: list[int], prefix: int = -1) -> int:
        """xxh64(seed 0) of [prefix as 8 LE bytes if given] + token ids as int64 LE (block_manager.py:36-42)."""
        h = xxhash.xxh64()
        if prefix != -1:
            h.update(prefix.to_bytes(8, "little"))
        h.update(np.asarray(token_ids, dtype=np.int64).tobytes())
        return h.intdigest()

    # -- free-list plumbing
    def _take(self, block_id: int) -> Block:
        blk = self.blocks[block_id]
        assert blk.ref_count == 0
        blk.reset()
        self.free_block_ids.remove(block_id)
        self.used_block_ids.add(block_id)
        return blk

    def _release(self, block_id: int):
        assert self.blocks[block_id].ref_count == 0
        self.used_block_ids.remove(block_id)
        self.free_block_ids.append(block_id)

    # -- prefill side
    def can_allocate(self, seq: Sequence) -> bool:
        return len(self.free_block_ids) >= seq.num_blocks

    def allocate(self, seq: Sequence):
        assert not seq.block_table
        chain = -1
        missed = False
        for i in range(seq.num_blocks):
            tokens = seq.block(i)
            full = len(tokens) == self.block_size
            chain = self.compute_hash(tokens, chain) if full else -1
            hit = self.hash_to_block_id.get(chain, -1)
            if hit == -1 or self.blocks[hit].token_ids != tokens:
                missed = True                      # once one block misses, every later block is fresh
            if missed:
                hit = self.free_block_ids[0]
                blk = self._take(hit)
            else:
                seq.num_cached_tokens += self.block_size
                if hit in self.used_block_ids:
                    blk = self.blocks[hit]
                    blk.ref_count += 1
                else:
                    blk = self._take(hit)          # revive a freed block whose content is still there
            if chain != -1:
                blk.update(chain, tokens)
                self.hash_to_block_id[chain] = hit
            seq.block_table.append(hit)
        # Deviation from the reference: when every block of the prompt is a cache hit the
        # reference prefills zero tokens and then samples from another sequence's row
        # (model_runner.py:175-181, embed_head.py:61).  Recompute the last block instead.
        if seq.num_cached_tokens >= len(seq):
            seq.num_cached_tokens -= self.block_size

    def deallocate(self, seq: Sequence):
        for block_id in reversed(seq.block_table):
            blk = self.blocks[block_id]
            blk.ref_count -= 1
            if blk.ref_count == 0:
                self._release(block_id)
        seq.num_cached_tokens = 0
        seq.block_table.clear()

    # -- without prefix caching (designs whose recurrent state a block does not hold): a sequence owns just the blocks
    #    its tokens need, whatever step they come in
    def can_grow(self, seq: Sequence) -> bool:
        return len(self.free_block_ids) >= seq.num_blocks - len(seq.block_table)

    def grow(self, seq: Sequence):
        while len(seq.block_table) < seq.num_blocks:
            block_id = self.free_block_ids[0]
            self._take(block_id)
            seq.block_table.append(block_id)

    # -- decode side
    def can_append(self, seq: Sequence) -> bool:
        return len(self.free_block_ids) >= (len(seq) % self.block_size == 1)

    def may_append(self, seq: Sequence):
        table = seq.block_table
        last = self.blocks[table[-1]]
        r = len(seq) % self.block_size
        if r == 1:                                 # the token to be written opens a new block
            assert last.hash != -1
            new_id = self.free_block_ids[0]
            self._take(new_id)
            table.append(new_id)
        elif r == 0:                               # the last block just became full: seal it
            assert last.hash == -1
            if seq.num_unknown:                    # ... once its tokens are known (seal_known)
                last.hash = self.PENDING
                self.unsealed.append((seq, seq.num_blocks - 1, last.block_id, table[-2] if len(table) > 1 else -1))
                return
            tokens = seq.block(seq.num_blocks - 1)
            prefix = self.blocks[table[-2]].hash if len(table) > 1 else -1
            h = self.compute_hash(tokens, prefix)
            last.update(h, tokens)
            self.hash_to_block_id[h] = last.block_id
        else:
            assert last.hash == -1

    PENDING = -2     # hash of a full block that waits for its tokens: neither free-to-seal (-1) nor sealed

    def seal_known(self):
        """Seal, oldest first, the full blocks whose tokens have all arrived.  A block that was freed and
        handed out again in between (its hash is no longer PENDING) is left alone: sealed in time it would
        have lost its hash to the same reset."""
        while self.unsealed:
            seq, index, block_id, before = self.unsealed[0]
            if (index + 1) * self.block_size > seq.num_known_tokens:
                return
            self.unsealed.popleft()
            blk = self.blocks[block_id]
            if blk.hash != self.PENDING:
                continue
            tokens = seq.block(index)
            prefix = self.blocks[before].hash if before != -1 else -1
            assert prefix != self.PENDING
            h = self.compute_hash(tokens, prefix)
            blk.update(h, tokens)
            self.hash_to_block_id[h] = block_id
