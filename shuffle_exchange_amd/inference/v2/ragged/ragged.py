"""Ragged-batch state for the FastGen-style engine: block allocator, blocked KV cache, sequence
descriptors, state manager and the per-forward ragged batch metadata.

Parity: reference inference/v2/ragged/ -- ``BlockedAllocator`` (blocked_allocator.py:11),
``BlockedKVCache`` (kv_cache.py:40), ``DSSequenceDescriptor`` (sequence_descriptor.py:59),
``DSStateManager`` (ragged_manager.py:19), ``RaggedBatchWrapper`` (ragged_wrapper.py:31).

MI355X-first sizing: the KV cache is one allocation per model ([layers, blocks, 2, nkv, bs, D]),
sized from a fraction of the free HBM (288 GB per GPU => hundreds of thousands of tokens of
Llama-3-8B KV at bf16); the batch metadata is built in pinned host buffers and crosses to the GPU
in one copy per dtype.
"""
import math
from dataclasses import dataclass, field
from typing import List

import torch


class BlockedAllocator:
    """Free-list allocator of KV block ids (host side, O(1) alloc/free)."""

    def __init__(self, num_blocks):
        if num_blocks < 1:
            raise ValueError("num_blocks must be positive")
        self._num_blocks = num_blocks
        self._free = list(range(num_blocks - 1, -1, -1))
        self._used = [False] * num_blocks

    @property
    def free_blocks(self):
        return len(self._free)

    @property
    def num_blocks(self):
        return self._num_blocks

    def allocate(self, num_blocks):
        if num_blocks > len(self._free):
            raise ValueError(f"not enough free KV blocks ({num_blocks} > {len(self._free)})")
        out = [self._free.pop() for _ in range(num_blocks)]
        for b in out:
            self._used[b] = True
        return torch.tensor(out, dtype=torch.int32)

    def free(self, blocks):
        for b in (blocks.tolist() if torch.is_tensor(blocks) else list(blocks)):
            if not (0 <= b < self._num_blocks) or not self._used[b]:
                raise ValueError(f"invalid free of block {b}")
            self._used[b] = False
            self._free.append(b)


class BlockedKVCache:
    """One block id addresses the same block in every layer. Uniform models: one allocation [layers,
    blocks, 2, nkv, bs, D]. ``layer_shapes`` (one (kv heads, k row, v row) per layer): an allocation
    per layer whose blocks hold that layer's k [nkv, bs, k row] then v [nkv, bs, v row]; a row length of 0
    (no separate values, or a layer that keeps no keys at all) takes no memory.

    ``states`` (RecurrentStates or None): the per-sequence state of recurrent layers."""

    KEYLESS_BLOCKS = 65536  # block count when no layer keeps keys: blocks then only count tokens

    def __init__(self, num_layers, num_blocks, block_size, n_kv_heads=0, head_dim=0, dtype=torch.bfloat16, device=None,
                 layer_shapes=None):
        self.num_layers, self.num_blocks, self.block_size = num_layers, num_blocks, block_size
        self.n_kv_heads, self.head_dim = n_kv_heads, head_dim
        self.layer_shapes = layer_shapes
        if layer_shapes is None:
            self.cache = torch.zeros(num_layers, num_blocks, 2, n_kv_heads, block_size, head_dim, dtype=dtype,
                                     device=device)
        else:
            assert len(layer_shapes) == num_layers, "one cache shape per layer"
            self.cache = None
            self._kv = []
            for nkv, dk, dv in layer_shapes:
                buf = torch.zeros(num_blocks, nkv * block_size * (dk + dv), dtype=dtype, device=device)
                n = nkv * block_size * dk
                self._kv.append((buf[:, :n].unflatten(1, (nkv, block_size, dk)),
                                 buf[:, n:].unflatten(1, (nkv, block_size, dv))))
        self.allocator = BlockedAllocator(num_blocks)
        self.states = None

    @staticmethod
    def blocks_for_budget(budget_bytes, num_layers, block_size, n_kv_heads=0, head_dim=0, dtype=torch.bfloat16,
                          layer_shapes=None):
        rows = (num_layers * 2 * n_kv_heads * head_dim if layer_shapes is None
                else sum(nkv * (dk + dv) for nkv, dk, dv in layer_shapes))
        per_block = rows * block_size * torch.tensor([], dtype=dtype).element_size()
        if per_block == 0:
            return BlockedKVCache.KEYLESS_BLOCKS
        return max(1, int(budget_bytes // per_block))

    def layer(self, i):
        return self.cache[i]

    def layer_kv(self, i):
        """(k, v) views [blocks, nkv, bs, row] of layer ``i``."""
        if self.layer_shapes is None:
            return self.cache[i][:, 0], self.cache[i][:, 1]
        return self._kv[i]

    def layer_state(self, i):
        """fp32 state [slots, *shape] of recurrent layer ``i``."""
        return self.states.layers[i]

    def reserve(self, n):
        return self.allocator.allocate(n)

    def free(self, blocks):
        self.allocator.free(blocks)

    @property
    def free_blocks(self):
        return self.allocator.free_blocks


class RecurrentStates:
    """State slots of recurrent layers: a sequence owns one slot, the same in every layer, from its first
    token until it is flushed. ``shapes``: per layer the state's shape, or None for a layer without one.
    States are fp32 and never cleared: kernels start from zero when a sequence has no earlier tokens."""

    def __init__(self, shapes, num_slots, device=None):
        self.num_slots = num_slots
        self.layers = [None if s is None else torch.empty(num_slots, *s, dtype=torch.float32, device=device) for s in shapes]
        self.allocator = BlockedAllocator(num_slots)

    @staticmethod
    def bytes_per_slot(shapes):
        return 4 * sum(math.prod(s) for s in shapes if s is not None)

    @property
    def free_slots(self):
        return self.allocator.free_blocks

    def reserve(self):
        return int(self.allocator.allocate(1)[0])

    def free(self, slot):
        self.allocator.free([slot])


@dataclass
class DSSequenceDescriptor:
    uid: int
    max_blocks: int
    state_slot: int = -1
    seen_tokens: int = 0
    in_flight_tokens: int = 0
    blocks: List[int] = field(default_factory=list)

    @property
    def cur_allocated_blocks(self):
        return len(self.blocks)

    def blocks_needed(self, new_tokens, block_size):
        total = self.seen_tokens + new_tokens
        return max(0, (total + block_size - 1) // block_size - len(self.blocks))

    def pre_forward(self, n):
        self.in_flight_tokens = n

    def post_forward(self):
        self.seen_tokens += self.in_flight_tokens
        self.in_flight_tokens = 0


class DSStateManager:
    def __init__(self, kv_cache: BlockedKVCache, max_tracked_sequences=2048, max_blocks_per_sequence=None):
        self.kv = kv_cache
        self.max_tracked = max_tracked_sequences
        self.max_blocks_per_seq = max_blocks_per_sequence or kv_cache.num_blocks
        self.seqs = {}

    @property
    def n_tracked_sequences(self):
        return len(self.seqs)

    @property
    def free_blocks(self):
        return self.kv.free_blocks

    def get_sequence(self, uid):
        return self.seqs.get(uid)

    def get_or_create_sequence(self, uid):
        s = self.seqs.get(uid)
        if s is None:
            if len(self.seqs) >= self.max_tracked:
                raise RuntimeError(f"tracking limit of {self.max_tracked} sequences reached")
            s = DSSequenceDescriptor(uid, self.max_blocks_per_seq)
            if self.kv.states is not None:
                s.state_slot = self.kv.states.reserve()
            self.seqs[uid] = s
        return s

    def allocate_blocks(self, seq, n_new_tokens):
        need = seq.blocks_needed(n_new_tokens, self.kv.block_size)
        if need:
            if len(seq.blocks) + need > seq.max_blocks:
                raise RuntimeError(f"sequence {seq.uid} exceeds {seq.max_blocks} KV blocks")
            seq.blocks.extend(self.kv.reserve(need).tolist())

    def flush_sequence(self, uid):
        s = self.seqs.pop(uid, None)
        if s is not None and s.blocks:
            self.kv.free(s.blocks)
        if s is not None and s.state_slot >= 0:
            self.kv.states.free(s.state_slot)


class RaggedBatch:
    """Device metadata of one forward over a ragged set of sequences (all int tensors on device).

    input_ids [T]; positions [T] (absolute); slots [T] (cache slot of every new token);
    q_start / q_len / kv_len / state_slots [S] int32; block_table [S, max_blocks] int32; last_idx int64: the rows whose
    logits are returned -- every sequence's last new token [S], or with ``want`` (per sequence, places
    among its new tokens) those places in order. Host copies of the small per-sequence ints are kept
    for scheduling decisions.
    """

    def __init__(self, seqs, tokens, block_size, device, want=None):
        S = len(seqs)
        lens = [int(t.numel()) for t in tokens]
        T = sum(lens)
        if want is None:
            want = [(n - 1,) for n in lens]
        n_want = sum(len(x) for x in want)
        maxb = max(1, max(len(s.blocks) for s in seqs))
        i64 = torch.empty(3 * T + n_want, dtype=torch.int64, pin_memory=torch.cuda.is_available() and device.type == "cuda")
        i32 = torch.zeros(4 * S + S * maxb, dtype=torch.int32,
                          pin_memory=torch.cuda.is_available() and device.type == "cuda")
        ids, pos, slots, last = i64[:T], i64[T:2 * T], i64[2 * T:3 * T], i64[3 * T:]
        qs, ql, kl, ss = i32[:S], i32[S:2 * S], i32[2 * S:3 * S], i32[3 * S:4 * S]
        bt = i32[4 * S:].view(S, maxb)
        t, nw = 0, 0
        self.host_q_len, self.host_kv_len, self.host_seen = [], [], []
        for i, (s, tk) in enumerate(zip(seqs, tokens)):
            n = lens[i]
            ids[t:t + n] = tk.to(torch.int64)
            p = torch.arange(s.seen_tokens, s.seen_tokens + n, dtype=torch.int64)
            pos[t:t + n] = p
            blk = torch.tensor(s.blocks, dtype=torch.int64)
            slots[t:t + n] = blk[p // block_size] * block_size + p % block_size
            qs[i], ql[i], kl[i], ss[i] = t, n, s.seen_tokens + n, s.state_slot
            bt[i, :len(s.blocks)] = torch.tensor(s.blocks, dtype=torch.int32)
            for j in want[i]:
                last[nw] = t + int(j)
                nw += 1
            self.host_q_len.append(n)
            self.host_kv_len.append(s.seen_tokens + n)
            self.host_seen.append(s.seen_tokens)
            t += n
        d64 = i64.to(device, non_blocking=True)
        d32 = i32.to(device, non_blocking=True)
        self.input_ids, self.positions, self.slots, self.last_idx = d64[:T], d64[T:2 * T], d64[2 * T:3 * T], d64[3 * T:]
        self.q_start, self.q_len, self.kv_len = d32[:S], d32[S:2 * S], d32[2 * S:3 * S]
        self.state_slots = d32[3 * S:4 * S]
        self.block_table = d32[4 * S:].view(S, maxb)
        self.num_tokens, self.num_seqs = T, S
        self.max_kv_len = max(self.host_kv_len) if S else 0
        self.host_q_start = [sum(lens[:i]) for i in range(S)]
        self.host_blocks = [s.blocks for s in seqs]
        self.block_size = block_size
        self._tables = {}

    def chunks(self, size, min_len=1):
        """int32 [n, 3] on the device: (sequence, first row, rows) of every chunk of up to ``size`` new
        tokens, sequence by sequence, of the sequences with at least ``min_len`` new tokens."""
        key = ("chunks", size, min_len)
        if key not in self._tables:
            rows = [(i, q + a, min(size, n - a)) for i, (q, n) in enumerate(zip(self.host_q_start, self.host_q_len))
                    if n >= min_len for a in range(0, n, size)]
            self._tables[key] = self._upload(rows, 3)
        return self._tables[key]

    def key_rows(self, window, min_len=1):
        """Keys in reach of the new tokens (window None: all earlier ones) of the sequences with at least
        ``min_len`` new tokens: (cache slots int64 [N], int32 [S, 2] (row of the list, position) of each
        sequence's first listed key; (0, 0) for the others)."""
        key = ("keys", window, min_len)
        if key not in self._tables:
            first, slots, at = [], [], 0
            for n, kl, seen, blocks in zip(self.host_q_len, self.host_kv_len, self.host_seen, self.host_blocks):
                if n < min_len:
                    first.append((0, 0))
                    continue
                lo = 0 if window is None else max(0, seen - window + 1)
                first.append((at, lo))
                p = torch.arange(lo, kl, dtype=torch.int64)
                slots.append(torch.tensor(blocks, dtype=torch.int64)[p // self.block_size] * self.block_size
                             + p % self.block_size)
                at += kl - lo
            slots = torch.cat(slots) if slots else torch.zeros(0, dtype=torch.int64)
            if self.slots.is_cuda:
                slots = slots.pin_memory().to(self.slots.device, non_blocking=True)
            self._tables[key] = (slots, self._upload(first, 2))
        return self._tables[key]

    def token_rows(self, below=None):
        """int32 [n, 2] on the device: (sequence, row) of every new token of the sequences with fewer than
        ``below`` new tokens (None: all)."""
        key = ("tokens", below)
        if key not in self._tables:
            rows = [(i, q + j) for i, (q, n) in enumerate(zip(self.host_q_start, self.host_q_len))
                    if below is None or n < below for j in range(n)]
            self._tables[key] = self._upload(rows, 2)
        return self._tables[key]

    def _upload(self, rows, n):
        t = torch.tensor(rows, dtype=torch.int32).reshape(-1, n)
        return t.pin_memory().to(self.slots.device, non_blocking=True) if self.slots.is_cuda else t
