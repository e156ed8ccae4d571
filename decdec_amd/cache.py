"""What a sequence leaves behind for its next tokens, layer by layer, and the manager that owns it.

A decoder creates one entry per layer run (layers that share weights do not share an entry) and wraps them in a
``SequenceState``.  Caches are indexed by position: a row beyond the sequence's length is never read, and writing a
position again replaces it.  Recurrent entries are updated in place, once per token; a call whose first position is 0
starts from an empty state whatever the memory holds, so giving a sequence back costs nothing."""
from __future__ import annotations

import torch
import torch.nn as nn


class KVCache(nn.Module):
    """Keys and values [batch, heads, positions, head_dim]."""

    def __init__(self, max_batch_size: int, max_seq_length: int, n_heads: int, head_dim: int, dtype, device):
        super().__init__()
        shape = (max_batch_size, n_heads, max_seq_length, head_dim)
        self.register_buffer("k_cache", torch.zeros(shape, dtype=dtype, device=device), persistent=False)
        self.register_buffer("v_cache", torch.zeros(shape, dtype=dtype, device=device), persistent=False)

    def update(self, input_pos: torch.Tensor, k: torch.Tensor, v: torch.Tensor):
        self.k_cache.index_copy_(2, input_pos, k)
        self.v_cache.index_copy_(2, input_pos, v)
        return self.k_cache, self.v_cache

    def recurrent(self):
        return []


class GroupedCache:
    """Keys by head [heads, positions, dim] and values transposed [heads * vdim, positions], as the attention products read
    them.  The positions come in multiples of 64 and are finite from the start (tiles read past the last one)."""

    def __init__(self, max_seq_length: int, kv_heads: int, dim: int, vdim: int, dtype, device):
        self.positions = (max_seq_length + 63) // 64 * 64
        self.keys = torch.zeros(kv_heads, self.positions, dim, dtype=dtype, device=device)
        self.values = torch.zeros(kv_heads * vdim, self.positions, dtype=dtype, device=device)

    def recurrent(self):
        return []


class JoinedState:
    """The entries of mixers that run side by side in one layer."""

    def __init__(self, parts):
        self.parts = list(parts)

    def recurrent(self):
        return [t for p in self.parts for t in p.recurrent()]


class LatentCache:
    """One row per position: a latent all heads' keys and values are linear in, and a rotated key part they share.
    The rows come in multiples of 64 and are finite from the start (tiles read past the last position)."""

    def __init__(self, max_seq_length: int, rank: int, rot: int, dtype, device):
        self.rows = torch.zeros((max_seq_length + 63) // 64 * 64, rank + rot, dtype=dtype, device=device)
        self.rank = rank

    def recurrent(self):
        return []


class RecurrentState:
    """A dim x vdim matrix per head in fp32 and, where the layer convolves its inputs, the last `taps` of them."""

    def __init__(self, heads: int, dim: int, vdim: int, device, taps: int = 0, channels: int = 0, dtype=None):
        self.state = torch.zeros(heads, dim, vdim, dtype=torch.float32, device=device)
        self.ring = torch.zeros(taps, channels, dtype=dtype, device=device) if taps else None

    def recurrent(self):
        return [t for t in (self.state, self.ring) if t is not None]


class SequenceState:
    """The entries of one sequence, in the order of the layer runs, and how many tokens they hold."""

    def __init__(self, entries, max_tokens: int):
        self.entries, self.max_tokens, self.length = list(entries), max_tokens, 0

    def release(self) -> None:
        """The sequence is finished: its memory is free for the next one."""
        self.length = 0

    def advance(self, start: int, count: int) -> None:
        if start != self.length:
            raise ValueError(f"tokens start at position {start}, the state holds {self.length}")
        if start + count > self.max_tokens:
            raise ValueError(f"{start + count} positions do not fit a cache of {self.max_tokens}")
        self.length = start + count

    def snapshot(self):
        """Copies of what a repeated step would change (caches are rewritten with the same values, states are not)."""
        return [t.clone() for e in self.entries for t in e.recurrent()]

    def restore(self, saved) -> None:
        for t, s in zip((t for e in self.entries for t in e.recurrent()), saved):
            t.copy_(s)
