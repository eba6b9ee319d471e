"""Blocked (paged) KV cache shared by the v1 kernel-injected engine and the v2 ragged engine
(reference `inference/v2/ragged/{kv_cache.py:40, blocked_allocator.py:11}` and the v1 in-workspace cache of
`csrc/transformer/inference/csrc/pt_binding.cpp:434-557`).

Per layer the cache is two tensors [num_blocks, kv_heads, block_size, head_dim] (head-major inside a block, so the
decode kernel reads one head's keys contiguously). Sequences own lists of block ids; the allocator is a simple
host-side free list (block ids are plain ints, the per-sequence block table is mirrored to a device int32 tensor).
Sized from free HBM: with 288 GB per MI355X even a 70B model leaves >100 GB of cache.
"""
import torch


class BlockedAllocator:

    def __init__(self, num_blocks):
        self.num_blocks = num_blocks
        self._free = list(range(num_blocks - 1, -1, -1))

    @property
    def free_blocks(self):
        return len(self._free)

    def allocate(self, n):
        if n > len(self._free):
            raise ValueError(f"KV cache exhausted: need {n} blocks, {len(self._free)} free")
        out = [self._free.pop() for _ in range(n)]
        return out

    def free(self, blocks):
        for b in blocks:
            self._free.append(int(b))


class BlockedKVCache:

    def __init__(self, num_layers, num_blocks, kv_heads, block_size, head_dim, dtype, device):
        self.num_layers = num_layers
        self.num_blocks = num_blocks
        self.kv_heads = kv_heads
        self.block_size = block_size
        self.head_dim = head_dim
        self.dtype = dtype
        self.device = device
        shape = (num_blocks, kv_heads, block_size, head_dim)
        self.k = [torch.zeros(shape, dtype=dtype, device=device) for _ in range(num_layers)]
        self.v = [torch.zeros(shape, dtype=dtype, device=device) for _ in range(num_layers)]
        self.allocator = BlockedAllocator(num_blocks)
        self.state, self.num_slots = [None] * num_layers, 0

    @classmethod
    def from_geometry(cls, geometry, num_blocks, block_size, dtype, device, state_geometry=None, num_slots=0):
        """A cache whose layers may differ. `geometry`: per layer (kv_heads, key width, value width) or None (no keys
        and values). `state_geometry`: per layer {name: (shape, dtype)} of a sequence's carried state, or None; every
        such layer gets `num_slots` slots of it. A slot is not cleared between owners: the kernels take a portion that
        starts at position 0 to start from zero state."""
        self = cls.__new__(cls)
        kv = [g for g in geometry if g is not None]
        self.num_layers, self.num_blocks, self.block_size = len(geometry), num_blocks, block_size
        self.kv_heads, self.head_dim = (kv[0][0], kv[0][1]) if kv else (0, 0)
        self.dtype, self.device = dtype, device
        kw = dict(dtype=dtype, device=device)
        self.k = [torch.zeros(num_blocks, g[0], block_size, g[1], **kw) if g else None for g in geometry]
        self.v = [torch.zeros(num_blocks, g[0], block_size, g[2], **kw) if g else None for g in geometry]
        self.allocator = BlockedAllocator(num_blocks)
        self.num_slots = num_slots
        self.state = [{n: torch.zeros((num_slots, ) + tuple(shape), dtype=dt, device=device)
                       for n, (shape, dt) in g.items()} if g else None
                      for g in (state_geometry or [None] * len(geometry))]
        return self

    @staticmethod
    def block_bytes(geometry, block_size, dtype):
        """Bytes of one block over all layers."""
        item = torch.tensor([], dtype=dtype).element_size()
        return sum(g[0] * block_size * (g[1] + g[2]) * item for g in geometry if g is not None)

    @staticmethod
    def slot_bytes(state_geometry):
        """Bytes of one sequence's carried state over all layers."""
        total = 0
        for g in state_geometry:
            for shape, dt in (g or {}).values():
                n = torch.tensor([], dtype=dt).element_size()
                for d in shape:
                    n *= d
                total += n
        return total

    @staticmethod
    def blocks_for_memory(bytes_avail, num_layers, kv_heads, block_size, head_dim, dtype):
        per_block = 2 * num_layers * kv_heads * block_size * head_dim * torch.tensor([], dtype=dtype).element_size()
        return max(int(bytes_avail // per_block), 1)

    def bytes(self):
        held = [t for t in self.k + self.v if t is not None] + [t for g in self.state if g for t in g.values()]
        return sum(t.numel() * t.element_size() for t in held)

    # ---- the reference's cache-object interface (`inference/v2/ragged/kv_cache.py:40-208`)
    @property
    def num_caches(self):
        """Cache groups (models with several attention geometries would hold one each): one here."""
        return 1

    @property
    def free_blocks(self):
        return torch.tensor([self.allocator.free_blocks], dtype=torch.int32)

    def reserve(self, num_blocks, cache_group=0):
        """Take `num_blocks` block ids out of the free list."""
        return torch.tensor(self.allocator.allocate(int(num_blocks)), dtype=torch.int32)

    def free(self, blocks, cache_group=0):
        self.allocator.free(blocks.tolist() if torch.is_tensor(blocks) else blocks)

    def get_cache(self, cache_id, cache_group=0):
        """(keys, values) of layer `cache_id`, each [blocks, kv_heads, block_size, head_dim]."""
        return self.k[cache_id], self.v[cache_id]

    def offload(self, blocks, cache_group=0):
        """Copy the given blocks of every layer to pinned host memory (the blocks stay allocated); returns the
        handle `restore` takes."""
        idx = torch.as_tensor(blocks, dtype=torch.long, device=self.device)
        pin = torch.device(self.device).type == "cuda" if self.device is not None else False
        host = []
        for k, v in zip(self.k, self.v):
            if k is None:
                host.append(None)
                continue
            hk = torch.empty((idx.numel(), ) + tuple(k.shape[1:]), dtype=k.dtype, pin_memory=pin)
            hv = torch.empty((idx.numel(), ) + tuple(v.shape[1:]), dtype=v.dtype, pin_memory=pin)
            hk.copy_(k.index_select(0, idx), non_blocking=pin)
            hv.copy_(v.index_select(0, idx), non_blocking=pin)
            host.append((hk, hv))
        if pin:
            torch.cuda.current_stream().synchronize()
        return {"blocks": idx.cpu(), "data": host}

    def restore(self, handle, blocks=None, cache_group=0):
        """Write offloaded blocks back, to their old ids or to `blocks` (same count)."""
        idx = torch.as_tensor(handle["blocks"] if blocks is None else blocks, dtype=torch.long, device=self.device)
        for held, k, v in zip(handle["data"], self.k, self.v):
            if held is None:
                continue
            hk, hv = held
            k.index_copy_(0, idx, hk.to(k.device, non_blocking=True))
            v.index_copy_(0, idx, hv.to(v.device, non_blocking=True))


def split_kv(kv_cache):
    """(keys, values) of a stacked [2, ...] cache tensor or an already split pair."""
    return kv_cache[0], kv_cache[1]


class SequenceState:
    """Per-sequence bookkeeping: tokens already in cache and owned block ids."""

    def __init__(self, uid, block_size):
        self.uid = uid
        self.seen_tokens = 0
        self.blocks = []
        self.block_size = block_size

    def blocks_needed(self, new_tokens):
        total = self.seen_tokens + new_tokens
        need = (total + self.block_size - 1) // self.block_size
        return max(0, need - len(self.blocks))
