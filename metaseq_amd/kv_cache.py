"""Preallocated contiguous per-layer caches: keys and values, and the latents and recurrent states
of hybrid decoders (``HybridCache``).

The reference grows its cache by ``torch.cat`` every step and every layer
(metaseq/modules/multihead_attention.py:449-479), re-copying the whole history.  Here each
layer owns one fp16 tensor ``[2, B, H, S_cap, hd]`` (K then V) that the QKV kernel appends to
in place; ``length`` counts the valid positions (columns of the token history).  A "ragged"
cache (prefilled from right-padded prompts, or filled slot by slot) stores every row without
pads and keeps the per-row lengths in ``lens`` (int32 [B] on the device, negative = empty
slot).  The object lives inside the caller-owned
``incremental_state`` dict, as the reference's per-module buffers do
(metaseq/incremental_decoding_utils.py:30-69), and is freed with it.
"""
import weakref

import torch


class KVCache:
    def __init__(self, n_layers, batch, heads, head_dim, capacity, device):
        self.n_layers, self.batch, self.heads, self.head_dim = n_layers, batch, heads, head_dim
        self.capacity = int(capacity)
        self.length = 0
        self.device = device
        self.has_pads = False
        self.ragged = False
        self.lens = None  # int32 [B] device tensor when ragged
        self.layers = [
            torch.empty(2, batch, heads, self.capacity, head_dim, dtype=torch.float16,
                        device=device)
            for _ in range(n_layers)
        ]

    def k(self, i):
        return self.layers[i][0]

    def v(self, i):
        return self.layers[i][1]

    def rows_view(self, b0, b1):
        """Rows b0 .. b1 - 1 as a cache of their own (a decode step taken in row chunks); the
        same object for the same range, so that work buffers kept on it persist."""
        views = self.__dict__.setdefault("_row_views", {})
        if (b0, b1) not in views:
            views[(b0, b1)] = _RowsView(self, b0, b1)
        return views[(b0, b1)]

    def grow(self, new_capacity):
        """Reallocates every layer to ``new_capacity`` positions, keeping the valid prefix."""
        new_capacity = int(new_capacity)
        if new_capacity <= self.capacity:
            return
        for i, old in enumerate(self.layers):
            new = torch.empty(2, self.batch, self.heads, new_capacity, self.head_dim,
                              dtype=torch.float16, device=self.device)
            new[:, :, :, :self.length].copy_(old[:, :, :, :self.length])
            self.layers[i] = new
        self.capacity = new_capacity

    def copy_row(self, src, dst, n):
        """Row ``dst`` takes the first ``n`` positions of row ``src``."""
        for layer in self.layers:
            layer[:, dst, :, :n].copy_(layer[:, src, :, :n])

    def bytes(self):
        return sum(t.numel() * 2 for t in self.layers)


class _RowsView:
    """Rows b0 .. b1 - 1 of a ``KVCache`` with what a decode step reads of a cache: ``k(i)``,
    ``v(i)`` (contiguous slices of the parent's current tensors), ``capacity``, ``device``."""

    def __init__(self, cache, b0, b1):
        # a weak reference: the cache keeps its views, and must still be freed by its last
        # outside reference going away, not by a later garbage-collection pass
        self._cache, self._b0, self._b1 = weakref.proxy(cache), b0, b1
        self.device = cache.device

    @property
    def capacity(self):
        return self._cache.capacity

    def k(self, i):
        return self._cache.layers[i][0][self._b0:self._b1]

    def v(self, i):
        return self._cache.layers[i][1][self._b0:self._b1]


class HybridCache:
    """What the layers of a hybrid decoder keep per slot (a row of a batch, or a serving slot):

    * attention layers that own a latent: ``latent`` [slots, capacity, rank], activation format;
    * attention layers with keys and values: ``keys`` and ``values`` [slots, kv_heads, rows, size],
      activation format; rows is the capacity, or one chunk where attention stays within chunks;
    * recurrent layers: ``conv`` [slots, taps - 1, channels], the short convolution's last inputs
      (activation format), and ``rec``, the fp32 recurrent state.

    A layer that runs several times keeps that much for each of its runs.

    ``lens`` (int32 [slots] on the device): positions each slot holds, negative = empty slot;
    ``host_lens``: the same on the host where the caller of the slot interface knows it.  Nothing
    has to be cleared when a slot is given to a new sequence: a segment that starts at position 0
    ignores what the slot held.  Lives in the caller's ``incremental_state`` like ``KVCache``."""

    has_pads = False
    ragged = True

    def __init__(self, layout, slots, capacity, dtype, device):
        """``layout``: per run of a layer {"latent": rank}, {"keys": size, "values": size,
        "kv_heads": n, "chunk": positions or None}, {"conv": (taps - 1, channels), "rec": shape}
        or several of them (what the layer keeps; an empty dict: nothing)."""
        self.layout, self.batch, self.capacity = layout, int(slots), int(capacity)
        self.dtype, self.device = dtype, device
        self.length = 0
        self.lens = torch.full((self.batch,), -1, dtype=torch.int32, device=device)
        self.host_lens = [-1] * self.batch
        self.layers = []
        for keep in layout:
            t = {}
            if "latent" in keep:
                t["latent"] = torch.zeros(self.batch, self.capacity, keep["latent"], dtype=dtype,
                                          device=device)
            for name in ("keys", "values"):
                if name in keep:
                    t[name] = torch.zeros(self.batch, keep["kv_heads"],
                                          self.kept_rows(keep, self.capacity), keep[name],
                                          dtype=dtype, device=device)
            if "rec" in keep:
                t["rec"] = torch.zeros((self.batch,) + tuple(keep["rec"]), dtype=torch.float32,
                                       device=device)
            if keep.get("conv", (0,))[0] > 0:
                t["conv"] = torch.zeros((self.batch,) + tuple(keep["conv"]), dtype=dtype,
                                        device=device)
            self.layers.append(t)

    @staticmethod
    def kept_rows(keep, capacity):
        """Positions whose keys and values a slot of that capacity keeps."""
        return min(capacity, keep["chunk"]) if keep.get("chunk") else capacity

    def grow(self, new_capacity):
        """Re-allocates latents, keys and values to ``new_capacity`` positions per slot."""
        new_capacity = int(new_capacity)
        if new_capacity <= self.capacity:
            return
        for keep, t in zip(self.layout, self.layers):
            for name in ("keys", "values"):
                if name not in t or self.kept_rows(keep, new_capacity) == t[name].shape[2]:
                    continue
                old = t[name]
                new = torch.zeros(old.shape[:2] + (self.kept_rows(keep, new_capacity),
                                                   old.shape[3]), dtype=self.dtype,
                                  device=self.device)
                new[:, :, :old.shape[2]].copy_(old)
                t[name] = new
            if "latent" in t:
                old = t["latent"]
                new = torch.zeros(self.batch, new_capacity, old.shape[2], dtype=self.dtype,
                                  device=self.device)
                new[:, :self.capacity].copy_(old)
                t["latent"] = new
        self.capacity = new_capacity

    def copy_row(self, src, dst, n):
        """Slot ``dst`` becomes slot ``src``, which holds ``n`` positions."""
        for t in self.layers:
            for name, x in t.items():
                if name == "latent":
                    x[dst, :n].copy_(x[src, :n])
                elif name in ("keys", "values"):
                    x[dst, :, :n].copy_(x[src, :, :n])
                else:
                    x[dst].copy_(x[src])
        self.host_lens[dst] = n

    def bytes(self):
        return sum(x.numel() * x.element_size() for t in self.layers for x in t.values())
