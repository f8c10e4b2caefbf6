"""What every model of the framework offers to the front end: the entry points by name, adapter types, the last rows of a
pass."""
from __future__ import annotations

import numpy as np
import torch


class CausalLM:
    dtypes = ("float16",)     # element types the model runs in
    native_step = False       # whether the C decode step (mlora_decode_step) serves it

    lora_types = ()

    def _ids(self, T, pairs, host=False):
        """Adapter rows per token and type; a model without adapters takes none."""
        if pairs:
            raise ValueError(f"{type(self).__name__} has no adapters")
        return {}

    def _last_rows(self, kv):
        lens = kv._cur[1]
        return torch.from_numpy(np.cumsum(lens).astype(np.int64) - 1).to(self.device)

    def prefill_no_adapter(self, h, kv):
        return self.forward(h, kv, None, self._last_rows(kv)), kv

    def decode_no_adapter(self, h, kv):
        return self.forward(h, kv, None), kv

    def __getitem__(self, name: str):
        """Entry points by the reference's VM function names."""
        if name in ("embed", "create_paged_kv_cache", "prefill_no_adapter", "decode_no_adapter"):
            return getattr(self, name)
        raise KeyError(f"unknown entry point {name}")

    @staticmethod
    def _cache_geometry(max_batch_size, max_total_seq_len, page_size, free_pages, max_seq_len):
        """(pages, blocks per sequence) of a pool of ceil(max_total_seq_len / page_size) + max_batch_size pages (one partial
        page per sequence), or of the given free pages."""
        n_pages = -(-max_total_seq_len // page_size) + max_batch_size
        if free_pages is not None:
            n_pages = len(free_pages)
        max_seq_len = max_seq_len or min(max_total_seq_len, n_pages * page_size)
        return n_pages, -(-max_seq_len // page_size)
