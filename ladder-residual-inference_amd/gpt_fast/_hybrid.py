"""What the families whose configuration lists every layer's mixer share: caches and states held by the mixers, a residual
stream in fp32, the buffers of one (batch, seq) shape, and the count of bytes a decode step moves."""
from typing import List

import torch
from torch import Tensor

from . import _hip
from ._model import GPTBase
from .mixers import pad8


class HybridWorkspace:
    """Activation buffers for one (batch, seq) shape."""

    def __init__(self, model: "GPTHybrid", B: int, S: int, dtype, device, all_logits: bool):
        cfg = model.config
        rows, D = B * S, cfg.dim
        mixers = [blk.mixer for blk in model.layers]
        e = self._empty = lambda *shape, dt=dtype: torch.empty(*shape, dtype=dt, device=device)
        self.B, self.S, self.rows = B, S, rows
        self.x = e(rows, D, dt=torch.float32)     # residual stream
        self.xc = e(rows, D)                      # in the compute type: the input of the next product
        self.d = e(rows, D)                       # what the current sublayer adds to the residual
        self.proj = e(rows, pad8(max(m.proj_cols for m in mixers)))
        n = max(m.scratch_bytes(B, S) for m in mixers)
        self.scratch = e(n, dt=torch.uint8) if n else None
        n = max((r * c for r, c in (m.window_rows(B, S) for m in mixers)), default=0)
        self._window = e(n) if n else None
        out_rows = S if all_logits else 1
        self.logits = e(B, out_rows, pad8(cfg.output_rows))[..., :cfg.output_rows]
        self.last_rows = None
        if S > 1 and not all_logits:
            self.last_rows = (torch.arange(1, B + 1, dtype=torch.int64, device=device) * S - 1).contiguous()
            self.xl = e(B, D, dt=torch.float32)
            self.xcl = e(B, D)
        self.next_token = torch.empty(B, 1, dtype=torch.int32, device=device)
        self.next_token_valid_for = None

    def window_buffers(self, n: int, rank: int, cols: int):
        cp = pad8(cols)
        return self._window[:n * rank].view(n, rank), self._window[n * rank:n * (rank + cp)].view(n, cp)[:, :cols]


class GPTHybrid(GPTBase):
    supports_fp8 = False
    supported_dtypes = (torch.bfloat16, torch.float32)
    workspace_class = HybridWorkspace

    # -- caches and states ------------------------------------------------------------------------
    def _check_caches(self, max_seq_length):
        pass

    def _build_caches(self, max_batch_size, max_seq_length, dtype, device):
        for blk in self.layers:
            blk.mixer.setup_cache(max_batch_size, max_seq_length, dtype, device)

    def recurrent_states(self) -> List[Tensor]:
        return [s for blk in self.layers for s in blk.mixer.states()]

    def _weights_per_step(self, batch_size: int) -> float:
        """Parameters a decode step reads, the embedding table's aside."""
        return sum(p.numel() for p in self.parameters()) - self.tok_embeddings.weight.numel()

    def decode_bytes(self, batch_size: int, pos: int) -> int:
        """Algorithmic HBM bytes of one decode step at `pos`: every weight and gain it needs once, embedding rows, what the
        caches and states read and write."""
        it = self.output.weight.element_size()
        carried = sum(blk.mixer.cache_bytes_per_step(batch_size, pos, it) for blk in self.layers)
        return int(it * (self._weights_per_step(batch_size) + batch_size * self.config.dim) + carried)

    # -- forward ----------------------------------------------------------------------------------
    def _new_workspace(self, B, S):
        w = self.output.weight
        return self.workspace_class(self, B, S, w.dtype, w.device, not self.last_logits_only)

    def _last(self, ws, table: Tensor):
        """The last row of every sequence of `table` (fp32 or the compute type), in both."""
        _hip.embed_residual(table, ws.last_rows, ws.xl, None if table.dtype != ws.xcl.dtype else ws.xcl, 1.0)
        return ws.xl, ws.xcl
