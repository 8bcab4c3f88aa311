"""Lasivik: a post-norm hybrid decoder on the gfx950 kernels.

Every layer is a token mixer (gated linear attention, retention or windowed latent attention, in the order the
configuration lists) and an optional gated feed-forward; the residual is re-normalised after each sum:
    x <- norm1(alpha x + mixer(x)),   x <- norm2(alpha x + ff(x))
with gains stored around zero.  The residual stream is fp32; projections, caches and activations are bf16, or fp32 when
the model's parameters are.  Recurrent states live in fp32.  A call at position 0 starts every sequence of the batch
anew, so a cache slot is reused without being cleared; later calls continue where the previous one ended (input_pos must
be consecutive)."""
from types import SimpleNamespace
from typing import List

import torch
import torch.nn as nn
from torch import Tensor

from . import _hip
from ._model import GPTBase
from .config import REGISTRIES, LasivikArgs, LayerArgs
from .mixers import MIXERS, pad8, project
from .utils import FeedForward, RMSNorm

transformer_configs = REGISTRIES["lasivik"]


class HybridWorkspace:
    """Activation buffers for one (batch, seq) shape."""

    def __init__(self, model: "GPTLasivik", B: int, S: int, dtype, device, all_logits: bool):
        cfg = model.config
        rows, D = B * S, cfg.dim
        mixers = [blk.mixer for blk in model.layers]
        e = lambda *shape, dt=dtype: torch.empty(*shape, dtype=dt, device=device)
        self.B, self.S, self.rows = B, S, rows
        self.x = e(rows, D, dt=torch.float32)     # residual stream
        self.xc = e(rows, D)                      # the same in the compute type: the input of the next product
        self.d = e(rows, D)                       # what the current sublayer adds to it
        self.proj = e(rows, pad8(max(m.proj_cols for m in mixers)))
        ff = max([blk.feed_forward.w2.in_features for blk in model.layers if blk.feed_forward is not None], default=0)
        self._h, self._act = e(rows * 2 * ff), e(rows * ff)
        # zeroed once: the padding columns of a mixer's output stay zero
        self._y = {}
        for m in mixers:
            key = (m.y_cols, m.args.heads * m.args.vdim)
            if key not in self._y:
                self._y[key] = torch.zeros(rows, m.y_cols, dtype=dtype, device=device)
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

    def y_of(self, cols: int, used: int) -> Tensor:
        return self._y[(cols, used)]

    def ffn(self, I: int):
        return self._h[:self.rows * 2 * I].view(self.rows, 2 * I), self._act[:self.rows * I].view(self.rows, I)

    def window_buffers(self, n: int, rank: int, cols: int):
        cp = pad8(cols)
        return self._window[:n * rank].view(n, rank), self._window[n * rank:n * (rank + cp)].view(n, cp)[:, :cols]


class HybridBlock(nn.Module):
    def __init__(self, config: LasivikArgs, layer: LayerArgs):
        super().__init__()
        self.mixer = MIXERS[layer.mixer.kind](config.dim, layer.mixer, config.norm_eps)
        self.mixer_norm = RMSNorm(config.dim, config.norm_eps)
        self.feed_forward = self.ffn_norm = None
        if layer.ffn is not None:
            self.feed_forward = FeedForward(SimpleNamespace(dim=config.dim, intermediate_size=pad8(layer.ffn),
                                                            tp_world_size=1))
            self.ffn_norm = RMSNorm(config.dim, config.norm_eps)


class GPTLasivik(GPTBase):
    family = "lasivik"
    supports_fp8 = False

    def _make_block(self, config, layer_idx):
        return HybridBlock(config, config.layers[layer_idx])

    # -- caches and states ------------------------------------------------------------------------
    def _check_caches(self, max_seq_length):
        pass

    def _build_caches(self, max_batch_size, max_seq_length, dtype, device):
        for blk in self.layers:
            blk.mixer.setup_cache(max_batch_size, max_seq_length, dtype, device)

    supported_dtypes = (torch.bfloat16, torch.float32)

    def recurrent_states(self) -> List[Tensor]:
        return [s for s in (blk.mixer.state() for blk in self.layers) if s is not None]

    def decode_bytes(self, batch_size: int, pos: int) -> int:
        """Algorithmic HBM bytes of one decode step at `pos`: every weight and gain once, embedding rows, what the
        caches and states read and write."""
        it = self.output.weight.element_size()
        weights = sum(p.numel() for p in self.parameters()) - self.tok_embeddings.weight.numel()
        carried = sum(blk.mixer.cache_bytes_per_step(batch_size, pos, it) for blk in self.layers)
        return it * (weights + batch_size * self.config.dim) + carried

    # -- forward ----------------------------------------------------------------------------------
    def _new_workspace(self, B, S):
        w = self.output.weight
        return HybridWorkspace(self, B, S, w.dtype, w.device, not self.last_logits_only)

    def _embed(self, ws, idx):
        _hip.embed_residual(self.tok_embeddings.weight, idx.contiguous(), ws.x, ws.xc, self.config.embedding_scale)

    def _norm_into(self, ws, norm: RMSNorm, alpha, d):
        """x <- norm(alpha x + d), in fp32 and in the compute type."""
        _hip.residual_rmsnorm(ws.x, alpha, d, norm.weight, ws.x, ws.xc, norm.eps, self.config.width, gain_offset=1.0)

    def _run_layers(self, ws, pos):
        alpha = self.config.residual_scale
        for blk in self.layers:
            blk.mixer.run(ws, pos)
            self._norm_into(ws, blk.mixer_norm, alpha, ws.d)
            if blk.feed_forward is not None:
                self._feed_forward(ws, blk.feed_forward)
                self._norm_into(ws, blk.ffn_norm, alpha, ws.d)
        return None, None

    def _feed_forward(self, ws, ff: FeedForward):
        h, act = ws.ffn(ff.w2.in_features)
        if ws.xc.dtype == torch.float32:
            _hip.linear(ws.xc, ff.w1.weight, h)
            _hip.swiglu(h, act)
        else:
            _hip.linear_swiglu_out(ws.xc, ff.w1.weight, act, h)
        project(act, ff.w2, ws.d)

    def _head(self, ws, d1, d2):
        cfg = self.config
        x, xc = ws.x, ws.xc
        if ws.last_rows is not None:
            x, xc = ws.xl, ws.xcl
            _hip.embed_residual(ws.x, ws.last_rows, x, None, 1.0)   # a row gather
        _hip.residual_rmsnorm(x, 1.0, None, self.norm.weight, None, xc, cfg.norm_eps, cfg.width, gain_offset=1.0)
        logits = ws.logits.flatten(0, 1)
        project(xc, self.output, logits)
        _hip.logit_cap(logits, cfg.logit_scale, cfg.logit_softcap)
        return ws.logits
