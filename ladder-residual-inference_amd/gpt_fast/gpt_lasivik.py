"""Lasivik: a post-norm hybrid decoder on the gfx950 kernels.

Every layer is a token mixer (gated linear attention, retention or windowed latent attention, in the order the
configuration lists) and an optional gated feed-forward; the residual is re-normalised after each sum:
    x <- norm1(alpha x + mixer(x)),   x <- norm2(alpha x + ff(x))
with gains stored around zero.  The residual stream is fp32; projections, caches and activations are bf16, or fp32 when
the model's parameters are.  Recurrent states live in fp32.  A call at position 0 starts every sequence of the batch
anew, so a cache slot is reused without being cleared; later calls continue where the previous one ended (input_pos must
be consecutive)."""
from types import SimpleNamespace

import torch
import torch.nn as nn
from torch import Tensor

from . import _hip
from ._hybrid import GPTHybrid, HybridWorkspace
from .config import REGISTRIES, LasivikArgs, LayerArgs
from .mixers import MIXERS, pad8, project
from .utils import FeedForward, RMSNorm

transformer_configs = REGISTRIES["lasivik"]


class LasivikWorkspace(HybridWorkspace):
    def __init__(self, model: "GPTLasivik", B: int, S: int, dtype, device, all_logits: bool):
        super().__init__(model, B, S, dtype, device, all_logits)
        e, rows = self._empty, self.rows
        ff = max([blk.feed_forward.w2.in_features for blk in model.layers if blk.feed_forward is not None], default=0)
        self._h, self._act = e(rows * 2 * ff), e(rows * ff)
        # zeroed once: the padding columns of a mixer's output stay zero
        self._y = {}
        for m in (blk.mixer for blk in model.layers):
            key = (m.y_cols, m.args.heads * m.args.vdim)
            if key not in self._y:
                self._y[key] = torch.zeros(rows, m.y_cols, dtype=dtype, device=device)

    def y_of(self, cols: int, used: int) -> Tensor:
        return self._y[(cols, used)]

    def ffn(self, I: int):
        return self._h[:self.rows * 2 * I].view(self.rows, 2 * I), self._act[:self.rows * I].view(self.rows, I)


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


class GPTLasivik(GPTHybrid):
    family = "lasivik"
    workspace_class = LasivikWorkspace

    def _make_block(self, config, layer_idx):
        return HybridBlock(config, config.layers[layer_idx])

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
            x, xc = self._last(ws, ws.x)
        _hip.residual_rmsnorm(x, 1.0, None, self.norm.weight, None, xc, cfg.norm_eps, cfg.width, gain_offset=1.0)
        logits = ws.logits.flatten(0, 1)
        project(xc, self.output, logits)
        _hip.logit_cap(logits, cfg.logit_scale, cfg.logit_softcap)
        return ws.logits
