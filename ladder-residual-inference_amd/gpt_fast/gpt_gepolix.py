"""Gepolix: a parallel hybrid decoder on the gfx950 kernels.

Both sublayers of a layer read one normalised input, and both results are added to the residual:
    h = norm(x),   x <- x + (mixer(h) + ff(h))
The norm is a scaled tanh, tanh(alpha x) w + b.  Mixers: a selective state space (Mamba-2) and grouped attention through a
sliding window, which may read another layer's keys and values; the feed-forward is dense, a mixture of experts (with or
without a shared expert) or absent.

The parallel form is used throughout: one launch projects h for mixer and feed-forward (decode batches), and the mixer's
output projection and the feed-forward's down projection are one product over the concatenated columns, whose fp32 sums are
the layer's update.  The norm needs no statistics, so residual, experts' weighted sum and the next layer's norm are one pass,
which in decode batches is the end of that product.
The residual stream is fp32; projections, caches and activations are bf16, or fp32 when the model's parameters are.  States
live in fp32.  A call at position 0 starts every sequence of the batch anew, so a cache slot is reused without being cleared;
later calls continue where the previous one ended (input_pos must be consecutive)."""
import torch
import torch.nn as nn

from . import _hip
from ._hybrid import GPTHybrid, HybridWorkspace
from .config import REGISTRIES, GepolixArgs, LayerArgs
from .mixers import MIXERS, pad8, project
from .utils import DynamicTanh, Experts

transformer_configs = REGISTRIES["gepolix"]


class ParallelWorkspace(HybridWorkspace):
    def __init__(self, model, B, S, dtype, device, all_logits):
        super().__init__(model, B, S, dtype, device, all_logits)
        e, rows = self._empty, self.rows
        # mixer output and feed-forward activation side by side, as the joint output projection reads them
        self._joint = {}
        for blk in model.layers:
            key = (blk.mixer.y_cols, blk.beside)
            if key not in self._joint:
                self._joint[key] = torch.zeros(rows, sum(key), dtype=dtype, device=device)
        self.h = e(rows * 2 * max(blk.beside for blk in model.layers))
        mix = [blk.experts for blk in model.layers if blk.experts is not None]
        if mix:
            top = max(m.top for m in mix)
            self._expert_out = e(rows * top * model.config.dim)
            self._expert_ids, self._expert_weights = e(rows * top, dt=torch.int32), e(rows * top, dt=torch.float32)
            self._gate = e(rows, dt=torch.float32)
            self._counts = torch.zeros(max(m.n for m in mix), dtype=torch.int32, device=device)
            self._expert_scratch = e(max(_hip.moe_scratch_bytes(rows, m.n, m.top, m.ff, dtype) for m in mix), dt=torch.uint8)

    def joint(self, blk):
        """(both, mixer's columns, feed-forward's columns)"""
        t = self._joint[(blk.mixer.y_cols, blk.beside)]
        return t, t[:, :blk.mixer.y_cols], t[:, blk.mixer.y_cols:]

    def expert_buffers(self, m: Experts, dim: int):
        n = self.rows * m.top
        return (self._expert_out[:n * dim].view(n, dim), self._expert_ids[:n].view(self.rows, m.top),
                self._expert_weights[:n].view(self.rows, m.top), self._gate, self._counts[:m.n], self._expert_scratch)


class ParallelBlock(nn.Module):
    def __init__(self, config: GepolixArgs, layer: LayerArgs):
        super().__init__()
        D, m = config.dim, layer.experts
        self.norm = DynamicTanh(D)
        self.mixer = MIXERS[layer.mixer.kind](D, layer.mixer, config.norm_eps)
        # the dense feed-forward, or the shared expert: its rows [up; gate], its down projection in the joint one
        dense = layer.ffn if m is None else m.shared
        self.beside = 0 if dense is None else pad8(dense)
        self.w1 = nn.Linear(D, 2 * self.beside, bias=False) if self.beside else None
        self.mixer.widen_out(self.beside)
        self.experts = None if m is None else Experts(D, m.experts, m.top, pad8(m.ff), m.shared is not None)


class GPTGepolix(GPTHybrid):
    family = "gepolix"
    workspace_class = ParallelWorkspace

    def __init__(self, config: GepolixArgs) -> None:
        super().__init__(config)
        self.norm = DynamicTanh(config.dim)
        for blk, layer in zip(self.layers, config.layers):
            if layer.mixer.kv_from is not None:
                blk.mixer.lend(self.layers[layer.mixer.kv_from].mixer)

    def _make_block(self, config, layer_idx):
        return ParallelBlock(config, config.layers[layer_idx])

    def _weights_per_step(self, batch_size):
        """Of a mixture, the experts a batch of independent choices is expected to touch."""
        n = super()._weights_per_step(batch_size)
        for blk in self.layers:
            m = blk.experts
            if m is not None:
                n -= (m.w1.numel() + m.w2.numel()) * (1 - m.top / m.n) ** batch_size
        return n

    # -- forward ----------------------------------------------------------------------------------
    def _embed(self, ws, idx):
        _hip.embed_residual(self.tok_embeddings.weight, idx.contiguous(), ws.x, None, 1.0)
        self.layers[0].norm.into(ws.x, None, None, ws.xc)

    def _run_layers(self, ws, pos):
        norms = [blk.norm for blk in self.layers[1:]] + [self.norm]
        for blk, following in zip(self.layers, norms):
            both, y, act = ws.joint(blk)
            m, experts, routed = blk.experts, None, None
            if m is not None:
                buffers = ws.expert_buffers(m, self.config.dim)
                routed, experts = m.on(ws.xc, act if m.shared else None, *buffers), (buffers[0], buffers[2])
            proj = self._project_in(ws, blk, act, routed)
            blk.mixer.mix(ws, pos, proj, y)
            if m is not None:
                _hip.moe(routed)
            following.after(both, blk.mixer.out_proj, ws.d, ws.x, ws.xc, experts)
        return None, None

    def _project_in(self, ws, blk, act, routed):
        """The mixer's projections of ws.xc; the feed-forward's activations into `act`.  A decode batch takes one launch, routing
        included."""
        proj = ws.proj[:, :blk.mixer.proj_cols]
        w = blk.mixer.in_proj.weight
        if ws.xc.dtype == torch.bfloat16 and ws.rows <= 64:
            todo = [(ws.xc, w, proj, _hip.EPI_NONE)]
            if blk.w1 is not None:
                todo.append((ws.xc, blk.w1.weight, act, _hip.EPI_SWIGLU))
            if routed is not None:
                _hip.linear_multi_route(routed, *todo)
            else:
                _hip.linear_multi(*todo)
            return proj
        if blk.w1 is None:
            return project(ws.xc, blk.mixer.in_proj, proj)
        h = ws.h[:ws.rows * 2 * blk.beside].view(ws.rows, -1)
        if ws.xc.dtype == torch.float32:
            _hip.linear(ws.xc, blk.w1.weight, h)
            _hip.swiglu(h, act)
            _hip.linear(ws.xc, w, proj)
        else:
            _hip.linear_swiglu_out(ws.xc, blk.w1.weight, act, h)
            _hip.linear(ws.xc, w, proj)
        return proj

    def _head(self, ws, d1, d2):
        xc = ws.xc if ws.last_rows is None else self._last(ws, ws.xc)[1]
        project(xc, self.output, ws.logits.flatten(0, 1))
        return ws.logits
