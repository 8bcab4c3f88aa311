"""Token mixers of hybrid models, on the gfx950 kernels: gated linear attention, retention, windowed latent attention.

A mixer is a module with its projections, its constants and -- after setup_cache -- what it carries from token to token:
a recurrent state in fp32 or a cache of latents.  run() mixes B * S rows of a workspace: it reads the layer's input in
the compute type and leaves the output projection in ws.d.  Sizes and constants come as arguments, so that another
design can use a mixer with other ones.  Column counts that are the inner dimension of a following product are padded
to a multiple of 8 (`pad8`); the padding is zero in weights and activations alike."""
import math
from dataclasses import dataclass
from typing import List, Optional

import torch
import torch.nn as nn
from torch import Tensor

from . import _hip
from .utils import RMSNorm


def pad8(n: int) -> int:
    return (n + 7) // 8 * 8


@dataclass
class MixerArgs:
    kind: str                       # a key of MIXERS
    heads: int
    dim: int                        # query / key dimensions per head
    vdim: int                       # value dimensions per head
    tau: float = 1.0                # gla: the decay is sigmoid(z)^(1 / tau)
    decay_rank: int = 16            # gla: rank of z's projection
    decay: Optional[List[float]] = None   # retention: per head
    rot_dims: int = 0               # retention: rotated dimensions per head ("rotate half" pairs), 0: none
    rot_base: float = 10000.0
    kv_rank: int = 0                # latent attention
    window: int = 0
    scale: float = 1.0


def project(x: Tensor, lin: nn.Linear, out: Tensor) -> Tensor:
    """lin(x) for the rows of a step: the weight-streaming kernel from two to 64 rows (as the other families' decode
    steps use it), what the shape picks otherwise."""
    if x.dtype == torch.bfloat16 and 2 <= x.shape[0] <= 64:
        _hip.linear_multi((x, lin.weight, out, _hip.EPI_NONE))
        return out
    return _hip.linear(x, lin.weight, out)


def rotate_half_table(length: int, dims: int, base: float) -> Tensor:
    """(cos, sin) of position * base^(-2 i / dims), fp32 [length, dims / 2, 2]; evaluated in double on the host."""
    with torch.device("cpu"):
        f = float(base) ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
        a = torch.outer(torch.arange(length, dtype=torch.float64), f)
        return torch.stack([a.cos(), a.sin()], dim=-1).float()


class Mixer(nn.Module):
    """What the mixers share: an input projection whose rows are the concatenated projections of the layer's input, and
    the output projection."""

    recurrent = False   # True: carries a state that a step changes, so running a step twice is not the same as once

    def __init__(self, width: int, args: MixerArgs, eps: float, in_rows: int):
        super().__init__()
        self.args, self.eps = args, eps
        self.y_cols = pad8(args.heads * args.vdim)
        self.proj_cols = in_rows
        self.in_proj = nn.Linear(width, in_rows, bias=False)
        self.out_proj = nn.Linear(self.y_cols, width, bias=False)

    def setup_cache(self, batch: int, length: int, dtype, device):
        raise NotImplementedError

    def state(self) -> Optional[Tensor]:
        """The recurrent state, None for a mixer whose cache is written by position."""
        return None

    def scratch_bytes(self, B: int, S: int) -> int:
        return 0

    def window_rows(self, B: int, S: int):
        """(rows, columns) of expanded keys and values a portion needs besides, (0, 0) for none."""
        return 0, 0

    def cache_bytes_per_step(self, B: int, pos: int, itemsize: int) -> int:
        """Bytes of cache or state one decode step at `pos` reads and writes."""
        raise NotImplementedError

    def _project_in(self, ws) -> Tensor:
        return project(ws.xc, self.in_proj, ws.proj[:, :self.proj_cols])

    def _y(self, ws) -> Tensor:
        return ws.y_of(self.y_cols, self.args.heads * self.args.vdim)

    def run(self, ws, pos: Tensor):
        raise NotImplementedError


class _LinearAttention(Mixer):
    recurrent = True

    def __init__(self, width, args: MixerArgs, eps, extra_rows: int = 0):
        super().__init__(width, args, eps, 2 * args.heads * (args.dim + args.vdim) + extra_rows)

    def setup_cache(self, batch, length, dtype, device):
        a = self.args
        self.register_buffer("recurrent_state", torch.zeros(batch, a.heads, a.dim, a.vdim, dtype=torch.float32,
                                                            device=device), persistent=False)

    def state(self):
        return self.recurrent_state

    def scratch_bytes(self, B, S):
        a = self.args
        return _hip.linear_attention_scratch_bytes(B, S, a.heads, a.dim, a.vdim, self._gated)

    def cache_bytes_per_step(self, B, pos, itemsize):
        a = self.args
        return 2 * B * a.heads * a.dim * a.vdim * 4

    def _attend(self, ws, pos, **kw):
        a = self.args
        _hip.linear_attention(self._project_in(ws), self._y(ws), self.recurrent_state, pos, ws.B, ws.S, a.heads, a.dim,
                              a.vdim, self.eps, scratch=ws.scratch, **kw)
        project(self._y(ws), self.out_proj, ws.d)


class GatedLinearAttention(_LinearAttention):
    """in_proj rows [q; k; v; g; low-rank decay input]; decay_up maps the latter to a decay per key channel."""
    _gated = True

    def __init__(self, width, args: MixerArgs, eps):
        super().__init__(width, args, eps, args.decay_rank)
        self.decay_up = nn.Linear(args.decay_rank, args.heads * args.dim, bias=True)
        self.norm = RMSNorm(args.vdim, eps)

    def run(self, ws, pos):
        a = self.args
        self._attend(ws, pos, q_scale=a.dim ** -0.5, norm=self.norm.weight,
                     gate=(self.decay_up.weight, self.decay_up.bias, a.tau))


class Retention(_LinearAttention):
    """in_proj rows [q; k; v; g]; a fixed decay per head, rotated q and k, an output norm without a gain."""
    _gated = False

    def setup_cache(self, batch, length, dtype, device):
        super().setup_cache(batch, length, dtype, device)
        a = self.args
        log_decay = [math.log(d) if d > 0 else -math.inf for d in a.decay]
        self.register_buffer("log_decay", torch.tensor(log_decay, dtype=torch.float32, device=device), persistent=False)
        table = rotate_half_table(length, a.rot_dims, a.rot_base).to(device) if a.rot_dims else None
        self.register_buffer("rope", table, persistent=False)

    def run(self, ws, pos):
        self._attend(ws, pos, k_scale=self.args.dim ** -0.5, head_decay=self.log_decay, rope=self.rope)


class LatentAttention(Mixer):
    """in_proj rows [q; latent]; kv_up rows [k of every head; v of every head].  Only the normalised latents are cached:
    [batch, length, rank padded to 8]."""

    # portions of up to this many tokens attend on the latents themselves; longer ones expand k and v of their window
    absorb_up_to = 8

    def __init__(self, width, args: MixerArgs, eps):
        super().__init__(width, args, eps, args.heads * args.dim + args.kv_rank)
        self.rank_p = pad8(args.kv_rank)
        self.norm = RMSNorm(args.kv_rank, eps)
        self.kv_up = nn.Linear(self.rank_p, args.heads * (args.dim + args.vdim), bias=False)

    def setup_cache(self, batch, length, dtype, device):
        self.register_buffer("latents", torch.zeros(batch, length, self.rank_p, dtype=dtype, device=device),
                             persistent=False)

    def _absorbs(self, S):
        return S <= self.absorb_up_to

    def _n_keys(self, S):
        return min(S + self.args.window - 1, self.latents.shape[1])

    def scratch_bytes(self, B, S):
        if not self._absorbs(S):
            return 0
        return _hip.latent_attention_scratch_bytes(B, S, self.args.heads, self.rank_p, self.args.window,
                                                   self.latents.shape[1])

    def window_rows(self, B, S):
        a = self.args
        return (0, 0) if self._absorbs(S) else (B * self._n_keys(S), self.rank_p + pad8(a.heads * (a.dim + a.vdim)))

    def cache_bytes_per_step(self, B, pos, itemsize):
        return B * self.rank_p * itemsize * (min(pos + 1, self.args.window) + 1)

    def run(self, ws, pos):
        a = self.args
        nq, cache = a.heads * a.dim, self.latents
        proj = self._project_in(ws)
        y = self._y(ws)
        if self._absorbs(ws.S):
            w = self.kv_up.weight
            _hip.latent_attention(proj[:, :nq], w[:nq], w[nq:], cache, y, pos, ws.scratch, ws.B, ws.S, a.heads, a.dim,
                                  a.vdim, a.window, a.scale, new=(proj[:, nq:], self.norm.weight, a.kv_rank, self.eps))
        else:
            _hip.latent_update(proj[:, nq:], self.norm.weight, pos, cache, ws.B, ws.S, a.kv_rank, self.eps)
            n = self._n_keys(ws.S)
            rows, kv = ws.window_buffers(ws.B * n, self.rank_p, a.heads * (a.dim + a.vdim))
            if n == cache.shape[1]:      # the window reaches over the whole cache: its rows as they lie
                rows = cache[:ws.B].view(ws.B * n, self.rank_p)
            else:
                _hip.latent_window(cache, pos, rows.view(ws.B, n, self.rank_p), ws.B, a.window)
            _hip.linear(rows, self.kv_up.weight, kv)
            _hip.window_attention(proj[:, :nq], kv, y, pos, ws.B, ws.S, a.heads, a.dim, a.vdim, a.window, n,
                                  cache.shape[1], a.scale)
        project(y, self.out_proj, ws.d)


MIXERS = {"gla": GatedLinearAttention, "retention": Retention, "latent_attention": LatentAttention}
