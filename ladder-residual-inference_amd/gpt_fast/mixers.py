"""Token mixers of hybrid models, on the gfx950 kernels: gated linear attention, retention, windowed latent attention, a
selective state space (Mamba-2), grouped attention through a sliding window.

A mixer is a module with its projections, its constants and -- after setup_cache -- what it carries from token to token:
a recurrent state in fp32 or a cache of latents.  run() mixes B * S rows of a workspace: it reads the layer's input in
the compute type and leaves the output projection in ws.d; mix() is its part between the two projections, for blocks that
project for several sublayers at once.  Sizes and constants come as arguments, so that another
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


def pad16(n: int) -> int:
    return (n + 15) // 16 * 16


@dataclass
class MixerArgs:
    kind: str                       # a key of MIXERS
    heads: int
    dim: int                        # query / key dimensions per head (mamba2: none)
    vdim: int                       # value dimensions per head
    tau: float = 1.0                # gla: the decay is sigmoid(z)^(1 / tau)
    decay_rank: int = 16            # gla: rank of z's projection
    decay: Optional[List[float]] = None   # retention: per head
    rot_dims: int = 0               # retention, attention: rotated dimensions per head ("rotate half" pairs), 0: none
    rot_base: float = 10000.0
    kv_rank: int = 0                # latent attention
    window: int = 0                 # latent attention, attention
    scale: float = 1.0
    kv_heads: int = 0               # attention: query head h reads head h // (heads / kv_heads)
    kv_from: Optional[int] = None   # attention: the layer whose keys and values it reads instead of its own
    bias: bool = False              # attention: biases of q, k and v
    state: int = 0                  # mamba2: rows of a head's state, shared by the heads of one of `groups`
    groups: int = 1
    norm_groups: int = 1            # mamba2: parts of the output norm
    taps: int = 1                   # mamba2: of the convolution ahead of the state space


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

    def __init__(self, width: int, args: MixerArgs, eps: float, in_rows: int, y_cols: Optional[int] = None, bias: bool = False):
        super().__init__()
        self.args, self.eps = args, eps
        self.y_cols = pad8(args.heads * args.vdim) if y_cols is None else y_cols
        self.proj_cols = in_rows
        self.in_proj = nn.Linear(width, in_rows, bias=bias)     # (a bias is added by what follows the product)
        self.out_proj = nn.Linear(self.y_cols, width, bias=False)

    def setup_cache(self, batch: int, length: int, dtype, device):
        raise NotImplementedError

    def states(self) -> List[Tensor]:
        """What a step changes so that running it twice is not the same as once; nothing for a mixer whose cache is written
        by position."""
        return []

    def widen_out(self, beside: int):
        """Output projection over y_cols + beside inner columns: another sublayer's result is projected in the same product."""
        if beside:
            self.out_proj = nn.Linear(self.y_cols + beside, self.out_proj.out_features, bias=False)

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

    def mix(self, ws, pos: Tensor, proj: Tensor, y: Tensor):
        """proj [rows, proj_cols] -> y [rows, >= y_cols]; a row of either may be part of a longer one."""
        raise NotImplementedError

    def run(self, ws, pos: Tensor):
        y = self._y(ws)
        self.mix(ws, pos, self._project_in(ws), y)
        project(y, self.out_proj, ws.d)


class _LinearAttention(Mixer):
    recurrent = True

    def __init__(self, width, args: MixerArgs, eps, extra_rows: int = 0):
        super().__init__(width, args, eps, 2 * args.heads * (args.dim + args.vdim) + extra_rows)

    def setup_cache(self, batch, length, dtype, device):
        a = self.args
        self.register_buffer("recurrent_state", torch.zeros(batch, a.heads, a.dim, a.vdim, dtype=torch.float32,
                                                            device=device), persistent=False)

    def states(self):
        return [self.recurrent_state]

    def scratch_bytes(self, B, S):
        a = self.args
        return _hip.linear_attention_scratch_bytes(B, S, a.heads, a.dim, a.vdim, self._gated)

    def cache_bytes_per_step(self, B, pos, itemsize):
        a = self.args
        return 2 * B * a.heads * a.dim * a.vdim * 4

    def _attend(self, ws, pos, proj, y, **kw):
        a = self.args
        _hip.linear_attention(proj, y, self.recurrent_state, pos, ws.B, ws.S, a.heads, a.dim, a.vdim, self.eps,
                              scratch=ws.scratch, **kw)


class GatedLinearAttention(_LinearAttention):
    """in_proj rows [q; k; v; g; low-rank decay input]; decay_up maps the latter to a decay per key channel."""
    _gated = True

    def __init__(self, width, args: MixerArgs, eps):
        super().__init__(width, args, eps, args.decay_rank)
        self.decay_up = nn.Linear(args.decay_rank, args.heads * args.dim, bias=True)
        self.norm = RMSNorm(args.vdim, eps)

    def mix(self, ws, pos, proj, y):
        a = self.args
        self._attend(ws, pos, proj, y, q_scale=a.dim ** -0.5, norm=self.norm.weight,
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

    def mix(self, ws, pos, proj, y):
        self._attend(ws, pos, proj, y, k_scale=self.args.dim ** -0.5, head_decay=self.log_decay, rope=self.rope)


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

    def mix(self, ws, pos, proj, y):
        a = self.args
        nq, cache = a.heads * a.dim, self.latents
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


class Mamba2(Mixer):
    """in_proj rows [z; x; B; C; dt].  Heads and state rows are padded to multiples of 16 with zeros; what a sequence carries
    is the state and the convolution's last inputs, a ring of `taps` rows in the compute type."""
    recurrent = True

    def __init__(self, width, args: MixerArgs, eps):
        P, N = pad16(args.vdim), pad16(args.state)
        inner, conv_cols = args.heads * P, args.heads * P + 2 * args.groups * N
        super().__init__(width, args, eps, inner + conv_cols + args.heads, y_cols=inner)
        self.P, self.N, self.inner, self.conv_cols = P, N, inner, conv_cols
        self.conv_weight = nn.Parameter(torch.zeros(self.conv_cols, args.taps))
        self.conv_bias = nn.Parameter(torch.zeros(self.conv_cols))
        self.dt_bias, self.a_log, self.d = (nn.Parameter(torch.zeros(args.heads)) for _ in range(3))
        self.norm = RMSNorm(self.inner, eps)

    def setup_cache(self, batch, length, dtype, device):
        a = self.args
        self.register_buffer("recurrent_state", torch.zeros(batch, a.heads, self.N, self.P, dtype=torch.float32, device=device),
                             persistent=False)
        self.register_buffer("conv_ring", torch.zeros(batch, a.taps, self.conv_cols, dtype=dtype, device=device), persistent=False)

    def states(self):
        return [self.recurrent_state, self.conv_ring]

    def _conv_bytes(self, B, S):
        return (B * S * self.conv_cols * self.in_proj.weight.element_size() + 255) // 256 * 256

    def scratch_bytes(self, B, S):
        if S == 1:
            return 0
        return self._conv_bytes(B, S) + _hip.ssd_scratch_bytes(B, S, self.args.heads, self.N, self.P, self.in_proj.weight.dtype)

    def cache_bytes_per_step(self, B, pos, itemsize):
        a = self.args
        return 2 * B * a.heads * a.state * a.vdim * 4 + B * a.taps * (a.heads * a.vdim + 2 * a.groups * a.state) * itemsize

    def mix(self, ws, pos, proj, y):
        a = self.args
        z, u, dt = proj[:, :self.inner], proj[:, self.inner:self.inner + self.conv_cols], proj[:, self.inner + self.conv_cols:]
        heads = (self.dt_bias, self.a_log, self.d, pos, self.recurrent_state, y)
        if ws.S == 1:
            _hip.ssd_step(z, u, dt, self.conv_weight, self.conv_bias, self.conv_ring, *heads, ws.B, a.heads, a.groups)
        else:
            n = self._conv_bytes(ws.B, ws.S)
            c = ws.scratch[:n].view(proj.dtype)[:ws.rows * self.conv_cols].view(ws.rows, self.conv_cols)
            _hip.causal_conv(u, self.conv_weight, self.conv_bias, self.conv_ring, pos, c, ws.B, ws.S)
            _hip.ssd(z, c, dt, *heads, ws.B, ws.S, a.heads, a.groups, scratch=ws.scratch[n:] if ws.scratch.numel() > n else None)
        _hip.parts_norm(y, self.norm.weight, a.norm_groups, a.heads, a.vdim, self.P, self.eps)


class GroupedAttention(Mixer):
    """in_proj rows [q; k; v] with biases, or q alone for a layer that reads another one's cache.  Heads are padded to multiples
    of 8 with zeros.  The cache holds rows [k of every kv head | v of every kv head], k rotated: [batch, length, columns]."""

    def __init__(self, width, args: MixerArgs, eps):
        dk, dv = pad8(args.dim), pad8(args.vdim)
        kv_cols = args.kv_heads * (dk + dv)
        super().__init__(width, args, eps, args.heads * dk + (kv_cols if args.kv_from is None else 0), y_cols=args.heads * dv,
                         bias=args.bias)
        self.dk, self.dv, self.kv_cols = dk, dv, kv_cols
        self._lender = None

    def lend(self, mixer: "GroupedAttention"):
        """Reads `mixer`'s keys and values."""
        assert (mixer.args.kv_heads, mixer.dk, mixer.dv) == (self.args.kv_heads, self.dk, self.dv)
        object.__setattr__(self, "_lender", mixer)      # (not a submodule: its parameters are the other layer's)

    @property
    def cache(self) -> Tensor:
        return self.kv if self._lender is None else self._lender.cache

    def setup_cache(self, batch, length, dtype, device):
        a = self.args
        if a.kv_from is None:
            self.register_buffer("kv", torch.zeros(batch, length, self.kv_cols, dtype=dtype, device=device), persistent=False)
        table = rotate_half_table(length, a.rot_dims, a.rot_base).to(device) if a.rot_dims else None
        self.register_buffer("rope", table, persistent=False)

    def scratch_bytes(self, B, S):
        if S > 1 or self.in_proj.weight.dtype != torch.bfloat16:
            return 0
        return _hip.window_decode_scratch_bytes(B, self.args.heads, self.args.kv_heads, self.dv, self.args.window, self.cache.shape[1])

    def cache_bytes_per_step(self, B, pos, itemsize):
        a = self.args
        return B * a.kv_heads * (a.dim + a.vdim) * itemsize * (min(pos + 1, a.window) + (a.kv_from is None))

    def mix(self, ws, pos, proj, y):
        a, cache = self.args, self.cache
        own = a.kv_from is None
        _hip.bias_rope_cache(proj, self.in_proj.bias, self.rope, pos, cache if own else (None, cache.shape[1]), ws.B, ws.S, a.heads,
                             a.kv_heads, self.dk, self.dv)
        q = proj[:, :a.heads * self.dk]
        if ws.S == 1 and q.dtype == torch.bfloat16:
            _hip.window_decode(q, cache, y, pos, ws.scratch, ws.B, a.heads, a.kv_heads, self.dk, self.dv, a.window, a.scale)
        else:
            L = cache.shape[1]
            _hip.window_attention(q, cache[:ws.B].view(ws.B * L, -1), y, pos, ws.B, ws.S, a.heads, self.dk, self.dv, a.window, L, L,
                                  a.scale, kv_heads=a.kv_heads)


MIXERS = {"gla": GatedLinearAttention, "retention": Retention, "latent_attention": LatentAttention, "mamba2": Mamba2,
          "attention": GroupedAttention}
