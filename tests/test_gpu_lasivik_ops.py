"""The kernels behind the Lasivik family, one by one, against the plain restatement in float64.

Inputs are made so that a fault shows: scores in which a single key stands out, placed just inside or just outside a
window or a chunk; decays from none at all to forgetting at once; sizes that are multiples of nothing."""
import math

import pytest
import torch

from oracle import lasivik_oracle as O

pytestmark = pytest.mark.gpu
DEV = "cuda"
BF, F32, F64 = torch.bfloat16, torch.float32, torch.float64
TOL = {F32: 3e-6, BF: 1.2e-2}      # of the largest value


@pytest.fixture(scope="module")
def hip():
    from gpt_fast import _hip

    _hip.load()
    return _hip


@pytest.fixture(autouse=True)
def _no_device_error():
    from gpt_fast import _hip

    yield
    _hip.raise_on_device_error()


def rnd(*shape, seed=0, dtype=F32):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g).to(dtype).to(DEV)


def close(got, want, dtype, what="", scale=1.0):
    want = want.to(DEV, F64)
    err = ((got.to(F64) - want).abs().max() / want.abs().max()).item()
    assert err <= TOL[dtype] * scale, f"{what}: {err:.2e} of the largest value"


d64 = lambda t: t.detach().cpu().to(F64)


# ------------------------------------------------------------------------------------------------ residual stream

@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("idx_dtype", [torch.int32, torch.int64])
def test_embed_residual(hip, dtype, idx_dtype):
    table = rnd(50, 72, dtype=dtype)
    idx = torch.tensor([3, 49, 0, 7, -1, 50], dtype=idx_dtype, device=DEV)
    x, xc = torch.empty(6, 72, device=DEV), torch.empty(6, 72, dtype=dtype, device=DEV)
    hip.embed_residual(table, idx, x, xc, 8.5)
    want = table[idx[:4].long()].float() * 8.5
    assert torch.equal(x[:4], want) and torch.equal(xc[:4], want.to(dtype)) and not x[4:].any()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("rows,dim,width", [(1, 8, 5), (7, 64, 64), (33, 200, 195), (3, 1024, 1024), (2, 4096, 4090), (2, 16384, 16384)])
def test_residual_rmsnorm(hip, dtype, rows, dim, width):
    x, d = rnd(rows, dim, seed=1), rnd(rows, dim, seed=2).to(dtype)
    gain = (0.3 * rnd(dim, seed=3)).to(dtype)
    for t in (x, d, gain):
        t[..., width:] = 0
    xo, xc = torch.empty_like(x), torch.full((rows, dim), float("nan"), dtype=dtype, device=DEV)
    hip.residual_rmsnorm(x, 2.5, d, gain, xo, xc, 1e-5, width, gain_offset=1.0)
    r = 2.5 * d64(x) + d64(d)
    want = O.zero_centred_norm(r[:, :width], d64(gain)[:width], 1e-5)
    close(xo[:, :width], want, F32)
    assert torch.equal(xc, xo.to(dtype)) and not xo[:, width:].any()
    # in place, without an addend, gain as it is, one output
    hip.residual_rmsnorm(x, 1.0, None, gain, x, None, 1e-5, width)
    r = d64(x)      # (already normed once: compare with the norm of the original below)
    ref = O.rms(d64(rnd(rows, dim, seed=1))[:, :width], 1e-5) * d64(gain)[:width]
    close(x[:, :width], ref, F32)
    assert r.shape == x.shape


@pytest.mark.parametrize("dtype", [F32, BF])
def test_logit_cap(hip, dtype):
    l = rnd(5, 104, seed=4, dtype=dtype) * 30
    view, before = l[:, :99], l.clone()
    hip.logit_cap(view, 0.5, 15.0)
    close(view, 15.0 * torch.tanh(0.5 * d64(before)[:, :99] / 15.0), dtype, scale=0.5)
    assert torch.equal(l[:, 99:], before[:, 99:])
    hip.logit_cap(l, 2.0, 0.0)
    assert torch.equal(l[:, 99:], (before[:, 99:].float() * 2).to(dtype))


@pytest.mark.parametrize("M,N,K", [(1, 1, 1), (1, 100, 45), (3, 67, 51), (64, 64, 64), (65, 130, 200), (200, 33, 19)])
def test_linear_f32(hip, M, N, K):
    x, w = rnd(M, K + 3, seed=5)[:, :K], rnd(N, K, seed=6)
    out = torch.full((M, N + 5), float("nan"), device=DEV)
    hip.linear(x, w, out[:, :N])
    close(out[:, :N], d64(x) @ d64(w).T, F32)
    assert torch.isnan(out[:, N:]).all()


def test_swiglu_and_argmax_f32(hip):
    h = rnd(7, 2 * 51, seed=7) * 4
    out = torch.empty(7, 51, device=DEV)
    hip.swiglu(h, out)
    u, g = d64(h).chunk(2, -1)
    close(out, O.silu(g) * u, F32)
    l = rnd(3, 5001, seed=8)
    l[1, 4096] = l[1, 77] = 50.0
    idx = torch.empty(3, dtype=torch.int32, device=DEV)
    hip.argmax(l, idx)
    assert idx.tolist() == [int(l[0].argmax()), 77, int(l[2].argmax())]


# ------------------------------------------------------------------------------------------------ linear attention

class LinearCase:
    """q | k | v | g | low-rank input of B sequences of T tokens, and what the restatement makes of it."""

    def __init__(self, B, T, H, dk, dv, gated, dtype, seed=0, dims=0, bias=2.0, tau=4.0, decay=None, rank=6, norm=True):
        self.B, self.T, self.H, self.dk, self.dv, self.dtype, self.gated = B, T, H, dk, dv, dtype, gated
        nq, nv = H * dk, H * dv
        r = lambda *s, i=0: rnd(*s, seed=seed * 100 + i)
        cols = 2 * nq + 2 * nv + (rank if gated else 0)
        self.ld = (cols + 7) // 8 * 8
        self.proj = torch.full((B * T, self.ld), float("nan"), dtype=dtype, device=DEV)
        self.proj[:, :cols] = r(B * T, cols).to(dtype)
        self.norm = (1 + 0.2 * r(dv, i=1)).to(dtype) if norm else None
        self.kw = dict(q_scale=0.7, k_scale=1.3, norm=self.norm)
        if gated:
            a2, b = r(nq, rank, i=2).to(dtype), (bias + r(nq, i=3)).to(dtype)
            self.kw["gate"] = (a2, b, tau)
        else:
            decay = [0.9, 0.99, 0.999, 0.5][:H] if decay is None else decay
            self.decay = torch.tensor(decay, dtype=F64)
            self.kw["head_decay"] = torch.tensor([math.log(d) if d > 0 else -math.inf for d in decay], dtype=F32, device=DEV)
        if dims:
            from gpt_fast.mixers import rotate_half_table

            self.kw["rope"] = rotate_half_table(4 * T + 64, dims, 100.0).to(DEV)
        self.dims, self.rank = dims, rank
        self.state = torch.full((B + 1, H, dk, dv), float("nan"), device=DEV)   # (what it holds before position 0 is nobody's)

    def want(self, pos0=0, states=None):
        B, T, H, dk, dv = self.B, self.T, self.H, self.dk, self.dv
        nq, nv = H * dk, H * dv
        P = d64(self.proj).view(B, T, -1)
        outs, ends = [], []
        for b in range(B):
            q, k = P[b, :, :nq].view(T, H, dk), P[b, :, nq:2 * nq].view(T, H, dk)
            v, g = P[b, :, 2 * nq:2 * nq + nv].view(T, H, dv), P[b, :, 2 * nq + nv:2 * nq + 2 * nv]
            if self.dims:
                at = torch.arange(pos0, pos0 + T)
                q, k = (O.rotate_half(x, at, self.dims, 100.0) for x in (q, k))
            if self.gated:
                a2, bias, tau = self.kw["gate"]
                t = P[b, :, 2 * nq + 2 * nv:2 * nq + 2 * nv + self.rank]
                a = O.gla_decay(t, torch.eye(self.rank, dtype=F64), d64(a2), d64(bias), tau).view(T, H, dk)
            else:
                a = self.decay[None, :, None].expand(T, H, dk)
            o, S = O.recurrence(q * self.kw["q_scale"], k * self.kw["k_scale"], v, a, None if states is None else states[b])
            o = O.rms(o, 1e-5)
            if self.norm is not None:
                o = o * d64(self.norm)
            outs.append(o.reshape(T, nv) * O.silu(g))
            ends.append(S)
        return torch.stack(outs), torch.stack(ends)

    def run(self, hip, cuts, pos0=0):
        """In portions of the sizes `cuts`; y [B, T, H dv]."""
        B, T, nv = self.B, self.T, self.H * self.dv
        P = self.proj.view(B, T, -1)
        ys, at = [], 0
        for n in cuts:
            y = torch.full((B * n, (nv + 7) // 8 * 8), float("nan"), dtype=self.dtype, device=DEV)
            need = hip.linear_attention_scratch_bytes(B, n, self.H, self.dk, self.dv, self.gated)
            scratch = torch.empty(need, dtype=torch.uint8, device=DEV) if need else None
            pos = torch.arange(pos0 + at, pos0 + at + n, dtype=torch.int32, device=DEV)
            hip.linear_attention(P[:, at:at + n].reshape(B * n, -1).contiguous(), y, self.state, pos, B, n, self.H, self.dk,
                                 self.dv, 1e-5, scratch=scratch, **self.kw)
            assert torch.isnan(y[:, nv:].float()).all(), "columns beyond the heads were written"
            ys.append(y[:, :nv].view(B, n, nv))
            at += n
        assert at == T
        return torch.cat(ys, 1)


SHAPES = [  # H, dk, dv
    (1, 8, 8), (2, 16, 32), (3, 24, 40), (2, 32, 16), (2, 48, 64), (1, 64, 33), (2, 128, 128), (1, 128, 256), (1, 256, 64),
    (3, 13, 9), (2, 22, 100), (1, 250, 255)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("gated", [True, False])
@pytest.mark.parametrize("H,dk,dv", SHAPES)
def test_linear_attention_sizes(hip, H, dk, dv, gated, dtype):
    dims = 0 if gated else (dk // 2 * 2 if dk < 64 else 32)
    c = LinearCase(2, 37, H, dk, dv, gated, dtype, seed=dk, dims=dims, norm=gated)
    want, S = c.want()
    close(c.run(hip, [37]), want, dtype, "prompt", 4)
    close(c.state[:2], S, F32 if dtype == F32 else BF, "state", 4)
    assert torch.isnan(c.state[2]).all()
    close(c.run(hip, [1] * 37), want, dtype, "token by token", 4)
    close(c.state[:2], S, F32 if dtype == F32 else BF, "state", 4)


@pytest.mark.parametrize("gated", [True, False])
@pytest.mark.parametrize("cuts", [[1], [2], [15], [16], [17], [2, 3, 12, 16, 1, 1, 17, 2], [31, 33, 32, 1, 63], [130, 200, 2]])
def test_linear_attention_portions(hip, cuts, gated):
    """Portions of any size, from a position of their own, continue the state exactly where it was left."""
    T = sum(cuts)
    c = LinearCase(2, T, 2, 40, 24, gated, F32, seed=T, dims=0 if gated else 16, bias=4.0)
    want, S = c.want()
    close(c.run(hip, cuts), want, F32, "outputs", 4)
    close(c.state[:2], S, F32, "state", 4)


def test_linear_attention_restarts_at_position_zero_and_continues_elsewhere(hip):
    c = LinearCase(2, 20, 2, 16, 24, False, F32, seed=9, dims=16)
    want, S = c.want()
    for _ in range(2):                                   # the second sequence finds the first one's state in its slot
        close(c.run(hip, [20]), want, F32)
    later, _ = c.want(pos0=20, states=S)
    close(c.run(hip, [7, 12, 1], pos0=20), later, F32)


@pytest.mark.parametrize("B,T,H", [(1, 64, 1), (1, 128, 1), (1, 777, 2), (3, 300, 2)])
def test_linear_attention_segments(hip, B, T, H):
    """Few heads and long prompts: segments side by side.  Slow decays, so that every segment matters to every later one."""
    for gated in (True, False):
        c = LinearCase(B, T, H, 32, 48, gated, F32, seed=T, dims=0 if gated else 32, bias=6.0, tau=16.0, decay=[0.9995, 0.998][:H])
        want, S = c.want()
        close(c.run(hip, [T]), want, F32, "outputs", 8)
        close(c.state[:B], S, F32, "state", 8)


@pytest.mark.parametrize("gated,kw", [
    (True, dict(bias=-3.0, tau=0.05)), (True, dict(bias=0.0, tau=0.2)), (True, dict(bias=-1.0, tau=1.0)),
    (True, dict(bias=30.0, tau=1.0)), (False, dict(decay=[0.0, 1e-30, 0.03])), (False, dict(decay=[0.12, 1.0, 0.3]))])
@pytest.mark.parametrize("T", [1, 16, 50])
def test_linear_attention_steep_and_absent_decay(hip, gated, kw, T):
    """From forgetting everything at once to forgetting nothing: the factors of a chunk must not leave fp32's range."""
    c = LinearCase(1, T, 3, 24, 16, gated, F32, seed=11, **kw)
    want, S = c.want()
    close(c.run(hip, [T]), want, F32, "prompt", 8)
    close(c.state[:1], S, F32, "state", 8)
    close(c.run(hip, [1] * T), want, F32, "token by token", 8)


@pytest.mark.parametrize("T,far", [(100, 0), (100, 15), (100, 16), (333, 5), (333, 200)])
def test_linear_attention_recalls_one_far_key(hip, T, far):
    """One key a thousand times the others: the last output is that token's value (normed and gated)."""
    c = LinearCase(1, T, 1, 32, 24, False, F32, seed=13, dims=32, decay=[0.9999], norm=False)
    c.proj[far, 32:64] *= 1000
    q = c.proj[T - 1, :32]
    # a query that meets the rotated key head on
    from gpt_fast.mixers import rotate_half_table  # noqa: F401
    k = O.rotate_half(d64(c.proj[far:far + 1, 32:64]).view(1, 1, 32), torch.tensor([far - (T - 1)]), 32, 100.0).view(-1)
    q.copy_(k.float() / 1000)
    y = c.run(hip, [T])[0, -1]
    g = d64(c.proj[T - 1, 64 + 24:64 + 48])
    want = O.rms(d64(c.proj[far, 64:64 + 24]), 1e-5) * O.silu(g)
    sign = (d64(y) * want).sum().sign()
    assert sign > 0
    close(y, want, F32, scale=2000)       # (the other keys' contributions are a few thousandths)
    close(c.run(hip, [T - 40] + [1] * 40)[0, -1], d64(y), F32, scale=4)


def test_linear_attention_reports_a_position_outside_the_rotation_table(hip):
    c = LinearCase(1, 4, 2, 16, 16, False, F32, dims=16)
    c.kw["rope"] = c.kw["rope"][:6].contiguous()
    for cuts in ([4], [1, 1, 1, 1]):
        c.run(hip, cuts, pos0=4)
        with pytest.raises(hip.LadderHipError):
            hip.raise_on_device_error(DEV)


# ------------------------------------------------------------------------------------------------ windowed latent attention

class LatentCase:
    def __init__(self, B, T, H, dk, dv, rank, window, dtype, seed=0, Smax=None):
        self.B, self.T, self.H, self.dk, self.dv, self.rank, self.window, self.dtype = B, T, H, dk, dv, rank, window, dtype
        self.ldr = (rank + 7) // 8 * 8
        self.Smax = Smax or T + 5
        r = lambda *s, i=0: rnd(*s, seed=seed * 100 + i)
        self.q = (1.5 * r(B, T, H * dk)).to(dtype)
        self.c = r(B, T, rank, i=1).to(dtype)
        self.gain = (1 + 0.2 * r(rank, i=2)).to(dtype)
        self.up = torch.zeros(H * (dk + dv), self.ldr, dtype=dtype, device=DEV)
        self.up[:, :rank] = (r(H * (dk + dv), rank, i=3) / math.sqrt(rank)).to(dtype)
        self.scale = dk ** -0.5
        self.cache = torch.full((B + 1, self.Smax, self.ldr), 50.0, dtype=dtype, device=DEV)   # stale rows stand out

    def want(self, lo=0):
        outs = []
        for b in range(self.B):
            lat = O.rms(d64(self.c[b]), 1e-5) * d64(self.gain)
            up = d64(self.up)[:, :self.rank]
            nq = self.H * self.dk
            k, v = (lat @ up[:nq].T).view(self.T, self.H, self.dk), (lat @ up[nq:].T).view(self.T, self.H, self.dv)
            at = torch.arange(self.T)
            outs.append(O.windowed_softmax_attention(d64(self.q[b]).view(self.T, self.H, self.dk)[lo:], k, v, at[lo:], at,
                                                     self.window, self.scale).reshape(self.T - lo, -1))
        return torch.stack(outs)

    def portion(self, hip, at, n, absorb):
        B, H, dk, dv = self.B, self.H, self.dk, self.dv
        nq = H * dk
        pos = torch.arange(at, at + n, dtype=torch.int32, device=DEV)
        ldq = (nq + 7) // 8 * 8
        q = torch.zeros(B * n, ldq, dtype=self.dtype, device=DEV)
        q[:, :nq] = self.q[:, at:at + n].reshape(B * n, nq)
        c = self.c[:, at:at + n].reshape(B * n, self.rank).contiguous()
        y = torch.full((B * n, (H * dv + 7) // 8 * 8), float("nan"), dtype=self.dtype, device=DEV)
        if absorb:
            need = hip.latent_attention_scratch_bytes(B, n, H, self.ldr, self.window, self.Smax)
            scratch = torch.full((need,), 255, dtype=torch.uint8, device=DEV)       # NaNs everywhere
            hip.latent_attention(q[:, :nq], self.up[:nq], self.up[nq:], self.cache, y, pos, scratch, B, n, H, dk, dv, self.window,
                                 self.scale, new=(c, self.gain, self.rank, 1e-5))
        else:
            hip.latent_update(c, self.gain, pos, self.cache, B, n, self.rank, 1e-5)
            nk = min(n + self.window - 1, self.Smax)
            rows = torch.empty(B, nk, self.ldr, dtype=self.dtype, device=DEV)
            hip.latent_window(self.cache, pos, rows, B, self.window)
            cols = H * (dk + dv)
            kv = torch.empty(B * nk, (cols + 7) // 8 * 8, dtype=self.dtype, device=DEV)[:, :cols]
            hip.linear(rows.view(B * nk, -1), self.up, kv)
            hip.window_attention(q[:, :nq], kv, y, pos, B, n, H, dk, dv, self.window, nk, self.Smax, self.scale)
        assert torch.isnan(y[:, H * dv:].float()).all()
        return y[:, :H * dv].view(B, n, H * dv)

    def run(self, hip, cuts, absorb):
        ys, at = [], 0
        for n in cuts:
            ys.append(self.portion(hip, at, n, absorb(n) if callable(absorb) else absorb))
            at += n
        return torch.cat(ys, 1)


LATENT = [  # H, dk, dv, rank, window, T
    (1, 32, 32, 32, 1, 45), (2, 16, 48, 24, 2, 70), (3, 32, 24, 40, 31, 100), (4, 64, 64, 64, 32, 150), (2, 64, 128, 72, 33, 150),
    (2, 128, 64, 128, 64, 200), (5, 19, 11, 21, 7, 60), (33, 16, 16, 136, 65, 140), (2, 128, 128, 512, 100, 300),
    (4, 96, 80, 256, 500, 260), (1, 160, 200, 64, 17, 50)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,dk,dv,rank,window,T", LATENT)
def test_latent_attention_sizes_and_windows(hip, H, dk, dv, rank, window, T, dtype):
    c = LatentCase(2, T, H, dk, dv, rank, window, dtype, seed=T)
    want = c.want()
    tol = 2.0 if dtype == BF else 4.0
    close(c.run(hip, [T], False), want, dtype, "whole prompt", tol)
    close(c.run(hip, [T - 20] + [3] * 4 + [8], lambda n: n <= 8), want, dtype, "prompt, then portions on the latents", tol)
    close(c.run(hip, [2, 17, T - 39, 20], lambda n: n <= 8), want, dtype, "portions", tol)
    close(c.run(hip, [T - 12] + [1] * 12, lambda n: n == 1)[:, -12:], want[:, -12:], dtype, "decoded", tol)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("window", [1, 16, 31, 32, 33, 64, 96, 129])
def test_a_standing_out_key_just_inside_and_just_outside_the_window(hip, window, dtype):
    """One latent meets every query head on and takes all the weight: it counts for exactly `window` queries."""
    H, d, rank, T, at = 2, 64, 64, 300, 100
    c = LatentCase(1, T, H, d, d, rank, window, dtype, seed=window)
    c.up[:H * d] = torch.cat([torch.eye(rank)] * H).to(DEV, dtype)           # k = the latent itself
    spike = torch.zeros(rank, device=DEV)
    spike[3] = 1.0
    c.c[0, at] = spike.to(dtype)
    c.c[0, :, 3] = torch.where(torch.arange(T, device=DEV) == at, 1.0, -0.1).to(dtype)
    c.q.zero_()
    c.q.view(1, T, H, d)[..., 3] = 20.0
    nq = H * d
    v = (O.rms(d64(c.c[0, at]), 1e-5) * d64(c.gain)) @ d64(c.up[nq:]).T
    for run in (c.run(hip, [T], False), c.run(hip, [at - 1] + [1] * (T - at + 1), lambda n: n <= 8), c.run(hip, [64, 37, 63, 136], False)):
        dist = (run[0].to(F64).cpu() - v).abs().max(-1).values / v.abs().max()
        near = dist < 0.05
        assert near.nonzero().flatten().tolist() == list(range(at, at + window)), window


def test_latents_land_at_their_positions_only(hip):
    c = LatentCase(2, 12, 2, 16, 16, 20, 4, F32)
    c.run(hip, [5, 1, 6], lambda n: n == 1)
    lat = torch.stack([O.rms(d64(c.c[b]), 1e-5) * d64(c.gain) for b in range(2)])
    close(c.cache[:2, :12, :20], lat, F32)
    assert not c.cache[:2, :12, 20:].any()
    assert (c.cache[:2, 12:] == 50).all() and (c.cache[2] == 50).all()


def test_latent_position_outside_the_cache_is_reported(hip):
    c = LatentCase(1, 12, 2, 16, 16, 16, 4, BF, Smax=8)
    for absorb in (True, False):
        c.portion(hip, 5, 4, absorb)
        with pytest.raises(hip.LadderHipError):
            hip.raise_on_device_error(DEV)
