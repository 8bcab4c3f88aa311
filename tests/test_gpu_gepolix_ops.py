"""The kernels behind the Gepolix family, one by one, against the plain restatement in float64.

Inputs are made so that a fault shows: one key or one token that stands out, placed just inside or just outside a window, a chunk
or a range; states from hardly forgetting to forgetting at once; choices of experts that are far apart; sizes of every kind."""
import math

import pytest
import torch

from oracle import gepolix_oracle as O

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
at_pos = lambda lo, n: torch.arange(lo, lo + n, dtype=torch.int32, device=DEV)


# ------------------------------------------------------------------------------------------------ residual and norm

@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("rows,dim,top", [(1, 8, 1), (5, 72, 3), (33, 1024, 2), (3, 4096, 9)])
def test_residual_tanh(hip, dtype, rows, dim, top):
    x, d = rnd(rows, dim, seed=1), rnd(rows, dim, seed=2, dtype=dtype)
    w, b, alpha = rnd(dim, seed=3, dtype=dtype), rnd(dim, seed=4, dtype=dtype), torch.tensor([0.625], dtype=dtype, device=DEV)
    eo, ew = rnd(rows * top, dim, seed=5, dtype=dtype), torch.softmax(rnd(rows, top, seed=6), -1)
    norm = lambda r: O.dynamic_tanh(r, d64(alpha), d64(w), d64(b))
    add = (d64(ew)[:, :, None] * d64(eo).view(rows, top, dim)).sum(1)
    for dd, experts in ((None, None), (d, None), (None, (eo, ew)), (d, (eo, ew))):
        xo, xc = torch.empty_like(x), torch.empty(rows, dim, dtype=dtype, device=DEV)
        hip.residual_tanh(x, dd, alpha, w, b, xo, xc, experts)
        r = d64(x) + (0 if dd is None else d64(d)) + (0 if experts is None else add)
        close(xo, r, F32)
        close(xc, norm(r), dtype)
    keep = x.clone()
    hip.residual_tanh(x, None, alpha, w, b, None, xc)          # the norm alone
    assert torch.equal(x, keep)
    close(xc, norm(d64(x)), dtype)
    hip.residual_tanh(x, d, alpha, w, b, x, None)              # in place, no norm
    close(x, d64(keep) + d64(d), F32)


@pytest.mark.parametrize("M", [1, 2, 8, 9, 16, 30, 64])
@pytest.mark.parametrize("N,K,top", [(72, 200, 0), (2048, 136, 3), (5000, 1000, 1)])
def test_linear_residual_tanh(hip, M, N, K, top):
    h, w = rnd(M, K + 8, seed=1, dtype=BF)[:, :K], (rnd(N, K, seed=2) / K ** 0.5).to(BF)
    x, gain, bias, alpha = rnd(M, N, seed=3), rnd(N, seed=4, dtype=BF), rnd(N, seed=5, dtype=BF), torch.tensor([0.75], dtype=BF, device=DEV)
    experts = (rnd(M * top, N, seed=6, dtype=BF), torch.softmax(rnd(M, top, seed=7), -1)) if top else None
    want = d64(x) + d64(h) @ d64(w).T
    if top:
        want += (d64(experts[1])[:, :, None] * d64(experts[0]).view(M, top, N)).sum(1)
    out = torch.full((M, N), float("nan"), dtype=BF, device=DEV)
    hip.linear_residual_tanh(h, w, x, alpha, gain, bias, out, experts)
    close(x, want, F32)
    close(out, O.dynamic_tanh(want, d64(alpha), d64(gain), d64(bias)), BF)


# ------------------------------------------------------------------------------------------------ convolution

@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 8])
def test_causal_conv_in_portions(hip, dtype, taps):
    B, T, Cc = 3, 75, 48
    wide = rnd(B, T, Cc + 16, seed=1, dtype=dtype)
    w, b = rnd(Cc, taps, seed=2, dtype=dtype), rnd(Cc, seed=3, dtype=dtype)
    ring = torch.full((B + 1, taps, Cc), float("nan"), dtype=dtype, device=DEV)   # whatever an earlier sequence left
    want = torch.stack([O.silu(O.causal_conv(d64(wide[i, :, 8:8 + Cc]), d64(w), d64(b), torch.zeros(taps - 1, Cc, dtype=F64))) for i in range(B)])
    for cuts in ([75], [1] * 20 + [55], [2, 3, 1, 40, 16, 1, 1, 11], [17, 58], [32, 43]):
        lo = 0
        for n in cuts:
            u = wide[:, lo:lo + n].contiguous().view(B * n, -1)[:, 8:8 + Cc]
            out = torch.full((B * n, Cc + 8), float("nan"), dtype=dtype, device=DEV)
            hip.causal_conv(u, w, b, ring, at_pos(lo, n), out[:, :Cc], B, n)
            close(out[:, :Cc].reshape(B, n, Cc), want[:, lo:lo + n], dtype, (cuts, lo))
            assert torch.isnan(out[:, Cc:]).all()
            lo += n


# ------------------------------------------------------------------------------------------------ state space

class Ssm:
    """Inputs of B sequences of T tokens and what the restatement makes of them (convolution aside)."""

    def __init__(self, B, T, H, G, N, P, dtype, seed=0, a_log=0.0, dt_bias=-1.0):
        self.B, self.T, self.H, self.G, self.N, self.P, self.dtype = B, T, H, G, N, P, dtype
        Cc = H * P + 2 * G * N
        self.u = rnd(B, T, Cc, seed=seed, dtype=dtype)
        self.rest = rnd(B, T, H * P + H + 8 - H % 8, seed=seed + 1, dtype=dtype)       # z | dt
        s = lambda k, around: (around + rnd(H, seed=seed + k)).to(dtype)
        self.heads = (s(2, dt_bias), s(3, a_log), s(4, 0.0))                          # dt_bias, A_log, D
        self.state = torch.full((B, H, N, P), float("nan"), device=DEV)

    def want(self, u=None):
        H, G, N, P = self.H, self.G, self.N, self.P
        db, al, D = (d64(t) for t in self.heads)
        ys, Ss = [], []
        for i in range(self.B):
            x, Bm, Cm = d64((self.u if u is None else u)[i]).split([H * P, G * N, G * N], -1)
            x, T = x.view(-1, H, P), self.T
            z, dt = d64(self.rest[i]).split([H * P, self.rest.shape[-1] - H * P], -1)
            y, S = O.selective_scan(x, Bm.view(T, G, N), Cm.view(T, G, N), O.softplus(dt[:, :H] + db), al, torch.zeros(H, N, P, dtype=F64))
            ys.append(((y + D[:, None] * x).reshape(T, H * P)) * O.silu(z))
            Ss.append(S)
        return torch.stack(ys), torch.stack(Ss)

    def run(self, hip, cuts, conv=None):
        """cuts: portion sizes; 0 stands for one token through the decode kernel (conv: its weights)."""
        out, lo = [], 0
        for c in cuts:
            n = max(c, 1)
            u, r = self.u[:, lo:lo + n].contiguous().view(self.B * n, -1), self.rest[:, lo:lo + n].contiguous().view(self.B * n, -1)
            z, dt = r[:, :self.H * self.P], r[:, self.H * self.P:]
            y = torch.full((self.B * n, self.H * self.P + 8), float("nan"), dtype=self.dtype, device=DEV)
            args = (*self.heads, at_pos(lo, n), self.state, y[:, :self.H * self.P], self.B)
            if c == 0:
                hip.ssd_step(z, u, dt, *conv, *args, self.H, self.G)
            else:
                need = hip.ssd_scratch_bytes(self.B, n, self.H, self.N, self.P, self.dtype)
                hip.ssd(z, u, dt, *args, n, self.H, self.G, scratch=torch.empty(need, dtype=torch.uint8, device=DEV) if need else None)
            assert torch.isnan(y[:, self.H * self.P:]).all()
            out.append(y[:, :self.H * self.P].reshape(self.B, n, -1))
            lo += n
        assert lo == self.T
        return torch.cat(out, 1)


SSM_SIZES = [(1, 1, 16, 16), (4, 2, 48, 48), (2, 1, 128, 64), (3, 3, 32, 128), (2, 2, 256, 16), (2, 1, 64, 80), (2, 1, 24, 40), (6, 2, 8, 8)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,G,N,P", SSM_SIZES)
@pytest.mark.parametrize("a_log,dt_bias", [(0.0, -1.0), (4.0, 3.0), (-4.0, -4.0)])
def test_ssd(hip, dtype, H, G, N, P, a_log, dt_bias):
    c = Ssm(2, 200, H, G, N, P, dtype, a_log=a_log, dt_bias=dt_bias)
    y, S = c.want()
    for cuts in ([200], [64, 64, 72], [1, 2, 61, 65, 2, 69], [63, 1, 136]):
        close(c.run(hip, cuts), y, dtype, cuts)
        close(c.state, S, dtype, cuts, scale=1.0 if dtype == F32 else 0.1)      # (nothing rounds the state to 16 bits)


def test_ssd_in_segments(hip):
    """Few heads: the prompt's segments run side by side, from the state an earlier portion left."""
    for T, cuts in ((1100, [1100]), (1400, [137, 1263]), (900, [640, 260])):
        c = Ssm(1, T, 2, 1, 128, 64, BF, seed=T, a_log=-3.0)
        y, S = c.want()
        assert hip.ssd_scratch_bytes(1, T, 2, 128, 64, BF) > 0
        close(c.run(hip, cuts), y, BF, cuts)
        close(c.state, S, BF, cuts, scale=0.1)


@pytest.mark.parametrize("far", [0, 1, 63, 64, 500])
def test_a_token_far_back_is_recalled(hip, far):
    """One token's input dwarfs the others'; the state hardly forgets; what a much later token reads is that input."""
    T, H, G, N, P = 700, 2, 1, 48, 48
    c = Ssm(1, T, H, G, N, P, BF, a_log=-7.0, dt_bias=-2.0)
    c.u[0, far, :H * P] *= 200
    y, S = c.want()
    without = c.u.clone()
    without[0, far] = 0
    y0, _ = c.want(without)
    shown = ((y - y0)[0, 650:].abs().max() / y.abs()[0, 650:].max()).item()
    assert shown > 0.5
    for cuts in ([700], [far + 1, 699 - far], [300, 2, 398]):
        got = c.run(hip, cuts)
        close(got[:, 650:], y[:, 650:], BF, cuts)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,G,N,P", SSM_SIZES)
@pytest.mark.parametrize("taps", [1, 4])
def test_ssd_step_with_its_convolution(hip, dtype, H, G, N, P, taps):
    c = Ssm(3, 40, H, G, N, P, dtype)
    Cc = c.u.shape[-1]
    w, b = rnd(Cc, taps, seed=8, dtype=dtype), rnd(Cc, seed=9, dtype=dtype)
    ring = torch.full((3, taps, Cc), float("nan"), dtype=dtype, device=DEV)
    u = torch.stack([O.silu(O.causal_conv(d64(c.u[i]), d64(w), d64(b), torch.zeros(taps - 1, Cc, dtype=F64))) for i in range(3)])
    y, S = c.want(u)
    close(c.run(hip, [0] * 40, (w, b, ring)), y, dtype)
    close(c.state, S, dtype, scale=1.0 if dtype == F32 else 0.1)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("heads,P,PP,parts", [(4, 16, 16, 1), (4, 16, 16, 4), (4, 9, 16, 3), (6, 24, 32, 2), (64, 64, 64, 8), (3, 7, 16, 7)])
def test_parts_norm(hip, dtype, heads, P, PP, parts):
    rows = 5
    y = torch.zeros(rows, heads * PP + 8, dtype=dtype, device=DEV)
    gain = torch.zeros(heads, PP, dtype=dtype, device=DEV)
    y[:, :heads * PP].view(rows, heads, PP)[:, :, :P] = 3 * rnd(rows, heads, P, seed=1).to(dtype)
    gain[:, :P] = rnd(heads, P, seed=2).to(dtype)
    inner = lambda t: t[:, :heads * PP].view(rows, heads, PP)[:, :, :P].reshape(rows, -1)
    want = O.parts_norm(d64(inner(y)), parts, 1e-5) * d64(gain[:, :P].reshape(-1))
    hip.parts_norm(y, gain.view(-1), parts, heads, P, PP, 1e-5)
    close(inner(y), want, dtype)
    y[:, :heads * PP].view(rows, heads, PP)[:, :, :P] = 0
    assert not y.any()


# ------------------------------------------------------------------------------------------------ attention

@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,G,dk,dv,rot", [(4, 2, 16, 24, 16), (3, 3, 24, 16, 10), (8, 1, 64, 64, 2), (6, 2, 40, 8, 0)])
def test_bias_rope_cache(hip, dtype, H, G, dk, dv, rot):
    from gpt_fast.mixers import rotate_half_table

    B, S, L, lo = 2, 9, 40, 21
    cols = H * dk + G * (dk + dv)
    proj, bias = rnd(B * S, cols + 8, seed=1, dtype=dtype), rnd(cols, seed=2, dtype=dtype)
    before = proj.clone()
    cache = torch.full((B + 1, L, G * (dk + dv) + 8), float("nan"), dtype=dtype, device=DEV)
    rope = rotate_half_table(L, rot, 100.0).to(DEV) if rot else None
    hip.bias_rope_cache(proj, bias, rope, at_pos(lo, S), cache, B, S, H, G, dk, dv)
    x = (d64(before[:, :cols]) + d64(bias)).view(B, S, cols)
    turn = lambda t, n: O.rotate_half(t.reshape(S, n, dk), torch.arange(lo, lo + S), rot, 100.0).reshape(S, n * dk)
    for b in range(B):
        q, k, v = x[b].split([H * dk, G * dk, G * dv], -1)
        close(proj.view(B, S, -1)[b, :, :H * dk], turn(q, H), dtype)
        close(cache[b, lo:lo + S, :G * dk], turn(k, G), dtype)
        close(cache[b, lo:lo + S, G * dk:G * (dk + dv)], v, dtype)
    assert torch.isnan(cache[:, :lo]).all() and torch.isnan(cache[:, lo + S:]).all() and torch.isnan(cache[B]).all()
    assert torch.isnan(cache[:B, lo:lo + S, G * (dk + dv):]).all()
    assert torch.equal(proj[:, H * dk:], before[:, H * dk:])
    # queries alone, no bias
    q = before.clone()
    hip.bias_rope_cache(q[:, :H * dk], None, rope, at_pos(lo, S), (None, L), B, S, H, G, dk, dv)
    close(q.view(B, S, -1)[0, :, :H * dk], turn(d64(before).view(B, S, -1)[0, :, :H * dk], H), dtype)
    assert torch.equal(q[:, H * dk:], before[:, H * dk:])


def test_a_position_outside_the_cache_is_reported(hip):
    proj, cache = rnd(2, 64, dtype=BF), torch.zeros(1, 8, 32, dtype=BF, device=DEV)
    before = proj.clone()
    hip.bias_rope_cache(proj, None, None, at_pos(7, 2), cache, 1, 2, 2, 1, 16, 16)
    with pytest.raises(hip.LadderHipError):
        hip.raise_on_device_error()
    assert torch.equal(proj[1], before[1]) and not cache[0, :7].any()


ATTENTION = [(4, 2, 16, 24, 7), (8, 2, 64, 64, 33), (3, 3, 40, 8, 20), (8, 1, 128, 128, 70), (20, 1, 64, 48, 64), (6, 3, 32, 136, 1), (4, 4, 8, 8, 1000),
             (2, 1, 200, 256, 130)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,G,dk,dv,window", ATTENTION)
def test_window_attention_over_a_cache(hip, dtype, H, G, dk, dv, window):
    """Portions of every size; in each, one key stands out for each query: the last it sees, or the first it does not."""
    B, L, T = 2, 320, 300
    cache = rnd(B, L, G * (dk + dv), seed=1, dtype=dtype)
    q = rnd(B, T, H * dk, seed=2, dtype=dtype)
    for i in range(T):        # an edge key, alternately just inside and just outside the window
        j = i - window + 1 - (i % 2)
        if j >= 0:
            for g in range(G):
                lead = q[:, i].view(B, H, dk)[:, g * (H // G)]
                cache[:, j, g * dk:(g + 1) * dk] = (lead * 3).to(dtype)
    want = torch.stack([O.grouped_window_attention(d64(q[b]).view(T, H, dk), d64(cache[b, :T, :G * dk]).reshape(T, G, dk),
                                                   d64(cache[b, :T, G * dk:]).reshape(T, G, dv), 0, window, dk ** -0.5).reshape(T, -1) for b in range(B)])
    cache[:, T:] = 3e4        # beyond the last position: must not be seen
    kv = cache.view(B * L, -1)
    for cuts in ([300], [2, 61, 3, 64, 33, 137], [128, 172], [16, 17, 267]):
        lo = 0
        for n in cuts:
            rows = q[:, lo:lo + n].contiguous().view(B * n, -1)
            y = torch.full((B * n, H * dv + 8), float("nan"), dtype=dtype, device=DEV)
            hip.window_attention(rows, kv, y[:, :H * dv], at_pos(lo, n), B, n, H, dk, dv, window, L, L, dk ** -0.5, kv_heads=G)
            close(y[:, :H * dv].reshape(B, n, -1), want[:, lo:lo + n], dtype, (cuts, lo))
            assert torch.isnan(y[:, H * dv:]).all()
            lo += n
    if dtype == BF:
        for p in sorted({0, 1, window - 1, window, window + 1, 127, 128, 255, 299} & set(range(T))):
            y = torch.full((B, H * dv + 8), float("nan"), dtype=dtype, device=DEV)
            need = hip.window_decode_scratch_bytes(B, H, G, dv, window, L)
            scratch = torch.full((need // 4,), float("nan"), device=DEV)
            hip.window_decode(q[:, p].contiguous(), cache, y[:, :H * dv], at_pos(p, 1), scratch, B, H, G, dk, dv, window, dk ** -0.5)
            close(y[:, :H * dv].reshape(B, 1, -1), want[:, p:p + 1], dtype, p)
            assert torch.isnan(y[:, H * dv:]).all()


def test_window_decode_cuts_long_windows_into_ranges(hip):
    B, H, G, d, L = 1, 4, 1, 64, 5000
    cache, q = rnd(B, L, 2 * d, seed=1, dtype=BF), rnd(B, H * d, seed=2, dtype=BF)
    for window in (4999, 4096, 130):
        for p in (4998, 4095, 129, 64):
            for edge in (p, max(0, p - window + 1)):
                c = cache.clone()
                c[:, edge, :d] = (q.view(B, H, d)[:, 0] * 4).to(BF)
                y, scratch = torch.empty(B, H * d, dtype=BF, device=DEV), torch.empty(hip.window_decode_scratch_bytes(B, H, G, d, window, L), dtype=torch.uint8, device=DEV)
                hip.window_decode(q, c, y, at_pos(p, 1), scratch, B, H, G, d, d, window, d ** -0.5)
                want = O.grouped_window_attention(d64(q).view(1, H, d), d64(c[0, :p + 1, :d])[:, None], d64(c[0, :p + 1, d:])[:, None], p, window, d ** -0.5)
                close(y, want.reshape(1, -1), BF, (window, p, edge))


# ------------------------------------------------------------------------------------------------ experts

class Mix:
    def __init__(self, D, I, E, top, shared, dtype, seed=0):
        self.D, self.I, self.E, self.top, self.dtype = D, I, E, top, dtype
        s = lambda *shape, k, f=1.0: (rnd(*shape, seed=seed + k) * f / math.sqrt(shape[-1])).to(dtype)
        self.router, self.bias = s(E + (shared > 0), D, k=1, f=4.0), rnd(E, seed=seed + 2, dtype=dtype)
        self.w1, self.w2 = s(E, 2 * I, D, k=3, f=2.0), s(E, D, I, k=4)
        self.shared = shared
        self.counts = torch.zeros(E, dtype=torch.int32, device=DEV)

    def desc(self, hip, x, shared=None):
        rows = x.shape[0]
        self.out = torch.full((rows * self.top, self.D), float("nan"), dtype=self.dtype, device=DEV)
        self.ids, self.wts = torch.full((rows, self.top), -1, dtype=torch.int32, device=DEV), torch.full((rows, self.top), float("nan"), device=DEV)
        self.gate = torch.full((rows,), float("nan"), device=DEV)
        self.scratch = torch.full((hip.moe_scratch_bytes(rows, self.E, self.top, self.I, self.dtype),), 255, dtype=torch.uint8, device=DEV)
        return hip.moe_desc(x, self.router, self.bias, self.w1, self.w2, self.out, self.ids, self.wts, self.gate, self.counts, self.scratch, shared)

    def check(self, x, act=None, act_before=None):
        rows = x.shape[0]
        idx, w = O.route(d64(x), d64(self.router[:self.E]), d64(self.bias), self.top)
        near = torch.topk(d64(x) @ d64(self.router[:self.E]).T + d64(self.bias), min(self.top + 1, self.E), -1)[0]
        clear = (near[:, :-1] - near[:, 1:]).amin(-1) > 1e-4 if near.shape[1] > 1 else torch.ones(rows, dtype=torch.bool)
        assert clear.float().mean() > 0.9
        assert torch.equal(self.ids.cpu().long()[clear], idx[clear])
        close(self.wts[clear], w[clear], F32, scale=10)
        x64, w1, w2 = x.to(F64), self.w1.to(F64), self.w2.to(F64)
        got = self.out.view(rows, self.top, self.D)
        for k in range(self.top):
            e = self.ids[:, k].long()
            want = torch.empty(rows, self.D, dtype=F64, device=DEV)
            for i in e.unique().tolist():
                up, g = (x64[e == i] @ w1[i].T).chunk(2, -1)
                want[e == i] = (up * g * torch.sigmoid(g)) @ w2[i].T
            close(got[:, k], want, self.dtype, ("slot", k))
        assert not self.counts.any()
        if act is not None:
            f = torch.sigmoid(x64 @ self.router[self.E].to(F64))
            close(act, act_before.to(F64) * f[:, None], self.dtype)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("rows", [1, 2, 17, 64, 65, 300])
@pytest.mark.parametrize("D,I,E,top,shared", [(64, 32, 5, 2, 24), (72, 40, 1, 1, 0), (128, 16, 70, 9, 8), (256, 64, 16, 16, 0), (200, 24, 33, 3, 64)])
def test_mixture(hip, dtype, rows, D, I, E, top, shared):
    m = Mix(D, I, E, top, shared, dtype, seed=rows)
    x = rnd(rows, D + 8, seed=rows + 50, dtype=dtype)[:, :D]
    act = rnd(rows, shared + 8, seed=7, dtype=dtype)[:, :shared] if shared else None
    before = None if act is None else act.clone()
    hip.moe(m.desc(hip, x, act))
    m.check(x, act, before)


def test_mixture_of_many_tokens(hip):
    """Enough entries for the 256-row tiles and the sort in several launches, spread very unevenly."""
    for rows, D, I, E, top in ((5000, 256, 136, 24, 6), (2600, 512, 1024, 4, 2), (4000, 128, 1088, 8, 4)):
        m = Mix(D, I, E, top, 16, BF, seed=rows)
        m.bias[E // 2] += 6
        x, act = rnd(rows, D, seed=3, dtype=BF), rnd(rows, 16, seed=4, dtype=BF)
        before = act.clone()
        for _ in range(2):
            act.copy_(before)
            hip.moe(m.desc(hip, x, act))
            m.check(x, act, before)


@pytest.mark.parametrize("rows", [3, 70])
def test_every_token_chooses_the_same_experts_and_equals_go_to_the_lower(hip, rows):
    m = Mix(64, 32, 9, 3, 0, BF)
    m.router.zero_()
    m.bias.zero_()
    m.bias[4] = m.bias[6] = 1.0
    x = rnd(rows, 64, seed=1, dtype=BF)
    hip.moe(m.desc(hip, x))
    assert (m.ids.cpu() == torch.tensor([4, 6, 0])).all()
    e = math.e
    close(m.wts, torch.tensor([e, e, 1.0]).expand(rows, 3) / (2 * e + 1), F32)


@pytest.mark.parametrize("M", [1, 2, 9, 16, 17, 40, 64])
@pytest.mark.parametrize("E,top", [(5, 2), (20, 4), (70, 9)])
def test_routing_beside_projections(hip, M, E, top):
    D, N, I = 136, 200, 72
    m = Mix(D, 16, E, top, 24, BF, seed=M)
    x, w, w1 = rnd(M, D, seed=1, dtype=BF), rnd(N, D, seed=2, dtype=BF), rnd(2 * I, D, seed=3, dtype=BF)
    act, before = rnd(M, 24, seed=4, dtype=BF), rnd(M, 24, seed=4, dtype=BF)
    y, a, y1, a1 = (torch.empty(M, n, dtype=BF, device=DEV) for n in (N, I, N, I))
    hip.linear_multi((x, w, y1, hip.EPI_NONE), (x, w1, a1, hip.EPI_SWIGLU))
    d = m.desc(hip, x, act)
    hip.linear_multi_route(d, (x, w, y, hip.EPI_NONE), (x, w1, a, hip.EPI_SWIGLU))
    assert torch.equal(act, before)            # gated by the experts' launches, not here
    hip.moe(d)
    m.check(x, act, before)
    close(y, d64(y1), BF)
    close(a, d64(a1), BF)
    ids = m.ids.clone()
    d = m.desc(hip, x, before.clone())
    hip.linear_multi_route(d, (x, w, y, hip.EPI_NONE))
    assert torch.equal(m.ids, ids)
    close(y, d64(y1), BF)


@pytest.mark.parametrize("rows", [40, 100])
def test_swiglu_into_part_of_a_wider_row(hip, rows):
    for dtype in (F32, BF):
        x, w1 = rnd(rows, 64, seed=1, dtype=dtype), rnd(2 * 40, 64, seed=2, dtype=dtype)
        wide, h = torch.full((rows, 64), float("nan"), dtype=dtype, device=DEV), torch.empty(rows, 80, dtype=dtype, device=DEV)
        if dtype == BF:
            hip.linear_swiglu_out(x, w1, wide[:, 8:48], h)
        else:
            hip.swiglu(hip.linear(x, w1, h), wide[:, 8:48])
        up, g = (d64(x) @ d64(w1).T).chunk(2, -1)
        close(wide[:, 8:48], up * O.silu(g), dtype)
        assert torch.isnan(wide[:, :8]).all() and torch.isnan(wide[:, 48:]).all()
