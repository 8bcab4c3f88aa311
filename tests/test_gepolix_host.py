"""The Gepolix family without a GPU: the plain restatement's mechanisms against closed forms, that the test models show a planted
mistake, configuration, checkpoint conversion (padding included) and the C ABI's argument checks."""
import ctypes
import json
import math

import pytest
import torch

import gepolix_cases as C
from oracle import gepolix_oracle as O

F64 = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


# ------------------------------------------------------------------------------------------------ mechanisms

def test_dynamic_tanh_and_softplus():
    x, w, b = rnd(5, 7), rnd(7, seed=1), rnd(7, seed=2)
    torch.testing.assert_close(O.dynamic_tanh(x, torch.tensor(0.7, dtype=F64), w, b), torch.tanh(0.7 * x) * w + b)
    z = torch.tensor([-800.0, -3.0, 0.0, 2.5, 800.0], dtype=F64)
    torch.testing.assert_close(O.softplus(z), torch.nn.functional.softplus(z, threshold=50))


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_causal_conv_is_a_convolution_and_continues(taps):
    u, w, b = rnd(11, 6), rnd(6, taps, seed=1), rnd(6, seed=2)
    before = rnd(taps - 1, 6, seed=3)
    want = torch.nn.functional.conv1d(torch.cat([before, u]).T[None], w[:, None], b, groups=6)[0].T
    torch.testing.assert_close(O.causal_conv(u, w, b, before), want)
    both = torch.cat([before, u])
    halves = torch.cat([O.causal_conv(u[:4], w, b, before), O.causal_conv(u[4:], w, b, both[4:4 + taps - 1])])
    torch.testing.assert_close(halves, want)


def test_selective_scan_is_the_decayed_sum():
    T, H, G, N, P = 9, 4, 2, 3, 5
    x, B, Cm = rnd(T, H, P), rnd(T, G, N, seed=1), rnd(T, G, N, seed=2)
    dt, A_log = O.softplus(rnd(T, H, seed=3)), rnd(H, seed=4)
    S0 = rnd(H, N, P, seed=5)
    y, S = O.selective_scan(x, B, Cm, dt, A_log, S0)
    for h in range(H):
        g = h // 2
        a = -torch.exp(A_log[h]) * dt[:, h]
        for t in range(T):
            want = torch.exp(a[:t + 1].sum()) * (S0[h].T @ Cm[t, g])
            for s in range(t + 1):
                want = want + torch.exp(a[s + 1:t + 1].sum()) * dt[s, h] * (B[s, g] @ Cm[t, g]) * x[s, h]
            torch.testing.assert_close(y[t, h], want)
    y1, S1 = O.selective_scan(x[:4], B[:4], Cm[:4], dt[:4], A_log, S0)
    y2, S2 = O.selective_scan(x[4:], B[4:], Cm[4:], dt[4:], A_log, S1)
    torch.testing.assert_close(torch.cat([y1, y2]), y)
    torch.testing.assert_close(S2, S)


def test_parts_norm_has_unit_parts():
    y = O.parts_norm(rnd(3, 12), 4, 0.0).view(3, 4, 3)
    torch.testing.assert_close(y.pow(2).mean(-1), torch.ones(3, 4, dtype=F64))


@pytest.mark.parametrize("size", [1, 3, 50])
def test_grouped_window_attention(size):
    H, G, T, d, dv, pos0 = 6, 2, 5, 4, 3, 7
    q, k, v = rnd(T, H, d), rnd(pos0 + T, G, d, seed=1), rnd(pos0 + T, G, dv, seed=2)
    got = O.grouped_window_attention(q, k, v, pos0, size, 0.3)
    for t in range(T):
        keys = list(range(max(0, pos0 + t - size + 1), pos0 + t + 1))
        for h in range(H):
            w = torch.softmax(k[keys, h // 3] @ q[t, h] * 0.3, 0)
            torch.testing.assert_close(got[t, h], w @ v[keys, h // 3])


def test_mixture_with_every_expert_is_the_softmax_average():
    cfg = C.config([C.ssm(mlp=C.moe(experts=4, top=4, ff=6, shared=None))], width=8)
    W = {k: v.to(F64) for k, v in C.weights(cfg, 1).items()}
    h, p = rnd(5, 8), "l0.mlp."
    w = torch.softmax(h @ W[p + "router"].T + W[p + "router.b"], -1)
    want = sum(w[:, e:e + 1] * O.feed_forward(h, W, f"{p}e{e}.") for e in range(4))
    torch.testing.assert_close(O.mixture(h, W, p, cfg["layers"][0]["mlp"]), want)
    idx, w1 = O.route(h, W[p + "router"], W[p + "router.b"], 1)
    assert torch.equal(w1, torch.ones_like(w1)) and torch.equal(idx[:, 0], (h @ W[p + "router"].T + W[p + "router.b"]).argmax(-1))


def test_oracle_portions_and_restart():
    cfg, kw = C.CASES["mixed"]
    o = O.Oracle(cfg, C.weights(cfg, 3, **kw))
    t = C.tokens(cfg, 45)
    whole = o.step(t)
    o.reset()
    parts = torch.cat([o.step(t[:2]), o.step(t[2:30]), *[o.step([x]) for x in t[30:]]])
    torch.testing.assert_close(parts, whole)
    assert o.residuals.shape == (len(cfg["layers"]), 1, cfg["width"])


def _mistakes(cfg, W):
    """name -> (configuration, weights) with one thing wrong."""
    copy = lambda: json.loads(json.dumps(cfg))
    out = {}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        if layer["type"] == "attention":
            for d in (-1, 1):
                c = copy()
                c["layers"][i]["mixer"]["mask"]["size"] += d
                out[f"{i}: window {d:+d}"] = (c, W)
            c = copy()
            c["layers"][i]["mixer"]["rot"]["dims"] -= 2
            out[f"{i}: fewer rotated dimensions"] = (c, W)
        else:
            for name in ("conv.b", "D"):
                out[f"{i}: {name} left out"] = (cfg, dict(W, **{p + "mix." + name: torch.zeros_like(W[p + "mix." + name])}))
            taps = W[p + "mix.conv"].clone()
            taps[:, 0] = 0
            if m["conv"] > 1:
                out[f"{i}: the oldest tap left out"] = (cfg, dict(W, **{p + "mix.conv": taps}))
            if m["norm_groups"] > 1:
                c = copy()
                c["layers"][i]["mixer"]["norm_groups"] = 1
                out[f"{i}: one norm part"] = (c, W)
        if layer["mlp"] is not None and layer["mlp"]["kind"] == "moe":
            if layer["mlp"]["router"]["top"] > 1:
                c = copy()
                c["layers"][i]["mlp"]["router"]["top"] -= 1
                out[f"{i}: an expert too few"] = (c, W)
            if "shared" in layer["mlp"]:
                out[f"{i}: shared expert's gate"] = (cfg, dict(W, **{p + "mlp.shared.sg": torch.zeros_like(W[p + "mlp.shared.sg"])}))
    return out


@pytest.mark.parametrize("case", ["mixed", "odd"])
def test_the_test_models_show_a_mistake(case):
    """What the GPU tests compare with tolerances of 2e-5 (fp32) moves by far more when one mechanism is off."""
    cfg, kw = C.CASES[case]
    W = C.weights(cfg, 1, **kw)
    t = C.tokens(cfg, 60)
    want = O.Oracle(cfg, W).step(t)
    for name, (c, w) in _mistakes(cfg, W).items():
        got = O.Oracle(c, w).step(t)
        err = ((got - want).pow(2).mean(-1).sqrt().max() / want.pow(2).mean().sqrt()).item()
        assert err > 2e-3, (name, err)


# ------------------------------------------------------------------------------------------------ configuration, loading

def folder(tmp_path, cfg, W):
    from safetensors.torch import save_file

    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(W, str(tmp_path / "model.safetensors"))
    return str(tmp_path)


@pytest.mark.parametrize("case", sorted(C.CASES))
def test_checkpoint_loads_with_padding(tmp_path, case):
    from gpt_fast import GPTGepolix
    from gpt_fast.checkpoint import load_pretrained, pretrained_class

    cfg, kw = C.CASES[case]
    W = C.weights(cfg, 5, **kw)
    path = folder(tmp_path, cfg, W)
    assert pretrained_class(path) is GPTGepolix
    model = load_pretrained(path, "cpu", torch.float32)
    D, Dp = cfg["width"], model.config.dim
    f = lambda name: W[name].float()
    assert torch.equal(model.norm.weight[:D], f("final.norm")) and torch.equal(model.norm.alpha, f("final.norm.alpha").view(1))
    assert torch.equal(model.output.weight[:, :D], f("head")) and not model.output.weight[:, D:].any()
    for i, (layer, blk) in enumerate(zip(cfg["layers"], model.layers)):
        m, mix, p = layer["mixer"], blk.mixer, f"l{i}.mix."
        H, P = m["heads"], m["vdim"]
        assert torch.equal(blk.norm.bias[:D], f(f"l{i}.norm1.b")) and not blk.norm.weight[D:].any() and not blk.norm.bias[D:].any()
        Pp = mix.y_cols // H
        o = mix.out_proj.weight[:D, :mix.y_cols].view(D, H, Pp)
        assert torch.equal(o[:, :, :P].reshape(D, -1), f(p + "o")) and not o[:, :, P:].any() and not mix.out_proj.weight[D:].any()
        if layer["type"] == "mamba2":
            N, G = m["state"], m["groups"]
            assert mix.P % 16 == 0 and mix.N % 16 == 0
            got = mix.in_proj.weight[:, :D]
            z, x, B, Cw, dt = got.split([mix.inner, mix.inner, G * mix.N, G * mix.N, H])
            want = f(p + "in").split([H * P, H * P, G * N, G * N, H])
            for have, w, n, size in ((z, want[0], H, P), (x, want[1], H, P), (B, want[2], G, N), (Cw, want[3], G, N)):
                have = have.reshape(n, -1, D)
                assert torch.equal(have[:, :size].reshape(-1, D), w) and not have[:, size:].any()
            assert torch.equal(dt, want[4]) and torch.equal(mix.a_log, f(p + "A_log"))
            conv = mix.conv_weight[:mix.inner].view(H, mix.P, -1)
            assert torch.equal(conv[:, :P].reshape(H * P, -1), f(p + "conv")[:H * P]) and not conv[:, P:].any()
        else:
            d = m["dim"]
            q = mix.in_proj.weight[:H * mix.dk, :D].view(H, mix.dk, D)
            assert torch.equal(q[:, :d].reshape(-1, D), f(p + "q")) and not q[:, d:].any()
            own = "kv_from" not in m
            assert mix.in_proj.weight.shape[0] == H * mix.dk + (mix.kv_cols if own else 0)
            bias = mix.in_proj.bias[:H * mix.dk].view(H, mix.dk)
            assert torch.equal(bias[:, :d].reshape(-1), f(p + "q.b")) and not bias[:, d:].any()
            if not own:
                assert mix._lender is model.layers[m["kv_from"]].mixer
        mlp, p = layer["mlp"], f"l{i}.mlp."
        dense = None if mlp is None else mlp["ff"] if mlp["kind"] == "dense" else mlp.get("shared", {}).get("ff")
        if dense is None:
            assert blk.w1 is None and mix.out_proj.in_features == mix.y_cols
        else:
            src = p if mlp["kind"] == "dense" else p + "shared."
            up, gate = blk.w1.weight.chunk(2)
            assert torch.equal(up[:dense, :D], f(src + "up")) and torch.equal(gate[:dense, :D], f(src + "gate")) and not up[dense:].any()
            assert torch.equal(mix.out_proj.weight[:D, mix.y_cols:mix.y_cols + dense], f(src + "down"))
        if mlp is not None and mlp["kind"] == "moe":
            x, I = blk.experts, mlp["expert"]["ff"]
            e = x.n - 1
            assert torch.equal(x.router[e, :D], f(p + "router")[e]) and torch.equal(x.router_bias, f(p + "router.b"))
            assert torch.equal(x.w1[e, x.ff:x.ff + I, :D], f(f"{p}e{e}.gate")) and torch.equal(x.w2[e, :D, :I], f(f"{p}e{e}.down"))
            assert not x.w2[:, :, I:].any() and not x.w1[:, I:x.ff].any()
            if x.shared:
                assert torch.equal(x.router[x.n, :D], f(p + "shared.sg")[0])


def test_checkpoint_is_checked(tmp_path):
    from gpt_fast import GPTLadder
    from gpt_fast.checkpoint import load_checkpoint, load_pretrained
    from gpt_fast.config import ModelArgs

    cfg, kw = C.CASES["mixed"]
    W = C.weights(cfg, 5, **kw)
    for name, change, error in (("missing", lambda w: w.pop("l0.mix.A_log"), KeyError),
                                ("more", lambda w: w.update({"l3.mix.k": torch.zeros(3)}), KeyError),
                                ("shape", lambda w: w.update({"l2.mlp.e3.up": w["l2.mlp.e3.up"][:-1].clone()}), ValueError)):
        d = tmp_path / name
        d.mkdir()
        w = dict(W)
        change(w)
        with pytest.raises(error):
            load_pretrained(folder(d, cfg, w), "cpu", torch.float32)
    with torch.device("meta"):
        other = GPTLadder(ModelArgs(n_layer=1, n_head=2, dim=64, vocab_size=64))
    with pytest.raises(ValueError, match="listed layers"):
        load_checkpoint(other, W)


def test_configuration_is_checked_and_named_shapes_build():
    from gpt_fast import GPTGepolix
    from gpt_fast.config import REGISTRIES, GepolixArgs, args_from_name

    cfg, _ = C.CASES["mixed"]

    def refused(change, match):
        bad = json.loads(json.dumps(cfg))
        change(bad["layers"])
        with pytest.raises(ValueError, match=match):
            GepolixArgs.from_config(bad)
    refused(lambda l: l[0].update(type="other"), "unknown mixer")
    refused(lambda l: l[0]["mlp"].update(kind="other"), "unknown feed-forward")
    refused(lambda l: l[3]["mixer"].update(kv_from=0), "keys and values of its own")
    refused(lambda l: l[3]["mixer"].update(kv_from=3), "keys and values of its own")
    refused(lambda l: l[3]["mixer"].update(kv_heads=3), "heads differ")
    with pytest.raises(KeyError):
        args_from_name("gepolix", "no-such-shape")
    for name in REGISTRIES["gepolix"]:
        with torch.device("meta"):
            model = GPTGepolix.from_name(name)
        assert {blk.mixer.args.kind for blk in model.layers} == {"mamba2", "attention"}
        assert any(blk.experts is not None for blk in model.layers)
        assert any(blk.mixer.args.kv_from is not None for blk in model.layers)


def test_rank_shards_and_quantisation_are_refused(monkeypatch):
    from gpt_fast import GPTGepolix, tp
    from gpt_fast.config import args_from_name
    from gpt_fast.quantize import quantize_model_fp8

    with torch.device("meta"):
        model = GPTGepolix.from_name("gepolix-1b")
    with pytest.raises(NotImplementedError):
        quantize_model_fp8(model)
    monkeypatch.setattr(tp, "_TP_WORLD_SIZE", 2)
    with pytest.raises(NotImplementedError):
        args_from_name("gepolix", "gepolix-1b")


def test_bytes_per_step_count_weights_states_caches_and_touched_experts():
    import benchmark as bm
    from gpt_fast import GPTGepolix
    from gpt_fast.config import GepolixArgs

    cfg = C.config([C.ssm(heads=2, vdim=16, state=16, groups=1, norm_groups=1, conv=4),
                    C.attention(heads=4, kv_heads=2, dim=16, vdim=24, window=10, dims=16, mlp=C.moe(experts=4, top=1, ff=8, shared=16))], width=64, ff=64)
    with torch.device("meta"):
        model = GPTGepolix(GepolixArgs.from_config(cfg)).to(torch.bfloat16)
    n = sum(p.numel() for p in model.parameters()) - model.tok_embeddings.weight.numel()
    untouched = 4 * 3 * 8 * 64 * (1 - 1 / 4) ** 3
    carried = 2 * 3 * 2 * 16 * 16 * 4 + 3 * 4 * (2 * 16 + 2 * 16) * 2 + 3 * 2 * (16 + 24) * 2 * 11
    assert bm.decode_bytes_per_step(model, 3, 100) == int(2 * (n - untouched + 3 * 64) + carried)


# ------------------------------------------------------------------------------------------------ C ABI argument checks

def test_new_entry_points_validate_before_any_device_work():
    from gpt_fast import _hip

    lib = _hip.load()
    NULL, ALIGN, SHAPE, UNSUP = -1, -2, -3, -4

    def vary(desc, call, cases):
        for field, value, code in cases:
            old = getattr(desc, field)
            setattr(desc, field, value)
            assert call() == code, (field, value)
            setattr(desc, field, old)

    assert lib.lr_residual_tanh(64, None, None, None, 0, 64, 64, 64, None, None, 1, 8, 0, None) == NULL
    assert lib.lr_residual_tanh(64, None, None, None, 0, None, 64, 64, None, 64, 1, 8, 0, None) == NULL
    assert lib.lr_residual_tanh(64, None, 64, None, 2, 64, 64, 64, 64, 64, 1, 8, 0, None) == NULL
    assert lib.lr_residual_tanh(64, None, None, None, 0, 64, 64, 64, 64, 64, 1, 12, 0, None) == ALIGN
    assert lib.lr_residual_tanh(64, None, None, None, 0, 64, 64, 64, 64, 64, 1, 8, 9, None) == UNSUP
    assert lib.lr_causal_conv(64, 8, 64, 64, 64, 64, 64, 8, 1, 1, 16, 4, 0, None) == SHAPE
    assert lib.lr_causal_conv(64, 16, 64, 64, 64, 64, 64, 16, 1, 1, 16, 9, 0, None) == UNSUP
    assert lib.lr_causal_conv(64, 16, 64, 64, 64, None, 64, 16, 1, 1, 16, 4, 0, None) == NULL
    s = _hip._Ssd(z=64, x=64, b=64, c=64, dt=64, ld=128, ldu=128, dt_bias=64, a_log=64, d=64, pos=64, state=64, y=64, ldy=64, B=1, S=4, H=2,
                  G=1, N=16, P=16, dtype=0)
    vary(s, lambda: lib.lr_ssd(ctypes.byref(s), None),
         (("z", None, NULL), ("state", 8, ALIGN), ("H", 0, SHAPE), ("G", 3, SHAPE), ("ldu", 24, SHAPE), ("N", 12, ALIGN), ("N", 264, SHAPE),
          ("dtype", 4, UNSUP)))
    s.ldu = 1024
    vary(s, lambda: lib.lr_ssd(ctypes.byref(s), None), (("N", 264, UNSUP),))
    assert lib.lr_ssd_step(ctypes.byref(s), 64, 64, 64, 4, None) == SHAPE          # more than one token
    s.S = 1
    assert lib.lr_ssd_step(ctypes.byref(s), 64, 64, 64, 9, None) == UNSUP
    assert lib.lr_ssd_step(ctypes.byref(s), None, 64, 64, 4, None) == NULL
    s.S, s.B, s.H = 4096, 1, 2
    assert lib.lr_ssd_scratch_bytes(1, 4096, 2, 16, 16, 0) > 0 and lib.lr_ssd_scratch_bytes(1, 4096, 2, 16, 16, 1) == 0
    assert lib.lr_ssd(ctypes.byref(s), None) == NULL                                # segments need scratch
    assert lib.lr_parts_norm(64, 64, 64, 1, 48, 5, 16, 16, 1e-5, 0, None) == SHAPE
    assert lib.lr_parts_norm(64, 32, 64, 1, 48, 2, 16, 16, 1e-5, 0, None) == SHAPE
    rope = lambda **k: lib.lr_bias_rope_cache(*[dict(proj=64, ld=64, bias=None, rope=64, pos=64, cache=64, B=1, S=1, H=2, G=1, dk=16, dv=16, rot=8,
                                                     rope_len=8, ldc=32, Smax=8, dtype=0, err=None, stream=None, **{})[n] if n not in k else k[n]
                                                for n in ("proj", "ld", "bias", "rope", "pos", "cache", "B", "S", "H", "G", "dk", "dv", "rot",
                                                          "rope_len", "ldc", "Smax", "dtype", "err", "stream")])
    assert rope(rot=18) == SHAPE and rope(rot=7) == SHAPE and rope(rope=None) == NULL and rope(ld=48) == SHAPE and rope(ldc=24) == SHAPE
    assert rope(dtype=3) == UNSUP and rope(H=3, G=2) == SHAPE
    win = lambda dk=16, G=1, scratch=1 << 20: lib.lr_window_decode(64, 64, 64, 64, 64, 64, 1, 2, G, dk, 16, 64, 8, 4, 1.0, 64, scratch, None)
    assert win(dk=12) == ALIGN and win(dk=40) == SHAPE and win(G=3) == SHAPE and win(scratch=4) == SHAPE
    assert lib.lr_window_decode_scratch_bytes(1, 2, 1, 16, 4, 8) > 0
    m = _hip._Moe(x=64, ldx=64, router=64, router_bias=64, w1=64, w2=64, out=64, experts=64, weights=64, gate=64, counts=64, shared=None, ld_shared=0,
                  scratch=64, scratch_bytes=1 << 30, rows=3, D=64, I=32, E=4, top=2, shared_cols=0, dtype=0, routed=0)
    cases = (("w1", None, NULL), ("experts", None, NULL), ("top", 5, SHAPE), ("ldx", 32, SHAPE), ("I", 20, ALIGN), ("E", 600, UNSUP),
             ("scratch_bytes", 8, SHAPE), ("dtype", 2, UNSUP), ("out", 8, ALIGN))
    vary(m, lambda: lib.lr_moe(ctypes.byref(m), None), cases)
    p = (_hip._Projection * 1)(_hip._Projection(64, 64, 64, 64, 64, 64, 64, 0, None))
    route = lambda M=3, n=1: lib.lr_linear_multi_route(ctypes.cast(p, ctypes.c_void_p), n, M, ctypes.byref(m), None)
    assert route(M=4) == SHAPE and route(n=3) == SHAPE
    vary(m, route, (("rows", 2, SHAPE), ("w2", None, NULL), ("dtype", 1, UNSUP)))
    m.rows = 65
    assert route(M=65) == UNSUP
    wa = _hip._WindowAttention(q=64, ldq=64, k=64, v=64, ldk=64, y=64, ldy=64, pos=64, B=1, S=4, H=4, dk=16, dv=16, window=3, n_keys=6, Smax=8,
                               dtype=0, kv_heads=3, scale=1.0)
    assert lib.lr_window_attention(ctypes.byref(wa), None) == SHAPE
