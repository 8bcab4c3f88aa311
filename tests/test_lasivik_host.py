"""The Lasivik family without a GPU: the plain restatement's mechanisms against closed forms, configuration, checkpoint
conversion (padding included), the trace replay's bookkeeping and refusals, and the C ABI's argument checks."""
import ctypes
import json
import math
import os
import subprocess
import sys

import pytest
import torch

import lasivik_cases as C
from oracle import lasivik_oracle as O

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64


# ------------------------------------------------------------------------------------------------ mechanisms

def test_recurrence_is_the_decayed_sum():
    g = torch.Generator().manual_seed(1)
    T, H, dk, dv = 9, 2, 3, 4
    q, k = (torch.randn(T, H, dk, generator=g, dtype=F64) for _ in range(2))
    v = torch.randn(T, H, dv, generator=g, dtype=F64)
    a = torch.rand(T, H, dk, generator=g, dtype=F64)
    o, S = O.recurrence(q, k, v, a)
    for t in range(T):
        want = torch.zeros(H, dv, dtype=F64)
        for s in range(t + 1):
            w = a[s + 1:t + 1].prod(0)                         # decays applied after s's key went in
            want += (q[t] * k[s] * w).sum(-1, keepdim=True) * v[s]
        torch.testing.assert_close(o[t], want)
    o1, S1 = O.recurrence(q[:4], k[:4], v[:4], a[:4])
    o2, S2 = O.recurrence(q[4:], k[4:], v[4:], a[4:], S1)
    torch.testing.assert_close(torch.cat([o1, o2]), o)
    torch.testing.assert_close(S2, S)


def test_gla_decay_is_the_root_of_a_sigmoid():
    g = torch.Generator().manual_seed(2)
    h, a1, a2 = (torch.randn(*s, generator=g, dtype=F64) for s in ((5, 8), (3, 8), (6, 3)))
    b = torch.randn(6, generator=g, dtype=F64)
    z = h @ a1.T @ a2.T + b
    torch.testing.assert_close(O.gla_decay(h, a1, a2, b, 16.0), torch.sigmoid(z) ** (1 / 16))


def test_rotation_keeps_pair_norms_depends_on_distance_and_leaves_the_rest():
    x = torch.randn(6, 2, 10, generator=torch.Generator().manual_seed(3), dtype=F64)
    at = torch.arange(7, 13)
    y = O.rotate_half(x, at, 6, 100.0)
    torch.testing.assert_close(y[..., 6:], x[..., 6:])
    for i in range(3):
        torch.testing.assert_close(y[..., i] ** 2 + y[..., i + 3] ** 2, x[..., i] ** 2 + x[..., i + 3] ** 2)
    a = 7 * 100.0 ** (-2 / 6)
    assert math.isclose(float(y[0, 0, 1]), float(x[0, 0, 1] * math.cos(a) - x[0, 0, 4] * math.sin(a)))
    q, k = x[:1], x[1:2]
    dot = lambda p, r: (O.rotate_half(q, torch.tensor([p]), 6, 100.0) * O.rotate_half(k, torch.tensor([r]), 6, 100.0)).sum()
    torch.testing.assert_close(dot(5, 2), dot(105, 102))


@pytest.mark.parametrize("size", [1, 2, 5, 50])
def test_window_edges(size):
    m = O.window_mask(torch.arange(12), torch.arange(12), size)
    for i in range(12):
        assert m[i].nonzero().flatten().tolist() == list(range(max(0, i - size + 1), i + 1))


def test_oracle_portions_and_restart():
    cfg, kw = C.CASES["mixed"]
    W = C.weights(cfg, 3, **kw)
    o = O.Oracle(cfg, W)
    t = C.tokens(cfg, 45)
    whole = o.step(t)
    o.reset()
    parts = torch.cat([o.step(t[:2]), o.step(t[2:30]), *[o.step([x]) for x in t[30:]]])
    torch.testing.assert_close(parts, whole)
    assert o.residuals.shape == (len(cfg["layers"]), 1, cfg["width"])


# ------------------------------------------------------------------------------------------------ configuration, loading

def folder(tmp_path, cfg, W):
    from safetensors.torch import save_file

    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(W, str(tmp_path / "model.safetensors"))
    return str(tmp_path)


@pytest.mark.parametrize("case", sorted(C.CASES))
def test_checkpoint_loads_with_padding(tmp_path, case):
    from gpt_fast import GPTLasivik
    from gpt_fast.checkpoint import load_pretrained, pretrained_class

    cfg, kw = C.CASES[case]
    W = C.weights(cfg, 5, **kw)
    path = folder(tmp_path, cfg, W)
    assert pretrained_class(path) is GPTLasivik
    model = load_pretrained(path, "cpu", torch.float32)
    D, Dp = cfg["width"], model.config.dim
    assert Dp % 8 == 0 and Dp - D < 8
    emb = model.tok_embeddings.weight
    assert torch.equal(emb[:, :D], W["embed"].float()) and not emb[:, D:].any()
    for i, (layer, blk) in enumerate(zip(cfg["layers"], model.layers)):
        m, mix = layer["mixer"], blk.mixer
        nq, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        assert torch.equal(mix.in_proj.weight[:nq, :D], W[f"l{i}.mix.q"].float())
        assert torch.equal(mix.out_proj.weight[:D, :nv], W[f"l{i}.mix.o"].float())
        assert not mix.out_proj.weight[:, nv:].any() and not mix.out_proj.weight[D:].any()
        if layer["type"] == "gla":
            assert mix.args.decay_rank == W[f"l{i}.mix.a1"].shape[0]
            assert torch.equal(mix.in_proj.weight[-mix.args.decay_rank:, :D], W[f"l{i}.mix.a1"].float())
        if layer["type"] == "latent_attention":
            assert torch.equal(mix.kv_up.weight[nq:, :m["kv_rank"]], W[f"l{i}.mix.uv"].float())
        if layer["mlp"] is None:
            assert blk.feed_forward is None
        else:
            I = layer["mlp"]["ff"]
            up, gate = blk.feed_forward.w1.weight.chunk(2)
            assert torch.equal(up[:I, :D], W[f"l{i}.mlp.up"].float()) and torch.equal(gate[:I, :D], W[f"l{i}.mlp.gate"].float())
            assert not up[I:].any() and not blk.feed_forward.w2.weight[:, I:].any()


def test_checkpoint_is_checked(tmp_path):
    from gpt_fast.checkpoint import load_pretrained

    cfg, kw = C.CASES["mixed"]
    W = C.weights(cfg, 5, **kw)
    for name, change, error in (("missing", lambda w: w.pop("l1.mix.a2"), KeyError),
                                ("more", lambda w: w.update(extra=torch.zeros(3)), KeyError),
                                ("shape", lambda w: w.update({"l0.mix.uk": w["l0.mix.uk"][:-1].clone()}), ValueError)):
        d = tmp_path / name
        d.mkdir()
        w = dict(W)
        change(w)
        with pytest.raises(error):
            load_pretrained(folder(d, cfg, w), "cpu", torch.float32)


def test_configuration_is_checked_and_named_shapes_build():
    from gpt_fast import GPTLasivik
    from gpt_fast.config import REGISTRIES, LasivikArgs, args_from_name

    cfg, _ = C.CASES["plain"]
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["type"] = "other"
    with pytest.raises(ValueError, match="unknown mixer"):
        LasivikArgs.from_config(bad)
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["mlp"]["kind"] = "routed"
    with pytest.raises(ValueError, match="unknown feed-forward"):
        LasivikArgs.from_config(bad)
    with pytest.raises(KeyError):
        args_from_name("lasivik", "no-such-shape")
    for name in REGISTRIES["lasivik"]:
        with torch.device("meta"):
            model = GPTLasivik.from_name(name)
        kinds = [blk.mixer.args.kind for blk in model.layers]
        assert len(kinds) == model.config.n_layer and set(kinds) == {"gla", "retention", "latent_attention"}


def test_rank_shards_are_refused(monkeypatch):
    from gpt_fast import tp
    from gpt_fast.config import args_from_name

    monkeypatch.setattr(tp, "_TP_WORLD_SIZE", 2)
    with pytest.raises(NotImplementedError):
        args_from_name("lasivik", "lasivik-1b")


def test_weight_only_quantisation_is_refused():
    from gpt_fast import GPTLasivik
    from gpt_fast.quantize import quantize_model_fp8

    with torch.device("meta"):
        model = GPTLasivik.from_name("lasivik-1b")
    with pytest.raises(NotImplementedError):
        quantize_model_fp8(model)


def test_bytes_per_step_count_weights_states_and_caches():
    import benchmark as bm
    from gpt_fast import GPTLasivik
    from gpt_fast.config import LasivikArgs

    cfg = C.config([C.latent(heads=2, dim=16, vdim=16, kv_rank=24, window=10), C.gla(heads=2, dim=16, vdim=8)], width=64, ff=64)
    with torch.device("meta"):
        model = GPTLasivik(LasivikArgs.from_config(cfg, {1: 8})).to(torch.bfloat16)
    n = sum(p.numel() for p in model.parameters()) - model.tok_embeddings.weight.numel()
    got = bm.decode_bytes_per_step(model, 3, 100)
    assert got == 2 * (n + 3 * 64) + 3 * 24 * 2 * 11 + 3 * 2 * 2 * 16 * 8 * 4


# ------------------------------------------------------------------------------------------------ trace replay

class _Recorder:
    """Stands in for a model: logits that say which token sat at which position."""

    def __init__(self):
        self.output = torch.nn.Linear(2, 2)
        self.calls = []

    def setup_caches(self, batch, length):
        self.shape = (batch, length)

    def check_device_errors(self):
        pass

    def __call__(self, idx, pos):
        self.calls.append((idx.tolist(), pos.tolist()))
        return torch.stack([idx.float(), pos.float().expand(idx.shape)], dim=-1)


def test_replay_continues_requests_and_frees_them():
    from trace_replay import Replay

    m = _Recorder()
    r = Replay(m, 8)
    assert m.shape == (1, 8)
    assert r.feed("a", [5, 6, 7], [0, 2]).tolist() == [[5, 0], [7, 2]]
    assert r.feed("a", [8], []) is None
    with pytest.raises(RuntimeError, match="follow one another"):
        r.feed("b", [1], [0])
    r.end("a")
    assert r.feed("b", [1, 2], [1]).tolist() == [[2, 1]]
    with pytest.raises(RuntimeError, match="max-tokens"):
        r.feed("b", [1] * 7, [])


def test_trace_run_refuses_fp32_for_a_family_that_has_none(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps(dict(hidden_size=64)))
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "8"], capture_output=True, text=True, timeout=300)
    assert r.returncode == 3, r.stderr
    assert os.access(os.path.join(ROOT, "bin", "trace_run"), os.X_OK)


# ------------------------------------------------------------------------------------------------ C ABI argument checks

def test_new_entry_points_validate_before_any_device_work():
    from gpt_fast import _hip

    lib = _hip.load()
    NULL, ALIGN, SHAPE, UNSUP = -1, -2, -3, -4
    assert lib.lr_embed_residual(None, 64, 0, 64, 64, 1, 8, 8, 1.0, 0, None) == NULL
    assert lib.lr_embed_residual(64, 64, 0, 64, 64, 1, 12, 8, 1.0, 0, None) == ALIGN
    assert lib.lr_residual_rmsnorm(64, 1.0, None, 64, 0.0, None, None, 1, 8, 8, 1e-5, 0, None) == NULL
    assert lib.lr_residual_rmsnorm(64, 1.0, None, 64, 0.0, 64, None, 1, 8, 9, 1e-5, 0, None) == SHAPE
    assert lib.lr_residual_rmsnorm(64, 1.0, None, 64, 0.0, 64, None, 1, 8, 8, 1e-5, 7, None) == UNSUP
    assert lib.lr_logit_cap(64, 4, 1, 8, 1.0, 1.0, 0, None) == SHAPE
    assert lib.lr_linear_f32(64, 4, 64, 64, 8, 1, 8, 8, None) == SHAPE
    assert lib.lr_swiglu_f32(None, 4, 64, 2, 1, 2, None) == NULL

    la = _hip._LinearAttention(q=64, k=64, v=64, g=64, ld=64, head_decay=64, pos=64, state=64, y=64, ldy=64, B=1, S=4, H=2, dk=16,
                               dv=16, rank=0, rot_dims=0, rope_len=0, dtype=0, tau=1.0, q_scale=1.0, k_scale=1.0, eps=1e-5)
    call = lambda: lib.lr_linear_attention(ctypes.byref(la), None)
    for field, value, code in (("q", None, NULL), ("head_decay", None, NULL), ("dk", 0, SHAPE), ("ld", 16, SHAPE),
                               ("ld", 68, ALIGN), ("dtype", 5, UNSUP), ("state", 8, ALIGN)):
        old = getattr(la, field)
        setattr(la, field, value)
        assert call() == code, field
        setattr(la, field, old)
    la.dv, la.ld, la.ldy = 300, 4096, 4096
    assert call() == UNSUP                                            # more than 256 dimensions per head
    la.dv, la.rope, la.rot_dims, la.rope_len = 16, 64, 18, 8
    assert call() == SHAPE                                            # more rotated dimensions than there are
    la.rope, la.lowrank, la.a2, la.a_bias, la.rank = None, 64, 64, 64, 4
    assert call() == NULL                                             # gated prefill needs scratch

    wa = _hip._WindowAttention(q=64, ldq=32, k=64, v=64, ldk=64, y=64, ldy=32, pos=64, B=1, S=4, H=2, dk=16, dv=16, window=3,
                               n_keys=6, Smax=8, dtype=0, scale=1.0)
    for field, value, code in (("k", None, NULL), ("window", 0, SHAPE), ("n_keys", 9, SHAPE), ("ldq", 16, SHAPE)):
        old = getattr(wa, field)
        setattr(wa, field, value)
        assert lib.lr_window_attention(ctypes.byref(wa), None) == code, field
        setattr(wa, field, old)
    assert lib.lr_latent_update(64, 8, 64, 64, 64, 1, 1, 12, 8, 4, 1e-5, 0, None, None) == SHAPE
    assert lib.lr_latent_window(64, 64, 64, 1, 9, 3, 8, 8, 0, None) == SHAPE
    assert lib.lr_latent_attention_scratch_bytes(1, 1, 2, 16, 5, 8) > 0
    at = _hip._LatentAttention(q=64, ldq=32, uk=64, uv=64, cache=64, y=64, ldy=32, pos=64, scratch=64, scratch_bytes=16, B=1, S=1,
                               H=2, dk=16, dv=16, ldr=16, rank=16, window=5, Smax=8, dtype=0, scale=1.0, eps=1e-5)
    assert lib.lr_latent_attention(ctypes.byref(at), None) == SHAPE   # too little scratch
    assert lib.lr_linear_attention_scratch_bytes(1, 1, 4, 16, 16, 1) == 0
    assert lib.lr_linear_attention_scratch_bytes(1, 2, 4, 16, 16, 1) == 2 * 4 * 16 * 4
    assert lib.lr_argmax_f32(None, 8, 64, 1, 8, None) == NULL
