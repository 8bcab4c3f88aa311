"""The Gepolix family end to end on a real GPU: the framework's model, caches, generation loop, graphs and trace replay against the
plain restatement in float64, on small random checkpoints."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import gepolix_cases as C
from oracle.gepolix_oracle import Oracle

pytestmark = pytest.mark.gpu
DEV = "cuda"
BF, F32 = torch.bfloat16, torch.float32
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {F32: 2e-5, BF: 6e-2}


class Served:
    """A case's model behind the framework's interface, and the restatement of it."""

    def __init__(self, cfg, W, dtype, batch=1, length=256):
        from gpt_fast import GPTGepolix
        from gpt_fast.checkpoint import load_checkpoint
        from gpt_fast.config import GepolixArgs

        with torch.device("meta"):
            m = GPTGepolix(GepolixArgs.from_config(cfg))
        self.model = m.to(dtype=dtype).to_empty(device=DEV).eval()
        load_checkpoint(self.model, W)
        self.model.setup_caches(batch, length)
        self.oracle = Oracle(cfg, W)
        self.dtype = dtype

    @torch.no_grad()
    def feed(self, rows, cuts, pos0=0):
        """rows: B token lists of one length; logits [B, T, V]."""
        idx = torch.tensor(rows, dtype=torch.int32, device=DEV)
        out, at = [], 0
        for n in cuts:
            pos = torch.arange(pos0 + at, pos0 + at + n, dtype=torch.int32, device=DEV)
            out.append(self.model(idx[:, at:at + n].contiguous(), pos).float().clone())
            at += n
        assert at == idx.shape[1]
        self.model.check_device_errors()
        return torch.cat(out, 1).cpu()

    def want(self, tokens):
        self.oracle.reset()
        return self.oracle.step(tokens).float()


def each(got, want):
    """Root mean square over the vocabulary at every position, relative to the logits' own."""
    d = (got - want).double()
    return d.pow(2).mean(-1).sqrt() / want.double().pow(2).mean().sqrt()


def agrees(got, want, dtype, what=""):
    """fp32: every position.  bf16: rounding may tip a close choice between two experts, after which a few positions differ by more
    than rounding: nearly all must agree closely."""
    e = each(got, want).flatten()
    if dtype == F32:
        assert e.max() < TOL[F32], (what, e.max())
    else:
        assert e.median() < TOL[BF] / 2 and (e < TOL[BF]).double().mean() >= 0.9, (what, e.median(), e.sort()[0][-8:])


def served(case, dtype, seed=1, **kw):
    cfg, wkw = C.CASES[case]
    return Served(cfg, C.weights(cfg, seed, **wkw), dtype, **kw), cfg


@pytest.mark.parametrize("case", sorted(C.CASES))
def test_prompt_decoding_and_portions_fp32(case):
    s, cfg = served(case, F32)
    t = C.tokens(cfg, 150)
    want = s.want(t)
    for cuts in ([150], [1] * 150, [2] * 75, [2, 3, 31, 9, 8, 7, 33, 57], [100] + [1] * 50, [64, 1, 1, 2, 82], [149, 1]):
        agrees(s.feed([t], cuts), want, F32, cuts)


@pytest.mark.parametrize("case", sorted(C.CASES))
def test_prompt_decoding_and_portions_bf16(case):
    s, cfg = served(case, BF)
    t = C.tokens(cfg, 150)
    want = s.want(t)
    for cuts in ([150], [1] * 150, [110] + [1] * 40, [2, 37, 3, 64, 9, 35], [65, 2, 63, 20]):
        agrees(s.feed([t], cuts), want, BF, cuts)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_residual_after_every_layer(dtype):
    """Layer by layer: the residual a model cut after its first n layers leaves."""
    cfg, kw = C.CASES["mixed"]
    W = C.weights(cfg, 4, **kw)
    t = C.tokens(cfg, 50)
    o = Oracle(cfg, W)
    o.step(t)
    for n in range(1, len(cfg["layers"]) + 1):
        part = dict(cfg, layers=cfg["layers"][:n])
        s = Served(part, {k: v for k, v in W.items() if not k.startswith("l") or int(k[1:].split(".")[0]) < n}, dtype)
        s.feed([t], [50])
        x = next(ws.x for k, ws in s.model._ws.items() if k[1] == 50)[:, :cfg["width"]]
        agrees(x.float().cpu(), o.residuals[n - 1].float(), dtype, n)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("case", ["mixed", "odd", "large", "experts"])
@pytest.mark.parametrize("batch", [5, 20])
def test_a_batch_gives_every_sequence_what_it_gets_alone(case, dtype, batch):
    s, cfg = served(case, dtype, batch=batch)
    rows = [C.tokens(cfg, 60, seed=i) for i in range(batch)]
    got = s.feed(rows, [41, 2] + [1] * 17)
    for r, g in list(zip(rows, got))[::4]:
        agrees(g, s.want(r), dtype)
        agrees(s.feed([r], [60])[0], g, dtype)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_a_slot_is_used_again_without_a_trace_of_the_last_sequence(dtype):
    s, cfg = served("mixed", dtype)
    a, b = C.tokens(cfg, 120, seed=1), C.tokens(cfg, 40, seed=2)
    first = s.feed([b], [30] + [1] * 10)
    s.feed([a], [100] + [1] * 20)                  # longer: leaves states, taps and keys behind
    assert torch.equal(first, s.feed([b], [30] + [1] * 10))
    agrees(first[0], s.want(b), dtype)
    s.feed([a[:3]], [3])
    assert torch.equal(s.feed([b], [1] * 40)[0], s.feed([b], [1] * 40)[0])
    agrees(s.feed([b], [1] * 40)[0], s.want(b), dtype)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_long_decoding_passes_windows_and_stays_exact(dtype):
    s, cfg = served("mixed", dtype, length=700)
    t = C.tokens(cfg, 600)
    want = s.want(t)
    got = s.feed([t], [5] + [1] * 595)[0]
    for lo in range(0, 600, 100):
        agrees(got[lo:lo + 100], want[lo:lo + 100], dtype, lo)


def test_long_prompt_runs_in_segments_and_tall_tiles():
    s, cfg = served("large", BF, length=1200)
    t = C.tokens(cfg, 1100)
    want = s.want(t)
    for cuts in ([1100], [700, 400], [513, 2, 585]):
        agrees(s.feed([t], cuts)[0], want, BF, cuts)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("window", [16, 17, 64])
def test_a_key_just_inside_and_just_outside_the_window(dtype, window):
    """One token whose key every query prefers: what follows depends on it exactly as long as the window reaches."""
    cfg = C.config([C.attention(heads=2, kv_heads=1, dim=16, vdim=16, window=window, dims=2, base=1e9, scale=1.0),
                    C.attention(heads=2, kv_heads=1, dim=16, vdim=16, window=window // 2, dims=2, base=1e9, scale=1.0, kv_from=0)], width=32, vocab=40, ff=32)
    W = C.weights(cfg, 2)
    # key 0 answers the bias of every query; token 7 alone has it
    W["l0.mix.q"][:], W["l1.mix.q"][:], W["l0.mix.k"][:] = 0, 0, 0
    W["l0.mix.q.b"][:], W["l1.mix.q.b"][:], W["l0.mix.k.b"][:] = 0, 0, 0
    for n in ("l0.mix.q.b", "l1.mix.q.b"):
        W[n][15::16] = 4
    W["embed"][:, 0] = -1
    W["embed"][7, 0] = 1
    W["l0.norm1"][0], W["l0.norm1.b"][0], W["l0.norm1.alpha"] = 3, 0, torch.tensor(2.0).bfloat16()
    W["l0.mix.k"][15, 0] = 1
    s = Served(cfg, W, dtype)
    t = [x if x != 7 else 8 for x in C.tokens(cfg, 120)]
    t[20] = 7
    other = list(t)
    other[20] = 9
    seen = each(s.want(t)[None], s.want(other)[None])[0]
    assert seen[20 + window - 1] > 0.1 and seen[20 + window:].max() < seen[20 + window - 1] / 10   # (only through the layer's own output)
    want = s.want(t)
    for cuts in ([120], [20 + window, 100 - window], [20 + window - 1, 2, 99 - window], [21] + [1] * 99):
        agrees(s.feed([t], cuts)[0], want, dtype, cuts)


def test_last_logits_only():
    for dtype in (F32, BF):
        s, cfg = served("mixed", dtype, batch=2)
        rows = [C.tokens(cfg, 33, seed=i) for i in range(2)]
        full = s.feed(rows, [33])
        s.model.last_logits_only = True
        idx, pos = torch.tensor(rows, dtype=torch.int32, device=DEV), torch.arange(33, dtype=torch.int32, device=DEV)
        with torch.no_grad():
            last = s.model(idx, pos)
        assert last.shape == (2, 1, cfg["vocab"])
        tol = dict(rtol=1e-5, atol=1e-5) if dtype == F32 else dict(rtol=2e-2, atol=6e-2)
        torch.testing.assert_close(last.float().cpu(), full[:, -1:], **tol)


@pytest.mark.parametrize("graphs", [False, True])
@pytest.mark.parametrize("B", [1, 3])
def test_greedy_generation_through_the_frameworks_loop(B, graphs, capsys):
    import benchmark as bm

    s, cfg = served("mixed", F32, batch=B)
    prompt, new = C.tokens(cfg, 37), 40
    s.oracle.reset()
    want = s.oracle.greedy(prompt, new)
    p = torch.tensor(prompt, dtype=torch.int64, device=DEV)
    for _ in range(2):                             # the second generation reuses the caches
        empty = torch.empty(B, len(prompt) + new, dtype=torch.int64, device=DEV)
        if graphs:
            g, x, pos, first = bm.get_cuda_graphs_for_prefill(s.model, p, B, greedy=True)
            dg = bm.get_cuda_graphs_for_decode(s.model, p, B, new, first, greedy=True)
            y, _, _ = bm.generate_using_cuda_graphs(g, x, pos, first, dg, p, B, empty, new)
        else:
            y, _, _ = bm.generate(s.model, p, new, B, empty, greedy=True)
        for row in y[:, len(prompt):].tolist():
            assert row == want


def test_graphs_of_a_bf16_decode_step_replay_what_eager_steps_give():
    import benchmark as bm

    s, cfg = served("large", BF, batch=2)
    t = C.tokens(cfg, 30)
    p = torch.tensor(t, device=DEV)

    def start():
        with torch.no_grad():
            return bm.prefill(s.model, p.view(1, -1).repeat(2, 1), torch.arange(30, device=DEV, dtype=torch.int32), greedy=True).clone()
    first = start()
    eager, cur, pos = [], first, torch.tensor([30], dtype=torch.int32, device=DEV)
    for _ in range(20):
        cur = bm.decode_one_token(s.model, cur, pos, greedy=True)[0].clone()
        pos += 1
        eager.append(cur[:, 0].tolist())
    first = start()
    before = [x.clone() for x in s.model.recurrent_states()]
    assert len(before) == 4                        # a state and the taps of two layers
    dg = bm.get_cuda_graphs_for_decode(s.model, p, 2, 21, first, greedy=True)
    assert all(torch.equal(x, y) for x, y in zip(before, s.model.recurrent_states()))      # the warm-up steps are undone
    for i in range(20):
        dg.replay()
        torch.cuda.synchronize()
        assert dg.cur_token[:, 0].tolist() == eager[i], i


def test_sampling_goes_through_the_device_sampler():
    import benchmark as bm

    s, cfg = served("mixed", BF)
    empty = torch.empty(1, 20 + 8, dtype=torch.int64, device=DEV)
    torch.manual_seed(5)
    y, _, _ = bm.generate(s.model, torch.tensor(C.tokens(cfg, 20), device=DEV), 8, 1, empty, temperature=0.8, top_k=5)
    assert ((y >= 0) & (y < cfg["vocab"])).all()


def write(folder, cfg, W):
    from safetensors.torch import save_file

    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file(W, str(folder / "model.safetensors"))
    return str(folder)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_replays_a_trace(tmp_path, dtype):
    cfg, kw = C.CASES["odd"]
    W = C.weights(cfg, 7, **kw)
    a, b = C.tokens(cfg, 30, seed=1), C.tokens(cfg, 11, seed=2)
    steps = [dict(step=0, entries=[dict(id="x", tokens=a[:20], want=[0, 19])], end=[]),
             dict(step=1, entries=[dict(id="x", tokens=a[20:29], want=[])], end=[]),
             dict(step=2, entries=[dict(id="x", tokens=a[29:], want=[0])], end=["x"]),
             dict(step=3, entries=[dict(id="y", tokens=b, want=[10, 3])], end=["y"])]
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", write(tmp_path / "m", cfg, W), "--dtype", dtype,
                        "--out", str(out), "--max-tokens", "40"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
    o = Oracle(cfg, W)
    wa = o.step(a).float()
    o.reset()
    wb = o.step(b).float()
    got, want = [], []
    for n, w in ((0, wa[[0, 19]]), (2, wa[[29]]), (3, wb[[10, 3]])):
        got.append(torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(len(w), -1)))
        want.append(w)
    e = each(torch.cat(got), torch.cat(want))
    assert e.max() < TOL[getattr(torch, dtype)], e


def test_benchmark_command_serves_a_checkpoint(tmp_path, capsys):
    import benchmark as bm

    cfg, kw = C.CASES["mixed"]
    path = write(tmp_path / "m", cfg, C.weights(cfg, 3, **kw))
    run = lambda graph: bm.main(None, prompt_length=12, num_samples=1, max_new_tokens=9, batch_size=2, compile=graph, greedy=True, seed=0, warmup=1,
                                device=DEV, precision=F32, checkpoint=path)
    res, eager = run(True), run(False)
    assert res["tokens"] == eager["tokens"] and len(res["tokens"]) == 9
    assert "tokens/sec" in capsys.readouterr().out


def test_errors_are_reported():
    from gpt_fast import _hip

    s, cfg = served("mixed", F32, length=40)
    with pytest.raises(_hip.LadderHipError):
        s.feed([C.tokens(cfg, 41)], [41])
    with pytest.raises(NotImplementedError):
        m = s.model.to(torch.float16)
        m.max_seq_length = -1
        m.setup_caches(1, 8)
