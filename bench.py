"""Headline benchmark: batch-1 greedy decode of one TP=8 rank shard of Ladder-70B on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch B] [--no-cpu-baseline]
    python bench.py --lasivik [SIZE ...]     # other workloads, see below
    python bench.py --gepolix [SIZE ...]

A "step" is one decode step (one new token per sequence) of the whole per-rank forward pass,
replayed as a captured hipGraph: embedding -> 80 ladder blocks -> final add/norm -> vocab-shard
lm_head -> argmax -> device-side token/position hand-over.  Weights are random N(0, 0.02) bf16
(seed 0), the prompt is 2048 uniform-random ids; the prompt is prefilled before the timed region
so the KV cache has its real length, and the timed steps start at position 2048.  Everything the
steps read is resident in HBM when the clock starts.

Prints ONE JSON line.  `value` = decoded tokens per second (whole job = the one GPU).
`roofline`   : the dominant kernel.  For the ladder model at batch <= 2 that is k_ladder_step, ONE
               persistent launch per decode step; `achieved` = algorithmic bytes per launch (all
               weights and gains once + valid KV + KV write + embedding rows + logits) / its mean
               launch duration, measured here with HIP events around back-to-back launches on the
               launch stream.  `traffic` = HBM bytes per launch from rocprofv3 FETCH_SIZE + WRITE_SIZE
               counter runs (a constant recorded from those runs, or null).  Other models / batches
               run the per-op path, whose dominant kernel is the up/gate projection (timed alone here:
               the GEMV up to batch 4, the matrix-core band kernel above).
               `measured_read_ceiling` = GB/s of a plain streaming read of 8 GiB by every CU
               (lr_stream_read) on this machine in the same run; `frac` is against the nominal
               8 TB/s, `frac_of_measured_ceiling` against that.
`step_roofline`: the same ratio for the whole decode step as replayed from the hipGraph (kernel +
               token hand-over): algorithmic bytes per step / measured step time.
`cpu_baseline`: the oracle (a PyTorch-CPU restatement of the reference; the reference itself cannot
               run without CUDA + NCCL) timed on this machine's host cores on the reference's
               CPU-sized case: Ladder-1B fp32, batch 1, 128-token prompt, greedy decode.  `cores` =
               threads used (the process's CPU share: OMP_NUM_THREADS when set, else every core),
               `host_cpus` = os.cpu_count().
Measured in the same run and reported as extra keys (not the headline; --no-extras skips them):
`batched`     : the same rank shard at batch 2 (one-kernel step), 4, 8 and 64, the 8B model at batch 1 (one-kernel
               step) and 16 (prompt 1024) and the 405B rank shard at batch 16 (context 4096) -- per-op kernels unless noted,
               hipGraph replay: ms per step, tok/s, algorithmic GB/s and its fraction of 8 TB/s; `traffic` = HBM
               bytes per step from counter runs where one was made.
`fp8`         : the same shard with weight-only e4m3 projections at batch 1 (the one-kernel step on e4m3 weights)
               and batch 8 (per-op kernels): ms per step and the fraction of 8 TB/s on ITS algorithmic bytes
               (one byte per weight + scales).
`--lasivik`   : instead of the above, the Lasivik hybrid beside the dense family at equal layer sizes (lasivik-1b /
               gpt_dense:ladder-1b, lasivik-8b / gpt_dense:ladder-8b; random weights): prefill and decode throughput at
               several batch sizes, and the kernels only one of the two has, each timed alone over data that does not
               fit the caches, with the fraction of its roofline.  One JSON line of its own.
`--gepolix`   : the same for the Gepolix hybrid beside the Lasivik one (gepolix-1b / lasivik-1b, gepolix-8b / lasivik-8b).
`prefill`     : Ladder-8B, batch 32 x 2048 prompt tokens, causal prefill with last-position logits:
               seconds, algorithmic TFLOP/s and the fraction of 2.5 PFLOP/s (dense bf16 MFMA peak)."""
import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, os.path.join(ROOT, "ladder-residual-inference_amd"))
sys.path.insert(0, ROOT)

HBM_PEAK_GBPS = 8000.0
MFMA_PEAK_TFLOPS = 2500.0   # dense bf16
# HBM bytes one launch of the dominant kernel moves, per workload (model, batch, prompt), from the rocprofv3
# FETCH_SIZE / WRITE_SIZE counter runs summarised under profiles/; workloads without a counter run report null.
TRAFFIC_BYTES_PER_LAUNCH = {
    ("gpt_ladder:ladder-70b-tp8", 1, 2048): 17.585e9,    # k_ladder_step, 1.007 x algorithmic
    # the up/gate projection alone (the kernel the batched workloads' roofline object is measured on):
    ("gpt_ladder:ladder-70b-tp8", 8, 2048): 118.75e6,    # k_stream_gemm<16,2>, 256 bands: 1.009 x algorithmic
    ("gpt_ladder:ladder-70b-tp8", 64, 2048): 126.46e6,   # k_stream_gemm<64,2>, the decode step's 224 bands: 1.06 x
}
# HBM bytes of a whole decode step through the per-op kernels (all its launches), from the same kind of counter runs
STEP_TRAFFIC_BYTES = {
    ("gpt_ladder:ladder-70b-tp8", 8, 2048): 22.41e9,     # 1.24 x algorithmic
    ("gpt_ladder:ladder-70b-tp8", 64, 2048): 30.46e9,    # 1.34 x algorithmic
}


def cpu_baseline(new_tokens=32, repeats=2):
    """Oracle on the host cores, config 1 of the benchmark set.  Returns the cpu_baseline object."""
    import torch

    from oracle import ladder_oracle as O

    host_cpus = os.cpu_count() or 1
    # the process may own only a share of the host (the harness exports it as OMP_NUM_THREADS): more threads than
    # that only fight each other
    cores = min(host_cpus, int(os.environ.get("OMP_NUM_THREADS", host_cpus)))
    torch.set_num_threads(cores)
    cfg = O.OracleConfig(block_size=2048, vocab_size=128256, n_layer=16, n_head=32, n_local_heads=8, dim=2048,
                         intermediate_size=8192, rope_base=500000)
    dev = "cuda" if torch.cuda.is_available() else "cpu"   # generate the random weights fast, compute on the CPU
    P = {k: v.float().cpu() for k, v in O.init_params(cfg, seed=0, dtype=torch.float32, device=dev).items()}
    g = torch.Generator()
    g.manual_seed(1)
    prompt = torch.randint(0, cfg.vocab_size, (128,), generator=g)
    O.generate(cfg, P, prompt, 2, 1)  # warm the allocator and thread pool
    dec, pre = [], []
    for _ in range(repeats):
        tm = {}
        O.generate(cfg, P, prompt, new_tokens, 1, timers=tm)
        dec.append(tm["decode_latency"] / (new_tokens - 1))
        pre.append(tm["prefill_latency"])
    ms = 1e3 * sum(dec) / len(dec)
    return {"value": round(1e3 / ms, 3), "unit": "tok/s", "cores": cores, "host_cpus": host_cpus, "kind": "port",
            "ms_per_token": round(ms, 3), "prefill_s": round(sum(pre) / len(pre), 3),
            "sample": f"oracle (PyTorch CPU fp32) on Ladder-1B (dim 2048, 16 layers, 32q/8kv, FFN 8192, vocab 128256), "
                      f"B=1, prompt 128, greedy decode of {new_tokens} tokens, {repeats} runs"}


def decode_run(bm, model, prompt, B, T, K, W):
    """Prefill the prompt at batch B, capture the decode step, run W untimed + K timed steps from position T.
    Returns (ms per step, first token tensor, DecodeGraph)."""
    import torch

    new = max(K, W) + 1
    model.max_seq_length = -1            # new caches for this batch size
    model.setup_caches(B, T + max(new, 128))
    rows = prompt.view(1, -1).repeat(B, 1)
    first = bm.prefill(model, rows, torch.arange(T, device=prompt.device, dtype=torch.int32), greedy=True).clone()
    dg = bm.get_cuda_graphs_for_decode(model, prompt, B, new, first, greedy=True)
    states = [(s, s.clone()) for s in model.recurrent_states()]
    dg.reset(first)
    for _ in range(W):
        dg.replay()
    dg.reset(first)
    for s, kept in states:               # the timed steps start where the prompt ended, here too
        s.copy_(kept)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(K):
        dg.replay()
    torch.cuda.synchronize()
    ms = 1e3 * (time.perf_counter() - t0) / K
    model.check_device_errors()
    return ms, first, dg


def extra_batched(bm, model, prompt, T, batches=(2, 4, 8, 64), K=32, W=5):
    """The headline shard at other batch sizes (2: the one-kernel step; from 3 on the per-op kernels; 4, 8 and 64 are
    those of the benchmark set)."""
    cfg = model.config
    out = []
    for B in batches:
        ms, _, dg = decode_run(bm, model, prompt, B, T, K, W)
        nbytes = sum(bm.decode_bytes_per_step(cfg, B, T + i) for i in range(K)) / K
        gbps = nbytes / (ms * 1e-3) / 1e9
        out.append({"model": "gpt_ladder:ladder-70b-tp8", "batch": B, "prompt_len": T, "ms_per_step": round(ms, 4),
                    "tok_per_s": round(B * 1e3 / ms, 1), "bytes_per_step": int(nbytes), "achieved_GBps": round(gbps, 1),
                    "frac": round(gbps / HBM_PEAK_GBPS, 4), "steps": K,
                    "traffic": STEP_TRAFFIC_BYTES.get(("gpt_ladder:ladder-70b-tp8", B, T))})
        del dg
    return out


def extra_model_decode(bm, name, B, T, K=16, W=3):
    """Another decode configuration of the benchmark set, on a model of its own (random weights)."""
    import torch

    model = bm._load_model(name, "cuda", torch.bfloat16, seed=0, verbose=False)
    model.last_logits_only = True
    g = torch.Generator(device="cuda")
    g.manual_seed(1)
    prompt = torch.randint(0, model.config.vocab_size, (T,), device="cuda", generator=g)
    ms, _, dg = decode_run(bm, model, prompt, B, T, K, W)
    nbytes = sum(bm.decode_bytes_per_step(model.config, B, T + i) for i in range(K)) / K
    gbps = nbytes / (ms * 1e-3) / 1e9
    del dg, model
    torch.cuda.empty_cache()
    return {"model": name, "batch": B, "prompt_len": T, "ms_per_step": round(ms, 4), "tok_per_s": round(B * 1e3 / ms, 1),
            "bytes_per_step": int(nbytes), "achieved_GBps": round(gbps, 1), "frac": round(gbps / HBM_PEAK_GBPS, 4),
            "steps": K}


def fp8_bytes_per_step(cfg, B, pos):
    """decode_bytes_per_step with one byte per projection weight plus a bf16 scale per output row."""
    D, L, hd = cfg.dim, cfg.n_layer, cfg.head_dim
    Hq, Hkv, I, V = cfg.n_head_local, cfg.n_kv_local, cfg.ffn_local, cfg.output_rows
    nqkv = (Hq + 2 * Hkv) * hd
    w = L * (D * nqkv + D * Hq * hd + D * 2 * I + I * D) + V * D                   # one byte each
    scales = 2 * (L * (nqkv + D + 2 * I + D) + V)
    gains = 2 * (L * 2 * D + D)
    kv = 2 * (L * B * 2 * Hkv * hd * (pos + 1) + L * B * 2 * Hkv * hd) + 2 * B * D
    return w + scales + gains + kv


def extra_fp8(bm, model, prompt, T, K=32, W=5):
    """Weight-only e4m3 projections on the headline shard, batch 1 and 8.  Quantises `model` in place (call it last)."""
    from gpt_fast.quantize import quantize_model_fp8

    quantize_model_fp8(model)
    res = []
    for B, kernels in ((1, "one-kernel step (lr_ladder_decode_step_fp8), hipGraph replay"),
                       (8, "per-op (fp8 matrix-core bands), hipGraph replay")):
        ms, _, dg = decode_run(bm, model, prompt, B, T, K, W)
        if B == 1 and model._fused_step(B) is None:
            kernels = "per-op (fp8 matrix-vector kernel), hipGraph replay"
        nbytes = sum(fp8_bytes_per_step(model.config, B, T + i) for i in range(K)) / K
        gbps = nbytes / (ms * 1e-3) / 1e9
        res.append({"batch": B, "ms_per_step": round(ms, 4), "tok_per_s": round(B * 1e3 / ms, 1),
                    "bytes_per_step": int(nbytes), "achieved_GBps": round(gbps, 1),
                    "frac": round(gbps / HBM_PEAK_GBPS, 4), "steps": K, "kernels": kernels})
        del dg
    out = res[0]
    out["batch8"] = res[1]
    return out


def extra_prefill(bm, B=32, T=2048, reps=2):
    """Config 4: Ladder-8B, B x T prompt tokens, causal prefill, logits of the last position."""
    import torch

    model = bm._load_model("gpt_ladder:ladder-8b", "cuda", torch.bfloat16, seed=0, verbose=False)
    model.last_logits_only = True
    c = model.config
    g = torch.Generator(device="cuda")
    g.manual_seed(1)
    rows = torch.randint(0, c.vocab_size, (T,), device="cuda", generator=g).view(1, -1).repeat(B, 1)
    pos = torch.arange(T, device="cuda", dtype=torch.int32)
    model.setup_caches(B, T + 8)
    bm.prefill(model, rows, pos, greedy=True)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(reps):
        bm.prefill(model, rows, pos, greedy=True)
    torch.cuda.synchronize()
    sec = (time.perf_counter() - t0) / reps
    model.check_device_errors()
    D, L, hd, Hq, Hkv, I, V = c.dim, c.n_layer, c.head_dim, c.n_head_local, c.n_kv_local, c.ffn_local, c.output_rows
    lin = 2 * B * T * L * (D * (Hq + 2 * Hkv) * hd + D * Hq * hd + 3 * D * I) + 2 * B * V * D
    att = L * B * Hq * 2 * hd * T * T
    tf = (lin + att) / sec / 1e12
    return {"workload": f"gpt_ladder:ladder-8b, batch {B} x {T} prompt tokens, causal prefill, last-position logits",
            "seconds": round(sec, 4), "flop": int(lin + att), "achieved_TFLOPs": round(tf, 1),
            "peak_TFLOPs": MFMA_PEAK_TFLOPS, "frac": round(tf / MFMA_PEAK_TFLOPS, 4),
            "prompt_tok_per_s": round(B * T / sec, 1)}


FP32_MATRIX_PEAK_TFLOPS = 157.3   # v_mfma_f32, the recurrences' products


def _graph_us(calls, reps=5):
    """Mean microseconds per call of a list of launches, captured into one hipGraph and replayed."""
    import torch

    for c in calls[:2]:
        c()
    torch.cuda.synchronize()
    calls = calls * max(1, 16 // len(calls))      # (the replay's own cost is spread over them)
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        for c in calls:
            c()
    g.replay()
    torch.cuda.synchronize()
    ev0, ev1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    ev0.record()
    for _ in range(reps):
        g.replay()
    ev1.record()
    torch.cuda.synchronize()
    return 1e3 * ev0.elapsed_time(ev1) / (reps * len(calls))


def _kernel_row(name, us, bound, work):
    """`work`: bytes (bound hbm) or FLOP (bound mfma: bf16, mfma_f32)."""
    peak = {"hbm": HBM_PEAK_GBPS * 1e9, "mfma": MFMA_PEAK_TFLOPS * 1e12, "mfma_f32": FP32_MATRIX_PEAK_TFLOPS * 1e12}[bound]
    return {"kernel": name, "us": round(us, 2), "bound": bound, "work": int(work), "frac": round(work / (us * 1e-6) / peak, 4)}


def _residual_norm_row(D, rows, copies):
    import torch

    from gpt_fast import _hip

    n = copies(rows * D * 12)
    rnd = lambda *s: torch.randn(*s, device="cuda")
    xs, ds = [rnd(rows, D) for _ in range(n)], [rnd(rows, D).bfloat16() for _ in range(n)]
    xc, gain = torch.empty(rows, D, dtype=torch.bfloat16, device="cuda"), rnd(D).bfloat16()
    us = _graph_us([lambda i=i: _hip.residual_rmsnorm(xs[i], 2.0, ds[i], gain, xs[i], xc, 1e-5, gain_offset=1.0) for i in range(n)])
    return _kernel_row("lr_residual_rmsnorm (fp32 residual)", us, "hbm", rows * D * (4 + 2 + 4 + 2))


def gepolix_kernels(model, lasivik, B, T, decode):
    """The kernels the Gepolix model does not share, then the like kernels of the Lasivik model, as in mixer_kernels."""
    import torch

    from gpt_fast import _hip

    dev, BF = "cuda", torch.bfloat16
    S = 1 if decode else T
    rows, L, D = B * S, T + 8, model.config.dim
    pos = torch.arange(T, T + 1, dtype=torch.int32, device=dev) if decode else torch.arange(T, dtype=torch.int32, device=dev)
    rnd = lambda *s, dt=BF: torch.randn(*s, device=dev, dtype=torch.float32).to(dt)
    copies = lambda nbytes: max(2, min(64, (600 << 20) // max(int(nbytes), 1))) if decode else 2
    bytes_of = lambda t, n: [torch.empty(max(n, 16), dtype=torch.uint8, device=dev) for _ in range(t)]
    out = []
    blocks = {}
    for blk in model.layers:
        blocks.setdefault(blk.mixer.args.kind, blk)
        blocks.setdefault("moe" if blk.experts is not None else "dense", blk)
    # state space
    m = blocks["mamba2"].mixer
    a = m.args
    proj, y = rnd(rows, (m.proj_cols + 7) // 8 * 8), torch.empty(rows, m.y_cols, dtype=BF, device=dev)
    z, u, dt = proj[:, :m.inner], proj[:, m.inner:m.inner + m.conv_cols], proj[:, m.inner + m.conv_cols:m.proj_cols]
    cw, cb = rnd(m.conv_cols, a.taps), rnd(m.conv_cols)
    db, al, dd = rnd(a.heads), rnd(a.heads), rnd(a.heads)
    carried = 2 * B * a.heads * m.N * m.P * 4
    n = copies(carried)
    states, rings = [torch.zeros(B, a.heads, m.N, m.P, device=dev) for _ in range(n)], torch.zeros(B, a.taps, m.conv_cols, dtype=BF, device=dev)
    name = f"{a.heads} heads of {m.N} x {m.P}"
    act_bytes = rows * 2 * (2 * m.inner + m.conv_cols + a.heads)
    if decode:
        us = _graph_us([lambda s=s: _hip.ssd_step(z, u, dt, cw, cb, rings, db, al, dd, pos, s, y, B, a.heads, a.groups) for s in states])
        out.append(_kernel_row(f"lr_ssd_step ({name}; convolution included)", us, "hbm", carried + act_bytes))
    else:
        c = rnd(rows, m.conv_cols)
        us = _graph_us([lambda: _hip.causal_conv(u, cw, cb, rings, pos, c, B, S)])
        out.append(_kernel_row("lr_causal_conv", us, "hbm", 4 * rows * m.conv_cols))
        scratch = bytes_of(1, _hip.ssd_scratch_bytes(B, S, a.heads, m.N, m.P, BF))[0]
        us = _graph_us([lambda s=s: _hip.ssd(z, c, dt, db, al, dd, pos, s, y, B, S, a.heads, a.groups, scratch=scratch) for s in states])
        out.append(_kernel_row(f"lr_ssd ({name})", us, "hbm", act_bytes))
        # per token and head: the state is multiplied by C and added B x^T to; inside a chunk of 64 the scores and their sums
        flop = rows * a.heads * (4 * m.N * m.P + 2 * 64 * (m.N + m.P) // 2)
        out.append(dict(out[-1], bound="mfma", work=int(flop), frac=round(flop / (us * 1e-6) / (MFMA_PEAK_TFLOPS * 1e12), 4)))
    gain = rnd(m.inner)
    us = _graph_us([lambda: _hip.parts_norm(y, gain, a.norm_groups, a.heads, a.vdim, m.P, 1e-5)])
    out.append(_kernel_row("lr_parts_norm", us, "hbm", 4 * rows * m.inner))
    del states, proj, y, z, u, dt
    # attention
    m = blocks["attention"].mixer
    a = m.args
    seen = min(T + 1, a.window)
    proj, y, bias = rnd(rows, m.proj_cols), torch.empty(rows, m.y_cols, dtype=BF, device=dev), rnd(m.proj_cols)
    nbytes = B * m.kv_cols * 2 * seen
    n = copies(nbytes)
    caches = [rnd(B, L, m.kv_cols) for _ in range(n)]
    rope = torch.zeros(L, a.rot_dims // 2, 2, device=dev)
    q = proj[:, :a.heads * m.dk]
    us = _graph_us([lambda c=c: _hip.bias_rope_cache(proj, bias, rope, pos, c, B, S, a.heads, a.kv_heads, m.dk, m.dv) for c in caches])
    out.append(_kernel_row("lr_bias_rope_cache", us, "hbm", 4 * rows * m.proj_cols))
    name = f"{a.heads} / {a.kv_heads} heads of {a.dim}, window {a.window}"
    if decode:
        scratch = bytes_of(1, _hip.window_decode_scratch_bytes(B, a.heads, a.kv_heads, m.dv, a.window, L))[0]
        us = _graph_us([lambda c=c: _hip.window_decode(q, c, y, pos, scratch, B, a.heads, a.kv_heads, m.dk, m.dv, a.window, a.scale)
                        for c in caches])
        out.append(_kernel_row(f"lr_window_decode ({name}; two launches)", us, "hbm", nbytes))
    else:
        kv = caches[0].view(B * L, -1)
        us = _graph_us([lambda: _hip.window_attention(q, kv, y, pos, B, S, a.heads, m.dk, m.dv, a.window, L, L, a.scale,
                                                      kv_heads=a.kv_heads)])
        keys = sum(min(i + 1, a.window) for i in range(T))
        out.append(_kernel_row(f"lr_window_attention ({name})", us, "mfma", B * a.heads * keys * 2 * (a.dim + a.vdim)))
    del caches, proj, y, q
    # feed-forwards: the mixture; the dense one of the same model (as the Lasivik model's, two launches) for comparison
    x = blocks["moe"].experts
    xc = rnd(rows, D)
    n = copies(x.n * 3 * x.ff * D * 2)
    w1s, w2s = [rnd(x.n, 2 * x.ff, D) for _ in range(n)], [rnd(x.n, D, x.ff) for _ in range(n)]
    router, rb = rnd(x.n + x.shared, D), rnd(x.n)
    eo, ids, wts = torch.empty(rows * x.top, D, dtype=BF, device=dev), torch.empty(rows, x.top, dtype=torch.int32, device=dev), torch.empty(rows, x.top, device=dev)
    counts, scratch = torch.zeros(x.n, dtype=torch.int32, device=dev), bytes_of(1, _hip.moe_scratch_bytes(rows, x.n, x.top, x.ff, BF))[0]
    shared = rnd(rows, blocks["moe"].beside) if x.shared else None
    gate = torch.empty(rows, device=dev)
    descs = [_hip.moe_desc(xc, router, rb, w1s[i], w2s[i], eo, ids, wts, gate, counts, scratch, shared) for i in range(n)]
    _hip.moe(descs[0])
    for d in descs:
        d.routed = int(decode)      # a decode step routes beside its projections
    us = _graph_us([lambda d=d: _hip.moe(d) for d in descs])
    name = f"{x.n} experts of {x.ff}, top {x.top}"
    if decode:
        wbytes = len(ids.unique()) * 3 * x.ff * D * 2
        out.append(_kernel_row(f"lr_moe ({name}; up, down)", us, "hbm", wbytes + 2 * rows * x.top * D))
    else:
        out.append(_kernel_row(f"lr_moe ({name})", us, "mfma", 6 * rows * x.top * x.ff * D))
    del w1s, w2s
    I = blocks["dense"].beside
    n = copies(3 * I * D * 2)
    w1s, w2s = [rnd(2 * I, D) for _ in range(n)], [rnd(D, I) for _ in range(n)]
    act, h, d = torch.empty(rows, I, dtype=BF, device=dev), torch.empty(rows, 2 * I, dtype=BF, device=dev), torch.empty(rows, D, dtype=BF, device=dev)

    def dense_ff(i):
        _hip.linear_swiglu_out(xc, w1s[i], act, h)
        _hip.linear(act, w2s[i], d)
    us = _graph_us([lambda i=i: dense_ff(i) for i in range(n)])
    out.append(_kernel_row(f"dense feed-forward of {I} (two launches)", us, "hbm" if decode else "mfma", 6 * I * D if decode else 6 * rows * I * D))
    del w1s, w2s, act, h
    # residual and norm
    n = copies(rows * D * (12 + 2 * x.top))
    xs, ds, es = ([rnd(rows, D, dt=torch.float32) for _ in range(n)], [rnd(rows, D) for _ in range(n)],
                  [rnd(rows * x.top, D) for _ in range(n)])
    one, g, b = rnd(1), rnd(D), rnd(D)
    us = _graph_us([lambda i=i: _hip.residual_tanh(xs[i], ds[i], one, g, b, xs[i], xc) for i in range(n)])
    out.append(_kernel_row("lr_residual_tanh", us, "hbm", rows * D * 12))
    us = _graph_us([lambda i=i: _hip.residual_tanh(xs[i], ds[i], one, g, b, xs[i], xc, (es[i], wts)) for i in range(n)])
    out.append(_kernel_row("lr_residual_tanh, experts' rows added", us, "hbm", rows * D * (12 + 2 * x.top)))
    del xs, ds, es, xc
    torch.cuda.empty_cache()
    return out + [dict(r, kernel="lasivik: " + r["kernel"]) for r in mixer_kernels(lasivik, None, B, T, decode)]


def mixer_kernels(hybrid, dense, B, T, decode):
    """The kernels the hybrid and the dense model do not share, at `B` sequences of `T` tokens (decode: one more token on
    top of them), on tensors of those models' shapes.  Inputs are rotated through copies that together exceed the caches."""
    import torch

    from gpt_fast import _hip
    from gpt_fast.mixers import rotate_half_table

    dev, BF = "cuda", torch.bfloat16
    S = 1 if decode else T
    rows = B * S
    pos = torch.arange(T, T + 1, dtype=torch.int32, device=dev) if decode else torch.arange(T, dtype=torch.int32, device=dev)
    rnd = lambda *s, dt=BF: torch.randn(*s, device=dev, dtype=torch.float32).to(dt)
    copies = lambda nbytes: max(2, min(64, (600 << 20) // max(int(nbytes), 1))) if decode else 2
    out = []
    mixers = {blk.mixer.args.kind: blk.mixer for blk in hybrid.layers}
    for kind in ("gla", "retention"):
        m = mixers[kind]
        a = m.args
        carried = 2 * B * a.heads * a.dim * a.vdim * 4
        n = copies(carried)
        states = [torch.zeros(B, a.heads, a.dim, a.vdim, device=dev) for _ in range(n)]
        proj, y = rnd(rows, (m.proj_cols + 7) // 8 * 8), torch.empty(rows, m.y_cols, dtype=BF, device=dev)
        need = _hip.linear_attention_scratch_bytes(B, S, a.heads, a.dim, a.vdim, kind == "gla")
        scratch = torch.empty(need, dtype=torch.uint8, device=dev) if need else None
        if kind == "gla":
            kw = dict(q_scale=a.dim ** -0.5, norm=rnd(a.vdim), gate=(rnd(a.heads * a.dim, a.decay_rank), rnd(a.heads * a.dim), a.tau))
        else:
            kw = dict(k_scale=a.dim ** -0.5, rope=rotate_half_table(T + 8, a.rot_dims, a.rot_base).to(dev),
                      head_decay=torch.tensor(a.decay, device=dev).log())
        us = _graph_us([lambda s=s: _hip.linear_attention(proj, y, s, pos, B, S, a.heads, a.dim, a.vdim, 1e-5, scratch=scratch, **kw)
                        for s in states])
        # per token and head: the state is multiplied by q and added k v^T to; inside a chunk of 16 the scores and their sums
        flop = rows * a.heads * (4 * a.dim * a.vdim + 2 * 16 * (a.dim + a.vdim) // 2)
        out.append(_kernel_row(f"lr_linear_attention ({kind}, {a.heads} heads of {a.dim} x {a.vdim})", us,
                               "hbm" if decode else "mfma_f32", carried + 2 * rows * (m.proj_cols + m.y_cols) if decode else flop))
        del states, proj, y, scratch
    m = mixers["latent_attention"]
    a = m.args
    L = T + 8
    nq, nv = a.heads * a.dim, a.heads * a.vdim
    seen = min(T + 1, a.window)
    if decode:
        nbytes = B * seen * m.rank_p * 2 + (nq + nv) * m.rank_p * 2
        n = copies(nbytes)
        caches, ups = [rnd(B, L, m.rank_p) for _ in range(n)], [rnd(nq + nv, m.rank_p) for _ in range(n)]
        q, c, gain = rnd(rows, nq), rnd(rows, m.rank_p), rnd(m.rank_p)
        y = torch.empty(rows, nv, dtype=BF, device=dev)
        scratch = torch.empty(_hip.latent_attention_scratch_bytes(B, 1, a.heads, m.rank_p, a.window, L), dtype=torch.uint8, device=dev)
        us = _graph_us([lambda i=i: _hip.latent_attention(q, ups[i][:nq], ups[i][nq:], caches[i], y, pos, scratch, B, 1, a.heads, a.dim,
                                                          a.vdim, a.window, a.scale, new=(c, gain, a.kv_rank, 1e-5)) for i in range(n)])
        out.append(_kernel_row(f"lr_latent_attention ({a.heads} heads, rank {a.kv_rank}, window {a.window}; three launches)", us, "hbm", nbytes))
        del caches, ups
    else:
        nk = min(T + a.window - 1, L)
        q, kv, y = rnd(rows, nq), rnd(B * nk, nq + nv), torch.empty(rows, nv, dtype=BF, device=dev)
        us = _graph_us([lambda: _hip.window_attention(q, kv, y, pos, B, T, a.heads, a.dim, a.vdim, a.window, nk, L, a.scale)] * 2)
        keys = sum(min(i + 1, a.window) for i in range(T))
        out.append(_kernel_row(f"lr_window_attention ({a.heads} heads of {a.dim}, window {a.window})", us, "mfma",
                               B * a.heads * keys * 2 * (a.dim + a.vdim)))
    if dense is None:
        out.append(_residual_norm_row(hybrid.config.dim, rows, copies))
        return out
    # the dense model's counterpart
    d = dense.config
    Hq, Hkv, hd = d.n_head_local, d.n_kv_local, d.head_dim
    nbytes = 2 * B * (T + 1) * Hkv * hd * 2
    n = copies(nbytes)
    kcs, vcs = [rnd(B, Hkv, L, hd) for _ in range(n)], [rnd(B, Hkv, L, hd) for _ in range(n)]
    q, y = rnd(rows, Hq * hd), torch.empty(rows, Hq * hd, dtype=BF, device=dev)
    if decode:
        scratch = torch.empty(_hip.attn_decode_scratch_bytes(B, Hq, hd, L) // 4, device=dev)
        us = _graph_us([lambda i=i: _hip.attn_decode(q, kcs[i], vcs[i], pos, y, scratch, B, Hq, Hkv, hd) for i in range(n)])
        out.append(_kernel_row(f"dense: lr_attn_decode ({Hq} / {Hkv} heads of {hd}; two launches)", us, "hbm", nbytes))
    else:
        us = _graph_us([lambda: _hip.attn_prefill(q, kcs[0], vcs[0], pos, y, B, T, Hq, Hkv, hd)] * 2)
        out.append(_kernel_row(f"dense: lr_attn_prefill ({Hq} / {Hkv} heads of {hd})", us, "mfma", B * Hq * (T * (T + 1) // 2) * 4 * hd))
    del kcs, vcs
    # the norms, a launch per sublayer in both
    out.append(_residual_norm_row(hybrid.config.dim, rows, copies))
    D = hybrid.config.dim
    n = copies(rows * D * 12)
    bs, ds = [rnd(rows, D) for _ in range(n)], [rnd(rows, D) for _ in range(n)]
    xc, gain = torch.empty(rows, D, dtype=BF, device=dev), rnd(D)
    us = _graph_us([lambda i=i: _hip.add_rmsnorm(bs[i], ds[i], None, gain, bs[i], xc, 1e-5) for i in range(n)])
    out.append(_kernel_row("dense: lr_add_rmsnorm", us, "hbm", rows * D * 8))
    torch.cuda.empty_cache()
    return out


GEPOLIX_PAIRS = {"1b": ("gpt_gepolix:gepolix-1b", "gpt_lasivik:lasivik-1b"), "8b": ("gpt_gepolix:gepolix-8b", "gpt_lasivik:lasivik-8b")}
LASIVIK_PAIRS = {"1b": ("gpt_lasivik:lasivik-1b", "gpt_dense:ladder-1b"), "8b": ("gpt_lasivik:lasivik-8b", "gpt_dense:ladder-8b")}


def family_compare(workload, pairs, kernels, sizes, T=1792, K=32, W=5):
    """Prefill and decode throughput of the models of each pair, and their kernels alone.  One JSON line."""
    import torch

    import benchmark as bm
    from gpt_fast import _hip

    _hip.load()
    out = {"workload": workload, "prompt_len": T, "data": "synthetic", "dtype": "bf16", "models": [], "kernels": []}
    for size in sizes:
        models = [bm._load_model(name, "cuda", torch.bfloat16, seed=0, verbose=False) for name in pairs[size]]
        g = torch.Generator(device="cuda")
        g.manual_seed(1)
        prompt = torch.randint(0, 100000, (T,), device="cuda", generator=g)
        for name, model in zip(pairs[size], models):
            model.last_logits_only = True
            row = {"model": name, "parameters": sum(p.numel() for p in model.parameters()), "prefill": [], "decode": []}
            count = sum(p.numel() for n, p in model.named_parameters() if p.dim() == 2 and not n.startswith(("tok_emb", "output")))
            for x in (blk.experts for blk in model.layers if getattr(blk, "experts", None) is not None):
                count += (x.w1.numel() + x.w2.numel()) * x.top // x.n
            for B in (1, 8):
                model.max_seq_length = -1
                model.setup_caches(B, T + 8)
                print(f"{name}: prefill, batch {B}", file=sys.stderr, flush=True)
                rows, pos = prompt.view(1, -1).repeat(B, 1), torch.arange(T, device="cuda", dtype=torch.int32)
                bm.prefill(model, rows, pos, greedy=True)
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                for _ in range(3):
                    bm.prefill(model, rows, pos, greedy=True)
                torch.cuda.synchronize()
                sec = (time.perf_counter() - t0) / 3
                row["prefill"].append({"batch": B, "ms": round(1e3 * sec, 3), "tok_per_s": round(B * T / sec, 1),
                                       "projection_TFLOPs": round(2 * count * B * T / sec / 1e12, 1)})
            for B in (1, 8, 32):
                ms, _, dg = decode_run(bm, model, prompt, B, T, K, W)
                nbytes = bm.decode_bytes_per_step(model if hasattr(model, "decode_bytes") else model.config, B, T + K // 2)
                row["decode"].append({"batch": B, "ms_per_step": round(ms, 4), "tok_per_s": round(B * 1e3 / ms, 1),
                                      "bytes_per_step": int(nbytes), "frac": round(nbytes / (ms * 1e-3) / 1e9 / HBM_PEAK_GBPS, 4)})
                del dg
            model.check_device_errors()
            model.release_workspace()
            out["models"].append(row)
        for B, decode in ((1, False), (8, False), (1, True), (8, True), (32, True)):
            out["kernels"].append({"size": size, "batch": B, "phase": "decode" if decode else "prefill",
                                   "rows": kernels(models[0], models[1], B, T, decode)})
            print(f"{size} kernels: batch {B}, {'decode' if decode else 'prefill'}", file=sys.stderr, flush=True)
        del models, model
        torch.cuda.empty_cache()
    print(json.dumps(out), flush=True)


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=127)
    ap.add_argument("--warmup", type=int, default=20)
    ap.add_argument("--batch", type=int, default=1)
    ap.add_argument("--prompt", type=int, default=2048)
    ap.add_argument("--model", type=str, default="gpt_ladder:ladder-70b-tp8")
    ap.add_argument("--no-cpu-baseline", action="store_true")
    ap.add_argument("--no-extras", action="store_true",
                    help="skip the extra keys (other batch sizes, fp8 weights, the prefill-heavy configuration)")
    ap.add_argument("--per-op", action="store_true",
                    help="decode with one kernel per operation (captured in the hipGraph) instead of the persistent "
                         "one-kernel step: the comparison point, not the headline")
    ap.add_argument("--fp8", action="store_true",
                    help="weight-only e4m3 projections (gpt_fast.quantize): a profiling aid, not the headline")
    ap.add_argument("--lasivik", nargs="*", choices=sorted(LASIVIK_PAIRS), metavar="SIZE",
                    help="the Lasivik family beside the dense one instead of the headline (sizes 1b and 8b; default both)")
    ap.add_argument("--gepolix", nargs="*", choices=sorted(GEPOLIX_PAIRS), metavar="SIZE",
                    help="the Gepolix family beside the Lasivik one instead of the headline (sizes 1b and 8b; default both)")
    ap.add_argument("--calibrate-copy", action="store_true",
                    help="also run a plain 1 GiB device copy (reads 1 GiB, writes 1 GiB) a few times: under "
                         "rocprofv3 --pmc its FETCH_SIZE / WRITE_SIZE readings calibrate the counters' unit")
    args = ap.parse_args()
    if args.gpus != 1 or int(os.environ.get("WORLD_SIZE", "1")) != 1:
        print("bench.py measures ONE tensor-parallel rank's shard on ONE GPU (partial sums stay local, no "
              "collectives); --gpus must be 1.", file=sys.stderr)
        sys.exit(2)

    import torch

    import benchmark as bm
    from gpt_fast import _hip

    assert torch.cuda.is_available(), "bench.py needs the MI355X"
    if args.lasivik is not None:
        return family_compare("lasivik beside dense", LASIVIK_PAIRS, mixer_kernels, args.lasivik or sorted(LASIVIK_PAIRS))
    if args.gepolix is not None:
        return family_compare("gepolix beside lasivik", GEPOLIX_PAIRS, gepolix_kernels, args.gepolix or sorted(GEPOLIX_PAIRS))
    _hip.load()
    dev = "cuda"
    B, T, K, W = args.batch, args.prompt, args.steps, args.warmup
    model = bm._load_model(args.model, dev, torch.bfloat16, seed=0, verbose=False)
    model.last_logits_only = True          # prefill is set-up here, not the timed region
    if args.per_op:
        model.use_fused_step = False
    if args.fp8:
        from gpt_fast.quantize import quantize_model_fp8

        quantize_model_fp8(model)
    cfg = model.config
    new = max(K, W, 127) + 1
    g = torch.Generator(device=dev)
    g.manual_seed(1)
    prompt = torch.randint(0, cfg.vocab_size, (T,), device=dev, generator=g)
    model.setup_caches(B, T + new)

    # ---- set-up: prefill the prompt (eager), capture the decode step
    rows = prompt.view(1, -1).repeat(B, 1)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    first = bm.prefill(model, rows, torch.arange(T, device=dev, dtype=torch.int32), greedy=True).clone()
    torch.cuda.synchronize()
    prefill_s = time.perf_counter() - t0
    dg = bm.get_cuda_graphs_for_decode(model, prompt, B, new, first, greedy=True)

    if args.calibrate_copy:
        src = torch.zeros(1 << 30, dtype=torch.uint8, device=dev)
        dst = torch.empty_like(src)
        for _ in range(3):
            dst.copy_(src)
        torch.cuda.synchronize()
        del src, dst

    # ---- W untimed steps, then exactly K timed steps from position T
    dg.reset(first)
    for _ in range(W):
        dg.replay()
    dg.reset(first)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(K):
        dg.replay()
    torch.cuda.synchronize()
    elapsed = time.perf_counter() - t0
    model.check_device_errors()   # raises if any timed step did not do its work (expired wait, position out of range)
    ms_per_step = 1e3 * elapsed / K
    tokens = dg.history[0, : min(K, 16)].tolist()

    bytes_per_step = fp8_bytes_per_step if args.fp8 else bm.decode_bytes_per_step
    step_bytes = sum(bytes_per_step(cfg, B, T + i) for i in range(K)) / K
    step_gbps = step_bytes / (ms_per_step * 1e-3) / 1e9

    # ---- dominant kernel, timed with HIP events on the stream it is launched on (torch's current stream)
    ev0, ev1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    fused = getattr(model, "use_fused_step", False) and hasattr(model, "decode_step_fused") and \
        model._fused_step(B) is not None
    if fused:
        # the whole step is ONE kernel (k_ladder_step): algorithmic bytes per launch = bytes per step
        pos = torch.tensor([T], dtype=torch.int32, device=dev)
        tok = first.view(B, 1).to(torch.int32).contiguous()
        for _ in range(3):
            model.decode_step_fused(tok, pos)
        reps = 30
        torch.cuda.synchronize()
        ev0.record()
        for _ in range(reps):
            model.decode_step_fused(tok, pos)
        ev1.record()
        torch.cuda.synchronize()
        k_us = 1e3 * ev0.elapsed_time(ev1) / reps
        model.check_device_errors()
        k_bytes = bytes_per_step(cfg, B, T)
        k_name = (f"k_ladder_step (one persistent launch = the whole decode step at position {T}: "
                  f"{cfg.n_layer} layers + lm_head, M={B}{', e4m3 weights' if args.fp8 else ''})")
    else:
        # per-op path: the weight-streaming GEMV on the w1 (up+gate) projection, a distinct matrix per launch
        w1s = [blk.feed_forward.w1.weight for blk in model.layers] if hasattr(model.layers[0], "feed_forward") else \
            [blk.attention.wqkv1.weight for blk in model.layers]
        N, Kdim = w1s[0].shape
        x = torch.randn(B, Kdim, device=dev).to(torch.bfloat16)
        y = torch.empty(B, N, device=dev, dtype=torch.bfloat16)
        if args.fp8:
            scs = [(blk.feed_forward.w1 if hasattr(blk, "feed_forward") else blk.attention.wqkv1).scales
                   for blk in model.layers]
            run = lambda i: _hip.linear_fp8_multi((x, w1s[i], scs[i], y, _hip.EPI_NONE)) if B <= 16 else \
                _hip.linear_fp8(x, w1s[i], scs[i], y)
        else:
            run = lambda i: _hip.linear(x, w1s[i], y)
        for i in range(8):
            run(i)
        reps = 3
        torch.cuda.synchronize()
        ev0.record()
        for _ in range(reps):
            for i in range(len(w1s)):
                run(i)
        ev1.record()
        torch.cuda.synchronize()
        k_us = 1e3 * ev0.elapsed_time(ev1) / (reps * len(w1s))
        wbytes = 1 if args.fp8 else 2
        k_bytes = wbytes * N * Kdim + 2 * (B * Kdim + B * N)
        kern = ("k_gemv_fp8_multi" if B == 1 else "k_stream_gemm (e4m3 bands)") if args.fp8 else \
            ("k_gemv" if B <= 4 else "k_stream_gemm")
        k_name = f"{kern} (w1 up+gate projection, [{N} x {Kdim}] {'e4m3' if args.fp8 else 'bf16'}, M={B})"
    k_gbps = k_bytes / (k_us * 1e-6) / 1e9

    # ---- the read rate this machine reaches: a plain streaming read of 8 GiB by every CU
    ceil_buf = torch.empty(8 << 30, dtype=torch.uint8, device=dev)
    ceil_buf.view(torch.int32).fill_(0x01010101)
    sink = torch.zeros(1, dtype=torch.int32, device=dev)
    for _ in range(2):
        _hip.stream_read(ceil_buf, sink)
    torch.cuda.synchronize()
    ev0.record()
    for _ in range(5):
        _hip.stream_read(ceil_buf, sink)
    ev1.record()
    torch.cuda.synchronize()
    ceiling_gbps = 5 * ceil_buf.numel() / (ev0.elapsed_time(ev1) * 1e-3) / 1e9
    del ceil_buf

    out = {
        "metric": "decode_tokens_per_sec", "value": round(B * 1e3 / ms_per_step, 2), "unit": "tok/s",
        "n_gpus": 1, "steps": K, "warmup": W, "ms_per_step": round(ms_per_step, 4), "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16 (e4m3 weights)" if args.fp8 else "bf16",
        "data": "synthetic",
        "config": {"workload": f"{args.model} rank shard (dim {cfg.dim}, {cfg.n_layer} layers, {cfg.n_head_local} q / "
                               f"{cfg.n_kv_local} kv heads, FFN {cfg.ffn_local}, lm_head rows {cfg.output_rows}), "
                               f"batch {B}, prompt {T}, greedy decode, hipGraph replay per step"
                               + (", one kernel per operation" if args.per_op else "")
                               + (", weight-only e4m3 projections" if args.fp8 else ""),
                   "batch": B, "prompt_len": T, "virtual_tp": cfg.tp_world_size},
        "ms_per_token": round(ms_per_step, 4),
        "prefill_s": round(prefill_s, 4),
        "roofline": {"bound": "hbm", "kernel": k_name,
                     "achieved": round(k_gbps, 1), "peak": HBM_PEAK_GBPS, "unit": "GB/s",
                     "frac": round(k_gbps / HBM_PEAK_GBPS, 4),
                     "traffic": TRAFFIC_BYTES_PER_LAUNCH.get((args.model, B, T)) if (fused or B > 4) and not args.fp8 else None,
                     "bytes_per_launch": int(k_bytes), "avg_launch_us": round(k_us, 3),
                     "measured_read_ceiling": round(ceiling_gbps, 1),
                     "frac_of_measured_ceiling": round(k_gbps / ceiling_gbps, 4)},
        "step_roofline": {"bound": "hbm", "achieved": round(step_gbps, 1), "peak": HBM_PEAK_GBPS, "unit": "GB/s",
                          "frac": round(step_gbps / HBM_PEAK_GBPS, 4), "bytes_per_step": int(step_bytes)},
        "first_tokens": tokens,
    }
    del dg
    if not args.no_extras and args.model == "gpt_ladder:ladder-70b-tp8" and B == 1:
        out["batched"] = extra_batched(bm, model, prompt, T)
        out["fp8"] = extra_fp8(bm, model, prompt, T)
        del model
        torch.cuda.empty_cache()
        out["prefill"] = extra_prefill(bm)
        # the other decode configurations of the benchmark set: the 8B model at batch 16, the 405B rank shard at batch 16
        out["batched"].append(extra_model_decode(bm, "gpt_ladder:ladder-8b", 1, 1024, K=32, W=5))   # one-kernel step
        out["batched"].append(extra_model_decode(bm, "gpt_ladder:ladder-8b", 16, 1024))
        out["batched"].append(extra_model_decode(bm, "gpt_ladder:ladder-405b-tp8", 16, 4096))
    else:
        del model
    torch.cuda.empty_cache()
    if not args.no_cpu_baseline:
        out["cpu_baseline"] = cpu_baseline()
    print(json.dumps(out), flush=True)


if __name__ == "__main__":
    main()
