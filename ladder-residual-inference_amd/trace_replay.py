"""Replay of recorded token steps: feeds given token ids to a checkpoint's model and writes the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps.jsonl

One step per line of standard input:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["a"]}
`tokens` are the request's next ones, continuing where its last step ended; `want` are places among them.  A step that
wants something writes <out>/<step>.f32 (fp32 [wanted, vocab], in the order of `want`); every step prints "done <step>".
Requests listed in `end` are finished and give their place in the cache back.  Nothing is sampled: the model's forward,
caches and kernels are those of generation.  Requests follow one another; two at a time are refused.

Exit code 3: the model's family does not run in the dtype asked for."""
import argparse
import json
import os
import sys

REFUSED = 3


def build_parser():
    p = argparse.ArgumentParser(description="Replay a trace of token steps and write logits.")
    p.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    p.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    p.add_argument("--out", required=True, help="folder for the logits")
    p.add_argument("--max-tokens", type=int, required=True, help="most tokens a live request holds")
    return p


class Replay:
    """One model with a cache for one sequence, and the request that holds it."""

    def __init__(self, model, max_tokens: int):
        self.model = model
        self.max_tokens = max_tokens
        model.setup_caches(1, max_tokens)
        self.live, self.length = None, 0

    def feed(self, rid, tokens, want):
        """Runs a request's next tokens; fp32 logits [len(want), vocab] on the host, None if nothing is wanted."""
        import torch

        if self.live is None:
            self.live, self.length = rid, 0
        if rid != self.live:
            raise RuntimeError(f"request {rid!r} while {self.live!r} is live: requests follow one another")
        n = len(tokens)
        if not n:
            return None
        if self.length + n > self.max_tokens:
            raise RuntimeError(f"request {rid!r} holds more than --max-tokens {self.max_tokens} tokens")
        dev = self.model.output.weight.device
        idx = torch.tensor([tokens], dtype=torch.int32, device=dev)
        pos = torch.arange(self.length, self.length + n, dtype=torch.int32, device=dev)
        with torch.no_grad():
            logits = self.model(idx, pos)
        self.length += n
        out = logits[0, torch.tensor(want, dtype=torch.int64, device=dev)].float().cpu() if want else None
        self.model.check_device_errors()
        return out

    def end(self, rid):
        if rid == self.live:
            self.live, self.length = None, 0


def main(argv=None) -> int:
    args = build_parser().parse_args(argv)
    import build
    import torch
    from gpt_fast import _hip
    from gpt_fast.checkpoint import load_pretrained, pretrained_class

    dtype = getattr(torch, args.dtype)
    cls = pretrained_class(args.model)
    if dtype not in cls.supported_dtypes:
        print(f"{cls.__name__} does not run in {args.dtype}", file=sys.stderr)
        return REFUSED
    _hip.use_library(build.ready_for(cls.family, verbose=False))
    replay = Replay(load_pretrained(args.model, "cuda", dtype), args.max_tokens)
    for line in iter(sys.stdin.readline, ""):
        if not line.strip():
            continue
        step = json.loads(line)
        rows = [replay.feed(e["id"], e["tokens"], e["want"]) for e in step["entries"]]
        rows = [r for r in rows if r is not None]
        if rows:
            with open(os.path.join(args.out, f"{step['step']}.f32"), "wb") as f:
                f.write(torch.cat(rows).numpy().astype("<f4").tobytes())
        for rid in step.get("end", []):
            replay.end(rid)
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
