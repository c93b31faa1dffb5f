"""Trace runner: replays given token ids through a model, step by step, and writes the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come as JSON lines on standard input,
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["a"]}
For every step in which logits are wanted DIR/<step>.f32 receives them (little-endian fp32, in the order of
the entries and their `want`), then "done <step>" is printed. The model, its step function, caches and
kernels are the ones generate() uses; requests keep their cache from step to step until they end."""
import argparse
import json
import os
import sys


def _parse(argv):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay token ids through a model and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the logits, <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=2048, help="capacity new caches start with (they grow when needed)")
    return ap.parse_args(argv)


def _write(path: str, rows) -> None:
    import torch

    data = torch.cat(rows).to(torch.float32).cpu().contiguous().numpy().astype("<f4").tobytes()
    part = path + ".part"
    with open(part, "wb") as f:
        f.write(data)
    os.replace(part, path)


def run(lm, device, lines, out_dir: str, max_tokens: int, say) -> None:
    """Replay `lines` (an iterable of JSON texts) through lm; say(text) reports finished steps."""
    import torch

    from .modules.kvcache.hybridcache import MuiCachePool

    pool = MuiCachePool(lambda: lm.create_cache(1, max(1, max_tokens)))
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = []
        for entry in step["entries"]:
            want = list(entry.get("want", ()))
            if not entry["tokens"]:
                continue
            ids = torch.tensor([entry["tokens"]], dtype=torch.int64, device=device)
            out = lm(input_ids=ids, past_key_values=pool.get(entry["id"]), use_cache=True, logits_positions=want)
            if want:
                rows.append(out.logits[0])
        if rows:
            _write(os.path.join(out_dir, f"{step['step']}.f32"), rows)
        else:
            torch.cuda.synchronize()
        for request in step.get("end", ()):
            pool.release(request)
        say(f"done {step['step']}")


def main(argv=None) -> int:
    args = _parse(argv)
    from . import _build

    _build.ensure_built()
    import torch

    from .modules.models.registry import load_model

    if not torch.cuda.is_available():
        print("trace_run: no GPU is visible", file=sys.stderr)
        return 1
    torch.backends.cuda.matmul.allow_tf32 = False
    device = torch.device("cuda", 0)
    with torch.no_grad():
        lm = load_model(args.model, dtype=getattr(torch, args.dtype), device=device)
        run(lm, device, sys.stdin, args.out, args.max_tokens, lambda text: print(text, flush=True))
    return 0
