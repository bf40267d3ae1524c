"""Trace replay (`bin/trace_run`) and plain generation (`python -m adam_amd`) from a model folder or file."""
import argparse
import json
import os
import sys

import numpy as np


def built_library():
    """The shared library, compiled first where a checkout has none."""
    from . import build
    if not os.environ.get("ADAMAH_LIB_PATH") and not os.path.exists(build.OUT):
        print("compiling the kernels for gfx950 ...", file=sys.stderr, flush=True)
        build.build(verbose=False)


def replay(engine, lines, out_dir, done):
    """Run every step of `lines`; `done(step)` after each."""
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        parts = [engine.score(e["id"], e["tokens"], e.get("want", ())) for e in step["entries"]]
        for name in step.get("end", ()):
            engine.release(name)
        logits = np.concatenate(parts) if parts else np.empty((0, 0), np.float32)
        if logits.shape[0]:
            final = os.path.join(out_dir, f"{step['step']}.f32")
            with open(final + ".part", "wb") as f:
                f.write(logits.astype("<f4").tobytes())
            os.replace(final + ".part", final)
        done(step["step"])


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token ids and write logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=0,
                    help="most tokens live requests hold together; what a sequence keeps does not grow with it")
    ap.add_argument("--slots", type=int, default=8, help="requests that may be live at once")
    a = ap.parse_args(argv)
    built_library()
    from . import adamah
    from .models import load_engine
    gpu = adamah.init()
    try:
        engine = load_engine(gpu, a.model, dtype=a.dtype, batch=a.slots)
        replay(engine, sys.stdin, a.out, lambda n: print(f"done {n}", flush=True))
    finally:
        gpu.shutdown()
    return 0


def generate_main(argv=None):
    ap = argparse.ArgumentParser(prog="python -m adam_amd", description="Generate token ids from a GGUF file or a model folder.")
    ap.add_argument("model")
    ap.add_argument("--tokens", required=True, help="prompt token ids, with commas between them; several prompts of equal "
                                                    "length with ';' between them decode in lockstep (greedy)")
    ap.add_argument("--max-tokens", type=int, default=32)
    ap.add_argument("--dtype", default=None, choices=["bfloat16", "float32"], help="model folders only")
    ap.add_argument("--prefill-chunk", type=int, default=512)
    ap.add_argument("--temperature", type=float, default=0.0)
    ap.add_argument("--top-k", type=int, default=1)
    ap.add_argument("--top-p", type=float, default=1.0)
    ap.add_argument("--repeat-penalty", type=float, default=1.0)
    ap.add_argument("--seed", type=int, default=None)
    ap.add_argument("--eos", default="", help="stop token ids")
    a = ap.parse_args(argv)
    ids = lambda t: [int(v) for v in t.split(",") if v.strip()]
    prompts = [ids(p) for p in a.tokens.split(";")]
    built_library()
    from . import adamah
    from .engine import GenerationConfig
    from .models import load_engine
    gpu = adamah.init()
    try:
        kw = {"prefill_chunk": a.prefill_chunk, "batch": len(prompts)}
        if os.path.isdir(a.model):
            kw["dtype"] = a.dtype or "bfloat16"
        else:
            kw.update(kv_cap=max(map(len, prompts)) + a.max_tokens + 1, kv_fp16=True, fusion_scheduler_mode="level_batched")
        engine = load_engine(gpu, a.model, **kw)
        if len(prompts) > 1:
            out, stats = engine.generate_batch(prompts, a.max_tokens)
        else:
            out, stats = engine.generate(prompts[0], GenerationConfig(
                max_tokens=a.max_tokens, temperature=a.temperature, top_k=a.top_k, top_p=a.top_p, repeat_penalty=a.repeat_penalty,
                seed=a.seed, eos_token_ids=tuple(ids(a.eos))))
        print(json.dumps({"tokens": out, "stats": {k: v for k, v in stats.items() if isinstance(v, (int, float, str))}}), flush=True)
    finally:
        gpu.shutdown()
    return 0
