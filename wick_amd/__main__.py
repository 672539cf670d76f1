"""Command line over the model handle:

    python -m wick_amd info --model PATH
    python -m wick_amd generate --model PATH --tokens 1,2,3 --max-new 16

PATH is a model folder (config.json + model.safetensors) or a GGUF file.  Prompts and output are token ids: tokenizers stay with the
host application.  A trace of requests is replayed with bin/trace_run."""
from __future__ import annotations

import argparse
import sys

import numpy as np

from . import model as M
from .rocm import RocmContext


def sampler(temperature: float, seed: int):
    """None (greedy, picked on the GPU), or a draw from softmax(logits / temperature)."""
    if temperature <= 0.0:
        return None
    rng = np.random.default_rng(seed)

    def draw(logits: np.ndarray) -> int:
        z = np.where(np.isnan(logits), -np.inf, logits).astype(np.float64) / temperature
        p = np.exp(z - z.max())
        return int(rng.choice(p.size, p=p / p.sum()))

    return draw


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="python -m wick_amd")
    sub = ap.add_subparsers(dest="command", required=True)
    for name in ("info", "generate"):
        p = sub.add_parser(name)
        p.add_argument("--model", required=True, help="model folder or GGUF file")
        p.add_argument("--dtype", choices=("native", "float32"), default="native", help="what the model computes in")
        p.add_argument("--context", type=int, default=4096, help="positions to keep room for")
        p.add_argument("--device", type=int, default=0)
        if name == "generate":
            p.add_argument("--tokens", required=True, help="prompt: token ids separated by commas")
            p.add_argument("--max-new", type=int, default=32)
            p.add_argument("--stop", default="", help="token ids that end the generation, separated by commas")
            p.add_argument("--ubatch", type=int, default=0, help="prompt tokens per chunk (0: all at once)")
            p.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
            p.add_argument("--seed", type=int, default=0)
    a = ap.parse_args(argv)
    ids = lambda text: [int(t) for t in text.split(",") if t.strip()]
    with RocmContext(a.device) as ctx, M.RocmModel(ctx, a.model, a.context, M.F32 if a.dtype == "float32" else M.NATIVE) as m:
        if a.command == "info":
            print(f"{m.architecture}: vocabulary {m.vocab_size}, width {m.hidden_size}, {m.layer_runs} layer runs, context {m.max_seq_len}, "
                  f"{m.gpu_memory_bytes() / 1e6:.1f} MB on {ctx.device_name}")
        else:
            out = M.generate(m, ids(a.tokens), a.max_new, stop=ids(a.stop), ubatch=a.ubatch, sample=sampler(a.temperature, a.seed))
            print(*out)
    return 0


if __name__ == "__main__":
    sys.exit(main())
