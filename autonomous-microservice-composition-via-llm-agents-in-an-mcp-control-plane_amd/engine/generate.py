"""Free generation with the serving engine, from Python or the command line.

    python -m mcp_amd.engine.generate --model llama3-8b --prompt "..." --max-new 32
    python -m mcp_amd.engine.generate --model DIR --ids 5,17,3 --temperature 0

``--model`` is a named configuration (random-init weights) or a checkpoint
directory of any served architecture (``models.registry``).
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import List, Optional, Sequence

from .decoders import TokenDecoder


def generate(engine, prompts: Sequence[Sequence[int]], max_new: int = 32,
             eos: Optional[int] = None) -> List[List[int]]:
    """Sampled ids of every prompt (one batch, the engine's temperature)."""
    seqs = [engine.submit(TokenDecoder(max_new, eos), list(p)) for p in prompts]
    engine.run()
    for q in seqs:
        if q.error:
            raise RuntimeError(q.error)
    return [q.result for q in seqs]


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(description="free generation on the serving engine")
    ap.add_argument("--model", default="llama3-8b", help="named configuration or checkpoint directory")
    ap.add_argument("--prompt", action="append", default=[], help="text prompt (repeatable)")
    ap.add_argument("--ids", action="append", default=[], help="prompt as comma-separated token ids")
    ap.add_argument("--max-new", type=int, default=32)
    ap.add_argument("--temperature", type=float, default=0.0)
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16",
                    help="checkpoints of families with a 32-bit mode")
    ap.add_argument("--blocks", type=int, default=1024, help="64-token KV cache blocks")
    ap.add_argument("--device", default="cuda:0")
    ap.add_argument("--seed", type=int, default=0)
    a = ap.parse_args(argv)
    import torch
    from ..models.registry import load_model, random_model
    from ..planner.tokenizer import tokenizer_for
    from .engine import LLMEngine
    tok = tokenizer_for(a.model) if a.prompt else None
    prompts = [tok.encode(p) for p in a.prompt] + [[int(t) for t in i.split(",")] for i in a.ids]
    if not prompts:
        ap.error("give --prompt or --ids")
    model = load_model(a.model, a.device, dtype=getattr(torch, a.dtype)) if os.path.isdir(a.model) \
        else random_model(a.model, a.device, seed=a.seed)
    V = model.cfg.vocab_size
    if any(not 0 <= t < V for p in prompts for t in p):
        ap.error(f"a prompt id is outside the model's vocabulary of {V}")
    eng = LLMEngine(model, num_blocks=a.blocks, max_batch=max(8, len(prompts)),
                    temperature=a.temperature, seed=a.seed)
    for p, out in zip(prompts, generate(eng, prompts, a.max_new)):
        line = {"prompt_ids": p, "ids": out}
        if tok is not None:
            line["text"] = tok.decode(out)
        print(json.dumps(line), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
