"""Generate from a checkpoint on the command line::

    python -m iron_amd DIR --prompt "The capital of France is" --count 32
    python -m iron_amd DIR --ids 5,17,3 --ids 8,1 --temperature 0.7 --top-k 50

The model class follows the folder's ``config.json``.  ``--ids`` prompts are token ids and come back as
token ids; several are served as one batch by a model that serves batches, one after the other by the rest.
"""

from __future__ import annotations

import argparse
import sys


def _ids(text: str) -> list[int]:
    return [int(t) for t in text.split(",")]


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="python -m iron_amd", description="Generate from a checkpoint.")
    ap.add_argument("model", help="a folder with config.json, the weights and, for text prompts, the tokenizer")
    asked = ap.add_mutually_exclusive_group(required=True)
    asked.add_argument("--prompt", action="append", help="a text prompt; may be given several times")
    asked.add_argument("--ids", action="append", type=_ids, help="a prompt as comma-separated token ids; may be given several times")
    ap.add_argument("--count", type=int, default=32, help="tokens to generate at most")
    ap.add_argument("--temperature", type=float, default=0.0, help="0 draws greedily")
    ap.add_argument("--top-k", type=int, default=50)
    ap.add_argument("--seed", type=int, default=0)
    ap.add_argument("--max-seq-len", type=int, default=None, help="positions a sequence may reach; the config's if not given")
    args = ap.parse_args(argv)

    from .applications import model_class
    from .lm import BatchedLM, Sampler

    cls, prompts = model_class(args.model), args.prompt or args.ids
    batched = issubclass(cls, BatchedLM) and args.ids is not None
    model = cls.load(args.model, max_seq_len=args.max_seq_len, **({"slots": len(prompts)} if batched else {}))
    samplers = [Sampler(args.temperature, args.top_k, seed=args.seed + i) if args.temperature else None for i in range(len(prompts))]
    try:
        if batched:
            made = model.generate_batch(prompts, args.count, samplers)
        else:
            made = [model.generate(p, args.count, s) for p, s in zip(prompts, samplers)]
    finally:
        model.release()
    for out in made:
        print(out if isinstance(out, str) else ",".join(map(str, out)), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
