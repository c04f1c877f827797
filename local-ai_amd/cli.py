"""Command line: generate tokens with a model folder, list the known architectures."""
from __future__ import annotations

import argparse
import sys

from . import generation, registry
from .trace import DTYPES


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="local-ai", description=__doc__)
    sub = ap.add_subparsers(dest="command", required=True)
    sub.add_parser("architectures", help="list the architectures a config.json may name")
    g = sub.add_parser("generate", help="continue prompts of token ids")
    g.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    g.add_argument("--prompt", required=True, action="append", help="token ids with commas between them; repeat for more requests")
    g.add_argument("--max-new-tokens", type=int, default=32)
    g.add_argument("--dtype", choices=sorted(DTYPES), default="bfloat16")
    g.add_argument("--sequences", type=int, default=4, help="requests that are live together")
    g.add_argument("--portion", type=int, default=512, help="prompt tokens per turn")
    g.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    g.add_argument("--top-k", type=int, default=0)
    g.add_argument("--top-p", type=float, default=1.0)
    g.add_argument("--seed", type=int, default=0)
    g.add_argument("--stop", default="", help="token ids that end a request")
    a = ap.parse_args(argv)
    if a.command == "architectures":
        print("\n".join(sorted(registry.ARCHITECTURES)))
        return 0

    def ids(text):
        return [int(t) for t in text.replace(",", " ").split()]
    prompts = [ids(p) for p in a.prompt]
    longest = max(len(p) for p in prompts) + a.max_new_tokens
    model = registry.load_model(a.model, longest, DTYPES[a.dtype], max_sequences=a.sequences)
    scheduler = generation.Scheduler(model, a.portion)
    requests = [scheduler.submit(generation.Request(p, a.max_new_tokens, generation.Sampler(a.temperature, a.top_k, a.top_p, a.seed + i), ids(a.stop)))
                for i, p in enumerate(prompts)]
    scheduler.run()
    for r in requests:
        print(",".join(str(t) for t in r.tokens))
    return 0


if __name__ == "__main__":
    sys.exit(main())
