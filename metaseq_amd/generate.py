"""Generates continuations of token-id prompts with any registered model.

    bin/generate --model DIR [--dtype NAME] [--max-tokens N] [--temperature T] [--top-p P]
                 [--logprobs K] [--seed S] [--slots N]

Standard input holds one prompt per line, token ids separated by blanks; one JSON record per
prompt is printed, in order ("tokens": the new ids, "token_scores", "top_logprobs").  With
--slots the prompts run through the continuous batching engine, otherwise as one batch."""
import argparse
import json
import sys


def main(argv=None, lines=None):
    ap = argparse.ArgumentParser(prog="generate", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default=None, help="compute format (default: the serving format)")
    ap.add_argument("--max-tokens", type=int, default=32)
    ap.add_argument("--min-tokens", type=int, default=0)
    ap.add_argument("--temperature", type=float, default=1.0)
    ap.add_argument("--top-p", type=float, default=-1.0, help="nucleus size (default: greedy)")
    ap.add_argument("--logprobs", type=int, default=0)
    ap.add_argument("--seed", type=int, default=None)
    ap.add_argument("--slots", type=int, default=0, help="continuous batching over this many slots")
    args = ap.parse_args(argv)
    import torch

    from .dictionary import Dictionary
    from .hub_utils import GeneratorInterface
    from .registry import load_model
    model = load_model(args.model, dtype=getattr(torch, args.dtype) if args.dtype else None)
    api = GeneratorInterface(model, Dictionary(model.decoder.cfg.vocab_size))
    prompts = [[int(t) for t in line.split()] for line in (sys.stdin if lines is None else lines)
               if line.strip()]
    if not prompts:
        return 0
    options = dict(temperature=args.temperature, top_p=args.top_p, logprobs=args.logprobs)
    if args.slots:
        from .service import ContinuousBatcher
        if args.seed:
            torch.manual_seed(args.seed)
            torch.cuda.manual_seed(args.seed)
        longest = max(len(p) for p in prompts) + 1 + args.max_tokens
        engine = ContinuousBatcher(api, slots=args.slots, capacity=longest)
        replies = [engine.submit(p, max_tokens=args.max_tokens, min_tokens=args.min_tokens, **options)
                   for p in prompts]
        while engine.step():
            pass
        results = [r.get_nowait()[1] for r in replies]
    else:
        results = api.generate(prompts, max_tokens=[args.max_tokens] * len(prompts),
                               min_tokens=[args.min_tokens] * len(prompts), seed=args.seed, **options)
    for result in results:
        if isinstance(result, Exception):
            raise result
        record = result[0]
        print(json.dumps({"tokens": [int(t) for t in record["tokens"]],
                          "token_scores": record["token_scores"],
                          "top_logprobs": record["top_logprobs"]}), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
