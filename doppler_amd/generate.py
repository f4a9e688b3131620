"""Command line: generates tokens with any model the registry knows (token ids in, token ids out).

    python -m doppler_amd.generate --model DIR --prompt 11,402,9 --max-tokens 32
    python -m doppler_amd.generate --model DIR --prompt 11,402,9 --temperature 0.8 --top-k 40 --seed 7
"""
import argparse
import json
import sys


def main(argv=None):
    ap = argparse.ArgumentParser(prog="doppler_amd.generate", description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True, help="model folder (RDRR artifact, or config.json + model.safetensors)")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default=None, help="default: what the model is served in")
    ap.add_argument("--prompt", required=True, help="token ids, separated by commas")
    ap.add_argument("--max-tokens", type=int, default=16)
    ap.add_argument("--max-seq", type=int, default=None, help="positions the cache holds")
    ap.add_argument("--chunk", type=int, default=2048, help="most prompt tokens per portion")
    ap.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    ap.add_argument("--top-k", type=int, default=40)
    ap.add_argument("--seed", type=int, default=0)
    args = ap.parse_args(argv)
    from . import models
    prompt = [int(t) for t in args.prompt.split(",")]
    max_seq = args.max_seq or max(len(prompt) + args.max_tokens, 1)
    dec = models.load(args.model, max_seq, args.dtype)
    bad = [t for t in prompt if not 0 <= t < dec.cfg["vocab"]]
    if bad:
        ap.error("token ids %s are outside the vocabulary of %d" % (bad, dec.cfg["vocab"]))
    sampling = dict(temperature=args.temperature, topK=args.top_k, seed=args.seed) if args.temperature > 0 else None
    tokens = dec.generate(prompt, args.max_tokens, sampling=sampling, chunk=args.chunk)
    print(json.dumps({"prompt": prompt, "tokens": tokens}))
    return 0


if __name__ == "__main__":
    sys.exit(main())
