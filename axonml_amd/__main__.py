"""Command line: `python -m axonml_amd generate|trace ...` for any model of the registry."""
import argparse
import sys


def _generate(args):
    from .generation import GenerationConfig
    from .quant import QuantType
    from .registry import load_model

    model = load_model(args.model, dtype=args.dtype, max_positions=args.max_positions,
                       quant_type=QuantType.from_str(args.quant_type) if args.quant_type else None)
    tokenizer = None
    if args.text is not None:
        from .tokenizer import HFTokenizer

        tokenizer = HFTokenizer.from_directory(args.model)
        prompt = [int(t) for t in tokenizer.encode(args.text)]
    else:
        prompt = [int(t) for t in args.tokens.replace(",", " ").split()]
    if args.temperature > 0:
        model.set_sampling(GenerationConfig(temperature=args.temperature, top_k=args.top_k, top_p=args.top_p,
                                            repetition_penalty=args.repetition_penalty), seed=args.seed)
    out, pre_ms, dec_ms = model.generate(prompt, args.max_new_tokens)
    print(tokenizer.decode(out.tolist()) if tokenizer else " ".join(str(t) for t in out.tolist()), flush=True)
    print(f"prompt {len(prompt)} tokens in {pre_ms:.2f} ms, {len(out)} tokens in {dec_ms:.2f} ms", file=sys.stderr)
    model.close()
    return 0


def main(argv=None):
    from . import trace

    ap = argparse.ArgumentParser(prog="python -m axonml_amd", description="run a model of the registry")
    sub = ap.add_subparsers(dest="command", required=True)
    g = sub.add_parser("generate", help="continue a prompt")
    g.add_argument("--model", required=True, help="directory with config.json and model.safetensors")
    g.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    g.add_argument("--quant-type", default=None, help="block type of models that are quantised as they are read (Q4_K, Q8_0, ...)")
    src = g.add_mutually_exclusive_group(required=True)
    src.add_argument("--tokens", help="prompt as token ids, separated by commas or spaces")
    src.add_argument("--text", help="prompt as text (needs a tokenizer in the directory)")
    g.add_argument("--max-new-tokens", type=int, default=50)
    g.add_argument("--max-positions", type=int, default=None)
    g.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    g.add_argument("--top-k", type=int, default=None)
    g.add_argument("--top-p", type=float, default=None)
    g.add_argument("--repetition-penalty", type=float, default=1.0)
    g.add_argument("--seed", type=int, default=0)
    trace.add_arguments(sub.add_parser("trace", help="replay a trace of token ids and write logits"))
    args = ap.parse_args(argv)
    return _generate(args) if args.command == "generate" else trace.main(args)


if __name__ == "__main__":
    sys.exit(main())
