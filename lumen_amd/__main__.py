"""Command line: python -m lumen_amd generate | trace.

generate: one turn on a model folder -- prompt token ids in, new token ids out (there is no tokenizer here).
trace:    the trace runner (also bin/trace_run).
"""
import argparse
import sys

from . import trace


def ids_of(text):
    return [int(t) for t in text.replace(",", " ").split()]


def generate(argv):
    from .registry import load_model
    ap = argparse.ArgumentParser(prog="lumen_amd generate")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16", help="storage of the weights")
    ap.add_argument("--prompt", required=True, type=ids_of, help="token ids, separated by commas or blanks")
    ap.add_argument("--max-new", type=int, default=64)
    ap.add_argument("--max-seq", type=int, default=None, help="tokens the sequence may hold")
    ap.add_argument("--greedy", action="store_true", help="always the most likely token")
    ap.add_argument("--temperature", type=float, default=0.8)
    ap.add_argument("--top-p", type=float, default=0.9)
    ap.add_argument("--repetition-penalty", type=float, default=1.05)
    ap.add_argument("--seed", type=int, default=0)
    ap.add_argument("--stop", type=ids_of, default=[], help="token ids that end the turn")
    a = ap.parse_args(argv)
    model = load_model(a.model, a.dtype, a.max_seq)
    # (a nucleus of no mass keeps the most likely token alone)
    top_p, penalty = (0.0, 1.0) if a.greedy else (a.top_p, a.repetition_penalty)
    out = model.generate_turn(a.prompt, temperature=a.temperature, top_p=top_p, repetition_penalty=penalty,
                              max_gen=a.max_new, seed=a.seed, stop_ids=a.stop)
    print(" ".join(str(int(t)) for t in out))
    return 0


def main(argv=None):
    argv = list(sys.argv[1:] if argv is None else argv)
    commands = {"generate": generate, "trace": trace.main}
    if not argv or argv[0] not in commands:
        print(__doc__.strip())
        return 0 if argv and argv[0] in ("-h", "--help") else 2
    return commands[argv[0]](argv[1:])


if __name__ == "__main__":
    sys.exit(main())
