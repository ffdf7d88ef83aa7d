"""Command line: greedy generation from token ids with any model the registry opens.

    python -m rust-model-inference_amd --model PATH --tokens 5,17,3 --max-new 32 [--dtype float32] [--stop 2,7]

PATH is a GGUF file (Qwen3 family) or a model folder (config.json, model.safetensors).  Prints the generated ids,
separated by commas, and the timing to standard error.
"""
import argparse
import sys

from . import hip, models


def ids(text):
    return [int(t) for t in text.replace(",", " ").split()]


def main(argv=None):
    p = argparse.ArgumentParser(prog="rust-model-inference_amd", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    p.add_argument("--model", required=True)
    p.add_argument("--tokens", required=True, type=ids, help="the prompt's token ids")
    p.add_argument("--max-new", type=int, default=32)
    p.add_argument("--stop", type=ids, default=[], help="ids that end the generation")
    p.add_argument("--dtype", choices=sorted(models.DTYPES), default="bfloat16", help="of a model folder's session")
    p.add_argument("--device", type=int, default=0)
    a = p.parse_args(argv)
    hip.init(a.device)
    session = models.open_session(a.model, len(a.tokens) + a.max_new, a.dtype)
    if a.stop:
        session.set_stop_ids(a.stop)
    r = session.generate(a.tokens, a.max_new)
    print(",".join(str(t) for t in r["tokens"]))
    print(f"{len(a.tokens)} prompt + {len(r['tokens'])} generated tokens in {r['seconds'] * 1e3:.2f} ms", file=sys.stderr)
    session.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
