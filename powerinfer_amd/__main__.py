"""Command line.

    python -m powerinfer_amd generate --model PATH --prompt 1,2,3 [--prompt ...] --new 16 [--dtype bfloat16|float32]
    python -m powerinfer_amd info --model PATH

PATH: a folder with config.json and model.safetensors, or a GGUF file.  Prompts are token ids."""
import argparse
import sys


def main(argv=None):
    ap = argparse.ArgumentParser(prog="powerinfer_amd")
    sub = ap.add_subparsers(dest="cmd", required=True)
    for name in ("generate", "info"):
        p = sub.add_parser(name)
        p.add_argument("--model", required=True)
        p.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
        p.add_argument("--ctx", type=int, default=4096)
        if name == "generate":
            p.add_argument("--prompt", action="append", required=True, help="token ids with commas between them; may be given several times")
            p.add_argument("--new", type=int, default=16)
            p.add_argument("--cells", type=int, default=0, help="cells of the shared cache (0: enough for every prompt at once)")
            p.add_argument("--budget", type=int, default=512, help="most tokens of one step")
    a = ap.parse_args(argv)
    from .registry import load_model
    m = load_model(a.model, a.dtype, a.ctx)
    if a.cmd == "info":
        print(" ".join(f"{k}={v}" for k, v in m.hp.items()))
        return 0
    from .serve import generate
    prompts = [[int(t) for t in p.split(",")] for p in a.prompt]
    for toks in generate(m, prompts, a.new, a.cells or None, budget=a.budget):
        print(",".join(map(str, toks)), flush=True)
    m.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
