"""Command line: python -m prometorch_amd generate --model PATH (--tokens IDS | --prompt TEXT) ...

PATH is a model folder or a .gguf file.  --tokens takes token ids and prints ids; --prompt runs one chat turn of a .gguf model
with the file's own tokenizer and template and prints the reply."""
from __future__ import annotations

import argparse
import re
import sys

from . import model as registry


def uniforms(seed: int, n: int) -> list:
    import ctypes as C
    from . import _lib
    out = (C.c_float * n)()
    _lib.check(_lib.load().ptm_mt19937_uniforms(seed, 0, n, out), "mt19937_uniforms")
    return list(out)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="prometorch_amd", description="Run a model on the GPU.")
    sub = ap.add_subparsers(dest="command", required=True)
    g = sub.add_parser("generate", help="continue a prompt")
    g.add_argument("--model", required=True, help="model folder (config.json, model.safetensors) or .gguf file")
    g.add_argument("--tokens", help="prompt as token ids, separated by commas or blanks")
    g.add_argument("--prompt", help="prompt as text (.gguf models)")
    g.add_argument("--max-new", type=int, default=64)
    g.add_argument("--dtype", choices=sorted(registry.PRECISIONS), default="bfloat16")
    g.add_argument("--temperature", type=float, default=0.7, help="0: greedy")
    g.add_argument("--top-k", type=int, default=40)
    g.add_argument("--top-p", type=float, default=0.9)
    g.add_argument("--repeat-penalty", type=float, default=1.0)
    g.add_argument("--seed", type=int, default=42)
    g.add_argument("--stop", help="token ids that end the output")
    g.add_argument("--context", type=int, default=4096, help="cache size for --prompt")
    a = ap.parse_args(argv)
    if (a.tokens is None) == (a.prompt is None):
        ap.error("give either --tokens or --prompt")

    def ids(text):
        try:
            return [int(t) for t in re.split(r"[,\s]+", text.strip()) if t]
        except ValueError:
            ap.error("not a list of token ids: %r" % text)

    if a.prompt is not None:
        m = registry.load(a.model, max_seq=a.context, precision=a.dtype)
        if not hasattr(m, "chat"):
            ap.error("%s has no tokenizer: give --tokens" % a.model)
        print(m.chat(a.prompt, max_new=a.max_new, temperature=a.temperature, top_k=a.top_k, top_p=a.top_p,
                     repeat_penalty=a.repeat_penalty, seed=a.seed))
    else:
        prompt = ids(a.tokens)
        if not prompt or a.max_new <= 0:
            ap.error("nothing to do: empty prompt or --max-new below 1")
        m = registry.load(a.model, max_seq=len(prompt) + a.max_new, precision=a.dtype)
        m.set_past_len(0)
        out = m.generate(prompt, uniforms(a.seed, a.max_new), temperature=a.temperature, top_k=a.top_k, top_p=a.top_p,
                         repeat_penalty=a.repeat_penalty, stop_ids=ids(a.stop or ""))
        print(" ".join(str(t) for t in out))
    m.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
