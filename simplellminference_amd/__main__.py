"""Command line: greedy generation from a model folder (``registry.py``), on token ids or text.

    python -m simplellminference_amd --model DIR --prompt "1 17 42" [--prompt "5 6"] --max-length 64
    python -m simplellminference_amd --model DIR --tokenizer tok.model --text "Once upon a time" --max-length 64

One line of token ids (the token fed at each position) per prompt; several prompts decode as one batch."""
from __future__ import annotations

import argparse
import sys

from .registry import architectures, load_model


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="python -m simplellminference_amd", description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True, help=f"folder with config.json and weights ({', '.join(architectures())})")
    ap.add_argument("--prompt", action="append", default=[], help="token ids, whitespace-separated (repeatable)")
    ap.add_argument("--text", action="append", default=[], help="text prompt (needs --tokenizer; repeatable)")
    ap.add_argument("--tokenizer", default="", help="sentencepiece model file")
    ap.add_argument("--max-length", type=int, default=64, help="positions per sequence, prompt included")
    ap.add_argument("--dtype", default="bfloat16", help="bfloat16 (16-bit serving) or float32")
    ap.add_argument("--no-prefill", action="store_true", help="feed the prompt token by token")
    a = ap.parse_args(argv)
    enc = None
    if a.tokenizer:
        from .encode import SPELayer
        enc = SPELayer(a.tokenizer)
    if a.text and enc is None:
        ap.error("--text needs --tokenizer")
    prompts = [[int(t) for t in p.split()] for p in a.prompt] + [enc.encode(t) for t in a.text]
    if not prompts or not all(prompts):
        ap.error("give at least one non-empty --prompt or --text")
    m = load_model(a.model, a.dtype, a.max_length, len(prompts))
    if hasattr(m, "predict_batch_prefill") and not a.no_prefill:
        out = m.predict_batch_prefill(prompts, a.max_length)
    elif len(prompts) == 1:
        out = [m.predict(prompts[0], a.max_length) if a.no_prefill else m.predict_prefill(prompts[0], a.max_length)]
    else:
        out = m.predict_batch(prompts, a.max_length)
    m.close()
    for ids in out:
        print(enc.decode([int(t) for t in ids]) if enc else " ".join(str(int(t)) for t in ids))
    return 0


if __name__ == "__main__":
    sys.exit(main())
