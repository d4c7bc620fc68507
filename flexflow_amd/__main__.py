"""Command line: greedy generation from a model folder.

    python -m flexflow_amd --model DIR --prompt "5 17 300" [--prompt ...] [options]

DIR holds config.json and the weights (HF LLaMA sizes with the converted
per-tensor files, or a family of the model registry with model.safetensors).
Prompts are token ids, or text with --tokenizer.
"""
import argparse
import json
import sys

from . import (Model, RequestManager, generate, load_config, set_device)


def main(argv=None):
    ap = argparse.ArgumentParser(prog="python -m flexflow_amd",
                                 description="greedy generation from a model folder")
    ap.add_argument("--model", required=True, help="folder with config.json and the weights")
    ap.add_argument("--prompt", action="append", required=True,
                    help="token ids separated by spaces, or text with --tokenizer; repeatable")
    ap.add_argument("--tokenizer", default=None, help="folder or file of the tokenizer")
    ap.add_argument("--max-length", type=int, default=-1, help="tokens in all, prompt included")
    ap.add_argument("--max-new-tokens", type=int, default=-1)
    ap.add_argument("--max-requests", type=int, default=8, help="requests decoded together")
    ap.add_argument("--max-tokens-per-batch", type=int, default=256)
    ap.add_argument("--max-sequence-length", type=int, default=1024)
    ap.add_argument("--kv-pool-tokens", type=int, default=0,
                    help="paged caches: tokens of the pool (0: every request at full length)")
    ap.add_argument("--bos", type=int, default=-1, help="token id put before prompts (-1: none)")
    ap.add_argument("--eos", type=int, action="append", default=[], help="token id that ends a request")
    ap.add_argument("--use-full-precision", action="store_true", help="32-bit model")
    ap.add_argument("--device", type=int, default=0)
    a = ap.parse_args(argv)
    config = load_config(a.model)
    seq = min(a.max_sequence_length, config.get("max_positions", a.max_sequence_length))
    set_device(a.device)
    rm = RequestManager(max_requests_per_batch=a.max_requests,
                        max_tokens_per_batch=a.max_tokens_per_batch, max_spec_tree_token_num=0,
                        max_sequence_length=seq, bos_token_id=a.bos, eos_token_ids=a.eos)
    if a.tokenizer:
        rm.register_tokenizer(a.tokenizer)
        prompts = a.prompt
    else:
        prompts = [[int(t) for t in p.replace(",", " ").split()] for p in a.prompt]
    llm = Model(config, "inc", max_requests=a.max_requests, max_tokens=a.max_tokens_per_batch,
                max_seq_len=seq, max_tree_tokens=0, weights_folder=a.model,
                full_precision=a.use_full_precision, kv_pool_tokens=a.kv_pool_tokens)
    for r in generate(rm, llm, prompts, max_length=a.max_length, max_new_tokens=a.max_new_tokens):
        out = {"error": "rejected: longer than the sequence limit"} if r is None else {
            "prompt_tokens": len(r.input_tokens), "tokens": r.output_tokens}
        if r is not None and a.tokenizer:
            out["text"] = r.output_text
        print(json.dumps(out), flush=True)
    llm.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
