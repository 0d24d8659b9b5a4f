"""python -m prima_cpp_amd MODEL --prompt 1,2,3 [--prompt ...] -n 32: greedy continuations of token-id prompts, batched (GGUF file or model folder)."""
import argparse
import json
import sys


def main(argv=None):
    ap = argparse.ArgumentParser(prog="prima_cpp_amd", description="greedy generation from token-id prompts")
    ap.add_argument("model", help="GGUF file (llama, qwen2) or a folder with config.json and model.safetensors")
    ap.add_argument("--prompt", action="append", required=True, help="token ids with commas between them; may be given several times")
    ap.add_argument("-n", "--n-predict", type=int, default=32)
    ap.add_argument("--dtype", default="bfloat16", choices=("bfloat16", "float32"), help="of dense models")
    ap.add_argument("--n-ctx", type=int, default=4096, help="tokens per sequence")
    ap.add_argument("--parallel", type=int, default=4, help="sequences in flight")
    ap.add_argument("--portion", type=int, default=512, help="prompt tokens of one request per step")
    a = ap.parse_args(argv)
    from . import registry, scheduler
    prompts = [[int(t) for t in p.split(",")] for p in a.prompt]
    model = registry.load(a.model, dtype=a.dtype, n_ctx=a.n_ctx)
    model.finalize_pool(2048, a.parallel, a.parallel * a.n_ctx)
    for p, t in zip(prompts, scheduler.generate(model, prompts, a.n_predict, portion=a.portion)):
        print(json.dumps({"prompt_tokens": len(p), "tokens": t}))
    model.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
