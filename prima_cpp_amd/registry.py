"""Model registry: what a model file says it is -> how it is configured and loaded. A GGUF file names its architecture in general.architecture, a folder in config.json
("architecture"). Every entry returns an engine.Model that the scheduler (scheduler.py) drives through the same calls."""
import json
import os

from .lib import BF16, F32, PM355Error

ARCHITECTURES = {}
DTYPES = {"bfloat16": BF16, "float32": F32}


def register(name):
    """Decorator: load(path, config, dtype) -> engine.Model for folders, load(path, gguf kv, n_ctx) for GGUF files."""
    def put(f):
        ARCHITECTURES[name] = f
        return f
    return put


def describe(path):
    """(architecture name, its configuration) without touching weights"""
    if os.path.isdir(path):
        with open(os.path.join(path, "config.json")) as f:
            config = json.load(f)
        return config.get("architecture"), config
    from . import gguf
    g = gguf.GGUFFile(path)
    kv = dict(g.kv)
    g.close()
    return kv.get("general.architecture"), kv


def load(path, dtype="bfloat16", n_ctx=4096):
    """The model at `path` on the current device, weights loaded, cache not made yet (Model.finalize_pool). dtype: dense models ("bfloat16", "float32");
    n_ctx: KV slab per sequence of the quantized layer windows."""
    name, config = describe(path)
    if name not in ARCHITECTURES:
        raise PM355Error(f"{path}: architecture {name!r} is not served ({', '.join(sorted(ARCHITECTURES))})")
    return ARCHITECTURES[name](path, config, dtype=dtype, n_ctx=n_ctx)


def _gguf_window(arch):
    def build(path, kv, dtype, n_ctx):
        from . import engine
        from .gguf import ARCH_NAMES

        def key(k, default=None):
            v = kv.get(f"{ARCH_NAMES[arch]}.{k}", default)
            if v is None:
                raise PM355Error(f"{path}: {ARCH_NAMES[arch]}.{k} is missing")
            return v
        heads, embd = key("attention.head_count"), key("embedding_length")
        n_vocab = kv.get(f"{ARCH_NAMES[arch]}.vocab_size") or len(kv.get("tokenizer.ggml.tokens", ()))
        hp = dict(arch=arch, n_layer=key("block_count"), n_embd=embd, n_head=heads, n_head_kv=key("attention.head_count_kv", heads),
                  head_dim=key("rope.dimension_count", embd // heads), n_ff=key("feed_forward_length"), n_vocab=n_vocab,
                  rms_eps=key("attention.layer_norm_rms_epsilon"), rope_freq_base=key("rope.freq_base", 10000.0), n_ctx_orig=key("context_length", 8192))
        w = engine.Window(hp, n_ctx=n_ctx)
        w.load_gguf(path)
        return w
    return build


register("llama")(_gguf_window(0))
register("qwen2")(_gguf_window(1))

from . import keranex, kudirax  # noqa: E402,F401  (they register themselves)
