"""bench.py --design keranex[:size,..]: throughput of the Keranex design (bf16, random weights, layer shapes of real models) beside the framework's closest model, Kudirax of the
same width, heads, layers and as many feed-forward values per token as the chosen experts have together. The kernels of both are timed inside the engine's own steps (a device
trace of a prompt and of decoded tokens, the launches of a step in order) and compared with the roofline that bounds each: HBM 8 TB/s, bf16 matrix cores 2.5 PFLOP/s, or the
vector pipe (39 T lane operations/s; an exponential takes four). One JSON line."""
import json

import torch

from . import keranex, kudirax
from .bench_design import CTX, HBM, MFMA, PROMPT, design_config, throughput_design

VALU = 256 * 64 * 2.4e9
WINDOW = 4096
SIZES = {"1b": dict(W=2048, H=32, G=8, d=64, rot=32, qr=768, kr=512, inner=4096, state=16, dt=128, E=32, top=4, ff=2048, layers=16, vocab=32000),
         "8b": dict(W=4096, H=32, G=8, d=128, rot=64, qr=1536, kr=512, inner=8192, state=16, dt=256, E=32, top=4, ff=3584, layers=8, vocab=32000),
         "70b": dict(W=8192, H=64, G=8, d=128, rot=64, qr=1536, kr=512, inner=16384, state=16, dt=512, E=16, top=4, ff=7168, layers=4, vocab=32000)}


def config(z):
    moe = {"kind": "moe", "expert": {"ff": z["ff"]}, "router": {"experts": z["E"], "top": z["top"], "groups": {"count": 4, "keep": 2}}}
    lat = dict(heads=z["H"], dim=z["d"], rot_dim=z["rot"], vdim=z["d"], q_rank=z["qr"], kv_rank=z["kr"], mask={"size": WINDOW}, rot={"base": 10000.0, "dims": z["rot"]},
               scale=(z["d"] + z["rot"]) ** -0.5)
    ssm = dict(inner=z["inner"], state=z["state"], dt_rank=z["dt"], conv=4)
    layers = [dict(type="mamba1", mixer=ssm, mlp=moe) if i % 2 else dict(type="latent_attention", mixer=dict(lat, kv_from=i - 2) if i % 4 else lat, mlp=moe) for i in range(z["layers"])]
    return dict(architecture="Keranex", width=z["W"], vocab=z["vocab"], norm={"eps": 1e-5}, embedding={"bigram": {"buckets": 50021, "mul_prev": 1009, "mul_cur": 31}}, layers=layers)


def mat(T, N, K, out=2):
    """(label's work) seconds at the roofline of a product of T rows"""
    return max(2.0 * T * N * K / MFMA, (N * K * 2 + T * K * 2 + T * N * out) / HBM)


def product(label, T, N, K, out=2):
    """a product's launches: prompts sum k ranges of products with few tiles in a launch of their own"""
    tiles = -(-T // 128) * -(-N // 128)
    split = T > 64 and tiles <= 128 and min(-(-K // 64) // 4, 256 // tiles) > 1
    yield label + ("_in_k_ranges" if split else ""), mat(T, N, K, out)
    if split:
        yield "sum_of_k_ranges", T * N * (4 * min(-(-K // 64) // 4, 256 // tiles) + out) / HBM


def keranex_launches(z, T):
    """(label, seconds at the roofline) of a step's launches, in order"""
    W, H, d, r, qr, kr, I, S, E, F = (z[k] for k in ("W", "H", "d", "rot", "qr", "kr", "inner", "state", "E", "ff"))
    one, fused, pairs = T == 1, T == 1 and W <= 2048, T * z["top"]
    raw = 4 if one else 2
    norm = ("norm", T * W * (12 + 2 + (4 if one else 2 * z["top"])) / HBM)
    yield "embedding", T * W * (2 + 2 + 4 + 2) / HBM
    yield "rotation_table", T * r * 4 / HBM
    for i in range(z["layers"]):
        if i and not fused:
            yield norm
        if i % 2 == 0:
            own = i % 4 == 0
            yield from product("latent_proj", T, qr + (kr + r if own else 0), W, raw)
            if one:
                yield from product("query", T, H * (d + r), qr)
                yield "absorb", mat(T, H * kr, d)
                yield "attention", CTX * (kr + r) * 2 / HBM
                yield "value", mat(T, H * d, kr)
            else:
                yield ("latent_norm_and_store" if own else "query_norm"), T * (qr + (kr + r if own else 0)) * 4 / HBM
                yield from product("query", T, H * (d + r), qr)
                yield "rotate", T * H * r * 6 / HBM
                yield "expand_keys", mat(T, H * d, kr)
                yield "expand_values", mat(T, H * d, kr)
                yield "spread_rotated", T * (H + 1) * r * 2 / HBM
                yield "attention", H * (2.0 * d + r) * T * (T + 1) / MFMA
            yield from product("out", T, W, H * d, 4)
        else:
            yield from product("scan_proj", T, 2 * I, W, raw)
            yield "convolution", T * I * (raw + 2) / HBM
            yield from product("scan_x", T, z["dt"] + 2 * S, I)
            if one:
                yield "scan_step", (I * S * 12 + I * z["dt"] * 2) / HBM
            else:
                yield from product("scan_dt", T, I, z["dt"], 4)
                yield "scan_ends", max(T * I * 6 / HBM, 7.0 * T * I * S / VALU)
                yield "scan_carry", T / 128 * I * S * 8 / HBM
                yield "scan", max(T * I * 10 / HBM, 8.0 * T * I * S / VALU)
            yield from product("out_scan", T, W, I, 4)
        if not fused:
            yield norm if one else ("norm", T * W * 18 / HBM)
        yield from product("router", T, E, W, 4)
        if not one:
            yield "route", T * E * 4 / HBM
            yield "place", pairs * 12 / HBM
        some = min(E, pairs)
        yield "up", max(2.0 * pairs * W * F / MFMA, (some * W * F + pairs * (W + F)) * 2 / HBM)
        yield "down", max(2.0 * pairs * W * F / MFMA, (some * W * F + pairs * (W + F)) * 2 / HBM)
    yield "final_add", norm[1]
    yield "final_norm", W * 6 / HBM
    yield from product("head", 1, z["vocab"], W, 4)
    yield "greedy", z["vocab"] * 4 / HBM


def kudirax_launches(z, T):
    W, H, G, d, F = z["W"], z["H"], z["G"], z["d"], z["top"] * z["ff"]
    one, fused = T == 1, T == 1 and W <= 2048
    raw, N = 4 if one else 2, 2 * H * d + 2 * G * d
    norm = ("norm", T * W * 18 / HBM)
    yield "embedding", T * W * (2 + 4 + 2) / HBM
    for i in range(z["layers"]):
        if i and not fused:
            yield norm
        yield from product("proj", T, N, W, raw)
        if not one:
            yield "norm_and_store", T * (N - H * d + H * d + 2 * G * d) * 2 / HBM
        yield "attention", 2 * CTX * G * d * 2 / HBM if one else 4.0 * d * H * T * (T + 1) / 2 / MFMA
        yield from product("out", T, W, H * d, 4)
        if not fused:
            yield norm
        yield from product("up", T, F, W)
        yield from product("down", T, W, F, 4)
    yield "final_add", norm[1]
    yield "final_norm", W * 6 / HBM
    yield from product("head", 1, z["vocab"], W, 4)
    yield "greedy", z["vocab"] * 4 / HBM


LIKE = {"latent_proj": "proj", "query": "proj", "absorb": "out", "value": "out", "out": "out", "up": "up", "down": "down", "attention": "attention", "scan_step": "attention",
        "norm": "norm", "embedding": "embedding", "head": "head", "latent_norm_and_store": "norm_and_store", "query_norm": "norm_and_store", "rotate": "norm_and_store",
        "spread_rotated": "norm_and_store", "expand_keys": "proj", "expand_values": "proj", "scan_proj": "proj", "scan_dt": "proj", "scan_x": "out", "out_scan": "out",
        "scan_x_in_k_ranges": "out", "latent_proj_in_k_ranges": "proj", "convolution": "norm_and_store", "scan_ends": "norm_and_store", "scan": "norm_and_store", "scan_carry": "norm_and_store"}


def traced(run, want, n):
    """{label: {us, of_roofline}}: medians over the launches of n steps"""
    from torch.profiler import ProfilerActivity, profile
    run()
    torch.cuda.synchronize()
    with profile(activities=[ProfilerActivity.CUDA]) as p:
        for _ in range(n):
            run()
        torch.cuda.synchronize()
    ev = sorted((e for e in p.events() if e.device_type == torch.autograd.DeviceType.CUDA and "Mem" not in e.name), key=lambda e: e.time_range.start)
    names = list(want) * n
    if len(ev) != len(names):
        raise RuntimeError("%d launches in the trace, %d expected: %s" % (len(ev), len(names), [(a, e.name[:60]) for (a, _), e in zip(names, ev)][:40]))
    seen = {}
    for (label, roof), e in zip(names, ev):
        seen.setdefault(label, []).append((e.device_time, roof))
    out = {}
    for label, v in seen.items():
        us, roof = sorted(v)[len(v) // 2]
        out[label] = {"us": round(us, 2), "of_roofline": round(roof * 1e6 / us, 4), "launches": len(v) // n}
    return out


def measure(m, z, launches, steps, warmup):
    toks = torch.randint(0, z["vocab"], (PROMPT,), generator=torch.Generator().manual_seed(1), dtype=torch.int32).numpy()
    am = torch.zeros(64, dtype=torch.int32, device="cuda")
    out = {"throughput": throughput_design(m, z, steps, warmup), "weight_bytes": m.weight_bytes}

    def prompt():
        s = m.seq_new()
        m.batch([(s, toks, [PROMPT - 1])], argmax=am)
        m.seq_free(s)
    s = m.seq_new()
    m.batch([(s, toks[:CTX - 32], [0])], argmax=am)
    out["kernels"] = {"prefill": traced(prompt, launches(z, PROMPT), 3), "decode": traced(lambda: m.batch([(s, None, (0,))], argmax=am), launches(z, 1), 1)}
    m.seq_free(s)
    return out


def main(sizes, steps, warmup):
    res = {}
    for size in sizes or list(SIZES):
        z, both = SIZES[size], []
        for build, launches in ((lambda: keranex.build(config(z)), keranex_launches), (lambda: kudirax.build(design_config(dict(z, F=z["top"] * z["ff"]))), kudirax_launches)):
            m = build()
            m.fill_synthetic()
            m.finalize_pool(PROMPT, 32, 32 * CTX + PROMPT)
            both.append(measure(m, z, launches, steps, warmup))
            m.close()
            torch.cuda.empty_cache()
        a, b = both
        far = {ph: {k: round(b["kernels"][ph][LIKE[k]]["of_roofline"] / v["of_roofline"], 2) for k, v in a["kernels"][ph].items() if LIKE.get(k) in b["kernels"][ph]} for ph in ("prefill", "decode")}
        res[size] = {"shape": z, "keranex": a, "kudirax_same_size": b, "times_further_from_roofline": far}
        print("design %s: %s" % (size, json.dumps(far)), flush=True)
    print(json.dumps({"metric": "keranex_decode_tokens_per_s", "value": next(iter(res.values()))["keranex"]["throughput"]["decode_1"]["tok/s"], "unit": "tokens/s", "n_gpus": 1, "steps": steps,
                      "warmup": warmup, "higher_is_better": True, "dtype": "bf16", "data": "synthetic", "config": {"design": "keranex", "context": CTX, "prompt": PROMPT}, "sizes": res}), flush=True)
