"""bench.py --design kudirax[:size,..]: throughput of the Kudirax design (bf16, random weights, layer shapes of real models) beside the framework's closest model, a llama
window of the same width, heads and feed-forward with Q8_0 weights, and both models' kernels one by one against the roofline that bounds them (HBM 8 TB/s or bf16 / f16
matrix cores 2.5 PFLOP/s). Kernels are timed from a captured graph over the layers' own weights, so that nothing stays in the caches. One JSON line."""
import ctypes as C
import json

import torch

from . import engine as E
from . import kudirax, ops
from . import lib as L
from .lib import Q8_0, check, ptr, row_size

HBM, MFMA = 8e12, 2.5e15
SIZES = {"1b": dict(W=2048, H=32, G=8, d=64, F=8192, layers=16, vocab=32000), "8b": dict(W=4096, H=32, G=8, d=128, F=14336, layers=16, vocab=32000),
         "70b": dict(W=8192, H=64, G=8, d=128, F=28672, layers=6, vocab=32000)}
CTX, PROMPT, CHUNK = 2048, 2048, 8192


def design_config(z):
    mixer = dict(heads=z["H"], kv_heads=z["G"], dim=z["d"], vdim=z["d"], mask={"size": CHUNK}, scale=12.0 / z["d"], softcap=50.0, v_mix=True)
    return dict(architecture="Kudirax", width=z["W"], vocab=z["vocab"], norm={"eps": 1e-5},
                layers=[dict(type="attention", mixer=mixer, mlp=dict(kind="dense", ff=z["F"]))] * z["layers"])


def timed(run, n=1, reps=5):
    """microseconds per call of run() (which makes n calls' worth of launches), best of `reps` replays of a captured graph"""
    side, g = torch.cuda.Stream(), torch.cuda.CUDAGraph()
    with torch.cuda.stream(side):
        run()
        torch.cuda.synchronize()
        with torch.cuda.graph(g, stream=side):
            run()
        e0, e1, best = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True), 1e30
        for _ in range(reps):
            e0.record(side)
            g.replay()
            e1.record(side)
            torch.cuda.synchronize()
            best = min(best, e0.elapsed_time(e1) * 1e3 / n)
    return best


def row(us, work, peak):
    return {"us": round(us, 2), ("GB/s" if peak == HBM else "TFLOP/s"): round(work / us / (1e3 if peak == HBM else 1e6), 1), "of_roofline": round(work / us * 1e6 / peak, 3)}


def wall(run, steps, warmup):
    for _ in range(warmup):
        run()
    torch.cuda.synchronize()
    e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    e0.record()
    for _ in range(steps):
        run()
    e1.record()
    torch.cuda.synchronize()
    return e0.elapsed_time(e1) / steps


def tensor_ptrs(m, kind, n):
    f = m.lib.pm355_model_tensor_ptr
    f.restype, f.argtypes = C.c_void_p, [C.c_void_p, C.c_int, C.c_int, C.c_void_p]
    return [f(m.h, kind, i, None) for i in range(n)]


def view(p, rows, cols, dtype=torch.bfloat16):
    """torch view of device memory that the engine owns"""
    class Mem:
        __cuda_array_interface__ = dict(shape=(rows * cols * 2,), typestr="|u1", data=(p, False), version=2)
    return torch.as_tensor(Mem(), device="cuda").view(dtype).view(rows, cols)


def design_model(z):
    m = kudirax.build(design_config(z), "bfloat16")
    m.fill_synthetic()
    m.finalize_pool(PROMPT, 32, 32 * CTX + PROMPT)
    return m


def throughput_design(m, z, steps, warmup):
    out, gen = {}, torch.Generator().manual_seed(1)
    toks = torch.randint(0, z["vocab"], (CTX,), generator=gen, dtype=torch.int32).numpy()

    def prompt():
        s = m.seq_new()
        m.batch([(s, toks[:PROMPT], [PROMPT - 1])], argmax=am)
        m.seq_free(s)
    am = torch.zeros(64, dtype=torch.int32, device="cuda")
    ms = wall(prompt, 4, 2)
    out["prefill"] = {"tokens": PROMPT, "ms": round(ms, 3), "tok/s": round(PROMPT / ms * 1e3, 1)}
    for n in (1, 8, 32):
        seqs = [m.seq_new() for _ in range(n)]
        ctx = CTX - steps - warmup - 8
        for s in seqs:
            m.batch([(s, toks[:ctx], [ctx - 1])], argmax=am)
        es = [(s, None, (0,)) for s in seqs]
        ms = wall(lambda: m.batch(es, argmax=am), steps, warmup)
        out["decode_%d" % n] = {"sequences": n, "context": ctx, "ms_per_step": round(ms, 4), "tok/s": round(n / ms * 1e3, 1)}
        for s in seqs:
            m.seq_free(s)
    return out


def kernels_design(m, z):
    W, H, G, d, F, n = z["W"], z["H"], z["G"], z["d"], z["F"], z["layers"]
    Np = H * d * 2 + 2 * G * d
    mats = {"proj": (E.T_WQ, Np, W), "out": (E.T_WO, W, H * d), "up": (E.T_FFN_UP, F, W), "down": (E.T_FFN_DOWN, W, F)}
    w = {k: [view(p, N, K) for p in tensor_ptrs(m, kind, n)] for k, (kind, N, K) in mats.items()}
    nw, nb = torch.ones(W, device="cuda"), torch.zeros(W, device="cuda")
    out = {"decode": {}, "prefill": {}}
    r, dl, r2 = (torch.randn(1, W, device="cuda") for _ in range(3))
    for k, (_, N, K) in mats.items():
        y = torch.empty(1, N, dtype=torch.bfloat16 if k == "up" else torch.float32, device="cuda")
        bias = torch.zeros(N, device="cuda") if k in ("up", "down") else None
        x = torch.randn(1, K, device="cuda").bfloat16()
        pro = k in ("proj", "up") and W <= 2048           # (wider rows: a norm launch of its own, as the engine does it)
        if pro:
            us = timed(lambda: [ops.dense_mul_mat_norm(a, r, dl, nw, nb, 1e-5, r2, y, W, bias=bias, act=int(k == "up")) for a in w[k]], n)
        else:
            us = timed(lambda: [ops.dense_mul_mat(a, x, y, bias=bias, act=int(k == "up")) for a in w[k]], n)
        out["decode"][k] = row(us, N * K * 2, HBM)
        y = torch.empty(PROMPT, N, dtype=torch.bfloat16 if k in ("up", "proj") else torch.float32, device="cuda")
        x = torch.randn(PROMPT, K, device="cuda").bfloat16()
        us = timed(lambda: [ops.dense_mul_mat(a, x, y, bias=bias, act=int(k == "up")) for a in w[k][:4]], min(n, 4))
        out["prefill"][k] = row(us, 2.0 * PROMPT * N * K, MFMA)
    # attention, caches of several layers in turn
    sets, pages = 8, CTX // 64
    dp = 64 if d <= 64 else 128
    kc = [torch.randn(pages * G * 64 * dp, device="cuda").bfloat16() for _ in range(sets)]
    vc = [torch.randn(pages * G * 64 * dp, device="cuda").bfloat16() for _ in range(sets)]
    table = torch.randperm(pages, device="cuda").int()
    pos = torch.arange(PROMPT, device="cuda", dtype=torch.int32)
    last = torch.tensor([CTX - 1], device="cuda", dtype=torch.int32)
    zero = torch.zeros(PROMPT, device="cuda", dtype=torch.int32)
    sink = torch.zeros(H, device="cuda")
    tiles = torch.tensor([[i, 128, i, 0] for i in range(0, PROMPT, 128)], device="cuda", dtype=torch.int32)
    q = torch.empty(PROMPT * H * dp, device="cuda", dtype=torch.bfloat16)
    o = torch.empty(PROMPT, H * d, device="cuda", dtype=torch.bfloat16)
    vf = torch.zeros(PROMPT, G * d, device="cuda")
    proj = {torch.float32: torch.randn(1, Np, device="cuda"), torch.bfloat16: torch.randn(PROMPT, Np, device="cuda").bfloat16()}
    nf = ops.attn_paged_scratch(1, H, G, dp)
    scratch, tk = torch.empty(nf, device="cuda"), torch.zeros(H, device="cuda", dtype=torch.int32)

    def attn(i, mode, T, cap=50.0):
        pr = proj[torch.float32 if T == 1 else torch.bfloat16]
        a = ops.AttnPagedArgs(type=L.BF16, n_head=H, n_head_kv=G, k_dim=d, v_dim=d, k_pad=dp, v_pad=dp, mix_flags=15, mask=1, mask_size=CHUNK, scale=12.0 / d, softcap=cap, eps=1e-5,
                              lam=0.5, mixes=1, sink=ptr(sink), k_pages=ptr(kc[i]), v_pages=ptr(vc[i]), v_first=ptr(vf), ld_v_first=G * d, proj=ptr(pr), ld_proj=Np,
                              proj_type=ops.pm_type(pr), q=ptr(q), out=ptr(o), ldo=H * d, d_pos=ptr(last if T == 1 else pos), d_seq=ptr(zero), d_table=ptr(table), table_ld=pages,
                              n_tokens=T, max_keys=CTX, d_tiles=ptr(tiles), n_tiles=len(tiles), scratch=ptr(scratch), scratch_floats=nf, tickets=ptr(tk))
        ops.attn_paged(a, mode)
    attn(0, 2, PROMPT)
    kv = 2 * CTX * G * d * 2
    out["decode"]["attention"] = dict(row(timed(lambda: [attn(i, 3, 1) for i in range(sets)], sets), kv, HBM), keys=CTX)
    flop = 4.0 * d * H * PROMPT * (PROMPT + 1) / 2
    out["prefill"]["attention"] = row(timed(lambda: [attn(i, 18, PROMPT) for i in range(4)], 4), flop, MFMA)
    out["prefill"]["attention_small_cap"] = row(timed(lambda: [attn(i, 18, PROMPT, 15.0) for i in range(4)], 4), flop, MFMA)
    byt = PROMPT * (Np - H * d + H * d + 2 * G * d) * 2
    out["prefill"]["unit_norm_and_store"] = row(timed(lambda: [attn(i, 0, PROMPT) for i in range(4)], 4), byt, HBM)
    r1, x1 = torch.randn(1, W, device="cuda"), torch.empty(1, W, dtype=torch.bfloat16, device="cuda")
    out["decode"]["add_norm"] = row(timed(lambda: [ops.add_layer_norm(r1, dl, nw, nb, 1e-5, W, x1) for _ in range(8)], 8), W * 22, HBM)
    rr, dd, xb = torch.randn(PROMPT, W, device="cuda"), torch.randn(PROMPT, W, device="cuda"), torch.empty(PROMPT, W, dtype=torch.bfloat16, device="cuda")
    out["prefill"]["add_norm"] = row(timed(lambda: [ops.add_layer_norm(rr, dd, nw, nb, 1e-5, W, xb) for _ in range(4)], 4), PROMPT * W * 14, HBM)
    return out


def window_model(z, n_ctx):
    hp = dict(arch=0, n_layer=z["layers"], n_embd=z["W"], n_head=z["H"], n_head_kv=z["G"], head_dim=z["d"], n_ff=z["F"], n_vocab=z["vocab"], rms_eps=1e-5, rope_freq_base=500000.0)
    w = E.Window(hp, n_ctx=n_ctx)
    w.fill_synthetic(lambda hp, il: {k: Q8_0 for k in (E.T_WQ, E.T_WK, E.T_WV, E.T_WO, E.T_FFN_GATE, E.T_FFN_UP, E.T_FFN_DOWN, E.T_TOK_EMBD)})
    w.finalize(max_tokens=PROMPT, n_seq=1)
    return w


def throughput_window(w, z, steps, warmup):
    toks = torch.randint(0, z["vocab"], (PROMPT,), dtype=torch.int32, device="cuda")
    ms = wall(lambda: w.decode(tokens=toks, pos0=0, want_hidden=False, want_argmax=True), 4, 2)
    out = {"prefill": {"tokens": PROMPT, "ms": round(ms, 3), "tok/s": round(PROMPT / ms * 1e3, 1)}}
    ctx = CTX - steps - warmup - 8
    w.decode(tokens=toks[:ctx].contiguous(), pos0=0, want_hidden=False)
    w.set_pos(ctx)
    io = torch.zeros(2, dtype=torch.int32, device="cuda")
    ms = wall(lambda: w.step(token=io[:1], argmax=io[:1]), steps, warmup)
    out["decode_1"] = {"sequences": 1, "context": ctx, "ms_per_step": round(ms, 4), "tok/s": round(1e3 / ms, 1)}
    return out


def kernels_window(w, z):
    lib, W, H, G, d, F, n = w.lib, z["W"], z["H"], z["G"], z["d"], z["F"], z["layers"]
    p = {k: tensor_ptrs(w, k, n) for k in (E.T_WQ, E.T_WK, E.T_WV, E.T_WO, E.T_FFN_GATE, E.T_FFN_UP, E.T_FFN_DOWN, E.T_ATTN_NORM)}
    fused = L.declare("pm355_mul_mat_vec_fused", C.c_int, [C.c_void_p, C.c_int, C.c_int64, C.c_void_p, C.c_void_p, C.c_float, C.c_void_p])
    multi = L.declare("pm355_mul_mat_q_mfma_multi", C.c_int, [C.c_void_p, C.c_int, C.c_int64, C.c_void_p, C.c_int64, C.c_void_p])
    pair = L.declare("pm355_mul_mat_q_mfma_pair", C.c_int, [C.c_int, C.c_void_p, C.c_void_p, C.c_int64, C.c_int64, C.c_void_p, C.c_int64, C.c_void_p, C.c_void_p])
    x, y = torch.randn(PROMPT, max(W, F, H * d), device="cuda"), torch.empty(PROMPT, 2 * max(F, H * d), device="cuda")
    y2 = [torch.empty(PROMPT, max(W, H * d), device="cuda") for _ in range(3)]
    cases = {"qkv": ([(E.T_WQ, H * d), (E.T_WK, G * d), (E.T_WV, G * d)], W, True), "out": ([(E.T_WO, W)], H * d, False), "gate|up": ([(E.T_FFN_GATE, F)], W, True),
             "down": ([(E.T_FFN_DOWN, W)], F, False)}
    out, keep = {"decode": {}, "prefill": {}}, []
    for name, (ms, K, norm) in cases.items():
        jobs, gj = [], []
        for i in range(n):
            a = (ops.MatvecJob * 3)()
            b = (ops.GemmJob * 3)()
            for j, (kind, N) in enumerate(ms):
                a[j] = ops.MatvecJob(Q8_0, 0, N, p[kind][i], p[E.T_FFN_UP][i] if name == "gate|up" else None, ptr(y2[j]) if N <= y2[j].shape[1] else ptr(y), None, None)
                b[j] = ops.GemmJob(Q8_0, N, p[kind][i], ptr(y2[j]) if N <= y2[j].shape[1] else ptr(y), None, None)
            jobs.append(a)
            gj.append(b)
        keep += [jobs, gj]
        byt = sum(row_size(Q8_0, K) * N for _, N in ms) * (2 if name == "gate|up" else 1)
        st = lambda: torch.cuda.current_stream().cuda_stream      # noqa: E731
        us = timed(lambda: [check(fused(C.addressof(a), len(ms), K, ptr(x), p[E.T_ATTN_NORM][0] if norm else None, 1e-5, st()), name) for a in jobs], n)
        out["decode"][name] = row(us, byt, HBM)
        flop = 2.0 * PROMPT * K * sum(N for _, N in ms) * (2 if name == "gate|up" else 1)
        if name == "gate|up":
            run = lambda: [check(pair(Q8_0, p[E.T_FFN_GATE][i], p[E.T_FFN_UP][i], K, F, ptr(x), PROMPT, ptr(y), st()), name) for i in range(4)]      # noqa: E731
        else:
            run = lambda: [check(multi(C.addressof(b), len(ms), K, ptr(x), PROMPT, st()), name) for b in gj[:4]]      # noqa: E731
        us = timed(run, 4)
        out["prefill"][name] = dict(row(us, flop, MFMA), note="with the f32 -> f16 pass over the activations")
    sets = 8
    kc = [torch.randn(CTX * G * d, device="cuda").half() for _ in range(sets)]
    vc = [torch.randn(CTX * G * d, device="cuda").half() for _ in range(sets)]
    q, o = torch.randn(PROMPT, H * d, device="cuda"), torch.empty(PROMPT, H * d, device="cuda")
    pos = torch.tensor([CTX - 1, 0], device="cuda", dtype=torch.int32)
    sf = L.declare("pm355_attn_split_scratch_floats", C.c_size_t, [C.c_int, C.c_int, C.c_int])(H, d, CTX)
    scratch = torch.zeros(max(sf, 1 << 22), device="cuda")
    long = L.declare("pm355_attn_cached_long", C.c_int, [C.c_void_p] * 8 + [C.c_int] * 4 + [C.c_float, C.c_int, C.c_int, C.c_void_p])
    pre = L.declare("pm355_attn_prefill", C.c_int, [C.c_void_p] * 5 + [C.c_int] * 5 + [C.c_float, C.c_void_p])
    us = timed(lambda: [check(long(ptr(q), ptr(kc[i]), ptr(vc[i]), ptr(pos), None, None, ptr(o), ptr(scratch), H, G, d, CTX, 0.1, CTX, 0, st()), "attention") for i in range(sets)], sets)
    out["decode"]["attention"] = dict(row(us, 2 * CTX * G * d * 2, HBM), keys=CTX)
    us = timed(lambda: [check(pre(ptr(q), ptr(kc[i]), ptr(vc[i]), ptr(pos[1:]), ptr(o), PROMPT, H, G, d, CTX, 0.1, st()), "attention") for i in range(4)], 4)
    out["prefill"]["attention"] = row(us, 4.0 * d * H * PROMPT * (PROMPT + 1) / 2, MFMA)
    rp = ops.RopeParams(n_dims=d, mode=0, n_ctx_orig=8192, freq_base=500000.0, freq_scale=1.0, ext_factor=0.0, attn_factor=1.0, beta_fast=32.0, beta_slow=1.0)
    rope = L.declare("pm355_rope_kv_store", C.c_int, [C.c_void_p] * 9 + [C.c_int] * 5 + [C.c_void_p, C.c_void_p])
    k, v = torch.randn(PROMPT, G * d, device="cuda"), torch.randn(PROMPT, G * d, device="cuda")
    us = timed(lambda: [check(rope(ptr(q), ptr(k), ptr(v), ptr(o), None, ptr(kc[i]), ptr(vc[i]), ptr(pos[1:]), None, PROMPT, H, G, d, CTX, C.addressof(rp), st()), "rope") for i in range(4)], 4)
    out["prefill"]["rope_and_store"] = row(us, PROMPT * (H * d * 8 + G * d * 12), HBM)
    norm = L.declare("pm355_rms_norm", C.c_int, [C.c_void_p] * 4 + [C.c_int64, C.c_int64, C.c_float, C.c_void_p])
    r, rn, nw = torch.randn(PROMPT, W, device="cuda"), torch.empty(PROMPT, W, device="cuda"), torch.ones(W, device="cuda")
    out["prefill"]["norm"] = row(timed(lambda: [check(norm(ptr(r), ptr(nw), ptr(rn), None, W, PROMPT, 1e-5, st()), "norm") for _ in range(4)], 4), PROMPT * W * 8, HBM)
    return out


LIKE = {"proj": "qkv", "out": "out", "up": "gate|up", "down": "down", "attention": "attention", "attention_small_cap": "attention", "unit_norm_and_store": "rope_and_store", "add_norm": "norm"}


def main(what, steps, warmup):
    name, _, sizes = what.partition(":")
    if name.lower() == "keranex":
        from . import bench_keranex
        return bench_keranex.main(sizes.split(",") if sizes else [], steps, warmup)
    if name.lower() != "kudirax":
        raise SystemExit(f"--design {name}: kudirax and keranex are measured")
    res = {}
    for size in (sizes.split(",") if sizes else list(SIZES)):
        z = SIZES[size]
        m = design_model(z)
        a = {"shape": z, "dtype": "bf16", "throughput": throughput_design(m, z, steps, warmup), "kernels": kernels_design(m, z), "weight_bytes": m.weight_bytes}
        m.close()
        torch.cuda.empty_cache()
        w = window_model(z, CTX)
        b = {"weights": "Q8_0", "throughput": throughput_window(w, z, steps, warmup), "kernels": kernels_window(w, z), "weight_bytes": w.weight_bytes}
        w.close()
        torch.cuda.empty_cache()
        far = {ph: {k: round(b["kernels"][ph][LIKE[k]]["of_roofline"] / v["of_roofline"], 2) for k, v in a["kernels"][ph].items() if LIKE.get(k) in b["kernels"][ph]} for ph in ("decode", "prefill")}
        res[size] = {"kudirax": a, "llama_same_size": b, "times_further_from_roofline_than_llama": far}
        print("design %s: %s" % (size, json.dumps(far)), flush=True)
    print(json.dumps({"metric": "kudirax_decode_tokens_per_s", "value": next(iter(res.values()))["kudirax"]["throughput"]["decode_1"]["tok/s"], "unit": "tokens/s", "n_gpus": 1, "steps": steps,
                      "warmup": warmup, "higher_is_better": True, "dtype": "bf16", "data": "synthetic", "config": {"design": name, "context": CTX, "prompt": PROMPT}, "sizes": res}), flush=True)
