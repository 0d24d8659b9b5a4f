"""Kudirax on the device against the plain restatement (tests/kudirax_plain.py): kernels, each mechanism alone, prompts, decoding, portions, batches, pages, the scheduler."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import kudirax_plain as P
from test_kudirax_cpu import small_config, write_model

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"float32": 3e-5, "bfloat16": 3e-2}


def layer(heads=4, kv=2, dim=32, vdim=48, size=40, scale=0.2, cap=10.0, mix=True, ff=96):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "mask": {"size": size}, "scale": scale, "softcap": cap, "v_mix": mix},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(*layers, width=96, vocab=101, eps=1e-5):
    return {"architecture": "Kudirax", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": list(layers)}


# sizes that share nothing with each other: head groups of 1, 3, 4 and 20, key and value sizes on both sides of 64 and 128 and above 256, chunks below a page, across
# pages and of one token, layers that forget, layers without feed-forward, values that stay unmixed
CONFIGS = {
    "mixed": config(layer(), layer(heads=6, kv=2, dim=24, vdim=48, size=100, cap=3.0, ff=72), layer(heads=2, kv=2, dim=80, vdim=48, size=64, scale=0.05, cap=50.0, ff=None)),
    "wide": config(layer(heads=2, kv=1, dim=136, vdim=72, size=150, scale=0.05, cap=20.0, mix=False, ff=200),
                   layer(heads=3, kv=3, dim=64, vdim=130, size=500, scale=0.4, cap=1.5, mix=False), width=136, vocab=75, eps=1e-3),
    "group": config(layer(heads=20, kv=1, dim=16, vdim=8, size=90), layer(heads=20, kv=1, dim=72, vdim=8, size=7, scale=0.3, cap=25.0), width=64, vocab=64),
    "huge_head": config(layer(heads=1, kv=1, dim=260, vdim=12, size=33, scale=0.06), layer(heads=2, kv=1, dim=8, vdim=12, size=1), width=40, vocab=33),
    "late_mix": config(layer(mix=False, vdim=20), layer(vdim=24), layer(heads=3, kv=1, vdim=64, mix=False, ff=None), layer(heads=6, kv=2, dim=48, vdim=24, size=70, scale=0.5, cap=4.0)),
    "broad": config(layer(heads=4, kv=2, dim=64, vdim=136, size=90, scale=0.1, ff=1200), width=600, vocab=140),
    "small": small_config(),
}
MODELS = {}


def model(name, dtype, cfg=None, seed=1, weights=None, fresh=False, **pool):
    """(configuration, weights, engine model with a cache of two prompts) - kept between tests unless `fresh`"""
    from prima_cpp_amd import kudirax
    key = (name, dtype, seed)
    if fresh or key not in MODELS:
        c = cfg or CONFIGS[name]
        w = P.random_model(c, seed) if weights is None else weights
        m = kudirax.load_arrays(c, w, dtype)
        p = dict(max_tokens=1024, n_seq=4, pool_tokens=2560)
        p.update(pool)
        m.finalize_pool(**p)
        if fresh:
            return c, w, m
        MODELS[key] = (c, w, m)
    return MODELS[key]


@pytest.fixture(scope="module", autouse=True)
def release():
    yield
    for _, _, m in MODELS.values():
        m.close()
    MODELS.clear()


def tokens(n, vocab, seed=0):
    return np.random.default_rng(seed).integers(0, vocab, n).astype(np.int32)


def feed(m, seq, toks, cuts):
    """logits of every token of `toks`, fed in portions that end at `cuts`"""
    out, at = [], 0
    for c in list(cuts) + [len(toks)]:
        if c > at:
            lg = torch.empty(c - at, m.n_vocab, device="cuda")
            m.batch([(seq, toks[at:c], np.arange(c - at))], logits=lg)
            out.append(lg.cpu().numpy())
            at = c
    return np.concatenate(out)


def alone(m, toks, cuts=()):
    s = m.seq_new()
    try:
        return feed(m, s, toks, cuts)
    finally:
        m.seq_free(s)


def close(got, want, dtype, rows=None):
    d = np.asarray(got, dtype=np.float64) - want
    err = np.sqrt((d * d).mean(-1)) / want.std()
    assert err.max() < TOL[dtype], (float(err.max()), int(err.argmax()) if rows is None else rows[int(err.argmax())])


# ---- kernels -------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,K,N,n_store", [(1, 64, 64, 64), (1, 4096, 192, 190), (3, 704, 1088, 1088), (16, 640, 64, 1), (17, 576, 192, 192), (40, 128, 320, 300), (64, 2048, 128, 128),
                                           (65, 192, 448, 448), (130, 320, 64, 50), (257, 1024, 576, 570), (700, 64, 1024, 1024)])
def test_dense_mul_mat(dtype, T, K, N, n_store):
    import prima_cpp_amd.ops as O
    g = torch.Generator().manual_seed(T + K)
    w = (torch.randn(N, K, generator=g) / K ** 0.5).to(dtype).cuda()
    x = torch.randn(T, K, generator=g).to(dtype).cuda()
    b = torch.randn(N, generator=g).cuda()
    ref = x.float().cpu().double() @ w.float().cpu().double().T
    for bias, act, ydt in ((None, 0, torch.float32), (b, 0, torch.float32), (b, 1, dtype)):
        y = torch.full((T, N), 7.0, dtype=ydt, device="cuda")
        O.dense_mul_mat(w, x, y, n_store=n_store, bias=bias, act=act)
        want = ref + (bias.cpu().double() if bias is not None else 0)
        if act:
            want = want.clamp(min=0) ** 2
        tol = 2e-6 * K ** 0.5 if ydt == torch.float32 else 1e-2
        assert ((y.cpu().double() - want)[:, :n_store].abs() <= tol * (1 + want[:, :n_store].abs())).all()
        assert (y[:, n_store:] == 7.0).all()               # nothing beyond the wanted columns is touched


@pytest.mark.parametrize("tiles", [(2048, 2048), (300, 4096)])
def test_dense_mul_mat_large_tiles(tiles):
    """shapes whose grid takes the 256 x 256 tiles, ragged in both directions"""
    import prima_cpp_amd.ops as O
    T, N = tiles[0] + 37, tiles[1] + 64
    g = torch.Generator(device="cuda").manual_seed(3)
    w, x = (torch.randn(n, 512, generator=g, device="cuda").bfloat16() for n in (N, T))
    y = torch.zeros(T, N, device="cuda")
    O.dense_mul_mat(w, x, y, n_store=N - 5)
    want = x.float() @ w.float().T
    assert (y - want)[:, :N - 5].abs().max() < 2e-3 and (y[:, N - 5:] == 0).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,width", [(1, 96), (1, 2000), (2, 300), (2, 1024), (3, 320), (4, 65), (4, 512)])
def test_norm_in_the_prologue_is_the_norm_launch(dtype, T, width):
    import prima_cpp_amd.ops as O
    K = (width + 63) // 64 * 64
    g = torch.Generator().manual_seed(width)
    r, d = (torch.zeros(T, K).index_copy_(1, torch.arange(width), torch.randn(T, width, generator=g) * s + 2).cuda() for s in (1.0, 30.0))
    nw, nb = torch.randn(width, generator=g).cuda(), torch.randn(width, generator=g).cuda()
    w = (torch.randn(128, K, generator=g) / K ** 0.5).to(dtype).cuda()
    want = P.layer_norm(d[:, :width].cpu().double().numpy(), nw.cpu().numpy(), nb.cpu().numpy(), 1e-5) + r[:, :width].cpu().numpy()
    r_out, y = torch.zeros_like(r), torch.zeros(T, 128, device="cuda")
    O.dense_mul_mat_norm(w, r, d, nw, nb, 1e-5, r_out, y, width)
    assert np.abs(r_out[:, :width].cpu().numpy() - want).max() < 1e-5 * np.abs(want).max()
    xb = torch.zeros(T, K, dtype=dtype, device="cuda")
    O.add_layer_norm(r, d, nw, nb, 1e-5, width, xb)
    assert np.abs(r[:, :width].cpu().numpy() - want).max() < 1e-5 * np.abs(want).max()
    y2 = torch.zeros(T, 128, device="cuda")
    O.dense_mul_mat(w, xb, y2)
    assert (y - y2).abs().max() <= (1e-5 if dtype == torch.float32 else 3e-2) * y2.abs().max()


@pytest.mark.parametrize("rows,width", [(3, 70), (3, 1024), (2, 3000), (600, 3000), (2, 8192), (5, 9000)])
def test_add_layer_norm(rows, width):
    import prima_cpp_amd.ops as O
    g = torch.Generator().manual_seed(width)
    r, d = torch.randn(rows, width + 3, generator=g) * 2, torch.randn(rows, width + 3, generator=g) * 9 + 4
    nw, nb = torch.randn(width, generator=g), torch.randn(width, generator=g)
    want = r[:, :width].double().numpy() + P.layer_norm(d[:, :width].double().numpy(), nw.numpy(), nb.numpy(), 1e-3)
    rd, xb = r.cuda(), torch.zeros(rows, width + 3, dtype=torch.bfloat16, device="cuda")
    O.add_layer_norm(rd, d.cuda(), nw.cuda(), nb.cuda(), 1e-3, width, xb)
    assert np.abs(rd[:, :width].cpu().numpy() - want).max() < 1e-5 * np.abs(want).max()
    assert (rd[:, :width].bfloat16() == xb[:, :width]).all() and (rd[:, width:].cpu() == r[:, width:]).all() and (xb[:, width:] == 0).all()


# ---- mechanisms ----------------------------------------------------------------------------------------------------------------------
SWITCHES = {"plain": {}, "unit_norm": {"unit_norm": 1}, "cap": {"softcap": 0.7}, "sink": {"has_sink": 1}, "gate": {"gate": 1}, "chunk": {"mask": {"size": 19}}, "mix": {"v_mix": 1},
            "all": {"unit_norm": 1, "softcap": 0.7, "has_sink": 1, "gate": 1, "mask": {"size": 19}, "v_mix": 1}}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(SWITCHES))
def test_a_mechanism_alone(name, dtype):
    """two layers with one mechanism switched on (the projections, causal softmax and feed-forward are always there): prompt, and the same token by token"""
    from prima_cpp_amd import engine as E, kudirax
    from prima_cpp_amd.lib import F32
    on = SWITCHES[name]
    c = config(layer(heads=4, kv=2, dim=24, vdim=40), layer(heads=2, kv=2, dim=72, vdim=40))
    for x in c["layers"]:
        x["mixer"].update(unit_norm=0, softcap=None, has_sink=0, gate=0, mask=None, v_mix=0, scale=0.15)
        x["mixer"].update(on)
    w = P.random_model(c, 5)
    specs = []
    for x in c["layers"]:
        s, m = kudirax.layer_spec(x), x["mixer"]
        s.mix_flags = (m["unit_norm"] and E.MIX_QK_NORM) | (m["has_sink"] and E.MIX_SINK) | (m["gate"] and E.MIX_OUT_GATE) | (m["v_mix"] and E.MIX_VALUE_MIX)
        specs.append(s)
    m = E.Stack("kudirax", specs, c["width"], c["vocab"], c["norm"]["eps"], kudirax.DTYPES[dtype])
    skip = {E.T_SINK: "has_sink", E.T_W_OUT_GATE: "gate", E.T_VALUE_MIX: "v_mix"}
    for kind, i, nm, shape in kudirax.tensors(c):
        if kind not in skip or c["layers"][i]["mixer"][skip[kind]]:
            m.set_tensor(kind, i, F32, w[nm])
    m.finalize_pool(256, 2, 512)
    toks = tokens(70, c["vocab"], 2)
    want = P.run(c, w, toks)
    close(alone(m, toks), want, dtype)
    close(alone(m, toks, range(1, 70)), want, dtype)
    if name != "plain":                                    # the mechanism shows: without it the result is another one
        off = copy.deepcopy(c)
        for x in off["layers"]:
            x["mixer"].update(unit_norm=0, softcap=None, has_sink=0, gate=0, mask=None, v_mix=0)
        other = P.run(off, w, toks)
        assert np.sqrt(((other - want) ** 2).mean(-1)).max() / want.std() > 4 * TOL[dtype]
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompts_decoding_and_portions(name, dtype):
    c, w, m = model(name, dtype)
    toks = tokens(230, c["vocab"], 1)
    want = P.run(c, w, toks)
    close(alone(m, toks), want, dtype)
    close(alone(m, toks, range(150, 230)), want, dtype)                                  # a prompt, then token by token
    close(alone(m, toks[:40], range(1, 40)), want[:40], dtype)                           # token by token from the first
    for step in (2, 3, 17, 63, 64, 65, 129):
        close(alone(m, toks, range(step, 230, step)), want, dtype)
    close(alone(m, toks, np.cumsum([1, 2, 61, 1, 64, 5, 31, 2, 1])), want, dtype)        # cuts inside and at the borders of pages and chunks


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_passes_that_do_not_hold_a_step(dtype):
    """a step longer than the engine's scratch runs in pieces; wanted rows in any order"""
    c, w, m = model("mixed", dtype, fresh=True, max_tokens=48)
    toks, toks2 = tokens(150, c["vocab"], 3), tokens(37, c["vocab"], 4)
    a, b = m.seq_new(), m.seq_new()
    order = np.random.default_rng(0).permutation(150).astype(np.int32)
    lg = torch.empty(150 + 2, c["vocab"], device="cuda")
    m.batch([(a, toks, order), (b, toks2, [36, 0])], logits=lg)
    close(lg[:150].cpu().numpy(), P.run(c, w, toks)[order], dtype)
    close(lg[150:].cpu().numpy(), P.run(c, w, toks2)[[36, 0]], dtype)
    m.close()


# ---- edges -----------------------------------------------------------------------------------------------------------------------------
def spot_model(size, cap=40.0, dim=32, heads=2, kv=1):
    """One layer in which a query on token 1 finds the keys of token 2 (and hardly anything else), whose value no other token has: the logits tell how many of them it sees."""
    W, V = 64, 16
    c = config(layer(heads=heads, kv=kv, dim=dim, vdim=16, size=size, scale=1.0, cap=cap, mix=False, ff=None), width=W, vocab=V)
    w = {k: np.array(v) for k, v in P.random_model(c, 9).items()}
    e = np.zeros((V, W))
    e[np.arange(V), np.arange(V)] = 4.0
    w["embed"] = e
    for nm, rows, col in (("q", heads * dim, 1), ("k", kv * dim, 2)):
        a = np.random.default_rng(3).normal(0, 0.02, (rows, W))
        a[:, col] = np.tile(np.resize([1.0, -1.0, 1.0, 1.0], dim), rows // dim)          # q of token 1 and k of token 2 point the same way
        w["l0.mix." + nm] = a
    v = np.random.default_rng(4).normal(0, 0.01, (kv * 16, W))
    v[:, 2] = np.linspace(1, 2, kv * 16)
    w["l0.mix.v"] = v
    w["l0.mix.sink"] = np.full(heads, 20.0)
    bf = torch.from_numpy
    return c, {k: bf(np.asarray(a, dtype=np.float32)).bfloat16().float().numpy() for k, a in w.items()}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("size,far", [(48, False), (64, False), (200, False), (700, True)])
def test_keys_at_every_edge(dtype, size, far):
    """the marked key just inside and just outside the chunk, at page borders and far back, asked for in a prompt, by a decoded token and in a short portion"""
    c, w = spot_model(size)
    _, _, m = model("spot%d" % size, dtype, c, 9, w)
    n = 2 * size + 9 if not far else 700
    seen = []
    for q in sorted({size - 1, size, 2 * size - 1, 2 * size, n - 1, 130 % n}):
        start = q - q % size
        for k in sorted({start - 1, start, start + 1, 63, 64, 127, 128, q - 1, 0}):
            if not 0 <= k < q:
                continue
            toks = np.full(q + 1, 5, dtype=np.int32)
            toks[k], toks[q] = 2, 1
            want = P.run(c, w, toks)[q:]
            for cuts in ((), (q,), (q - 1,), (q // 2, q)):
                close(alone(m, toks, cuts)[q:], want, dtype, ["query %d key %d cuts %s" % (q, k, cuts)])
            seen.append((start <= k, want[0]))
    inside, outside = ([x for ok, x in seen if ok == s] for s in (True, False))
    assert inside and np.std(inside[0]) > 0
    if outside:                                            # the two kinds of place give different answers, by far more than the tolerance
        assert np.sqrt(((inside[0] - outside[0]) ** 2).mean()) / np.std(inside) > 4 * TOL[dtype]


def test_the_edge_test_would_see_a_chunk_that_is_one_token_off():
    """a mistake planted in the restatement: chunks one token longer"""
    c, w = spot_model(64)
    toks = np.full(65, 5, dtype=np.int32)
    toks[63], toks[64] = 2, 1
    off = copy.deepcopy(c)
    off["layers"][0]["mixer"]["mask"]["size"] = 65
    a, b = P.run(c, w, toks)[64], P.run(off, w, toks)[64]
    assert np.sqrt(((a - b) ** 2).mean()) / a.std() > 4 * TOL["bfloat16"]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens_and_sinks(dtype):
    """the first tokens of a sequence, where a sink weighs most: every one of them alone in a portion, and sinks from negligible to overwhelming"""
    c = CONFIGS["mixed"]
    for value in (-30.0, 0.0, 6.0, 60.0):
        w = dict(P.random_model(c, 6))
        for i in range(3):
            w["l%d.mix.sink" % i] = np.full_like(w["l%d.mix.sink" % i], value)
        _, _, m = model("sink", dtype, c, 6, w, fresh=True)
        toks = tokens(5, c["vocab"], 8)
        want = P.run(c, w, toks)
        for cuts in ((), (1, 2, 3, 4), (2,), (1, 3)):
            close(alone(m, toks, cuts), want, dtype)
        m.close()


# ---- batches, pages, slots ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "group", "wide"])
def test_unequal_requests_together(name, dtype):
    """portions of some requests beside single tokens of others; each against itself alone and against the restatement"""
    c, w, m = model(name, dtype)
    reqs = [tokens(n, c["vocab"], 20 + n) for n in (190, 77, 1, 140)]
    want = [P.run(c, w, t) for t in reqs]
    seqs, at, got = [m.seq_new() for _ in reqs], [0] * 4, [[] for _ in reqs]
    plan = [(64, 0, 0, 3), (1, 20, 0, 1), (37, 1, 1, 60), (1, 1, 0, 2), (0, 55, 0, 1), (87, 0, 0, 73)]
    for step in plan:
        es = [(seqs[i], reqs[i][at[i]:at[i] + n], np.arange(n)) for i, n in enumerate(step) if n]
        lg = torch.empty(sum(step), c["vocab"], device="cuda")
        m.batch(es, logits=lg)
        row = 0
        for i, n in enumerate(step):
            got[i].append(lg[row:row + n].cpu().numpy())
            row, at[i] = row + n, at[i] + n
    for i, s in enumerate(seqs):
        g = np.concatenate(got[i])
        assert len(g) == len(reqs[i])
        close(g, want[i], dtype)
        m.seq_free(s)
        close(g, np.asarray(alone(m, reqs[i]), dtype=np.float64), dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decoding_many_sequences_at_once(dtype):
    """1 .. 70 tokens per step, repeated so that the captured step graph replays; every replay against the restatement"""
    c, w, m = model("mixed", dtype, fresh=True, n_seq=70, pool_tokens=70 * 192)
    reqs = [tokens(100, c["vocab"], i) for i in range(70)]
    want = [P.run(c, w, t) if i in (0, 1, 5, 16, 33, 63, 69) else None for i, t in enumerate(reqs)]
    seqs, at = [m.seq_new() for _ in reqs], [30 + i % 9 for i in range(70)]
    m.batch([(s, t[:a], []) for s, t, a in zip(seqs, reqs, at)])
    lg = torch.empty(70, c["vocab"], device="cuda")
    for n, reps in ((1, 4), (2, 4), (3, 4), (6, 4), (17, 5), (34, 5), (64, 5), (70, 4)):
        for _ in range(reps):
            m.batch([(seqs[i], reqs[i][at[i]:at[i] + 1], [0]) for i in range(n)], logits=lg)
            for i in range(n):
                if want[i] is not None:
                    close(lg[i:i + 1].cpu().numpy(), want[i][at[i]:at[i] + 1], dtype, ["sequence %d of %d at %d" % (i, n, at[i])])
                at[i] += 1
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_pages_and_slots_are_used_again(dtype):
    """a pool with room for little more than the live requests: stale pages of all kinds lie under every new one"""
    c, w, m = model("wide", dtype, fresh=True, pool_tokens=512, n_seq=2)
    rng = np.random.default_rng(5)
    live = {}
    want = {}
    for step in range(40):
        if len(live) < 2:
            n = int(rng.integers(3, 200))
            key = step
            live[key] = [m.seq_new(), tokens(n, c["vocab"], 100 + step), 0]
            want[key] = P.run(c, w, live[key][1])
        es, keys = [], []
        for key, (s, t, a) in live.items():
            n = min(int(rng.choice([1, 2, 33, 70])), len(t) - a)
            es.append((s, t[a:a + n], [n - 1]))
            keys.append(key)
            live[key][2] += n
        lg = torch.empty(len(es), c["vocab"], device="cuda")
        m.batch(es, logits=lg)
        for i, key in enumerate(keys):
            s, t, a = live[key]
            close(lg[i:i + 1].cpu().numpy(), want[key][a - 1:a], dtype, ["request %d at %d" % (key, a - 1)])
            if a == len(t):
                m.seq_free(s)
                del live[key]
    assert len(want) > 5
    m.close()


def test_pool_limits_are_errors_and_change_nothing():
    from prima_cpp_amd.lib import PM355Error
    c, w, m = model("mixed", "bfloat16", fresh=True, pool_tokens=128, n_seq=2)
    a, b = m.seq_new(), m.seq_new()
    with pytest.raises(PM355Error):
        m.seq_new()
    toks = tokens(120, c["vocab"])
    m.batch([(a, toks[:70], [])])
    assert m.pool_info().free_pages in (0, 1)              # (two pages, or one where the first lies in front of every chunk)
    before = (m.pool_info().free_pages, m.seq_len(a))
    for bad in ([(b, tokens(129, c["vocab"]), [])], [(a, [c["vocab"]], [])], [(a, [1], [1])], [(7, [1], [])], [(a, [1], []), (a, [1], [])]):
        with pytest.raises(PM355Error):
            m.batch(bad)
    assert (m.pool_info().free_pages, m.seq_len(a)) == before
    lg = torch.empty(1, c["vocab"], device="cuda")
    m.batch([(a, toks[70:71], [0])], logits=lg)
    close(lg.cpu().numpy(), P.run(c, w, toks[:71])[70:], "bfloat16")
    m.seq_free(a)
    m.seq_free(b)
    assert m.pool_info().free_pages == 2
    m.close()


def test_a_sequence_outgrows_the_pool_when_every_layer_forgets():
    """long decoding: pages in front of every layer's chunk go back to the pool while the sequence goes on"""
    c = config(layer(size=48), layer(heads=2, kv=2, size=130), width=64, vocab=50)
    _, w, m = model("forgets", "bfloat16", c, fresh=True, pool_tokens=256, n_seq=1)
    toks = tokens(700, 50, 3)
    want = P.run(c, w, toks)
    s = m.seq_new()
    close(feed(m, s, toks, list(range(90, 360, 90)) + list(range(360, 700))), want, "bfloat16")
    m.close()


@pytest.mark.parametrize("heads,kv,dim,vdim,size", [(8, 2, 128, 128, None), (4, 4, 64, 64, 3000), (2, 1, 256, 200, None), (5, 5, 100, 64, 1500)])
def test_attention_over_thousands_of_keys(heads, kv, dim, vdim, size):
    """keys split over workgroups (merge in the launch), prompt tiles over many pages: one marked key far back decides the answer"""
    c, w = spot_model(size, dim=dim, heads=heads, kv=kv)
    c["layers"][0]["mixer"].update(vdim=16, scale=0.35)
    rng = np.random.default_rng(1)
    if vdim != 16:
        c["layers"][0]["mixer"]["vdim"] = vdim
        full = P.random_model(c, 9)
        for nm in ("l0.mix.v", "l0.mix.g", "l0.mix.o"):
            w[nm] = full[nm]
    _, _, m = model("long", "bfloat16", c, 9, w, fresh=True, max_tokens=2048, pool_tokens=4096, n_seq=2)
    n = 2900
    toks = rng.integers(3, 16, n).astype(np.int32)
    toks[[5, 700, 1490, 1510, 2700]] = 2
    qs = [1400, 1600, 2890, 2896, 2897, 2898, 2899]
    toks[qs] = 1
    want = P.run(c, w, toks)
    got = alone(m, toks, [1000, 1001, 2895, 2896, 2897, 2898, 2899])
    close(got[qs], want[qs], "bfloat16", qs)
    m.close()


# ---- generation ----------------------------------------------------------------------------------------------------------------------------
def greedy(c, w, prompt, n):
    """greedy tokens of the restatement, and the smallest lead of a winner over the runner-up"""
    t, lead = list(prompt), np.inf
    for _ in range(n):
        lg = np.sort(P.run(c, w, t)[-1])
        lead = min(lead, (lg[-1] - lg[-2]) / lg.std())
        t.append(int(np.argmax(P.run(c, w, t)[-1])))
    return t[len(prompt):], lead


@pytest.mark.parametrize("lag", [0, 1, 3])
def test_scheduler_generates_what_the_restatement_generates(lag):
    from prima_cpp_amd import scheduler
    c, w, m = model("mixed", "float32", fresh=True, n_seq=3, pool_tokens=512)
    prompts = [tokens(n, c["vocab"], 40 + n).tolist() for n in (5, 130, 61, 64, 1, 33)]
    got = scheduler.generate(m, prompts, 12, portion=50, step_tokens=64, lag=lag)
    for p, g in zip(prompts, got):
        want, lead = greedy(c, w, p, 12)
        assert g == want or lead < 1e-4, (p, g, want)
    info = m.pool_info()
    assert info.free_seqs == 3 and info.free_pages == info.n_pages
    m.close()


def test_scheduler_serves_quantized_windows_too(tmp_path):
    """the same scheduler over a GGUF layer window: same tokens as its own device-resident greedy loop"""
    from prima_cpp_amd import gguf, registry, scheduler
    path = str(tmp_path / "m.gguf")
    gguf.write_synthetic_model(path, arch=0, n_layer=2, n_embd=256, n_head=4, n_head_kv=2, n_ff=512, n_vocab=320)
    m = registry.load(path, n_ctx=128)
    m.finalize_pool(64, 2, 256)
    prompts = [tokens(n, 320, n).tolist() for n in (9, 20, 4)]
    got = scheduler.generate(m, prompts, 8, portion=64)
    for p, g in zip(prompts, got):
        _, _, am = m.decode(tokens=torch.tensor(p, dtype=torch.int32, device="cuda"), pos0=0, want_hidden=False, want_logits=False, want_argmax=True)
        io = torch.zeros(9, dtype=torch.int32, device="cuda")
        io[0] = am[0]
        m.generate(io, len(p), 7)
        assert g == io[:8].cpu().tolist()
    m.close()


def test_device_resident_greedy_loop():
    c, w, m = model("small", "float32", fresh=True)
    prompt = tokens(20, c["vocab"], 2)
    s = m.seq_new()
    first = torch.zeros(1, dtype=torch.int32, device="cuda")
    m.batch([(s, prompt, [19])], argmax=first)
    io = torch.zeros(11, dtype=torch.int32, device="cuda")
    io[0] = first[0]
    m._chk(m.lib.pm355_model_generate(m.h, io.data_ptr(), 20, 10, 1, torch.cuda.current_stream().cuda_stream), "generate")
    want, lead = greedy(c, w, prompt.tolist(), 11)
    assert io.cpu().tolist() == want or lead < 1e-4
    m.close()


def test_command_line_and_trace_replay(tmp_path):
    """a model folder on disk through `python -m prima_cpp_amd` and bin/trace_run"""
    c = small_config()
    w = P.random_model(c, 12)
    path = write_model(tmp_path / "m", c, w)
    prompt = tokens(9, c["vocab"], 1).tolist()
    r = subprocess.run([sys.executable, "-m", "prima_cpp_amd", path, "--prompt", ",".join(map(str, prompt)), "-n", "5", "--dtype", "float32"], cwd=ROOT, capture_output=True, text=True,
                       timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    got = json.loads(r.stdout.strip().splitlines()[-1])["tokens"]
    want, lead = greedy(c, w, prompt, 5)
    assert got == want or lead < 1e-4
    toks = {"a": tokens(70, c["vocab"], 3), "b": tokens(40, c["vocab"], 4)}
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks["a"][:66].tolist(), "want": [0, 65]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": toks["b"][:39].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": toks["a"][66:67].tolist(), "want": [0]}, {"id": "b", "tokens": toks["b"][39:].tolist(), "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": toks["a"][67:].tolist(), "want": [2, 0]}], "end": ["a"]}]
    full = {k: P.run(c, w, t) for k, t in toks.items()}
    rows = {0: full["a"][[0, 65]], 2: np.stack([full["a"][66], full["b"][39]]), 3: full["a"][[69, 67]]}
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / dtype
        out.mkdir()
        r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out), "--max-tokens", "192"],
                           input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done %d" % i for i in range(4)]
        assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
        for s, want in rows.items():
            close(np.fromfile(out / ("%d.f32" % s), dtype="<f4").reshape(want.shape), want, dtype)
