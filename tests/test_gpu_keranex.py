"""Keranex on the device against the plain restatement (tests/keranex_plain.py): each mechanism alone, prompts, decoding, portions, batches, pages, slots, the scheduler."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import keranex_plain as P
from test_gpu_kudirax import ROOT, alone, feed, tokens
from test_keranex_cpu import config, latent, moe, scan, small_config
from test_kudirax_cpu import write_model

pytestmark = pytest.mark.gpu
TOL, TYPICAL = {"float32": 3e-5, "bfloat16": 8e-2}, {"float32": 3e-6, "bfloat16": 2e-2}      # of the worst position, of the median one
DTYPES = ["float32", "bfloat16"]

# sizes that share nothing with each other: heads below, at and above 16, key, value and latent sizes on both sides of 64, 128, 192 and 256, states that need padding,
# convolutions of one to seven taps, windows of one token, inside a page and across pages, layers that read an earlier layer's latents, without feed-forward, experts of all
# counts that a wave's lanes do not divide
CONFIGS = {
    "mixed": config(latent(mlp=moe()), scan(mlp=moe(4, 3, 1, 1, 40)), latent(heads=5, dim=40, vdim=72, size=100, kv_from=0, q_rank=17, scale=0.15, mlp=None), scan(inner=200, state=20, dt_rank=70, conv=3),
                    latent(heads=2, dim=8, rot_dim=16, vdim=24, kv_rank=64, size=7, base=300.0, mlp=moe(5, 5, 1, 1, 24))),
    "scan_first": config(scan(inner=130, state=1, dt_rank=1, conv=1, mlp=moe(9, 1, 3, 2, 130)), scan(inner=64, state=40, dt_rank=30, conv=7), scan(inner=65, state=64, dt_rank=64, conv=2),
                         latent(heads=1, dim=1, rot_dim=2, vdim=17, q_rank=19, kv_rank=22, size=64, scale=1.0), width=70, vocab=65, eps=1e-3, bigram=(13, 5, 3)),
    "wide": config(latent(heads=2, dim=136, rot_dim=64, vdim=130, q_rank=100, kv_rank=160, size=150, scale=0.08, mlp=moe(12, 5, 4, 2, 200)),
                   latent(heads=3, dim=150, rot_dim=64, vdim=64, q_rank=200, kv_rank=160, size=500, scale=0.05, kv_from=0), width=136, vocab=75, bigram=None),
    "many_heads": config(latent(heads=20, dim=16, rot_dim=4, vdim=8, kv_rank=130, size=90, mlp=moe(70, 9, 7, 3, 30)), latent(heads=33, dim=32, rot_dim=4, vdim=16, q_rank=64, kv_rank=130, size=1, kv_from=0),
                         latent(heads=16, dim=64, rot_dim=64, vdim=64, q_rank=64, kv_rank=300, size=65, scale=0.1), width=64, vocab=64),
    "huge": config(latent(heads=1, dim=260, rot_dim=12, vdim=300, q_rank=70, kv_rank=1100, size=33, scale=0.06), scan(inner=80, state=300, dt_rank=7, conv=4),
                   latent(heads=2, dim=180, rot_dim=70, vdim=20, q_rank=30, kv_rank=520, size=200, scale=0.06, mlp=moe(3, 2, 1, 1, 600)), width=48, vocab=33),
    "broad": config(scan(inner=1100, state=24, dt_rank=40), latent(heads=4, dim=72, vdim=136, q_rank=560, kv_rank=250, size=120, mlp=moe(7, 3, 1, 1, 300)), width=600, vocab=140),
    "small": small_config(),
}
MODELS = {}


def weights_for(c, dtype, seed):
    return P.random_model(c, seed, decisive=dtype == "bfloat16")


def model(name, dtype, cfg=None, seed=1, weights=None, fresh=False, **pool):
    """(configuration, weights, engine model with a cache of two prompts) - kept between tests unless `fresh`"""
    from prima_cpp_amd import keranex
    key = (name, dtype, seed)
    if fresh or key not in MODELS:
        c = cfg or CONFIGS[name]
        w = weights_for(c, dtype, seed) if weights is None else weights
        m = keranex.load_arrays(c, w, dtype)
        p = dict(max_tokens=1024, n_seq=4, pool_tokens=2560)
        p.update(pool)
        m.finalize_pool(**p)
        if fresh:
            return c, w, m
        MODELS[key] = (c, w, m)
    return MODELS[key]


@pytest.fixture(scope="module", autouse=True)
def release_models():
    yield
    for _, _, m in MODELS.values():
        m.close()
    MODELS.clear()


def error(got, want):
    """per row: root mean square of the difference over the vocabulary, in units of the wanted logits' spread"""
    d = np.asarray(got, dtype=np.float64) - want
    return np.sqrt((d * d).mean(-1)) / want.std()


def close(got, want, dtype, rows=None):
    e = error(got, want)
    worst, typical, at = float(e.max()), float(np.median(e)), int(e.argmax())
    assert worst < TOL[dtype], (worst, typical, rows[at % len(rows)] if rows else at)
    assert len(e) < 20 or typical < TYPICAL[dtype], (worst, typical)


# ---- mechanisms ----------------------------------------------------------------------------------------------------------------------
def silent(w, layer, ff=False):
    """the layer's mixer (or feed-forward) adds nothing"""
    k = "l%d.%s" % (layer, "norm2b" if ff else "norm1b")
    return dict(w, **{k: np.zeros_like(w[k])})


def one(layer, **kw):
    kw.setdefault("bigram", None)
    return config(layer, **kw)


MECHANISMS = {
    "embedding": (one(scan()), lambda w: silent(w, 0), None),
    "bigram": (one(scan(), bigram=(97, 31, 7)), lambda w: silent(w, 0), lambda c: c["embedding"]["bigram"].update(mul_prev=0)),
    "bigram_large": (one(scan(), bigram=(3001, 2147483629, 1999999973)), lambda w: silent(w, 0), lambda c: c["embedding"]["bigram"].update(mul_cur=1)),
    "latent": (one(latent(size=1000, base=1e30)), None, lambda c: c["layers"][0]["mixer"].update(scale=0.0)),
    "rotation": (one(latent(dim=4, rot_dim=32, size=1000)), None, lambda c: c["layers"][0]["mixer"]["rot"].update(base=5500.0)),
    "window": (one(latent(size=19)), None, lambda c: c["layers"][0]["mixer"]["mask"].update(size=20)),
    "shared_latents": (config(latent(), latent(heads=4, size=30, kv_from=0), latent(size=9, kv_from=0), bigram=None), None, lambda c: c["layers"][1]["mixer"]["mask"].update(size=31)),
    "scan": (one(scan(conv=1)), None, None),
    "convolution": (one(scan(conv=6, state=4)), None, None),
    "experts": (one(scan(mlp=moe(8, 3, 1, 1))), lambda w: silent(w, 0), lambda c: c["layers"][0]["mlp"]["router"].update(top=2)),
    "groups": (one(scan(mlp=moe(24, 4, 6, 2))), lambda w: silent(w, 0), lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=3)),
    "eps": (one(latent(mlp=moe()), eps=0.5), None, lambda c: c["norm"].update(eps=0.4)),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_a_mechanism_alone(name, dtype):
    """one mechanism at work (the others add nothing): a prompt, and the same token by token; a slightly different mechanism gives another result"""
    c, edit, other = MECHANISMS[name]
    w = weights_for(c, dtype, 5)
    w = edit(w) if edit else w
    _, _, m = model(name, dtype, c, 5, w, fresh=True, max_tokens=256, n_seq=2, pool_tokens=512)
    toks = tokens(70, c["vocab"], 2)
    want = P.run(c, w, toks)
    close(alone(m, toks), want, dtype)
    close(alone(m, toks, range(1, 70)), want, dtype)
    if other:                                              # the mistake is planted in the restatement
        off = copy.deepcopy(c)
        other(off)
        if name.startswith("bigram"):
            off["embedding"]["bigram"]["buckets"] = c["embedding"]["bigram"]["buckets"]
        assert error(P.run(off, w, toks), want).max() > 4 * TOL["float32"]
    m.close()


@pytest.mark.parametrize("E,top,count,keep", [(1, 1, 1, 1), (2, 2, 2, 2), (64, 64, 1, 1), (65, 3, 5, 1), (96, 12, 8, 4), (300, 10, 100, 7)])
def test_routing_picks_the_same_experts(E, top, count, keep):
    """true 32-bit: random router logits, from one token to a batch beyond every routing kernel's size"""
    c = one(scan(inner=64, mlp=moe(E, top, count, keep, 16)), width=64, vocab=200)
    w = silent(P.random_model(c, 3), 0)
    _, _, m = model("route", "float32", c, 3, w, fresh=True, max_tokens=512, n_seq=2, pool_tokens=1024)
    toks = tokens(300, 200, 5)
    want = P.run(c, w, toks)
    for n in (1, 2, 4, 5, 64, 65, 300):
        close(alone(m, toks[:n]), want[:n], "float32")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff,E,top", [(4700, 3, 2), (1030, 5, 1), (576, 2, 2)])
def test_wide_experts(ff, E, top, dtype):
    """hidden layers too long for the small-batch kernels' on-chip copies, and of block counts that leave some waves without work"""
    c = one(scan(inner=64, mlp=moe(E, top, 1, 1, ff)), width=72)
    w = silent(weights_for(c, dtype, 8), 0)
    _, _, m = model("experts", dtype, c, 8, w, fresh=True, max_tokens=512, n_seq=2, pool_tokens=1024)
    toks = tokens(150, c["vocab"], 5)
    want = P.run(c, w, toks)
    for n in (1, 4, 5, 33, 64, 150):
        close(alone(m, toks[:n]), want[:n], dtype)
    if E == 2:                                             # enough pairs per expert for the large tiles
        toks = tokens(900, c["vocab"], 6)
        close(alone(m, toks, (450,)), P.run(c, w, toks), dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_decay_reaches_as_far_as_it_should(dtype):
    """scan states from forgotten at once to kept for the whole sequence, steps from tiny to large (the softplus's linear end)"""
    c = one(scan(inner=64, state=16, conv=2), width=64)
    w = dict(weights_for(c, dtype, 4))
    a, b = np.meshgrid(np.linspace(-9, 4, 16), np.linspace(-12, 25, 64))
    w["l0.mix.A_log"], w["l0.mix.dt.b"] = P.bf16(a), P.bf16(b[:, 0])
    _, _, m = model("decay", dtype, c, 4, w, fresh=True)
    toks = tokens(500, c["vocab"], 6)
    want = P.run(c, w, toks)
    for cuts in ((), (128, 256, 384), (1, 130, 131, 300), range(2, 500, 2)):
        close(alone(m, toks, cuts), want, dtype)
    m.close()


# ---- prompts, decoding, portions ---------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompts_decoding_and_portions(name, dtype):
    c, w, m = model(name, dtype)
    toks = tokens(300, c["vocab"], 1)
    want = P.run(c, w, toks)
    close(alone(m, toks), want, dtype)
    close(alone(m, toks, range(200, 300)), want, dtype)                                  # a prompt, then token by token
    close(alone(m, toks[:40], range(1, 40)), want[:40], dtype)                           # token by token from the first
    for step in (2, 3, 17, 32, 33, 63, 64, 65, 127, 129):
        close(alone(m, toks, range(step, 300, step)), want, dtype)
    close(alone(m, toks, np.cumsum([1, 2, 61, 1, 64, 5, 31, 2, 1])), want, dtype)        # cuts inside and at the borders of pages, windows and chunks


@pytest.mark.parametrize("name", ["mixed", "many_heads"])
def test_unfused_kernels_give_the_same(name, monkeypatch):
    """PM355_STACK_PLAIN=1: every step as launches of its own, attention on the vector pipe"""
    monkeypatch.setenv("PM355_STACK_PLAIN", "1")
    c, w, m = model(name, "bfloat16", fresh=True)
    toks = tokens(120, c["vocab"], 1)
    close(alone(m, toks, (70, 71, 72, 110)), P.run(c, w, toks), "bfloat16")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_passes_that_do_not_hold_a_step(dtype):
    """a step longer than the engine's scratch runs in pieces (states and previous tokens go from one to the next); wanted rows in any order"""
    c, w, m = model("mixed", dtype, fresh=True, max_tokens=48)
    toks, toks2 = tokens(150, c["vocab"], 3), tokens(37, c["vocab"], 4)
    a, b = m.seq_new(), m.seq_new()
    order = np.random.default_rng(0).permutation(150).astype(np.int32)
    lg = torch.empty(150 + 2, c["vocab"], device="cuda")
    m.batch([(a, toks, order), (b, toks2, [36, 0])], logits=lg)
    close(lg[:150].cpu().numpy(), P.run(c, w, toks)[order], dtype)
    close(lg[150:].cpu().numpy(), P.run(c, w, toks2)[[36, 0]], dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens(dtype):
    """the first tokens of a sequence, alone in portions and together: empty states, zeros in front of the convolutions, the table row of a token without a predecessor"""
    c, w, m = model("mixed", dtype)
    for seed in range(3):
        toks = tokens(6, c["vocab"], 80 + seed)
        want = P.run(c, w, toks)
        for cuts in ((), (1, 2, 3, 4, 5), (2,), (1, 3), (3, 4)):
            close(alone(m, toks, cuts), want, dtype)


# ---- edges -----------------------------------------------------------------------------------------------------------------------------
def spot_model(size, heads=2, dim=32, rot_dim=8, vdim=16, q_rank=48, kv_rank=48, kv_from=False, peak=16.0):
    """A layer in which a query on token 1 finds the keys of token 2 and hardly anything else, and the value of token 2 is one that no other token has. kv_from: two layers
    in front, so that the finding layer reads the first one's latents."""
    W, V = 64, 16
    layers = [latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, size, scale=1.0)]
    if kv_from:
        layers = [latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, 3, scale=0.1), scan(inner=64), latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, size, scale=1.0, kv_from=0)]
    c = config(*layers, width=W, vocab=V, bigram=None)
    w, rng, f, s = dict(P.random_model(c, 9)), np.random.default_rng(3), "l%d.mix." % (len(layers) - 1), "l0.mix."
    if kv_from:
        w = silent(silent(w, 0), 1)
    w["embed"] = 4.0 * np.eye(V, W)
    for n in ("l%d.norm1" % (len(layers) - 1), "l0.norm1"):
        w[n] = np.ones(W)
    for p, key, nm, tok in ((f, "dq", q_rank, 1), (s, "dkv", kv_rank, 2)):
        a = rng.normal(0, 1, (nm, W))
        a[0], a[:, tok] = 0.0, 0.0                         # the first entry of the latent: the marked token and nobody else
        a[0, tok] = 1.0
        w[p + key] = np.concatenate([a, np.zeros((rot_dim, W))]) if key == "dkv" else a
        w[p + key + ".norm"] = np.ones(nm)
    uq, uk = np.zeros((heads, dim + rot_dim, q_rank)), np.zeros((heads, dim, kv_rank))
    g = np.resize([1.0, -1.0, 1.0, 1.0], dim)
    uq[:, :dim, 0] = g / np.sqrt(q_rank)
    uk[:, :, 0] = g * peak / dim / np.sqrt(kv_rank)
    uv = rng.normal(0, 0.05, (heads * vdim, kv_rank))
    uv[:, 0] = np.linspace(1, 2, heads * vdim)
    w.update({f + "uq": uq.reshape(-1, q_rank), f + "uk": uk.reshape(-1, kv_rank), f + "uv": uv})
    return c, {k: P.bf16(a) for k, a in w.items()}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size,kv_from", [(1, False), (2, False), (33, False), (64, True), (100, False), (200, True), (700, False)])
def test_keys_at_every_edge(dtype, size, kv_from):
    """the marked key just inside and just outside the window, at page borders and far back, asked for in a prompt, by a decoded token and in short and long portions"""
    c, w = spot_model(size, kv_from=kv_from)
    _, _, m = model("spot%d" % size, dtype, c, 9, w)
    seen = []
    for q in sorted({size - 1, size, size + 1, 2 * size + 63, 130, 192, 640}):
        if q > 2 * size + 200 or q < 1:
            continue
        for k in sorted({q - size - 1, q - size, q - size + 1, 63, 64, 127, 128, q - 1, 0}):
            if not 0 <= k < q:
                continue
            toks = np.full(q + 1, 5, dtype=np.int32)
            toks[k], toks[q] = 2, 1
            want = P.run(c, w, toks)[q:]
            for cuts in ((), (q,), (q - 1,), (q // 2, q), (max(q - 40, 1),)):
                close(alone(m, toks, cuts)[q:], want, dtype, ["query %d key %d cuts %s" % (q, k, cuts)])
            seen.append((q - k < size, want[0]))
    inside, outside = ([x for ok, x in seen if ok == s] for s in (True, False))
    for a in inside[:1]:
        for b in outside[:1]:                              # the two kinds of place give different answers, by far more than the tolerance
            assert np.sqrt(((a - b) ** 2).mean()) / a.std() > 4 * TOL[dtype]


def test_the_edge_test_would_see_a_window_that_is_one_token_off():
    """a mistake planted in the restatement"""
    c, w = spot_model(64)
    toks = np.full(90, 5, dtype=np.int32)
    toks[25], toks[89] = 2, 1
    off = copy.deepcopy(c)
    off["layers"][0]["mixer"]["mask"]["size"] = 65
    a, b = P.run(c, w, toks)[89], P.run(off, w, toks)[89]
    assert np.sqrt(((a - b) ** 2).mean()) / a.std() > 4 * TOL["bfloat16"]


@pytest.mark.parametrize("heads,dim,rot_dim,vdim,kv_rank,size", [(8, 128, 64, 128, 512, 5000), (16, 64, 32, 64, 256, 1500), (3, 100, 20, 72, 100, 2500), (40, 32, 64, 32, 700, 1400)])
def test_attention_over_thousands_of_keys(heads, dim, rot_dim, vdim, kv_rank, size):
    """keys split over workgroups (merge in the launch), prompt tiles over many pages: one marked key far back decides the answer"""
    c, w = spot_model(size, heads, dim, rot_dim, vdim, 96, kv_rank, peak=30.0)
    _, _, m = model("long", "bfloat16", c, 9, w, fresh=True, max_tokens=2048, pool_tokens=4096, n_seq=2)
    n = 2900
    toks = np.random.default_rng(1).integers(3, 16, n).astype(np.int32)
    toks[[5, 700, 1490, 1510, 2700]] = 2
    qs = [1400, 1600, 2890, 2896, 2897, 2898, 2899]
    toks[qs] = 1
    want = P.run(c, w, toks)
    got = alone(m, toks, [1000, 1001, 2895, 2896, 2897, 2898, 2899])
    close(got[qs], want[qs], "bfloat16", qs)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_far_into_a_sequence(dtype):
    """scores that depend on angles alone, thousands of tokens in"""
    c = one(latent(heads=2, dim=1, rot_dim=32, vdim=32, kv_rank=64, size=90, base=10000.0, scale=0.5), width=64)
    w = weights_for(c, dtype, 7)
    _, _, m = model("far", dtype, c, 7, w, fresh=True, max_tokens=2048, pool_tokens=4096, n_seq=1)
    toks = tokens(3000, c["vocab"], 2)
    close(alone(m, toks, [2000, 2990] + list(range(2991, 3000)))[-60:], P.run(c, w, toks)[-60:], dtype)
    m.close()


# ---- batches, pages, slots ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "scan_first", "many_heads", "wide"])
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


@pytest.mark.parametrize("dtype", DTYPES)
def test_decoding_many_sequences_at_once(dtype):
    """1 .. 70 tokens per step, repeated so that the captured step graph replays; every replay against the restatement"""
    c, w, m = model("mixed", dtype, fresh=True, n_seq=70, pool_tokens=70 * 192)
    reqs = [tokens(100, c["vocab"], i) for i in range(70)]
    want = [P.run(c, w, t) if i in (0, 1, 5, 16, 33, 63, 69) else None for i, t in enumerate(reqs)]
    seqs, at = [m.seq_new() for _ in reqs], [30 + i % 9 for i in range(70)]
    m.batch([(s, t[:a], []) for s, t, a in zip(seqs, reqs, at)])
    lg = torch.empty(70, c["vocab"], device="cuda")
    for n, reps in ((1, 4), (2, 4), (3, 4), (4, 4), (5, 4), (17, 5), (34, 5), (64, 5), (70, 4)):
        for _ in range(reps):
            m.batch([(seqs[i], reqs[i][at[i]:at[i] + 1], [0]) for i in range(n)], logits=lg)
            for i in range(n):
                if want[i] is not None:
                    close(lg[i:i + 1].cpu().numpy(), want[i][at[i]:at[i] + 1], dtype, ["sequence %d of %d at %d" % (i, n, at[i])])
                at[i] += 1
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_pages_and_slots_are_used_again(name, dtype):
    """a pool with room for little more than the live requests: stale pages, states and previous tokens of all kinds lie under every new one"""
    c, w, m = model(name, dtype, fresh=True, pool_tokens=512, n_seq=2)
    rng = np.random.default_rng(5)
    live, want = {}, {}
    for step in range(40):
        if len(live) < 2:
            live[step] = [m.seq_new(), tokens(int(rng.integers(3, 200)), c["vocab"], 100 + step), 0]
            want[step] = P.run(c, w, live[step][1])
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
    c, w, m = model("mixed", "float32", fresh=True, pool_tokens=192, n_seq=2)
    a, b = m.seq_new(), m.seq_new()
    with pytest.raises(PM355Error):
        m.seq_new()
    toks = tokens(120, c["vocab"])
    m.batch([(a, toks[:70], [])])
    before = (m.pool_info().free_pages, m.seq_len(a))
    for bad in ([(b, tokens(200, c["vocab"]), [])], [(a, [c["vocab"]], [])], [(a, [1], [1])], [(7, [1], [])], [(a, [1], []), (a, [1], [])]):
        with pytest.raises(PM355Error):
            m.batch(bad)
    assert (m.pool_info().free_pages, m.seq_len(a)) == before
    lg = torch.empty(1, c["vocab"], device="cuda")
    m.batch([(a, toks[70:71], [0])], logits=lg)
    close(lg.cpu().numpy(), P.run(c, w, toks[:71])[70:], "float32")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_outgrows_the_pool(dtype):
    """pages in front of every layer's window go back to the pool while the sequence goes on; states are carried for hundreds of tokens"""
    c = config(latent(size=48), scan(mlp=moe()), latent(heads=2, size=130, kv_from=0), width=64, vocab=50)
    _, w, m = model("forgets", dtype, c, fresh=True, pool_tokens=320, n_seq=1)
    toks = tokens(700, 50, 3)
    close(feed(m, m.seq_new(), toks, list(range(90, 360, 90)) + list(range(360, 700))), P.run(c, w, toks), dtype)
    m.close()


def test_a_missing_or_wrong_tensor_is_an_error():
    from prima_cpp_amd import keranex
    from prima_cpp_amd.lib import F32, PM355Error
    c = small_config()
    w = P.random_model(c, 2)
    m = keranex.build(c, "float32")
    todo = list(keranex.tensors(c))
    left = next(t for t in todo if t[3] == "l1.mlp.e2.down")
    for kind, layer, part, name, shape in todo:
        if name != left[3]:
            m.set_tensor(kind, layer, F32, w[name], part)
    with pytest.raises(PM355Error):
        m.finalize_pool(64, 1, 64)
    with pytest.raises(PM355Error):
        m.set_tensor(left[0], left[1], F32, w[left[3]], 4)           # (layer 1 has four experts)
    with pytest.raises(PM355Error):
        m.set_tensor(left[0], left[1], F32, w[left[3]][:-1], left[2])
    m.set_tensor(left[0], left[1], F32, w[left[3]], left[2])
    m.finalize_pool(64, 1, 64)
    toks = tokens(20, c["vocab"], 1)
    close(alone(m, toks), P.run(c, w, toks), "float32")
    m.close()


@pytest.mark.parametrize("change", [{"kv_from": 1}, {"kv_from": 2}, {"kv_rank": 57, "kv_from": 0}, {"rot_dim": 6, "kv_from": 0}, {"heads": 0}])
def test_descriptors_that_cannot_run_are_refused(change):
    from prima_cpp_amd import keranex
    from prima_cpp_amd.lib import PM355Error
    c = small_config()
    c["layers"][2]["mixer"].update(change)
    with pytest.raises(PM355Error):
        keranex.build(c)


# ---- generation ----------------------------------------------------------------------------------------------------------------------------
def greedy(c, w, prompt, n):
    """greedy tokens of the restatement, and the smallest lead of a winner over the runner-up"""
    t, lead = list(prompt), np.inf
    for _ in range(n):
        row = P.run(c, w, t)[-1]
        top = np.sort(row)[-2:]
        lead = min(lead, (top[1] - top[0]) / row.std())
        t.append(int(np.argmax(row)))
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
    w = P.random_model(c, 12, decisive=True)
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
    for dtype in DTYPES:
        out = tmp_path / dtype
        out.mkdir()
        r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out), "--max-tokens", "192"],
                           input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done %d" % i for i in range(4)]
        assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
        for s, rows_want in rows.items():
            close(np.fromfile(out / ("%d.f32" % s), dtype="<f4").reshape(rows_want.shape), rows_want, dtype)
