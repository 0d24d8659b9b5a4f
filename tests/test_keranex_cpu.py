"""Keranex without a GPU: the plain restatement on small closed cases, configuration, tensor names, registry."""
import copy

import numpy as np
import pytest

import keranex_plain as P
from test_kudirax_cpu import write_model


def latent(heads=3, dim=24, rot_dim=8, vdim=20, q_rank=40, kv_rank=56, size=40, base=5000.0, scale=0.2, kv_from=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "mask": {"size": size}, "rot": {"base": base, "dims": rot_dim}, "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def scan(inner=96, state=16, dt_rank=8, conv=4, mlp=None):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}, "mlp": mlp}


def moe(experts=6, top=2, count=2, keep=1, ff=72):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}}}


def config(*layers, width=96, vocab=101, eps=1e-5, bigram=(211, 31, 7)):
    c = {"architecture": "Keranex", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": list(layers)}
    if bigram:
        c["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}
    return c


def small_config():
    return config(latent(mlp=moe()), scan(inner=72, state=12, dt_rank=5, conv=3, mlp=moe(4, 3, 1, 1, 40)), latent(heads=2, size=70, vdim=36, dim=12, kv_from=0), width=80, vocab=90)


# ---- the plain restatement itself, on cases that can be written down ---------------------------------------------------------------
def test_plain_norm_has_eps_inside_the_root():
    assert np.allclose(P.rms_norm(np.full((1, 4), 1e-3), np.full(4, 2.0), 3e-6), 2e-3 / np.sqrt(1e-6 + 3e-6))


def test_plain_bigram_rows():
    assert P.bigram_rows([4, 9, 0], 10, 3, 5).tolist() == [10, (4 * 3 + 9 * 5) % 10, 27 % 10]


def test_plain_rotation_pairs_halves():
    x = np.arange(1.0, 6.0).reshape(1, 5)                   # four rotated entries, one that stays
    y = P.rotate_half(x, [3], 100.0, 4)
    c, s = np.cos([3.0, 0.3]), np.sin([3.0, 0.3])
    assert np.allclose(y, [[1 * c[0] - 3 * s[0], 2 * c[1] - 4 * s[1], 3 * c[0] + 1 * s[0], 4 * c[1] + 2 * s[1], 5]])
    a, b = np.random.default_rng(0).normal(size=(2, 1, 6))
    dots = [(P.rotate_half(a, [p + 5], 9.0, 6) @ P.rotate_half(b, [p], 9.0, 6).T).item() for p in (0, 7, 900)]
    assert np.allclose(dots, dots[0])                       # scores depend on the distance


def test_plain_window_counts_the_token_itself():
    v = P.window_visible(5, 2)
    assert [list(np.nonzero(r)[0]) for r in v] == [[0], [0, 1], [1, 2], [2, 3], [3, 4]]
    assert P.window_visible(4, None).sum() == 10


def test_plain_convolution_looks_back():
    y = P.causal_conv(np.array([[1.0], [10.0], [100.0]]), np.array([[3.0, 2.0]]), np.array([0.5]))
    assert y[:, 0].tolist() == [2.5, 23.5, 230.5]


def test_plain_scan_is_the_recurrence():
    y = P.selective_scan(np.array([[2.0], [3.0]]), np.array([[0.5], [1.0]]), np.array([[-1.0, -2.0]]), np.array([[1.0, 2.0], [0.5, 1.0]]), np.array([[1.0, 1.0], [1.0, -1.0]]), np.array([10.0]))
    s = np.array([1.0, 2.0])
    t = np.exp([-1.0, -2.0]) * s + 3.0 * np.array([0.5, 1.0])
    assert np.allclose(y[:, 0], [s.sum() + 20, t[0] - t[1] + 30])


def test_plain_routing_keeps_groups_and_does_not_renormalize():
    z = np.log(np.array([[0.05, 0.40, 0.30, 0.02, 0.20, 0.03]]))
    ids, w = P.route(z, 2, 3, 2)                            # groups {0, 1} {2, 3} {4, 5}: the first two stay
    assert ids.tolist() == [[1, 2]] and np.allclose(w, [[0.4, 0.3]])
    ids, w = P.route(z, 2, 3, 1)
    assert ids.tolist() == [[1, 0]] and np.allclose(w, [[0.4, 0.05]])
    assert P.route(z, 3)[0].tolist() == [[1, 2, 4]]


def test_plain_model_is_causal_and_shares_latents():
    c = small_config()
    w = P.random_model(c, 1)
    t = np.random.default_rng(0).integers(0, 90, 30)
    a = P.run(c, w, t)
    assert np.allclose(P.run(c, w, t[:17]), a[:17])
    w2 = dict(w, **{"l0.mix.uk": w["l0.mix.uk"] * 0, "l0.norm1b": w["l0.norm1b"] * 0})       # layer 0 adds nothing, but its latents still feed layer 2
    w3 = dict(w2, **{"l0.mix.dkv": w["l0.mix.dkv"][::-1].copy()})
    assert not np.allclose(P.run(c, w2, t), P.run(c, w3, t))


def test_decisive_routers_have_clear_winners():
    c = config(latent(mlp=moe(12, 5, 4, 2)), scan(mlp=moe()))
    w, x = P.random_model(c, 3, decisive=True), []
    t = np.arange(40) % 101
    P.run(c, w, t, x)
    z = np.sort(P.rms_norm(x[0], w["l1.norm2"], 1e-5) @ w["l1.mlp.router"].astype(np.float64).T, axis=-1)
    assert np.diff(z).min() > 0.02 and len({tuple(r) for r in P.route(z, 2)[0].tolist()}) >= 1


# ---- configuration, names, registry ----------------------------------------------------------------------------------------------------
def test_configuration_becomes_layer_descriptors():
    from prima_cpp_amd import engine as E, keranex
    from prima_cpp_amd.lib import PM355Error
    c = small_config()
    a, b, d = (keranex.layer_spec(x) for x in c["layers"])
    assert (a.mixer, a.n_head, a.k_dim, a.v_dim, a.rot_dim, a.rot_dims, a.q_rank, a.kv_rank, a.mask, a.mask_size, a.kv_from) == (E.MIXER_LATENT, 3, 24, 20, 8, 8, 40, 56, E.MASK_WINDOW, 40, -1)
    assert (a.ff, a.n_ff, a.act, a.n_expert, a.n_expert_used, a.n_group, a.n_group_keep) == (E.FF_EXPERTS, 72, E.ACT_RELU2, 6, 2, 2, 1) and np.isclose(a.rot_base, 5000.0)
    assert (b.mixer, b.inner, b.state, b.dt_rank, b.conv, b.n_expert, b.n_expert_used) == (E.MIXER_SSM, 72, 12, 5, 3, 4, 3)
    assert d.kv_from == 0 and d.ff == E.FF_NONE and d.mask_size == 70
    names = [t[3] for t in keranex.tensors(c)]
    assert len(names) == len(set(names)) and set(names) == set(P.random_model(c, 0))
    assert "l0.mix.dkv" in names and "l2.mix.dkv" not in names and "l2.norm2" not in names and "l1.mlp.e3.down" in names and "l1.mlp.e4.down" not in names
    shapes = {k: np.shape(v) for k, v in P.random_model(c, 0).items()}
    assert all(shapes[n] == s for _, _, _, n, s in keranex.tensors(c))
    for change in (lambda x: x.update(type="attention"), lambda x: x["mlp"].update(kind="dense")):
        bad = copy.deepcopy(c["layers"][0])
        change(bad)
        with pytest.raises(PM355Error):
            keranex.layer_spec(bad)
    no_bigram = dict(c, embedding={})
    assert keranex.bigram(no_bigram) is None and "bigram" not in [t[3] for t in keranex.tensors(no_bigram)]


def test_registry_serves_the_design(tmp_path):
    import prima_cpp_amd
    from prima_cpp_amd import registry
    assert "Keranex" in registry.ARCHITECTURES
    path = write_model(tmp_path / "m", small_config(), {"embed": np.zeros((2, 2))})
    assert registry.describe(path)[0] == "Keranex"
    assert prima_cpp_amd.load().pm355_arch_id(b"keranex") >= 0
