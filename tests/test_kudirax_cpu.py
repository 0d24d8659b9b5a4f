"""Kudirax without a GPU: the plain restatement on small closed cases, the page pool, file readers, registry and configuration, the scheduler's bookkeeping."""
import ctypes as C
import json
import struct

import numpy as np
import pytest

import kudirax_plain as P


# ---- the plain restatement itself, on cases that can be written down ---------------------------------------------------------------
def test_plain_unit_norm_and_layer_norm():
    x = np.array([[3.0, 4.0]])
    assert np.allclose(P.rms_unit(x, 0.0), x / np.sqrt(12.5))
    assert np.allclose(P.rms_unit(np.zeros((1, 4)), 1e-5), 0.0)                       # eps stands inside the root
    assert np.allclose(P.rms_unit(np.full((1, 4), 1e-3), 3e-6), 1e-3 / np.sqrt(1e-6 + 3e-6))
    y = P.layer_norm(np.array([[1.0, 3.0]]), np.array([2.0, 2.0]), np.array([0.5, -0.5]), 0.0)
    assert np.allclose(y, [[-1.5, 1.5]])


def test_plain_chunks_count_from_position_zero():
    v = P.chunk_visible(7, 3)
    assert [list(np.nonzero(r)[0]) for r in v] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]
    assert P.chunk_visible(4, None).sum() == 10


def test_plain_sink_takes_its_share_once():
    w = P.sink_softmax(np.array([[0.0, 0.0, 5.0]]), np.array([[True, True, False]]), np.log(2.0))
    assert np.allclose(w, [[0.25, 0.25, 0.0]])


def test_plain_cap_and_mix():
    assert np.isclose(P.cap_scores(np.array(1e9), 7.0), 7.0) and np.isclose(P.cap_scores(np.array(0.01), 7.0), 0.01, rtol=1e-5)
    assert np.allclose(P.mix_values(np.array([4.0]), np.array([8.0]), 0.25), [5.0])
    assert P.squared_relu(np.array([-2.0, 3.0])).tolist() == [0.0, 9.0]


# ---- page pool ---------------------------------------------------------------------------------------------------------------------
@pytest.fixture
def pool():
    import prima_cpp_amd
    lib = prima_cpp_amd.load()
    lib.pm355_page_pool_new.restype = C.c_void_p
    for n in ("free", "open", "close", "grow", "drop_before", "page", "free_pages"):
        getattr(lib, "pm355_page_pool_" + n).argtypes = [C.c_void_p] + [C.c_int] * {"close": 1, "grow": 2, "drop_before": 2, "page": 2}.get(n, 0)
    made = []

    def new(pages, seqs, limit=1000):
        made.append(lib.pm355_page_pool_new(pages, seqs, limit))
        return lambda name, *a: getattr(lib, "pm355_page_pool_" + name)(made[-1], *a)
    yield new
    for p in made:
        lib.pm355_page_pool_free(p)


def test_pool_grows_by_whole_pages_all_or_nothing(pool):
    p = pool(5, 2)
    a, b = p("open"), p("open")
    assert p("open") == -11 and {a, b} == {0, 1}
    assert p("grow", a, 64) == 0 and p("free_pages") == 4
    assert p("grow", a, 65) == 0 and p("free_pages") == 3
    assert p("grow", a, 100) == 0 and p("free_pages") == 3
    assert p("grow", b, 4 * 64) == -11 and p("free_pages") == 3 and p("page", b, 0) == -1
    assert p("grow", b, 3 * 64) == 0 and p("free_pages") == 0
    assert len({p("page", s, i) for s, i in ((a, 0), (a, 1), (b, 0), (b, 1), (b, 2))}) == 5


def test_pool_pages_come_back(pool):
    p = pool(4, 2)
    a = p("open")
    p("grow", a, 200)
    held = [p("page", a, i) for i in range(4)]
    assert p("close", a) == 0 and p("close", a) != 0 and p("free_pages") == 4
    b = p("open")
    p("grow", b, 256)
    assert b == a and [p("page", b, i) for i in range(4)] == held


def test_pool_drops_pages_that_lie_wholly_in_front(pool):
    p = pool(3, 1, 1000)
    a = p("open")
    p("grow", a, 192)
    assert p("drop_before", a, 63) == 0 and p("free_pages") == 0
    assert p("drop_before", a, 64) == 0 and p("free_pages") == 1 and p("page", a, 0) == -1 and p("page", a, 1) >= 0
    for n in range(4, 40):                                  # a sequence that forgets outgrows the pool
        assert p("grow", a, n * 64) == 0 and p("drop_before", a, (n - 2) * 64) == 0
    assert p("free_pages") == 1


def test_pool_refuses_a_sequence_beyond_its_table(pool):
    p = pool(8, 1, 2)
    a = p("open")
    assert p("grow", a, 128) == 0 and p("grow", a, 129) == -4


# ---- files, registry, configuration ------------------------------------------------------------------------------------------------
def small_config():
    return {"architecture": "Kudirax", "width": 80, "vocab": 90, "norm": {"eps": 1e-5}, "layers": [
        {"type": "attention", "mixer": {"heads": 6, "kv_heads": 2, "dim": 24, "vdim": 40, "mask": {"size": 37}, "scale": 0.2, "softcap": 9.0, "v_mix": False}, "mlp": {"kind": "dense", "ff": 112}},
        {"type": "attention", "mixer": {"heads": 4, "kv_heads": 4, "dim": 32, "vdim": 16, "mask": {"size": 100}, "scale": 0.3, "softcap": 30.0, "v_mix": True}, "mlp": None}]}


def write_safetensors(path, weights, drop=()):
    import torch
    header, blobs, at = {}, [], 0
    for name, a in weights.items():
        if name in drop:
            continue
        b = torch.from_numpy(np.ascontiguousarray(a, dtype=np.float32)).bfloat16().contiguous().view(torch.uint16).numpy().tobytes()
        header[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    h = json.dumps(header).encode()
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))


def write_model(folder, config, weights):
    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(config))
    write_safetensors(folder / "model.safetensors", weights)
    return str(folder)


def test_safetensors_reader(tmp_path):
    from prima_cpp_amd.lib import BF16, PM355Error
    from prima_cpp_amd.safetensors_file import SafetensorsFile
    write_safetensors(tmp_path / "a", {"m": np.arange(6).reshape(2, 3), "s": np.float32(0.5)})
    f = SafetensorsFile(tmp_path / "a")
    t, data = f.get("m", (2, 3))
    assert t == BF16 and (data.view(np.uint16).astype(np.uint32) << 16).view(np.float32).tolist() == [0, 1, 2, 3, 4, 5]
    assert f.get("s", ())[1].size == 2
    for bad in (("m", (3, 2)), ("x", (1,))):
        with pytest.raises(PM355Error):
            f.get(*bad)
    raw = bytearray((tmp_path / "a").read_bytes())
    (tmp_path / "b").write_bytes(raw[:-1])                  # a tensor that reaches beyond the file
    with pytest.raises(PM355Error):
        SafetensorsFile(tmp_path / "b")


def test_registry_knows_every_architecture(tmp_path):
    from prima_cpp_amd import gguf, registry
    from prima_cpp_amd.lib import PM355Error
    assert {"llama", "qwen2", "Kudirax"} <= set(registry.ARCHITECTURES)
    path = write_model(tmp_path / "m", small_config(), {"embed": np.zeros((2, 2))})
    assert registry.describe(path)[0] == "Kudirax"
    gguf.write_synthetic_model(str(tmp_path / "x.gguf"), arch=1, n_layer=1, n_embd=256, n_head=4, n_head_kv=2, n_ff=512, n_vocab=64)
    assert registry.describe(str(tmp_path / "x.gguf"))[0] == "qwen2"
    (tmp_path / "m" / "config.json").write_text(json.dumps({"architecture": "unheard of"}))
    with pytest.raises(PM355Error):
        registry.load(path)


def test_configuration_becomes_layer_descriptors():
    from prima_cpp_amd import engine as E, kudirax
    from prima_cpp_amd.lib import PM355Error
    c = small_config()
    a, b = (kudirax.layer_spec(x) for x in c["layers"])
    assert (a.n_head, a.n_head_kv, a.k_dim, a.v_dim, a.mask, a.mask_size, a.n_ff, a.act) == (6, 2, 24, 40, E.MASK_CHUNK, 37, 112, E.ACT_RELU2)
    assert not a.mix_flags & E.MIX_VALUE_MIX and b.mix_flags & E.MIX_VALUE_MIX and b.ff == E.FF_NONE and b.mask_size == 100
    names = [t[2] for t in kudirax.tensors(c)]
    assert "l0.mlp.up.b" in names and "l0.mix.vmix" not in names and "l1.mix.vmix" in names and "l1.norm2" not in names and len(names) == len(set(names))
    assert set(names) <= set(P.random_model(c, 0))
    for path, value in ((("type",), "recurrent"), (("mlp", "kind"), "experts")):
        layer = json.loads(json.dumps(c["layers"][0]))
        (layer if len(path) == 1 else layer[path[0]])[path[-1]] = value
        with pytest.raises(PM355Error):
            kudirax.layer_spec(layer)


def test_library_registers_architectures():
    import prima_cpp_amd
    lib = prima_cpp_amd.load()
    assert lib.pm355_arch_id(b"kudirax") >= 0 and lib.pm355_arch_id(b"nothing") < 0


# ---- the small build -----------------------------------------------------------------------------------------------------------------
def test_dense_subset_links_without_the_quantized_kernels():
    """the library of a fresh checkout that serves a dense model: no symbol of the rest of the library may be missing from it"""
    import os
    import subprocess
    from prima_cpp_amd import build
    if not os.path.exists(build.DENSE_LIB):
        pytest.skip("libprima_mi355_dense.so is not built")
    code = "import torch, ctypes; l = ctypes.CDLL(%r); assert l.pm355_arch_id(b'kudirax') >= 0 and l.pm355_arch_id(b'llama') < 0" % build.DENSE_LIB
    subprocess.run(["python3", "-c", code], check=True, timeout=120)
