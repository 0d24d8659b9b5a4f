"""Keranex: a decoder-only model of latent-attention layers (sliding windows; a layer may read the cached rows of an earlier one) and selective-scan layers, each followed by a
mixture of experts, with RMS norms in front of and behind every sublayer and a bigram embedding. This file reads its configuration and names its tensors; the mechanisms are the
engine's (csrc/stack.hip)."""
import os

from . import engine as E
from .lib import F32, PM355Error
from .registry import DTYPES, register
from .safetensors_file import SafetensorsFile


def layer_spec(layer):
    """engine.LayerSpec of one entry of config["layers"]"""
    m, ff, kw = layer["mixer"], layer.get("mlp"), {}
    if ff is not None:
        if ff.get("kind") != "moe":
            raise PM355Error(f"keranex: feed-forward {ff.get('kind')!r} is not part of the design")
        r = ff["router"]
        g = r.get("groups") or {}
        kw.update(ff=E.FF_EXPERTS, n_ff=ff["expert"]["ff"], act=E.ACT_RELU2, n_expert=r["experts"], n_expert_used=r["top"], n_group=g.get("count", 1), n_group_keep=g.get("keep", 1))
    if layer.get("type") == "latent_attention":
        size, src = (m.get("mask") or {}).get("size"), m.get("kv_from")
        kw.update(mixer=E.MIXER_LATENT, n_head=m["heads"], k_dim=m["dim"], v_dim=m["vdim"], q_rank=m["q_rank"], kv_rank=m["kv_rank"], rot_dim=m["rot_dim"], rot_dims=m["rot"]["dims"],
                  rot_base=m["rot"]["base"], kv_from=-1 if src is None else src, scale=m["scale"], mask=E.MASK_WINDOW if size else E.MASK_CAUSAL, mask_size=size or 0)
    elif layer.get("type") == "mamba1":
        kw.update(mixer=E.MIXER_SSM, inner=m["inner"], state=m["state"], dt_rank=m["dt_rank"], conv=m["conv"])
    else:
        raise PM355Error(f"keranex: mixer {layer.get('type')!r} is not part of the design")
    return E.LayerSpec(**kw)


def bigram(config):
    """(buckets, mul_prev, mul_cur) or None"""
    b = (config.get("embedding") or {}).get("bigram")
    return (b["buckets"], b["mul_prev"], b["mul_cur"]) if b else None


def tensors(config):
    """(engine tensor kind, layer or -1, part, name in the file, shape) of every tensor the model reads"""
    W, V = config["width"], config["vocab"]
    yield E.T_TOK_EMBD, -1, 0, "embed", (V, W)
    if bigram(config):
        yield E.T_BIGRAM, -1, 0, "bigram", (bigram(config)[0] + 1, W)
    yield E.T_OUT_NORM, -1, 0, "final.norm", (W,)
    yield E.T_OUTPUT, -1, 0, "head", (V, W)
    for i, layer in enumerate(config["layers"]):
        m, ff, p = layer["mixer"], layer.get("mlp"), f"l{i}."
        rows = [(E.T_ATTN_PRE_NORM, "norm1", (W,)), (E.T_ATTN_NORM, "norm1b", (W,))]
        if layer["type"] == "latent_attention":
            H, dn, dr, dv, qr, kr = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
            rows += [(E.T_DQ, "mix.dq", (qr, W)), (E.T_DQ_NORM, "mix.dq.norm", (qr,)), (E.T_UQ, "mix.uq", (H * (dn + dr), qr)), (E.T_UK, "mix.uk", (H * dn, kr)),
                     (E.T_UV, "mix.uv", (H * dv, kr)), (E.T_WO, "mix.o", (W, H * dv))]
            if m.get("kv_from") is None:
                rows += [(E.T_DKV, "mix.dkv", (kr + dr, W)), (E.T_DKV_NORM, "mix.dkv.norm", (kr,))]
        else:
            inner, S, r, taps = (m[k] for k in ("inner", "state", "dt_rank", "conv"))
            rows += [(E.T_SSM_IN, "mix.in", (2 * inner, W)), (E.T_SSM_CONV, "mix.conv", (inner, taps)), (E.T_SSM_CONV_B, "mix.conv.b", (inner,)), (E.T_SSM_X, "mix.x", (r + 2 * S, inner)),
                     (E.T_SSM_DT, "mix.dt", (inner, r)), (E.T_SSM_DT_B, "mix.dt.b", (inner,)), (E.T_SSM_A_LOG, "mix.A_log", (inner, S)), (E.T_SSM_D, "mix.D", (inner,)),
                     (E.T_WO, "mix.o", (W, inner))]
        if ff:
            rows += [(E.T_FFN_PRE_NORM, "norm2", (W,)), (E.T_FFN_NORM, "norm2b", (W,)), (E.T_ROUTER, "mlp.router", (ff["router"]["experts"], W))]
        for kind, name, shape in rows:
            yield kind, i, 0, p + name, shape
        for e in range(ff["router"]["experts"] if ff else 0):
            F = ff["expert"]["ff"]
            yield E.T_EXP_UP, i, e, f"{p}mlp.e{e}.up", (F, W)
            yield E.T_EXP_DOWN, i, e, f"{p}mlp.e{e}.down", (W, F)


def build(config, dtype="bfloat16"):
    """the model without weights"""
    if dtype not in DTYPES:
        raise PM355Error(f"keranex: dtype {dtype!r} is not served ({', '.join(DTYPES)})")
    return E.Stack("keranex", [layer_spec(x) for x in config["layers"]], config["width"], config["vocab"], config["norm"]["eps"], DTYPES[dtype], norm=E.NORM_RMS, pre_norm=True,
                   bigram=bigram(config))


@register("Keranex")
def load(path, config, dtype="bfloat16", n_ctx=None):
    model = build(config, dtype)
    f = SafetensorsFile(os.path.join(path, "model.safetensors"))
    for kind, layer, part, name, shape in tensors(config):
        t, data = f.get(name, shape)
        model.set_tensor(kind, layer, t, data, part)
    return model


def load_arrays(config, weights, dtype="bfloat16"):
    """the same from a dict name -> f32 array"""
    import numpy as np
    model = build(config, dtype)
    for kind, layer, part, name, shape in tensors(config):
        model.set_tensor(kind, layer, F32, np.asarray(weights[name], dtype=np.float32).reshape(shape), part)
    return model
