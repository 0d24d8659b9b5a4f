"""Kudirax: a decoder-only model of chunked-attention layers (unit-norm q / k, capped scores, a softmax sink, values mixed with the first layer's, output gate), squared-relu
feed-forwards and layer norms on the sublayers' outputs. This file reads its configuration and names its tensors; the mechanisms are the engine's (csrc/stack.hip)."""
import os

from . import engine as E
from .lib import F32, PM355Error
from .registry import DTYPES, register
from .safetensors_file import SafetensorsFile


def layer_spec(layer):
    """engine.LayerSpec of one entry of config["layers"]"""
    if layer.get("type") != "attention":
        raise PM355Error(f"kudirax: mixer {layer.get('type')!r} is not part of the design")
    m, ff = layer["mixer"], layer.get("mlp")
    if ff is not None and ff.get("kind") != "dense":
        raise PM355Error(f"kudirax: feed-forward {ff.get('kind')!r} is not part of the design")
    size = (m.get("mask") or {}).get("size")
    flags = E.MIX_QK_NORM | E.MIX_SINK | E.MIX_OUT_GATE | (E.MIX_VALUE_MIX if m.get("v_mix") else 0)
    return E.LayerSpec(n_head=m["heads"], n_head_kv=m["kv_heads"], k_dim=m["dim"], v_dim=m["vdim"], mix_flags=flags,
                       mask=E.MASK_CHUNK if size else E.MASK_CAUSAL, mask_size=size or 0, scale=m["scale"], softcap=m.get("softcap") or 0.0,
                       ff=E.FF_DENSE if ff else E.FF_NONE, n_ff=ff["ff"] if ff else 0, act=E.ACT_RELU2 if ff else E.ACT_NONE)


def tensors(config):
    """(engine tensor kind, layer or -1, name in the file, shape) of every tensor the model reads"""
    W, V = config["width"], config["vocab"]
    yield E.T_TOK_EMBD, -1, "embed", (V, W)
    yield E.T_OUT_NORM, -1, "final.norm", (W,)
    yield E.T_OUT_NORM_B, -1, "final.norm.b", (W,)
    yield E.T_OUTPUT, -1, "head", (V, W)
    for i, layer in enumerate(config["layers"]):
        m, ff, p = layer["mixer"], layer.get("mlp"), f"l{i}."
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for kind, name, shape in ((E.T_WQ, "q", (H * dk, W)), (E.T_WK, "k", (G * dk, W)), (E.T_WV, "v", (G * dv, W)), (E.T_W_OUT_GATE, "g", (H * dv, W)),
                                  (E.T_WO, "o", (W, H * dv)), (E.T_SINK, "sink", (H,))):
            yield kind, i, p + "mix." + name, shape
        if m.get("v_mix"):
            yield E.T_VALUE_MIX, i, p + "mix.vmix", ()
        yield E.T_ATTN_NORM, i, p + "norm1", (W,)
        yield E.T_ATTN_NORM_B, i, p + "norm1.b", (W,)
        if ff:
            F = ff["ff"]
            for kind, name, shape in ((E.T_FFN_UP, "mlp.up", (F, W)), (E.T_FFN_UP_B, "mlp.up.b", (F,)), (E.T_FFN_DOWN, "mlp.down", (W, F)), (E.T_FFN_DOWN_B, "mlp.down.b", (W,)),
                                      (E.T_FFN_NORM, "norm2", (W,)), (E.T_FFN_NORM_B, "norm2.b", (W,))):
                yield kind, i, p + name, shape


def build(config, dtype="bfloat16"):
    """the model without weights"""
    if dtype not in DTYPES:
        raise PM355Error(f"kudirax: dtype {dtype!r} is not served ({', '.join(DTYPES)})")
    return E.Stack("kudirax", [layer_spec(x) for x in config["layers"]], config["width"], config["vocab"], config["norm"]["eps"], DTYPES[dtype])


@register("Kudirax")
def load(path, config, dtype="bfloat16", n_ctx=None):
    model = build(config, dtype)
    f = SafetensorsFile(os.path.join(path, "model.safetensors"))
    for kind, layer, name, shape in tensors(config):
        if kind == E.T_VALUE_MIX and f.tensors.get(name, (0, None))[1] == (1,):
            shape = (1,)
        t, data = f.get(name, shape)
        model.set_tensor(kind, layer, t, data)
    return model


def load_arrays(config, weights, dtype="bfloat16"):
    """the same from a dict name -> f32 array"""
    import numpy as np
    model = build(config, dtype)
    for kind, layer, name, shape in tensors(config):
        model.set_tensor(kind, layer, F32, np.asarray(weights[name], dtype=np.float32).reshape(shape))
    return model
