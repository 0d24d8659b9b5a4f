"""Plain, slow restatement of the Kudirax equations for tests: numpy float64, one function per mechanism, one sequence at a time, no cache, no batching and
nothing shared with the product path. Weights arrive as a dict name -> array (any float dtype) next to the parsed configuration."""
import numpy as np


def rms_unit(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis"""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, w, b, eps):
    mu = np.mean(x, axis=-1, keepdims=True)
    d = x - mu
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w + b


def squared_relu(z):
    return np.square(np.maximum(z, 0.0))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def cap_scores(s, cap):
    return cap * np.tanh(s / cap) if cap else s


def chunk_visible(n, size):
    """[n, n] bool: row i may look at column j (causal; with size: only inside its own chunk, chunks counted from position 0)"""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    ok = j <= i
    return ok & (i // size == j // size) if size else ok


def sink_softmax(s, visible, sink):
    """softmax over the visible columns with exp(sink) added to the denominator"""
    s = np.where(visible, s, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - m))


def mix_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def attention(h, w, p, cfg, eps, first_values):
    """returns (mixer output, first_values or this layer's own values where it is the first one that mixes). The design has every mechanism; tests of one alone switch the
    others off (unit_norm, has_sink, gate)."""
    n = h.shape[0]
    H, G, dk, dv = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q, k = (h @ w[p + "q"].T).reshape(n, H, dk), (h @ w[p + "k"].T).reshape(n, G, dk)
    if cfg.get("unit_norm", True):
        q, k = rms_unit(q, eps), rms_unit(k, eps)
    v = (h @ w[p + "v"].T).reshape(n, G, dv)
    if cfg.get("v_mix"):
        if first_values is None:
            first_values = v
        else:
            v = mix_values(v, first_values, float(np.reshape(w[p + "vmix"], ())))
    visible = chunk_visible(n, (cfg.get("mask") or {}).get("size"))
    out = np.empty((n, H, dv))
    for a in range(H):
        g = a // (H // G)
        s = cap_scores(q[:, a] @ k[:, g].T * cfg["scale"], cfg.get("softcap"))
        out[:, a] = sink_softmax(s, visible, w[p + "sink"][a] if cfg.get("has_sink", True) else -np.inf) @ v[:, g]
    out = out.reshape(n, H * dv)
    if cfg.get("gate", True):
        out = out * sigmoid(h @ w[p + "g"].T)
    return out @ w[p + "o"].T, first_values


def feed_forward(h, w, p):
    return squared_relu(h @ w[p + "up"].T + w[p + "up.b"]) @ w[p + "down"].T + w[p + "down.b"]


def run(config, weights, tokens, want_layers=False):
    """logits [n, vocab] (and the residual stream after every layer)"""
    w = {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)]
    first, stream = None, []
    for i, layer in enumerate(config["layers"]):
        l = "l%d." % i
        y, first = attention(x, w, l + "mix.", layer["mixer"], eps, first)
        x = x + layer_norm(y, w[l + "norm1"], w[l + "norm1.b"], eps)
        if layer.get("mlp"):
            x = x + layer_norm(feed_forward(x, w, l + "mlp."), w[l + "norm2"], w[l + "norm2.b"], eps)
        stream.append(x)
    logits = layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T
    return (logits, np.stack(stream)) if want_layers else logits


def random_model(config, seed, bf16=True):
    """Random weights for a configuration, strong enough that every mechanism shows in the logits; values representable in bfloat16 by default."""
    import torch
    g = torch.Generator().manual_seed(seed)

    def t(*shape, scale=1.0, mean=0.0):
        a = torch.randn(tuple(shape), generator=g) * scale + mean
        return (a.bfloat16() if bf16 else a).float().numpy()

    W = config["width"]
    w = {"embed": t(config["vocab"], W), "head": t(config["vocab"], W, scale=W ** -0.5),
         "final.norm": t(W, scale=0.2, mean=1.0), "final.norm.b": t(W, scale=0.2)}
    for i, layer in enumerate(config["layers"]):
        l, m = "l%d." % i, layer["mixer"]
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for name, rows, cols in (("q", H * dk, W), ("k", G * dk, W), ("v", G * dv, W), ("g", H * dv, W), ("o", W, H * dv)):
            w[l + "mix." + name] = t(rows, cols, scale=cols ** -0.5)
        w[l + "mix.sink"] = t(H, scale=1.0, mean=1.0)
        w[l + "mix.vmix"] = t(scale=0.2, mean=0.5)
        for nm in ("norm1", "norm2"):
            if nm == "norm2" and not layer.get("mlp"):
                continue
            w[l + nm] = t(W, scale=0.2, mean=0.7)
            w[l + nm + ".b"] = t(W, scale=0.2)
        if layer.get("mlp"):
            F = layer["mlp"]["ff"]
            w[l + "mlp.up"], w[l + "mlp.up.b"] = t(F, W, scale=W ** -0.5), t(F, scale=0.3)
            w[l + "mlp.down"], w[l + "mlp.down.b"] = t(W, F, scale=F ** -0.5), t(W, scale=0.3)
    return w
