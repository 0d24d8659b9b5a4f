"""Plain, slow restatement of the Keranex equations for tests: numpy float64, one function per mechanism, one sequence at a time, no cache, no batching and nothing shared
with the product path. Weights arrive as a dict name -> array (any float dtype) next to the parsed configuration."""
import numpy as np


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis"""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def silu(z):
    return z / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def squared_relu(z):
    return np.square(np.maximum(z, 0.0))


def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """row of the bigram table per token: a hash of the token and the one before it; the first token of a sequence has the table's last row"""
    t = [int(x) for x in tokens]
    return np.array([buckets if i == 0 else (t[i - 1] * mul_prev + t[i] * mul_cur) % buckets for i in range(len(t))])


def embed(tokens, w, cfg):
    x = w["embed"][np.asarray(tokens)].astype(np.float64)
    b = (cfg.get("embedding") or {}).get("bigram")
    return x + w["bigram"][bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])] if b else x


def rotate_half(x, positions, base, dims):
    """the first `dims` entries of the last axis as pairs (i, i + dims / 2), turned by position * base^(-2 i / dims); x [n, .., d]"""
    half = dims // 2
    a = np.asarray(positions, dtype=np.float64)[:, None] * np.power(float(base), -2.0 * np.arange(half) / dims)
    a = a.reshape((len(a),) + (1,) * (x.ndim - 2) + (half,))
    u, v, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), rest], axis=-1)


def window_visible(n, size):
    """[n, n] bool: row i may look at column j (itself and the size - 1 tokens before it; everything before it without a size)"""
    d = np.arange(n)[:, None] - np.arange(n)[None, :]
    return (d >= 0) & (d < size) if size else d >= 0


def softmax(s, visible=None):
    s = s if visible is None else np.where(visible, s, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def latent_keys(h, w, p, m, eps):
    """what a layer caches per token: the normed latent, and the rotated key part that all heads share"""
    d = h @ w[p + "dkv"].T
    c = rms_norm(d[:, :m["kv_rank"]], w[p + "dkv.norm"], eps)
    return c, rotate_half(d[:, m["kv_rank"]:], range(len(h)), m["rot"]["base"], m["rot"]["dims"])


def latent_attention(h, w, p, m, eps, cached):
    """mixer output from the latents `cached` (of this layer or of the one it shares with)"""
    n, H, dn, dr, dv = len(h), m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, k_rot = cached
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(n, H, dn + dr)
    q_rot = rotate_half(q[..., dn:], range(n), m["rot"]["base"], m["rot"]["dims"])
    k, v = (c @ w[p + "uk"].T).reshape(n, H, dn), (c @ w[p + "uv"].T).reshape(n, H, dv)
    visible = window_visible(n, (m.get("mask") or {}).get("size"))
    out = np.empty((n, H, dv))
    for a in range(H):
        out[:, a] = softmax((q[:, a, :dn] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * m["scale"], visible) @ v[:, a]
    return out.reshape(n, H * dv) @ w[p + "o"].T


def causal_conv(x, taps, bias):
    """per channel: bias + sum of the last len(taps) inputs, the current one with the last column; zeros before the start"""
    k = taps.shape[1]
    pad = np.concatenate([np.zeros((k - 1, x.shape[1])), x])
    return bias + sum(pad[j:j + len(x)] * taps[:, j] for j in range(k))


def selective_scan(x, dt, A, B, C, D):
    """S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n; y_c = S[c, :] . C + D_c x_c, token by token from zero"""
    S, y = np.zeros(A.shape), np.empty_like(x)
    for t in range(len(x)):
        S = np.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba(h, w, p, m):
    inner, r, st = m["inner"], m["dt_rank"], m["state"]
    xz = h @ w[p + "in"].T
    x = silu(causal_conv(xz[:, :inner], w[p + "conv"], w[p + "conv.b"]))
    f = x @ w[p + "x"].T
    dt = softplus(f[:, :r] @ w[p + "dt"].T + w[p + "dt.b"])
    y = selective_scan(x, dt, -np.exp(w[p + "A_log"]), f[:, r:r + st], f[:, r + st:], w[p + "D"])
    return (y * silu(xz[:, inner:])) @ w[p + "o"].T


def route(z, top, count=1, keep=1):
    """router logits [n, experts] -> (chosen experts [n, top], their weights): softmax over all experts; only the `keep` of `count` groups of neighbours with the largest
    single score take part; weights are the scores themselves"""
    s = softmax(z)
    g = s.reshape(len(z), count, -1).max(axis=-1)
    ok = np.zeros(g.shape, dtype=bool)
    np.put_along_axis(ok, np.argsort(-g, axis=-1, kind="stable")[:, :keep], True, axis=-1)
    masked = np.where(np.repeat(ok, z.shape[1] // count, axis=-1), s, -1.0)
    ids = np.argsort(-masked, axis=-1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, axis=-1)


def experts(h, w, p, ff):
    r = ff["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    ids, weights = route(h @ w[p + "router"].T, r["top"], g["count"], g["keep"])
    out = np.zeros_like(h)
    for t in range(len(h)):
        for e, s in zip(ids[t], weights[t]):
            out[t] += s * (squared_relu(h[t] @ w[p + "e%d.up" % e].T) @ w[p + "e%d.down" % e].T)
    return out


def run(cfg, weights, tokens, layers=None):
    """logits [n, vocab] of a whole sequence; `layers` (a list) receives the residual stream after every layer"""
    w = {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}
    eps, caches = cfg["norm"]["eps"], {}
    x = embed(tokens, w, cfg)
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = "l%d." % i, layer["mixer"], layer.get("mlp")
        h = rms_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "latent_attention":
            src = m.get("kv_from")
            if src is None:
                src, caches[i] = i, latent_keys(h, w, p + "mix.", m, eps)
            y = latent_attention(h, w, p + "mix.", m, eps, caches[src])
        else:
            y = mamba(h, w, p + "mix.", m)
        x = x + rms_norm(y, w[p + "norm1b"], eps)
        if ff:
            x = x + rms_norm(experts(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", ff), w[p + "norm2b"], eps)
        if layers is not None:
            layers.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


def bf16(a):
    """float32 array rounded to bfloat16 (nearest, ties to even)"""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)).view(np.float32)


def random_model(cfg, seed, decisive=False):
    """weights name -> float32 array of bfloat16 values, of a size at which every mechanism matters. decisive: a few entries of the residual stream tell the routers (and nobody
    else) which class a token has, and no sublayer changes them, so that rounding cannot turn a choice of experts around"""
    rng = np.random.default_rng(seed)
    W, V, w = cfg["width"], cfg["vocab"], {}

    def mat(name, n, k, gain=1.0):
        w[name] = rng.normal(0, gain / np.sqrt(k), (n, k))

    def vec(name, n, mean=1.0, amp=0.2):
        w[name] = mean + amp * rng.normal(0, 1, n)
    w["embed"] = rng.normal(0, 1, (V, W))
    b = (cfg.get("embedding") or {}).get("bigram")
    if b:
        w["bigram"] = rng.normal(0, 0.7, (b["buckets"] + 1, W))
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = "l%d." % i, layer["mixer"], layer.get("mlp")
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if ff else ()):
            vec(p + n, W)
        if layer["type"] == "latent_attention":
            H, dn, dr, dv, qr, kr = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
            mat(p + "mix.dq", qr, W)
            vec(p + "mix.dq.norm", qr)
            mat(p + "mix.uq", H * (dn + dr), qr, 1.5)
            if m.get("kv_from") is None:
                mat(p + "mix.dkv", kr + dr, W)
                vec(p + "mix.dkv.norm", kr)
            mat(p + "mix.uk", H * dn, kr, 1.5)
            mat(p + "mix.uv", H * dv, kr)
            mat(p + "mix.o", W, H * dv)
        else:
            I, S, r, k = (m[n] for n in ("inner", "state", "dt_rank", "conv"))
            mat(p + "mix.in", 2 * I, W)
            w[p + "mix.conv"] = rng.normal(0, 0.6, (I, k))
            vec(p + "mix.conv.b", I, 0.0, 0.1)
            mat(p + "mix.x", r + 2 * S, I, 1.5)
            mat(p + "mix.dt", I, r, 1.0)
            vec(p + "mix.dt.b", I, -2.5, 1.0)
            w[p + "mix.A_log"] = np.log(rng.uniform(0.3, 6.0, (I, S)))
            vec(p + "mix.D", I)
            mat(p + "mix.o", W, I)
        if ff:
            E, F = ff["router"]["experts"], ff["expert"]["ff"]
            mat(p + "mlp.router", E, W, 2.0)
            for e in range(E):
                mat(p + "mlp.e%d.up" % e, F, W, 1.4)
                mat(p + "mlp.e%d.down" % e, W, F)
    vec("final.norm", W)
    mat("head", V, W, 2.0)
    if decisive:
        n, code = 5, slice(0, 5)
        w["embed"][:, code] = 0.0
        w["embed"][np.arange(V), np.arange(V) % n] = 0.5 * np.sqrt(W)
        if b:
            w["bigram"][:, code] = 0.0
        w["head"][:, code] = 0.0
        for k in w:
            if k.endswith(("norm1b", "norm2b")):
                w[k][code] = 0.0
            elif k.endswith((".dq", ".dkv", "mix.in", ".up")):
                w[k][:, code] = 0.0
            elif k.endswith("router"):
                w[k] *= 0.02
                w[k][:, code] = np.stack([rng.permutation(np.linspace(-1, 1, len(w[k]))) for _ in range(n)], axis=1) * (0.5 * len(w[k]) / np.sqrt(W))
    return {k: bf16(v) for k, v in w.items()}
