"""Plain numpy (float64) restatement of the Keronex design, one function per mechanism, whole sequences only (no cache, no state
between calls): the slow restatement that the device path is compared with.  It shares no code with tinygpt_amd.

A model is (cfg, tensors): cfg the dictionary of the checkpoint's config.json, tensors name -> float array.
Notation: T tokens, W width, n streams, H heads, G key / value heads, D key size, E value size.
"""
import numpy as np


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis"""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    """the stored weight is the distance of the factor from one"""
    return unit_rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.where(z > 30, z, np.log1p(np.exp(np.minimum(z, 30))))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


# ---- the embedding ---------------------------------------------------------------------------------------------------------------------
def bigram_row(before, token, b):
    """row of the pair table; a sequence's first token (before None) takes the row behind the buckets"""
    return b["buckets"] if before is None else (before * b["mul_prev"] + token * b["mul_cur"]) % b["buckets"]


def embed(ids, e, t):
    x = t["embed"][np.asarray(ids)] * e.get("scale", 1.0)
    if e.get("bigram"):
        x = x + t["bigram"][[bigram_row(ids[i - 1] if i else None, ids[i], e["bigram"]) for i in range(len(ids))]]
    return x


# ---- hyper-connections -----------------------------------------------------------------------------------------------------------------
def streams_in(xs, w_in):
    """xs [n][T][W] -> the sublayer's input"""
    return sum(w_in[s] * xs[s] for s in range(len(xs)))


def streams_out(xs, mix, w_out, y):
    """every new stream t from all old ones: sum_s mix[s][t] x_s + out[t] y"""
    n = len(xs)
    return np.stack([sum(mix[s, k] * xs[s] for s in range(n)) + w_out[k] * y for k in range(n)])


# ---- rotation ----------------------------------------------------------------------------------------------------------------------------
def rotate(x, rot):
    """x [T][heads][D]: dimension i of the first rot.dims turns with dimension i + dims / 2 by position * base^(-2 i / dims)"""
    if not rot:
        return x
    T, half = x.shape[0], rot["dims"] // 2
    a = np.arange(T)[:, None] * float(rot["base"]) ** (-2.0 * np.arange(half) / rot["dims"])
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * half:]], axis=-1)


# ---- mixers ------------------------------------------------------------------------------------------------------------------------------
def softmax_attention(q, k, v, scale):
    """one map: q, k [T][D], v [T][E], causal"""
    T = q.shape[0]
    s = q @ k.T * scale
    s[np.triu_indices(T, 1)] = -np.inf
    p = np.exp(s - s.max(axis=1, keepdims=True))
    return p @ v / p.sum(axis=1, keepdims=True)


def map_weight(t, pre, diff):
    return np.exp(np.sum(t[pre + "lq1"] * t[pre + "lk1"])) - np.exp(np.sum(t[pre + "lq2"] * t[pre + "lk2"])) + diff


def two_map_attention(h, m, t, pre, eps):
    T = h.shape[0]
    H, G, D, E, diff = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"], m["diff"]
    q = rotate((h @ t[pre + "q"].T).reshape(T, 2 * H, D), m.get("rot"))      # (head, map) in one axis, maps of a head side by side
    k = rotate((h @ t[pre + "k"].T).reshape(T, 2 * G, D), m.get("rot"))
    v = (h @ t[pre + "v"].T).reshape(T, G, E)
    lam = map_weight(t, pre, diff)
    out = np.zeros((T, H, E))
    for a in range(H):
        g = a // (H // G)
        o1, o2 = (softmax_attention(q[:, 2 * a + i], k[:, 2 * g + i], v[:, g], m["scale"]) for i in (0, 1))
        out[:, a] = unit_rms(o1 - lam * o2, eps) * (1.0 - diff)
    return out.reshape(T, H * E) @ t[pre + "o"].T


def decaying_memory(q, k, v, decay):
    """one head: S <- decay S + k v^T, o = S^T q"""
    S, out = np.zeros((k.shape[1], v.shape[1])), np.zeros_like(v)
    for i in range(len(q)):
        S = decay * S + np.outer(k[i], v[i])
        out[i] = S.T @ q[i]
    return out


def retention(h, m, t, pre, eps):
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    q = rotate((h @ t[pre + "q"].T).reshape(T, H, D), m.get("rot"))
    k = rotate((h @ t[pre + "k"].T).reshape(T, H, D), m.get("rot")) * D ** -0.5
    v = (h @ t[pre + "v"].T).reshape(T, H, E)
    o = np.stack([unit_rms(decaying_memory(q[:, a], k[:, a], v[:, a], m["decay"][a]), eps) for a in range(H)], axis=1)
    return (o.reshape(T, H * E) * silu(h @ t[pre + "g"].T)) @ t[pre + "o"].T


def short_conv(x, w):
    """x [T][C], w [C][taps] (last column: the current token), zeros before the start"""
    T, taps = x.shape[0], w.shape[1]
    out = np.zeros_like(x)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            out[back:] += x[:T - back] * w[:, j]
    return out


def delta_memory(q, k, v, beta, g):
    """one head: the rows of S decay by g [T][D] each, the error of the recalled value is written, the read sees the write"""
    S, out = np.zeros((k.shape[1], v.shape[1])), np.zeros_like(v)
    for i in range(len(q)):
        S = g[i][:, None] * S
        S = S + np.outer(k[i], beta[i] * (v[i] - S.T @ k[i]))
        out[i] = S.T @ q[i]
    return out


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def channel_decays(h, t, pre, H, D):
    z = h @ t[pre + "a1"].T @ t[pre + "a2"].T + t[pre + "dt_bias"]
    return np.exp(-np.exp(t[pre + "A_log"])[None, :, None] * softplus(z).reshape(-1, H, D))


def channel_delta(h, m, t, pre, eps):
    T = h.shape[0]
    H, G, D, E = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ t[pre + n].T, t[pre + n + ".conv"])) for n in "qkv")
    q, k, v = unit(q.reshape(T, G, D)) * D ** -0.5, unit(k.reshape(T, G, D)), v.reshape(T, H, E)
    beta, g = sigmoid(h @ t[pre + "b"].T), channel_decays(h, t, pre, H, D)
    o = np.stack([delta_memory(q[:, a // (H // G)], k[:, a // (H // G)], v[:, a], beta[:, a], g[:, a]) for a in range(H)], axis=1)
    o = unit_rms(o, eps) * t[pre + "norm"] * sigmoid(h @ t[pre + "g1"].T @ t[pre + "g2"].T).reshape(T, H, E)
    return o.reshape(T, H * E) @ t[pre + "o"].T


MIXERS = {"retention": retention, "attention": two_map_attention, "channel_delta": channel_delta}


# ---- feed-forwards -----------------------------------------------------------------------------------------------------------------------
def gated_gelu_ff(h, t, pre):
    return (gelu_tanh(h @ t[pre + "gate"].T) * (h @ t[pre + "up"].T)) @ t[pre + "down"].T


def squared_relu_ff(h, t, pre):
    return np.maximum(h @ t[pre + "up"].T, 0.0) ** 2 @ t[pre + "down"].T


def chosen_experts(h, t, pre, top):
    """[T][top] expert indices and their (not renormalised) scores"""
    s = sigmoid(h @ t[pre + "router"].T)
    sel = np.argsort(-s, axis=1, kind="stable")[:, :top]
    return sel, np.take_along_axis(s, sel, axis=1)


def experts_ff(h, f, t, pre):
    """a weight multiplies what its expert reads"""
    sel, w = chosen_experts(h, t, pre, f["router"]["top"])
    out = np.zeros_like(h)
    for i in range(len(h)):
        for e, we in zip(sel[i], w[i]):
            out[i] += squared_relu_ff(we * h[i], t, f"{pre}e{e}.")
    return out + squared_relu_ff(h, t, pre + "shared.") if f.get("shared") else out


def feed_forward(h, f, t, pre):
    return gated_gelu_ff(h, t, pre) if f["kind"] == "dense" else experts_ff(h, f, t, pre)


# ---- the model ---------------------------------------------------------------------------------------------------------------------
def weights_layer(cfg, i):
    """the layer whose tensors layer i uses"""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(cfg, t, ids, layers_out=None):
    """logits [T][vocab] of one sequence; layers_out (a list) receives the sum of the streams after every layer"""
    t = {k: np.asarray(v, np.float64) for k, v in t.items()}
    eps = cfg["norm"]["eps"]
    e = embed([int(i) for i in ids], cfg.get("embedding") or {}, t)
    xs = np.stack([e] * cfg["streams"])
    for i, L in enumerate(cfg["layers"]):
        p = f"l{weights_layer(cfg, i)}."
        u = norm(streams_in(xs, t[p + "hc1.in"]), t[p + "norm1"], eps)
        xs = streams_out(xs, t[p + "hc1.mix"], t[p + "hc1.out"], MIXERS[L["type"]](u, L["mixer"], t, p + "mix.", eps))
        if L.get("mlp"):
            u = norm(streams_in(xs, t[p + "hc2.in"]), t[p + "norm2"], eps)
            xs = streams_out(xs, t[p + "hc2.mix"], t[p + "hc2.out"], feed_forward(u, L["mlp"], t, p + "mlp."))
        if layers_out is not None:
            layers_out.append(xs.sum(axis=0))
    return norm(xs.sum(axis=0), t["final.norm"], eps) @ t["head"].T


# ---- random models -----------------------------------------------------------------------------------------------------------------
def tensor_shapes(cfg, rank_a=5, rank_g=7):
    """checkpoint name -> shape; the inner sizes of the two low-rank products are not part of the configuration (the tensors carry them)"""
    W, n, out = cfg["width"], cfg["streams"], {"embed": (cfg["vocab"], cfg["width"])}
    b = (cfg.get("embedding") or {}).get("bigram")
    if b:
        out["bigram"] = (b["buckets"] + 1, W)
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        out[p + "norm1"] = (W,)
        if f:
            out[p + "norm2"] = (W,)
        q, H, G, D, E = p + "mix.", m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
        if L["type"] == "retention":
            out.update({q + "q": (H * D, W), q + "k": (H * D, W), q + "v": (H * E, W), q + "g": (H * E, W)})
        elif L["type"] == "attention":
            out.update({q + "q": (2 * H * D, W), q + "k": (2 * G * D, W), q + "v": (G * E, W)})
            out.update({q + s: (D,) for s in ("lq1", "lk1", "lq2", "lk2")})
        else:
            for s, c in (("q", G * D), ("k", G * D), ("v", H * E)):
                out.update({q + s: (c, W), q + s + ".conv": (c, m["conv"])})
            out.update({q + "b": (H, W), q + "A_log": (H,), q + "norm": (E,), q + "a1": (rank_a, W), q + "a2": (H * D, rank_a), q + "dt_bias": (H * D,),
                        q + "g1": (rank_g, W), q + "g2": (H * E, rank_g)})
        out[q + "o"] = (W, H * E)
        if f and f["kind"] == "dense":
            out.update({p + "mlp.gate": (f["ff"], W), p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"])})
        elif f:
            F = f["expert"]["ff"]
            for e in range(f["router"]["experts"]):
                out.update({p + f"mlp.e{e}.up": (F, W), p + f"mlp.e{e}.down": (W, F)})
            out[p + "mlp.router"] = (f["router"]["experts"], W)
            if f.get("shared"):
                out.update({p + "mlp.shared.up": (f["shared"]["ff"], W), p + "mlp.shared.down": (W, f["shared"]["ff"])})
        for s in ("hc1", "hc2") if f else ("hc1",):
            out.update({p + s + ".in": (n,), p + s + ".out": (n,), p + s + ".mix": (n, n)})
    out["final.norm"] = (W,)
    out["head"] = (cfg["vocab"], W)
    return out


def bf16_round(a):
    """round-to-nearest-even onto the bfloat16 grid, so that every storage dtype of the library holds the same numbers"""
    u = np.asarray(a, np.float32).view(np.uint32).astype(np.uint64)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16
    return u.astype(np.uint32).view(np.float32).reshape(np.shape(a))


def random_tensors(cfg, seed=0, overrides=None, rank_a=5, rank_g=7):
    """weights on the bfloat16 grid, scaled so that every mechanism matters: projections ~ 1 / sqrt(inputs), decays spread over (0, 1), stream mixes near the
    identity with every entry different"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, rank_a, rank_g).items():
        leaf = name.split(".")[-1]
        if name in ("embed", "bigram"):
            v = rng.standard_normal(shape)
        elif leaf == "conv":
            v = rng.standard_normal(shape) * 0.6
        elif leaf == "A_log":
            v = rng.uniform(-2.5, 0.5, shape)
        elif leaf == "mix":
            v = np.eye(shape[0]) + rng.standard_normal(shape) * 0.15
        elif leaf == "in":
            v = rng.uniform(0.2, 1.0, shape) / shape[0] * 1.6
        elif leaf == "out":
            v = rng.uniform(0.5, 1.5, shape)
        elif len(shape) == 2:
            v = rng.standard_normal(shape) / np.sqrt(shape[1])
        elif name.endswith("mix.norm"):
            v = rng.uniform(0.5, 1.5, shape)
        elif "norm" in leaf:
            v = rng.uniform(-0.4, 0.4, shape)
        elif leaf == "dt_bias":
            v = rng.uniform(-3.0, 0.5, shape)
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            v = rng.standard_normal(shape) * 0.8 / np.sqrt(shape[0]) ** 0.5
        else:
            v = rng.standard_normal(shape) * 0.3
        out[name] = bf16_round(v)
    for k, v in (overrides or {}).items():
        out[k] = bf16_round(v)
    return out
