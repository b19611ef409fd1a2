"""Plain numpy (float64) restatement of the Nusovik design, one function per mechanism, whole sequences only (no cache, no state
between calls): the slow restatement that the device path is compared with.  It shares no code with tinygpt_amd.

A model is (cfg, tensors): cfg the dictionary of the checkpoint's config.json, tensors name -> float array.
Notation: T tokens, W width, H heads, G key / value heads or groups, D key size, E value size, N state size, C channels.
"""
import math

import numpy as np


def rms(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis"""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.where(z > 30, z, np.log1p(np.exp(np.minimum(z, 30))))


def sinusoids(T, W):
    """[T][W]: channel 2i holds sin(p f_i), channel 2i + 1 cos(p f_i), f_i = 10000^(-2i / W)"""
    out = np.zeros((T, W))
    for c in range(W):
        a = np.arange(T) * 10000.0 ** (-2.0 * (c // 2) / W)
        out[:, c] = np.cos(a) if c % 2 else np.sin(a)
    return out


def squared_relu_ff(h, up, down):
    return np.maximum(h @ up.T, 0.0) ** 2 @ down.T


# ---- attention: chunks, bucketed distance bias, per-head sink and gate -----------------------------------------------------------------
def chunk_mask(T, size):
    """visible[i][j]: j not behind i's block of `size` positions and not ahead of i (size None: plain causal)"""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) if size is None else (j <= i) & (i // size == j // size)


def bucket(n, B, D):
    """row of the distance table for a distance n >= 0: exact below B // 2, then logarithmic up to D, the last row beyond"""
    half = B // 2
    if n < half:
        return n
    return min(B - 1, half + math.floor(math.log(n / half) / math.log(D / half) * (B - half) + 1e-9))


def distance_bias(rel, T, D):
    """rel [B][H] -> [H][T] by distance"""
    return np.stack([rel[bucket(n, rel.shape[0], D)] for n in range(T)], axis=1)


def sink_attention(q, k, v, visible, scale, bias, sink):
    """q [T][H][E], k, v [T][G][E], bias [H][distance], sink [H] -> [T][H][E]: the sink is one more term of the softmax's denominator"""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            js = np.nonzero(visible[i])[0]
            s = k[js, g] @ q[i, h] * scale + bias[h][i - js]
            top = max(s.max(), sink[h])
            p = np.exp(s - top)
            out[i, h] = p @ v[js, g] / (p.sum() + math.exp(sink[h] - top))
    return out


def keys_as_values_attention(h, m, t, pre, eps):
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q = (h @ t[pre + "q"].T + t[pre + "q.b"]).reshape(T, H, D)
    k = (h @ t[pre + "k"].T + t[pre + "k.b"]).reshape(T, G, D)
    v = k                                                  # the projection itself, before its norm
    q, k = rms(q, t[pre + "q.norm"], eps), rms(k, t[pre + "k.norm"], eps)
    bias = distance_bias(t[pre + "rel"], T, m["bias_max"])
    o = sink_attention(q, k, v, chunk_mask(T, m["mask"]["size"] if m.get("mask") else None), m["scale"], bias, t[pre + "sink"])
    o = o * sigmoid(h @ t[pre + "g"].T)[:, :, None]
    return o.reshape(T, H * D) @ t[pre + "o"].T


# ---- the two state-space mixers ----------------------------------------------------------------------------------------------------------
def short_conv(x, w, b):
    """x [T][C], w [C][taps] (last column: the current token), b [C]; zeros before the start"""
    T, taps = x.shape[0], w.shape[1]
    out = np.tile(b, (T, 1)).astype(np.float64)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            out[back:] += x[:T - back] * w[:, j]
    return out


def scalar_decay_scan(dt, A_log, B, C, x, D):
    """dt [T][H], B, C [T][G][N], x [T][H][E]: per head a state [N][E] that decays by one number a token"""
    T, H, E = x.shape
    G, N = B.shape[1], B.shape[2]
    y = np.zeros((T, H, E))
    for h in range(H):
        g = h // (H // G)
        S = np.zeros((N, E))
        for i in range(T):
            S = np.exp(-np.exp(A_log[h]) * dt[i, h]) * S + dt[i, h] * np.outer(B[i, g], x[i, h])
            y[i, h] = S.T @ C[i, g] + D[h] * x[i, h]
    return y


def gated_part_norm(y, z, w, parts, eps):
    """(y silu(z)) in `parts` equal parts, each divided by its own root mean square, times w"""
    y = y * silu(z)
    T, I = y.shape
    y = y.reshape(T, parts, I // parts)
    y = y / np.sqrt(np.mean(y * y, axis=-1, keepdims=True) + eps)
    return y.reshape(T, I) * w


def mamba2(h, m, t, pre, eps):
    T = h.shape[0]
    H, E, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    I = H * E
    p = h @ t[pre + "in"].T
    z, xbc, dt = p[:, :I], p[:, I:2 * I + 2 * G * N], p[:, 2 * I + 2 * G * N:]
    xbc = silu(short_conv(xbc, t[pre + "conv"], t[pre + "conv.b"]))
    x, B, C = xbc[:, :I].reshape(T, H, E), xbc[:, I:I + G * N].reshape(T, G, N), xbc[:, I + G * N:].reshape(T, G, N)
    y = scalar_decay_scan(softplus(dt + t[pre + "dt_bias"]), t[pre + "A_log"], B, C, x, t[pre + "D"])
    return gated_part_norm(y.reshape(T, I), z, t[pre + "norm"], m["norm_groups"], eps) @ t[pre + "o"].T


def selective_scan(dt, A, B, C, x, D):
    """dt, x [T][C], A [C][N], B, C [T][N]: every (channel, state) pair decays on its own"""
    S = np.zeros_like(A)
    y = np.zeros_like(x)
    for i in range(x.shape[0]):
        S = np.exp(dt[i][:, None] * A) * S + (dt[i] * x[i])[:, None] * B[i][None, :]
        y[i] = S @ C[i] + D * x[i]
    return y


def mamba1(h, m, t, pre):
    I, N, R = m["inner"], m["state"], m["dt_rank"]
    p = h @ t[pre + "in"].T
    x, z = p[:, :I], p[:, I:]
    x = silu(short_conv(x, t[pre + "conv"], t[pre + "conv.b"]))
    q = x @ t[pre + "x"].T
    dt = softplus(q[:, :R] @ t[pre + "dt"].T + t[pre + "dt.b"])
    y = selective_scan(dt, -np.exp(t[pre + "A_log"]), q[:, R:R + N], q[:, R + N:], x, t[pre + "D"])
    return (y * silu(z)) @ t[pre + "o"].T


def parallel_mixer(h, m, t, pre, eps):
    return m["left_scale"] * keys_as_values_attention(h, m["left"], t, pre + "left.", eps) + m["right_scale"] * mamba2(h, m["right"], t, pre + "right.", eps)


# ---- the model ---------------------------------------------------------------------------------------------------------------------
def forward(cfg, t, ids, layers_out=None):
    """logits [T][vocab] of one sequence; layers_out (a list) receives the stream after every layer"""
    t = {k: np.asarray(v, np.float64) for k, v in t.items()}
    eps = cfg["norm"]["eps"]
    x = t["embed"][np.asarray(ids)] * cfg["embedding"]["scale"]
    x = x + sinusoids(*x.shape)
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        if L["type"] == "parallel":
            y = parallel_mixer(x, L["mixer"], t, p + "mix.", eps)
        elif L["type"] == "mamba1":
            y = mamba1(x, L["mixer"], t, p + "mix.")
        else:
            raise ValueError(L["type"])
        x = x + rms(y, t[p + "norm1"], eps)
        if L.get("mlp"):
            x = x + rms(squared_relu_ff(x, t[p + "mlp.up"], t[p + "mlp.down"]), t[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return rms(x, t["final.norm"], eps) @ t["head"].T * cfg["logit_scale"]


# ---- random models -----------------------------------------------------------------------------------------------------------------
def tensor_shapes(cfg, buckets=8):
    """checkpoint name -> shape; the number of distance buckets is not part of the configuration (the tensor carries it)"""
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        out[p + "norm1"] = (W,)
        if L.get("mlp"):
            out[p + "norm2"] = (W,)
        q = p + "mix."
        if L["type"] == "mamba1":
            I, N, R = m["inner"], m["state"], m["dt_rank"]
            out.update({q + "in": (2 * I, W), q + "conv": (I, m["conv"]), q + "conv.b": (I,), q + "x": (R + 2 * N, I), q + "dt": (I, R), q + "dt.b": (I,),
                        q + "A_log": (I, N), q + "D": (I,), q + "o": (W, I)})
        else:
            l, r = m["left"], m["right"]
            H, G, D = l["heads"], l["kv_heads"], l["dim"]
            a = q + "left."
            out.update({a + "q": (H * D, W), a + "q.b": (H * D,), a + "k": (G * D, W), a + "k.b": (G * D,), a + "q.norm": (D,), a + "k.norm": (D,),
                        a + "rel": (buckets, H), a + "sink": (H,), a + "g": (H, W), a + "o": (W, H * D)})
            I, gn = r["heads"] * r["vdim"], r["groups"] * r["state"]
            a = q + "right."
            out.update({a + "in": (2 * I + 2 * gn + r["heads"], W), a + "conv": (I + 2 * gn, r["conv"]), a + "conv.b": (I + 2 * gn,), a + "dt_bias": (r["heads"],),
                        a + "A_log": (r["heads"],), a + "D": (r["heads"],), a + "norm": (I,), a + "o": (W, I)})
        if L.get("mlp"):
            F = L["mlp"]["ff"]
            out.update({p + "mlp.up": (F, W), p + "mlp.down": (W, F)})
    out["final.norm"] = (W,)
    out["head"] = (cfg["vocab"], W)
    return out


def bf16_round(a):
    """round-to-nearest-even onto the bfloat16 grid, so that every storage dtype of the library holds the same numbers"""
    u = np.asarray(a, np.float32).view(np.uint32).astype(np.uint64)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16
    return u.astype(np.uint32).view(np.float32).reshape(np.shape(a))


def random_tensors(cfg, seed=0, overrides=None, buckets=8):
    """weights on the bfloat16 grid, scaled so that every mechanism matters: projections ~ 1 / sqrt(inputs), decays spread over (0, 1), sinks and distance rows
    of the size of the scores"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, buckets).items():
        leaf = name.split(".")[-1]
        if name == "embed":
            v = rng.standard_normal(shape)
        elif leaf == "conv":
            v = rng.standard_normal(shape) * 0.6
        elif leaf == "A_log":
            v = rng.uniform(-2.5, 0.5, shape)
        elif leaf == "rel":
            v = rng.standard_normal(shape)
        elif len(shape) == 2:
            v = rng.standard_normal(shape) / np.sqrt(shape[1])
        elif "norm" in leaf:
            v = rng.uniform(0.5, 1.5, shape)
        elif leaf == "dt_bias" or name.endswith("dt.b"):
            v = rng.uniform(-2.0, 0.5, shape)
        elif leaf == "sink":
            v = rng.uniform(-1.0, 2.0, shape)
        elif leaf == "D":
            v = rng.uniform(0.3, 1.5, shape)
        else:
            v = rng.standard_normal(shape) * 0.3
        out[name] = bf16_round(v)
    for k, v in (overrides or {}).items():
        out[k] = bf16_round(v)
    return out
