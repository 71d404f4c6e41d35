"""Plain, slow reference of the hybrid decoder (the Nilivik design) in numpy: one function per mechanism, a whole sequence at a
time, float64 unless said otherwise.  Test infrastructure only -- it shares nothing with crabml_amd/, and every function takes
arrays and numbers, so a test can plant a mistake by swapping one of them.

A model here is (config, tensors): the dictionary of config.json and a dictionary of float arrays by tensor name."""
import numpy as np

POSITION_BASE = 10000.0


def rms_scale(x, eps):
    """x / root mean square along the last axis, eps under the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.log1p(np.exp(-np.abs(z))) + np.maximum(z, 0.0)


def xielu(z, p, q):
    """a quadratic with slope 1/2 at the origin on the right, an exponential one on the left; the curvatures come from p and q"""
    neg = np.minimum(z, 0.0)
    right = softplus(p) * z * z
    left = (0.5 + softplus(q)) * (np.exp(neg) - 1.0 - neg)
    return np.where(z > 0, right, left) + 0.5 * z


def position_vectors(positions, width, dtype=np.float64):
    """interleaved sin / cos at geometrically falling frequencies"""
    out = np.zeros((len(positions), width), dtype)
    for c in range(width):
        ang = np.asarray(positions, np.float64) * POSITION_BASE ** (-2.0 * (c // 2) / width)
        out[:, c] = np.cos(ang) if c % 2 else np.sin(ang)
    return out


def softmax_attention(q, k, v, score_scale, chunk, bias_amp=None, bias_rate=None, sink=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv]: causal inside chunks of `chunk` positions, a log-distance penalty per head, and a
    sink logit per head in the denominator.  Returns [T, H, dv]."""
    T, H, _ = q.shape
    group = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]), q.dtype)
    i = np.arange(T)
    seen = (i[None, :] <= i[:, None]) & (i[None, :] // chunk == i[:, None] // chunk)
    dist = np.maximum(i[:, None] - i[None, :], 0).astype(q.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h // group].T) * score_scale
        if bias_amp is not None:
            s = s - bias_amp[h] * np.log(1.0 + bias_rate[h] * dist)
        s = np.where(seen, s, -np.inf)
        top = s.max(axis=1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, sink[h])
        e = np.exp(s - top)
        den = e.sum(axis=1, keepdims=True)
        if sink is not None:
            den = den + np.exp(sink[h] - top)
        out[:, h] = (e / den) @ v[:, h // group]
    return out


def decaying_linear_attention(q, k, v, decay, state=None):
    """q, k [T, H, d], v [T, H, dv]: S <- decay S + k v^T, o = S^T q, token by token.  Returns ([T, H, dv], S)."""
    T, H, d = q.shape
    s = np.zeros((H, d, v.shape[2]), q.dtype) if state is None else state.copy()
    dec = np.asarray(decay, q.dtype)[:, None, None]
    out = np.zeros((T, H, v.shape[2]), q.dtype)
    for t in range(T):
        s = dec * s + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hdv,hd->hv", s, q[t])
    return out, s


def attention_branch(h, w, pre, m):
    T = h.shape[0]
    H, G = m["heads"], m["kv_heads"]
    q = (h @ w[pre + "q"].T).reshape(T, H, m["dim"])
    k = (h @ w[pre + "k"].T).reshape(T, G, m["dim"])
    v = (h @ w[pre + "v"].T).reshape(T, G, m["vdim"])
    a = softmax_attention(q, k, v, m["scale"], m["mask"]["size"], w[pre + "r1"], w[pre + "r2"], w[pre + "sink"])
    a = a.reshape(T, -1) * sigmoid(h @ w[pre + "g"].T)
    return a @ w[pre + "o"].T


def linear_branch(h, w, pre, m, eps):
    T = h.shape[0]
    H = m["heads"]
    q = silu(h @ w[pre + "q"].T).reshape(T, H, m["dim"])
    k = silu(h @ w[pre + "k"].T).reshape(T, H, m["dim"])
    v = silu(h @ w[pre + "v"].T).reshape(T, H, m["vdim"])
    o, _ = decaying_linear_attention(q, k, v, m["decay"])
    o = rms_scale(o.reshape(T, -1), eps) * w[pre + "norm"] * sigmoid(h @ w[pre + "g"].T)
    return o @ w[pre + "o"].T


def feed_forward(h, w, pre):
    p, q = w[pre + "act"]
    return xielu(h @ w[pre + "up"].T, p, q) @ w[pre + "down"].T


def run_order(config):
    """[(layer, pass number or None, first of its pass)] of one forward"""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, None, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, None, False) for i in range(a)]
    for t in range(loop["times"]):
        runs += [(i, t, i == a) for i in range(a, b)]
    return runs + [(i, None, False) for i in range(b, n)]


def layer(x, w, spec, pre, eps):
    m = spec["mixer"]
    h = rms_scale(x, eps) * w[pre + "norm1"]
    x = x + m["left_scale"] * attention_branch(h, w, pre + "mix.left.", m["left"]) \
        + m["right_scale"] * linear_branch(h, w, pre + "mix.right.", m["right"], eps)
    if spec.get("mlp"):
        h = rms_scale(x, eps) * w[pre + "norm2"]
        x = x + feed_forward(h, w, pre + "mlp.")
    return x


def forward(config, tensors, tokens, dtype=np.float64, trace=None):
    """logits [T, vocab] of one sequence; trace (a list): the residual stream after every layer run is appended"""
    w = {k: np.asarray(v, dtype) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    emb = w["embed"][np.asarray(tokens)] * dtype(config["embedding"]["scale"])
    emb = emb + position_vectors(np.arange(len(tokens)), config["width"], dtype)
    x = emb
    for i, t, first in run_order(config):
        if first:
            if t > 0:
                x = x + emb
            x = x + w["loop.step"][t]
        x = layer(x, w, config["layers"][i], "l%d." % i, eps)
        if trace is not None:
            trace.append(x)
    y = (rms_scale(x, eps) * w["final.norm"]) @ w["head"].T
    cap = config["logit_softcap"]
    return cap * np.tanh(y / cap)
