"""Plain, slow reference of the Bifazen design in numpy: one function per mechanism, a whole sequence at a time, float64 unless said
otherwise.  Test infrastructure only -- it shares nothing with crabml_amd/, and every function takes arrays and numbers, so a test can
plant a mistake by swapping one of them.

A model here is (config, tensors): the dictionary of config.json and a dictionary of float arrays by tensor name."""
import numpy as np


def rms_norm(x, gain, eps):
    """x over its root mean square (eps under the root), times a gain per element"""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * gain


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rotate_pairs(x, positions, base, dims):
    """x [T, ..., n]: elements 2 i and 2 i + 1 of the first `dims` turned by position * base^(-2 i / dims)"""
    out = x.copy()
    for t, p in enumerate(positions):
        for i in range(dims // 2):
            a = float(p) * float(base) ** (-2.0 * i / dims)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            out[t, ..., 2 * i] = u * np.cos(a) - v * np.sin(a)
            out[t, ..., 2 * i + 1] = v * np.cos(a) + u * np.sin(a)
    return out


def window_mask(n, size):
    """[query, key]: a query sees itself and the size - 1 tokens before it"""
    d = np.arange(n)[:, None] - np.arange(n)[None, :]
    return (d >= 0) & (d < size)


def softmax_attention(scores, values, mask):
    """scores [T, T], values [T, dv]"""
    s = np.where(mask, scores, -np.inf)
    e = np.exp(s - s.max(axis=1, keepdims=True))
    return (e / e.sum(axis=1, keepdims=True)) @ values


def latent_attention(h, w, pre, m, eps):
    T, H = h.shape[0], m["heads"]
    dim, rot, rank = m["dim"], m["rot_dim"], m["kv_rank"]
    pos = range(T)
    q = (h @ w[pre + "q"].T).reshape(T, H, dim + rot)
    down = h @ w[pre + "dkv"].T
    c = rms_norm(down[:, :rank], w[pre + "dkv.norm"], eps)
    q_rot = rotate_pairs(q[:, :, dim:], pos, m["rot"]["base"], rot)
    k_rot = rotate_pairs(down[:, rank:], pos, m["rot"]["base"], rot)
    k = (c @ w[pre + "uk"].T).reshape(T, H, dim)
    v = (c @ w[pre + "uv"].T).reshape(T, H, m["vdim"])
    mask = window_mask(T, m["mask"]["size"])
    heads = [softmax_attention((q[:, i, :dim] @ k[:, i].T + q_rot[:, i] @ k_rot.T) * m["scale"], v[:, i], mask) for i in range(H)]
    return np.concatenate(heads, axis=1) @ w[pre + "o"].T


def grouped_attention(h, w, pre, m, eps, v_first):
    """returns (output, the values that later layers mix in)"""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = rms_norm(h @ w[pre + "q"].T + w[pre + "q.b"], w[pre + "q.norm"], eps).reshape(T, H, m["dim"])
    k = rms_norm(h @ w[pre + "k"].T + w[pre + "k.b"], w[pre + "k.norm"], eps).reshape(T, G, m["dim"])
    v = h @ w[pre + "v"].T + w[pre + "v.b"]
    if m.get("v_mix"):
        if v_first is None:
            v_first = v
        else:
            lam = w[pre + "vmix"]
            v = (1.0 - lam) * v + lam * v_first
    v = v.reshape(T, G, m["vdim"])
    gate = sigmoid(h @ w[pre + "g"].T)
    mask = window_mask(T, m["mask"]["size"])
    heads = [softmax_attention((q[:, i] @ k[:, i // (H // G)].T) * m["scale"], v[:, i // (H // G)], mask) * gate[:, i:i + 1] for i in range(H)]
    return np.concatenate(heads, axis=1) @ w[pre + "o"].T + w[pre + "o.b"], v_first


def gated_feed_forward(h, w, pre):
    return (gelu_tanh(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def hyper_connection(xs, w, pre, sublayer):
    """xs [streams, T, width]: the sublayer reads a weighted sum; every stream becomes a mixture of all plus its share of the result"""
    y = sublayer(np.einsum("s,stw->tw", w[pre + "in"], xs))
    return np.einsum("sd,stw->dtw", w[pre + "mix"], xs) + w[pre + "out"][:, None, None] * y


def forward(config, tensors, tokens, dtype=np.float64, trace=None):
    """logits [T, vocab] of one sequence; trace (a list): the sum of the streams after every layer is appended"""
    w = {k: np.asarray(v, dtype) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    emb = w["embed"][np.asarray(tokens)]
    xs = np.stack([emb] * config["streams"])
    v_first = None
    for i, spec in enumerate(config["layers"]):
        pre, m = "l%d." % i, spec["mixer"]

        def mixer(u):
            nonlocal v_first
            h = rms_norm(u, 1.0 + w[pre + "norm1"], eps)
            if spec["type"] == "latent_attention":
                return latent_attention(h, w, pre + "mix.", m, eps)
            y, v_first = grouped_attention(h, w, pre + "mix.", m, eps, v_first)
            return y
        xs = hyper_connection(xs, w, pre + "hc1.", mixer)
        if spec.get("mlp"):
            xs = hyper_connection(xs, w, pre + "hc2.", lambda u: gated_feed_forward(rms_norm(u, 1.0 + w[pre + "norm2"], eps), w, pre + "mlp."))
        if trace is not None:
            trace.append(xs.sum(axis=0))
    return rms_norm(xs.sum(axis=0), 1.0 + w["final.norm"], eps) @ w["embed"].T
