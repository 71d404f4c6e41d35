"""Synthetic models of the Bifazen design (random weights) for the bench, the tests and demos: a configuration dictionary as
config.json holds it, and bfloat16 tensors by name (synth_hybrid.write_model makes the folder).  Pure numpy."""
from __future__ import annotations

from typing import Dict, List, Optional

import numpy as np

from .synth_hybrid import to_bf16


def _layer(kind: str, mixer: dict, ff: Optional[int]) -> dict:
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def latent(heads, dim, rot_dim, vdim, kv_rank, window, ff: Optional[int], base=10000.0, scale: Optional[float] = None) -> dict:
    return _layer("latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": window},
                                       "rot": {"base": base, "dims": rot_dim}, "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}, ff)


def attention(heads, kv_heads, dim, vdim, window, ff: Optional[int], v_mix=True, scale: Optional[float] = None) -> dict:
    return _layer("attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
                                "scale": scale if scale is not None else dim ** -0.5, "v_mix": v_mix}, ff)


def config(width: int, vocab: int, layers: List[dict], streams: int = 2, eps=1e-5) -> dict:
    return {"architecture": "Bifazen", "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps}, "layers": layers}


def tensor_shapes(c: dict) -> Dict[str, tuple]:
    W, S = c["width"], c["streams"]
    s = {"embed": (c["vocab"], W), "final.norm": (W,)}
    for i, l in enumerate(c["layers"]):
        p, m = "l%d." % i, l["mixer"]
        x, H = p + "mix.", l["mixer"]["heads"]
        s.update({p + "norm1": (W,), p + "hc1.in": (S,), p + "hc1.out": (S,), p + "hc1.mix": (S, S), x + "o": (W, H * m["vdim"])})
        if l["type"] == "latent_attention":
            s.update({x + "q": (H * (m["dim"] + m["rot_dim"]), W), x + "dkv": (m["kv_rank"] + m["rot_dim"], W), x + "dkv.norm": (m["kv_rank"],),
                      x + "uk": (H * m["dim"], m["kv_rank"]), x + "uv": (H * m["vdim"], m["kv_rank"])})
        else:
            q, k, v = H * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"]
            s.update({x + "q": (q, W), x + "q.b": (q,), x + "q.norm": (q,), x + "k": (k, W), x + "k.b": (k,), x + "k.norm": (k,), x + "v": (v, W),
                      x + "v.b": (v,), x + "g": (H, W), x + "o.b": (W,)})
            if m.get("v_mix"):
                s[x + "vmix"] = ()
        if l.get("mlp"):
            f = l["mlp"]["ff"]
            s.update({p + "norm2": (W,), p + "hc2.in": (S,), p + "hc2.out": (S,), p + "hc2.mix": (S, S), p + "mlp.gate": (f, W), p + "mlp.up": (f, W),
                      p + "mlp.down": (W, f)})
    return s


def random_tensors(c: dict, seed: int = 0, pool: int = 0) -> Dict[str, np.ndarray]:
    """bfloat16 bits of every tensor.  pool > 0: matrices are cut out of one pool of that many numbers (large models)"""
    rng = np.random.default_rng(seed)
    base = rng.standard_normal(pool).astype(np.float32) if pool else None
    S = c["streams"]
    out = {}
    for name, shape in tensor_shapes(c).items():
        n = int(np.prod(shape, dtype=np.int64))
        tail = name.split(".")[-1]
        if ".hc" in name:
            v = rng.standard_normal(n) * 0.15 + {"in": 1.0 / S, "out": 1.0, "mix": 0.0}[tail]
            if tail == "mix":
                v = v / S + np.eye(S).reshape(-1) * 0.9
        elif len(shape) == 2:
            sd = 1.0 if name == "embed" else (1.3 if tail in ("q", "k", "uk", "gate") else 1.0) / np.sqrt(shape[1])
            if base is not None:
                out[name] = np.resize(np.roll(to_bf16(base * np.float32(sd)), int(rng.integers(pool))), n).reshape(shape)
                continue
            v = rng.standard_normal(n) * sd
        elif name.endswith((".q.norm", ".k.norm", ".dkv.norm")):
            v = rng.uniform(0.5, 1.5, n)
        elif tail in ("norm1", "norm2", "norm"):
            v = rng.standard_normal(n) * 0.3  # around zero: the gain is one more
        elif tail == "vmix":
            v = rng.uniform(0.2, 0.8, n)
        else:  # biases
            v = rng.standard_normal(n) * 0.4
        out[name] = to_bf16(np.asarray(v, np.float32)).reshape(shape)
    return out
