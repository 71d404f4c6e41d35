"""Synthetic models of the Nilivik design (random weights) for the bench, the tests and demos: a configuration dictionary as
config.json holds it, bfloat16-representable tensors by name, and the model folder (config.json + model.safetensors).  Pure numpy."""
from __future__ import annotations

import json
import os
import struct
from typing import Dict, List, Optional

import numpy as np


def to_bf16(a: np.ndarray) -> np.ndarray:
    """f32 -> bfloat16 bits, to nearest even"""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def from_bf16(b: np.ndarray) -> np.ndarray:
    return (b.astype(np.uint32) << 16).view(np.float32)


def layer(heads, kv_heads, dim, vdim, chunk, lin_heads, lin_dim, lin_vdim, ff: Optional[int], decay: Optional[List[float]] = None,
          scale: Optional[float] = None, left_scale=0.7, right_scale=0.55) -> dict:
    decay = decay if decay is not None else [float(1.0 - 2.0 ** (-1.0 - 8.0 * (h + 1) / lin_heads)) for h in range(lin_heads)]
    return {"type": "parallel",
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk},
                               "scale": scale if scale is not None else dim ** -0.5},
                      "left_scale": left_scale,
                      "right": {"heads": lin_heads, "dim": lin_dim, "vdim": lin_vdim, "decay": decay},
                      "right_scale": right_scale},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width: int, vocab: int, layers: List[dict], loop: Optional[dict] = None, embed_scale=2.5, eps=1e-5, softcap=25.0) -> dict:
    return {"architecture": "Nilivik", "width": width, "vocab": vocab, "embedding": {"scale": embed_scale}, "norm": {"eps": eps},
            "logit_softcap": softcap, "loop": loop, "layers": layers}


def tensor_shapes(c: dict) -> Dict[str, tuple]:
    W = c["width"]
    s = {"embed": (c["vocab"], W), "head": (c["vocab"], W), "final.norm": ()}
    if c.get("loop"):
        s["loop.step"] = (c["loop"]["times"], W)
    for i, l in enumerate(c["layers"]):
        p, a, r = "l%d." % i, l["mixer"]["left"], l["mixer"]["right"]
        H, G, R = a["heads"], a["kv_heads"], r["heads"]
        s[p + "norm1"] = ()
        q = p + "mix.left."
        s.update({q + "q": (H * a["dim"], W), q + "k": (G * a["dim"], W), q + "v": (G * a["vdim"], W), q + "g": (H * a["vdim"], W),
                  q + "o": (W, H * a["vdim"]), q + "r1": (H,), q + "r2": (H,), q + "sink": (H,)})
        q = p + "mix.right."
        s.update({q + "q": (R * r["dim"], W), q + "k": (R * r["dim"], W), q + "v": (R * r["vdim"], W), q + "g": (R * r["vdim"], W),
                  q + "o": (W, R * r["vdim"]), q + "norm": (R * r["vdim"],)})
        if l.get("mlp"):
            s.update({p + "norm2": (), p + "mlp.up": (l["mlp"]["ff"], W), p + "mlp.down": (W, l["mlp"]["ff"]), p + "mlp.act": (2,)})
    return s


def random_tensors(c: dict, seed: int = 0, pool: int = 0) -> Dict[str, np.ndarray]:
    """bfloat16 bits of every tensor.  pool > 0: matrices are cut out of one pool of that many numbers (large models: the generator
    would otherwise take longer than the run)"""
    rng = np.random.default_rng(seed)
    base = rng.standard_normal(pool).astype(np.float32) if pool else None
    out = {}
    for name, shape in tensor_shapes(c).items():
        n = int(np.prod(shape, dtype=np.int64))
        tail = name.split(".")[-1]
        if len(shape) == 2 and name not in ("embed", "loop.step"):
            sd = (1.3 if tail in ("q", "k") else 1.0) / np.sqrt(shape[1])
            if base is not None:
                b = to_bf16(base * np.float32(sd))
                out[name] = np.resize(np.roll(b, int(rng.integers(pool))), n).reshape(shape)
                continue
            v = rng.standard_normal(n) * sd
        elif name == "embed":
            v = np.resize(base, n) if base is not None else rng.standard_normal(n)
        elif tail in ("norm1", "norm2") or name == "final.norm":
            v = rng.uniform(0.6, 1.4, n)
        elif tail == "norm":
            v = rng.uniform(0.5, 1.5, n)
        elif tail == "r1":
            v = rng.uniform(0.1, 1.6, n)
        elif tail == "r2":
            v = rng.uniform(0.05, 0.5, n)
        elif tail == "sink":
            v = rng.normal(1.0, 1.5, n)
        else:  # loop.step, act
            v = rng.standard_normal(n) * (0.5 if name == "loop.step" else 1.0)
        out[name] = to_bf16(np.asarray(v, np.float32)).reshape(shape)
    return out


def write_safetensors(tensors: Dict[str, np.ndarray], path: str) -> None:
    """uint16 arrays (bfloat16 bits) by name"""
    head, at = {}, 0
    for name, t in tensors.items():
        head[name] = {"dtype": "BF16", "shape": list(t.shape), "data_offsets": [at, at + t.nbytes]}
        at += t.nbytes
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(h)))
        f.write(h)
        for t in tensors.values():
            f.write(np.ascontiguousarray(t).data)


def write_model(c: dict, tensors: Dict[str, np.ndarray], folder: str) -> str:
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(c, f)
    write_safetensors(tensors, os.path.join(folder, "model.safetensors"))
    return folder
