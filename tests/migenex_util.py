"""Helpers of the Migenex tests: configurations and random weights made here, written as checkpoints (config.json +
model.safetensors), run through the package's own loader, executor and trace replay, and compared with the plain model of
`migenex_oracle`."""
from __future__ import annotations

from typing import Dict, List, Optional

import numpy as np
import torch

import migenex_oracle as O
from letarax_util import random_tokens, rel_err, replay, save_model, session  # noqa: F401  (shared checkpoint / replay helpers)


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def moe(experts: int, top: int, ff: int, shared: int = 0) -> dict:
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def full(heads: int, kv_heads: int, dim: int, vdim: int, rot: Optional[int] = None, base: float = 5000.0, scale: Optional[float] = None,
         cap: float = 20.0, mlp: Optional[dict] = None) -> dict:
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": dim if rot is None else rot},
         "scale": dim ** -0.5 if scale is None else scale, "softcap": cap}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def keyed(heads: int, kv_heads: int, dim: int, window: int, rot: Optional[int] = None, base: float = 5000.0, scale: Optional[float] = None,
          mlp: Optional[dict] = None) -> dict:
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": {"base": base, "dims": dim if rot is None else rot},
         "scale": dim ** -0.5 if scale is None else scale, "mask": {"size": window}}
    return {"type": "attention_2", "mixer": m, "mlp": mlp}


def make_config(layers: List[dict], vocab: int, width: int, loop: Optional[tuple] = None, mult: float = 0.5, scale: float = 3.0,
                bigram: Optional[tuple] = (53, 7, 11), eps: float = 1e-5) -> dict:
    cfg = {"architecture": "Migenex", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps}, "residual_mult": mult,
           "vocab": vocab, "width": width}
    if bigram:
        cfg["embedding"]["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """bf16 tensors under the checkpoint's names, scaled so that every mechanism matters: projections at about 1 / sqrt(fan-in),
    norm weights around one, the bigram rows as large as the scaled embedding rows."""
    g = torch.Generator().manual_seed(seed)
    rn = lambda *shape, std=1.0: torch.randn(*shape, generator=g) * std
    W, H, V = {}, cfg["width"], cfg["vocab"]
    W["embed"], W["head"], W["final.norm"] = rn(V, H, std=1.0 / cfg["embedding"]["scale"]), rn(V, H, std=H ** -0.5), 1.0 + rn(H, std=0.2)
    if cfg["embedding"].get("bigram"):
        W["bigram"] = rn(cfg["embedding"]["bigram"]["buckets"] + 1, H, std=0.8)
    if cfg.get("loop"):
        W["loop.in"] = rn(H, 2 * H, std=1.2 * (2 * H) ** -0.5)
    for i, l in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", l["mixer"], l.get("mlp")
        x, qn, kn, vn, on = p + "mix.", m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"], m["heads"] * m["vdim"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ()):
            W[p + n] = 1.0 + rn(H, std=0.25)
        W[x + "q"], W[x + "k"], W[x + "o"] = rn(qn, H, std=1.5 * H ** -0.5), rn(kn, H, std=1.5 * H ** -0.5), rn(H, on, std=on ** -0.5)
        if l["type"] == "attention":
            W[x + "v"] = rn(vn, H, std=H ** -0.5)
            W[x + "q.norm"], W[x + "k.norm"] = 1.5 + rn(m["dim"], std=0.4), 1.0 + rn(m["dim"], std=0.3)
        else:
            W[x + "g"] = rn(on, H, std=1.5 * H ** -0.5)
        if mlp is None:
            continue
        x = p + "mlp."
        if mlp["kind"] == "dense":
            ff = mlp["ff"]
            W[x + "gate"], W[x + "up"], W[x + "down"] = rn(ff, H, std=H ** -0.5), rn(ff, H, std=H ** -0.5), rn(H, ff, std=ff ** -0.5)
        else:
            E = mlp["router"]["experts"]
            W[x + "router"] = rn(E, H, std=2.0 * H ** -0.5)
            for e in [f"e{j}." for j in range(E)] + (["shared."] if mlp.get("shared") else []):
                f = mlp["shared"]["ff"] if e == "shared." else mlp["expert"]["ff"]
                W[x + e + "up"], W[x + e + "down"] = rn(f, H, std=1.5 * H ** -0.5), rn(H, f, std=(0.5 if e == "shared." else 1.5) * f ** -0.5)
    return {k: v.to(torch.bfloat16) for k, v in W.items()}


def oracle_logits(cfg: dict, W, tokens: List[int]) -> np.ndarray:
    return O.forward(cfg, W, tokens)[0].numpy()


# Against the plain model: fp32 executors agree to rounding. In bf16 a router is a discontinuity (where two experts nearly tie, one
# rounding moves a whole position), so the sharp check of a bf16 run is `SAME`: however a request was cut into steps and whatever
# shared its batches, its logits agree with the same executor's run of the whole prompt alone to a few roundings.
TOL = {"fp32": 2e-4, "bf16": 0.1}
SAME = {"fp32": 1e-4, "bf16": 6e-2}


def alone(model_dir: str, backend: str, dtype: str, tokens: List[int]) -> np.ndarray:
    sess = session(model_dir, backend, dtype, max_tokens=len(tokens) + 64, slots=1)
    out = replay(sess, {"x": tokens}, [[("x", len(tokens))]])["x"]
    sess.close()
    return out


# Stacks that differ in everything a config can say: order and kind of the layers, head counts and groups down to one, key and value
# sizes (equal, unequal, not powers of two, no multiples of 8), rotations of a part of the head and of none, windows of one token,
# shorter and longer than a cache block or the prompts, caps that bite and caps that do not, scales, the loop (absent, at the start, in
# the middle, up to the end, once and several times), the bigram table (absent, one bucket, many), the residual multiplier, the
# embedding's scale, the feed-forward of every layer (none, dense, routed with or without a shared expert, all experts chosen, one
# expert of one), widths that are no multiple of 8, eps.
STACKS = {
    "mixed": make_config([keyed(4, 2, 24, 20, rot=16, mlp=moe(5, 2, 24, shared=40)), full(6, 3, 16, 24, cap=5.0, mlp=dense(40)),
                          keyed(3, 1, 12, 33, mlp=None), full(4, 4, 20, 8, rot=8, base=300.0, mlp=moe(6, 1, 16)),
                          keyed(2, 2, 16, 7, scale=0.7, mlp=dense(24))], vocab=96, width=48, loop=(1, 3, 2)),
    "odd_sizes": make_config([full(1, 1, 10, 9, rot=6, base=100.0, scale=0.6, cap=2.0, mlp=moe(1, 1, 12)), keyed(5, 1, 6, 1, rot=2, mlp=dense(33)),
                              keyed(2, 1, 14, 70, mlp=moe(4, 4, 10, shared=9)), full(3, 3, 7, 11, rot=0, mlp=None)],
                             vocab=51, width=37, loop=(0, 4, 2), mult=1.0, scale=1.0, bigram=(1, 0, 1), eps=1e-6),
    "plain": make_config([full(2, 1, 24, 36, mlp=dense(56)), keyed(4, 4, 8, 5, mlp=moe(3, 2, 16, shared=24))], vocab=40, width=64, bigram=None, scale=0.5),
    # widths and inner sizes that the packed-weight GEMMs and the matrix-core attention take in bf16
    "packed": make_config([keyed(4, 2, 64, 44, mlp=dense(256)), full(8, 2, 64, 64, cap=8.0, mlp=moe(8, 2, 64, shared=128)),
                           keyed(2, 1, 128, 100, rot=64, mlp=moe(4, 1, 128)), full(6, 2, 64, 64, rot=32, base=500000.0, cap=30.0, mlp=None),
                           full(4, 1, 128, 128, mlp=dense(128)), full(4, 2, 96, 32, mlp=moe(6, 2, 32, shared=64))],
                          vocab=90, width=128, loop=(2, 6, 2), mult=0.35, scale=8.0, bigram=(211, 31, 5)),
    # the same without a router's close calls: every position of a bf16 run has to hold
    "packed_dense": make_config([full(4, 2, 64, 64, cap=6.0, mlp=dense(128)), keyed(6, 2, 128, 40, mlp=dense(256)), keyed(4, 4, 64, 33, rot=32, mlp=moe(2, 2, 64, shared=32)),
                                 keyed(8, 2, 80, 50, mlp=None), full(2, 1, 32, 96, rot=16, mlp=dense(64))],
                                vocab=100, width=128, loop=(1, 4, 2), mult=0.6, scale=5.0, bigram=(97, 3, 8)),
}
