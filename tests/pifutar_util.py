"""Helpers of the Pifutar tests: configurations and random weights made here, written as checkpoints (config.json +
model.safetensors), run through the package's own loader, executor and trace replay, and compared with the plain model of
`pifutar_oracle`."""
from __future__ import annotations

from typing import Dict, List, Optional

import numpy as np
import torch

import pifutar_oracle as O
from letarax_util import random_tokens, rel_err, replay, save_model, session  # noqa: F401  (shared checkpoint / replay helpers)


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def moe(experts: int, top: int, ff: int, limit: float = 1.5, shared: int = 0, shared_limit: Optional[float] = None) -> dict:
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared, "limit": limit if shared_limit is None else shared_limit}
    return m


def gla(heads: int, dim: int, vdim: int, tau: float = 8.0, rank: int = 6, mlp: Optional[dict] = None) -> dict:
    """`rank` is the size of the tensors drawn by `random_weights`; a checkpoint's config does not carry it."""
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": mlp, "rank": rank}


def retention(heads: int, dim: int, vdim: int, decay: Optional[List[float]] = None, mlp: Optional[dict] = None) -> dict:
    decay = decay or [1.0 - 0.3 * 0.25 ** i for i in range(heads)]
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": mlp}


def latent(heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, window: int = 0, base: float = 5000.0, scale: Optional[float] = None,
           kv_from: Optional[int] = None, mlp: Optional[dict] = None) -> dict:
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "rot": {"base": base, "dims": rot_dim},
         "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def make_config(layers: List[dict], vocab: int, width: int, taps: int = 3, eps: float = 1e-5) -> dict:
    return {"architecture": "Pifutar", "layers": layers, "canon": {"taps": taps}, "norm": {"eps": eps}, "vocab": vocab, "width": width}


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """bf16 tensors (tables int32) under the checkpoint's names, scaled so that every mechanism matters: projections at about
    1 / sqrt(fan-in), convolution taps, depth weights and polynomial coefficients of order one, decays short and long."""
    g = torch.Generator().manual_seed(seed)
    rn = lambda *shape, std=1.0: torch.randn(*shape, generator=g) * std
    W, H, V = {}, cfg["width"], cfg["vocab"]
    W["embed"], W["final.norm"] = rn(V, H), rn(H, std=0.1)
    for i, l in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", l["mixer"], l.get("mlp")
        x, hd, dv = p + "mix.", m["heads"] * m["dim"], m["heads"] * m["vdim"]
        W[p + "norm1"], W[p + "canon1"] = rn(H, std=0.2), rn(H, cfg["canon"]["taps"], std=0.4)
        W[p + "dwa"] = rn(i + 2, std=0.2) + torch.tensor([0.2] * (i + 1) + [0.8])
        W[x + "o"] = rn(H, dv, std=dv ** -0.5)
        if l["type"] == "latent_attention":
            R, dr = m["kv_rank"], m["rot_dim"]
            W[x + "q"] = rn(m["heads"] * (m["dim"] + dr), H, std=1.5 * H ** -0.5)
            W[x + "uk"], W[x + "uv"] = rn(hd, R, std=R ** -0.5), rn(dv, R, std=R ** -0.5)
            if m.get("kv_from") is None:
                W[x + "dkv"], W[x + "dkv.norm"] = rn(R + dr, H, std=1.5 * H ** -0.5), 1.0 + rn(R, std=0.2)
        else:
            W[x + "q"], W[x + "k"], W[x + "v"], W[x + "g"] = (rn(n, H, std=H ** -0.5) for n in (hd, hd, dv, dv))
            if l["type"] == "gla":
                r = l["rank"]
                W[x + "a1"], W[x + "a2"], W[x + "a2.b"] = rn(r, H, std=H ** -0.5), rn(hd, r, std=2.0 * r ** -0.5), rn(hd, std=1.5)
                W[x + "norm"] = 1.0 + rn(m["vdim"], std=0.2)
        if mlp is None:
            continue
        W[p + "norm2"], W[p + "canon2"] = rn(H, std=0.2), rn(H, cfg["canon"]["taps"], std=0.4)
        x = p + "mlp."
        if mlp["kind"] == "dense":
            ff = mlp["ff"]
            W[x + "up"], W[x + "down"] = rn(ff, H, std=H ** -0.5), rn(H, ff, std=ff ** -0.5)
            W[x + "act"] = torch.tensor([0.6, -0.4, 0.5, 0.2]) + rn(4, std=0.2)
        else:
            E, top = mlp["router"]["experts"], mlp["router"]["top"]
            W[x + "table"] = torch.argsort(torch.rand(V, E, generator=g), dim=-1)[:, :top].to(torch.int32)
            for e in [f"e{j}." for j in range(E)] + (["shared."] if mlp.get("shared") else []):
                f = mlp["shared"]["ff"] if e == "shared." else mlp["expert"]["ff"]
                W[x + e + "gate"], W[x + e + "up"], W[x + e + "down"] = rn(f, H, std=1.5 * H ** -0.5), rn(f, H, std=1.5 * H ** -0.5), rn(H, f, std=f ** -0.5)
            if mlp.get("shared"):
                W[x + "shared.sg"] = rn(1, H, std=2.0 * H ** -0.5)
    return {k: (v.to(torch.bfloat16) if v.is_floating_point() else v) for k, v in W.items()}


def oracle_logits(cfg: dict, W, tokens: List[int]) -> np.ndarray:
    return O.forward(cfg, W, tokens)[0].numpy()


# Against the plain model: fp32 executors agree to rounding. In bf16 a tiny random model's worst position carries several per cent
# of rounding noise, so the sharp check of a bf16 run is `SAME`: however a request was cut into steps and whatever shared its
# batches, its logits agree with the same executor's run of the whole prompt alone to a few roundings.
TOL = {"fp32": 2e-4, "bf16": 0.3}
SAME = {"fp32": 1e-4, "bf16": 8e-2}


def alone(model_dir: str, backend: str, dtype: str, tokens: List[int]) -> np.ndarray:
    sess = session(model_dir, backend, dtype, max_tokens=len(tokens) + 64, slots=1)
    out = replay(sess, {"x": tokens}, [[("x", len(tokens))]])["x"]
    sess.close()
    return out


# Stacks that differ in everything a config can say: order and kind of the layers, head counts down to one, key and value sizes
# (equal, unequal, not powers of two, no multiples of 8), decays of one and zero and in between, tau of one and large, windows of
# one token, shorter and longer than a cache block or the prompts or absent, latents read by several layers with windows, heads
# and value sizes of their own, convolutions of one to five taps, the feed-forward of every layer (none, dense, routed with or
# without a shared expert, one expert of one), limits that clip, widths that are no multiple of 8, eps.
STACKS = {
    "mixed": make_config([retention(3, 16, 24, mlp=moe(5, 2, 24, shared=40, shared_limit=0.7)), latent(4, 16, 8, 12, 24, window=20, mlp=dense(40)),
                          gla(2, 12, 20, tau=4.0, mlp=moe(6, 3, 16, limit=0.5)), latent(2, 16, 8, 16, 24, window=33, kv_from=1, mlp=None),
                          latent(3, 8, 8, 8, 24, window=0, kv_from=1, mlp=moe(3, 1, 24, shared=16)), gla(4, 8, 8, tau=1.0, rank=3, mlp=dense(24))],
                         vocab=96, width=48, taps=3),
    "odd_sizes": make_config([latent(1, 10, 6, 9, 14, window=1, base=100.0, scale=0.6, mlp=moe(1, 1, 12)), gla(3, 7, 5, tau=16.0, rank=1, mlp=None),
                              retention(2, 9, 11, decay=[1.0, 0.0], mlp=dense(33)), latent(5, 6, 2, 7, 10, window=70, mlp=moe(4, 4, 10, limit=3.0, shared=9))],
                             vocab=51, width=37, taps=5, eps=1e-6),
    "plain": make_config([gla(1, 20, 36, tau=2.0, rank=9, mlp=dense(56)), retention(5, 24, 8, mlp=None), latent(2, 8, 4, 16, 12, window=5, mlp=None)],
                         vocab=40, width=64, taps=1),
    # widths and inner sizes that the packed-weight GEMMs and the matrix-core attention take in bf16
    "packed": make_config([latent(4, 32, 16, 32, 96, window=44, base=500000.0, mlp=dense(256)), retention(2, 64, 64, mlp=moe(8, 2, 64, limit=2.0, shared=128)),
                           gla(2, 128, 64, tau=16.0, rank=16, mlp=moe(4, 2, 128)), latent(8, 16, 16, 64, 96, window=100, base=500000.0, kv_from=0, mlp=moe(6, 2, 32, shared=64)),
                           latent(16, 24, 32, 16, 160, window=0, mlp=None)],
                          vocab=90, width=128, taps=4),
}
