"""Small random models of the Purusun architecture for the tests."""

from __future__ import annotations

import torch


def attention(heads: int = 4, kv_heads: int = 2, dim: int = 16, rot: int = 8, base: float = 300.0, scaling: dict | None = None,
              scale: float | None = None, window: int | None = 11, keep: int = 3, ff: int | None = 56) -> dict:
    return {"type": "attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale or 1.3 * dim ** -0.5,
                      "mask": {"size": window, "keep_first": keep} if window else None,
                      "rot": {"base": base, "dims": rot, "scaling": scaling}}}


def scan(inner: int = 48, state: int = 8, rank: int = 6, conv: int = 4, ff: int | None = 40) -> dict:
    return {"type": "mamba1", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"inner": inner, "state": state, "dt_rank": rank, "conv": conv}}


SCALING = {"factor": 6.0, "low": 1.5, "high": 5.0, "original": 40}


def config(layers: list[dict] | None = None, width: int = 48, vocab: int = 67, streams: int = 3, eps: float = 2e-5,
           loop: dict | None = {"start": 1, "stop": 3, "times": 2}) -> dict:
    layers = layers or [attention(scaling=SCALING), scan(), attention(window=7, keep=2), scan(conv=3)]
    return {"architecture": "Purusun", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "layers": layers, "loop": loop}


def random_weights(cfg: dict, seed: int, spread: float = 1.0) -> dict[str, torch.Tensor]:
    """Seeded weights, values exactly representable in bf16.  ``spread`` scales the key norms (larger: sharper scores)."""
    g = torch.Generator().manual_seed(seed)

    def normal(*shape: int, std: float = 1.0) -> torch.Tensor:
        return torch.randn(shape, generator=g) * std

    d, s = cfg["width"], cfg["streams"]
    w = {"embed": normal(cfg["vocab"], d), "final.norm": normal(d, std=0.1)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, mix = f"l{i}.", layer["mixer"], {}
        if layer["type"] == "attention":
            n, k, dim = m["heads"], m["kv_heads"], m["dim"]
            mix = {"q": normal(n * dim, d, std=d ** -0.5), "k": normal(k * dim, d, std=d ** -0.5), "g": normal(n * dim, d, std=d ** -0.5),
                   "q.norm": 1 + normal(dim, std=0.2), "k.norm": spread * (1 + normal(dim, std=0.2)),
                   "o": normal(d, n * dim, std=(n * dim) ** -0.5)}
        else:
            inner, state, rank, conv = (m[x] for x in ("inner", "state", "dt_rank", "conv"))
            mix = {"in": normal(2 * inner, d, std=d ** -0.5), "conv": normal(inner, conv, std=conv ** -0.5), "conv.b": normal(inner, std=0.2),
                   "x": normal(rank + 2 * state, inner, std=inner ** -0.5), "dt": normal(inner, rank, std=rank ** -0.5),
                   "dt.b": -2 + normal(inner, std=1.5), "A_log": normal(inner, state), "D": 1 + normal(inner, std=0.3),
                   "o": normal(d, inner, std=inner ** -0.5)}
        w.update({p + "mix." + name: t for name, t in mix.items()})
        if layer["mlp"] is not None:
            f = layer["mlp"]["ff"]
            w[p + "mlp.up"], w[p + "mlp.down"] = normal(f, d, std=d ** -0.5), normal(d, f, std=f ** -0.5)
        for q in ("1", "2") if layer["mlp"] is not None else ("1",):
            w[p + "norm" + q] = normal(d, std=0.2)
            w[p + "ls" + q] = 0.6 + normal(d, std=0.2)
            w[p + f"hc{q}.in"] = 1 / s + normal(s, std=0.3)
            w[p + f"hc{q}.out"] = 1 + normal(s, std=0.3)
            w[p + f"hc{q}.mix"] = torch.eye(s) + normal(s, s, std=0.15)
    return {k: v.to(torch.bfloat16).float() for k, v in w.items()}
