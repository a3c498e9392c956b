"""Small random models of the Dorutar architecture for the tests."""

from __future__ import annotations

import torch


def config(layers: int = 3, width: int = 48, heads: int = 4, dim: int = 16, rot: int = 8, vdim: int = 24, rank: int = 32,
           ff: int = 56, vocab: int = 67, positions: int = 512, window=11, base: float = 900.0, eps: float = 2e-5,
           loop: dict | None = {"start": 1, "stop": 2, "times": 3}, mlp_missing: tuple[int, ...] = (), scale: float | None = None) -> dict:
    """``window``: one for all layers or a list."""
    windows = window if isinstance(window, list) else [window] * layers
    out = {
        "architecture": "Dorutar", "vocab": vocab, "width": width, "max_positions": positions, "norm": {"eps": eps},
        "layers": [{"type": "latent_attention",
                    "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
                              "scale": scale or 1.3 * (dim + rot) ** -0.5, "mask": {"size": windows[i]},
                              "rot": {"base": base, "dims": rot}},
                    "mlp": None if i in mlp_missing else {"kind": "dense", "ff": ff}} for i in range(layers)],
        "loop": loop,
    }
    return out


def random_weights(cfg: dict, seed: int, spread: float = 1.0) -> dict[str, torch.Tensor]:
    """Seeded weights, values exactly representable in bf16.  ``spread`` scales queries and keys (larger: sharper scores)."""
    g = torch.Generator().manual_seed(seed)

    def normal(*shape: int, std: float = 1.0) -> torch.Tensor:
        return (torch.randn(shape, generator=g) * std).to(torch.bfloat16).float()

    d = cfg["width"]
    w = {"embed": normal(cfg["vocab"], d), "pos": normal(cfg["max_positions"], d, std=0.3),
         "final.norm": 1 + normal(d, std=0.1), "head": normal(cfg["vocab"], d, std=d ** -0.5)}
    if cfg.get("loop"):
        w["loop.step"] = normal(cfg["loop"]["times"], d, std=0.5)
    for i, layer in enumerate(cfg["layers"]):
        m = layer["mixer"]
        h, dim, rot, vdim, rank = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        p = f"l{i}."
        w[p + "norm1"] = 1 + normal(d, std=0.2)
        w[p + "mix.q"] = normal(h * (dim + rot), d, std=spread * d ** -0.5)
        w[p + "mix.dkv"] = normal(rank + rot, d, std=spread * d ** -0.5)
        w[p + "mix.dkv.norm"] = 1 + normal(rank, std=0.2)
        w[p + "mix.uk"] = normal(h * dim, rank, std=spread * rank ** -0.5)
        w[p + "mix.uv"] = normal(h * vdim, rank, std=rank ** -0.5)
        w[p + "mix.sink"] = normal(h)
        w[p + "mix.g"] = normal(h, d, std=d ** -0.5)
        w[p + "mix.o"] = normal(d, h * vdim, std=(h * vdim) ** -0.5)
        if layer["mlp"] is not None:
            f = layer["mlp"]["ff"]
            w[p + "norm2"] = 1 + normal(d, std=0.2)
            w[p + "mlp.gate"] = normal(f, d, std=d ** -0.5)
            w[p + "mlp.up"] = normal(f, d, std=d ** -0.5)
            w[p + "mlp.down"] = normal(d, f, std=f ** -0.5)
    return {k: v.to(torch.bfloat16).float() for k, v in w.items()}
