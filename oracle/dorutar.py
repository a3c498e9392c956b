"""Plain statement of the Dorutar decoder: one function per mechanism, a loop over everything, no cache.

TEST INFRASTRUCTURE ONLY (see the package docstring).  Every function takes explicit tensors and computes in
the dtype it is given (the tests use float64); nothing is fused, absorbed, windowed by slicing or shared with
``ajllm_amd``.  Tensor names are those of a checkpoint: ``embed``, ``pos``, ``loop.step``, ``l<i>.norm1``,
``l<i>.mix.q`` and so on.
"""

from __future__ import annotations

import math

import torch


def embedding(tokens: list[int], table: torch.Tensor, positions: torch.Tensor, first: int = 0) -> torch.Tensor:
    """E[token] + P[position], row by row."""
    return torch.stack([table[t] + positions[first + i] for i, t in enumerate(tokens)])


def layer_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """d / sqrt(mean(d^2) + eps) * weight with d = row - mean(row)."""
    out = []
    for row in x:
        deviation = row - row.sum() / len(row)
        out.append(deviation / torch.sqrt((deviation * deviation).sum() / len(row) + eps) * weight)
    return torch.stack(out)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    out = []
    for row in x:
        out.append(row / torch.sqrt((row * row).sum() / len(row) + eps) * weight)
    return torch.stack(out)


def rotate_halves(v: torch.Tensor, position: int, base: float, dims: int) -> torch.Tensor:
    """Rotate component i against component i + dims / 2 by ``position * base^(-2 i / dims)``; the rest passes."""
    out = v.clone()
    half = dims // 2
    for i in range(half):
        angle = position * base ** (-2.0 * i / dims)
        c, s = math.cos(angle), math.sin(angle)
        out[i] = v[i] * c - v[i + half] * s
        out[i + half] = v[i + half] * c + v[i] * s
    return out


def rotate_sequence(v: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """``rotate_halves`` of every row of ``v [T, ...]`` at its own position (vectorised over the rest)."""
    half = dims // 2
    t = torch.arange(v.shape[0], dtype=torch.float64)
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    angle = (t[:, None] * freq).view(v.shape[0], *([1] * (v.dim() - 2)), half)
    c, s = torch.cos(angle).to(v.dtype), torch.sin(angle).to(v.dtype)
    a, b = v[..., :half], v[..., half:dims]
    return torch.cat((a * c - b * s, b * c + a * s, v[..., dims:]), dim=-1)


def visible(i: int, j: int, window: int) -> bool:
    """Whether the query at position i reads the key at position j: the last ``window`` positions up to and including i."""
    return 0 <= i - j < window


def window_mask(count: int, window: int) -> torch.Tensor:
    i = torch.arange(count)
    distance = i[:, None] - i[None, :]
    return (distance >= 0) & (distance < window)


def softmax_with_sink(scores: torch.Tensor, sink: torch.Tensor | float) -> torch.Tensor:
    """Softmax of (scores, sink) along the last dimension without the sink's own weight; ``sink`` broadcasts over the rest."""
    sink = torch.as_tensor(sink, dtype=scores.dtype)
    top = torch.maximum(scores.amax(dim=-1), sink)
    weights = torch.exp(scores - top.unsqueeze(-1))
    return weights / (weights.sum(dim=-1) + torch.exp(sink - top)).unsqueeze(-1)


def latent_attention(h: torch.Tensor, w: dict[str, torch.Tensor], mixer: dict, eps: float) -> torch.Tensor:
    """The mixer on a whole sequence ``h [T, width]``; ``w``: its tensors by short name."""
    heads, dim, rot, vdim, rank = (mixer[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    count = h.shape[0]
    q = (h @ w["q"].T).view(count, heads, dim + rot)
    down = h @ w["dkv"].T
    latent = rms_norm(down[:, :rank], w["dkv.norm"], eps)
    key_rot = rotate_sequence(down[:, rank:], mixer["rot"]["base"], mixer["rot"]["dims"])
    q_rot = rotate_sequence(q[:, :, dim:], mixer["rot"]["base"], mixer["rot"]["dims"])
    key = (latent @ w["uk"].T).view(count, heads, dim)
    value = (latent @ w["uv"].T).view(count, heads, vdim)
    gate = torch.sigmoid(h @ w["g"].T)
    mask = window_mask(count, mixer["mask"]["size"])
    joined = []
    for n in range(heads):
        scores = (q[:, n, :dim] @ key[:, n].T + q_rot[:, n] @ key_rot.T) * mixer["scale"]
        weights = softmax_with_sink(scores.masked_fill(~mask, float("-inf")), w["sink"][n])
        joined.append((weights @ value[:, n]) * gate[:, n:n + 1])
    return torch.cat(joined, dim=1) @ w["o"].T


def gated_relu(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor) -> torch.Tensor:
    return (torch.relu(h @ gate.T) * (h @ up.T)) @ down.T


def parallel_layer(x: torch.Tensor, w: dict[str, torch.Tensor], layer: dict, eps: float) -> torch.Tensor:
    """Attention and feed-forward read the incoming stream, each through its own norm; both results join it at the end."""
    mix = {k[len("mix."):]: v for k, v in w.items() if k.startswith("mix.")}
    added = latent_attention(layer_norm(x, w["norm1"], eps), mix, layer["mixer"], eps)
    if layer.get("mlp") is not None:
        added = added + gated_relu(layer_norm(x, w["norm2"], eps), w["mlp.gate"], w["mlp.up"], w["mlp.down"])
    return x + added


def layer_runs(layers: int, loop: dict | None) -> list[tuple[int, int | None]]:
    """(layer, pass that starts with it or None) in the order they run."""
    if not loop:
        return [(i, None) for i in range(layers)]
    runs: list[tuple[int, int | None]] = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], layers)]


def forward(config: dict, weights: dict[str, torch.Tensor], tokens: list[int], dtype: torch.dtype = torch.float64,
            residuals: list[torch.Tensor] | None = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of a whole sequence; ``residuals`` collects the stream after every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x = embedding(tokens, w["embed"], w["pos"])
    embedded = x
    for index, begins in layer_runs(len(config["layers"]), config.get("loop")):
        if begins is not None:
            if begins > 0:
                x = x + embedded
            x = x + w["loop.step"][begins]
        prefix = f"l{index}."
        x = parallel_layer(x, {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)},
                           config["layers"][index], eps)
        if residuals is not None:
            residuals.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T
