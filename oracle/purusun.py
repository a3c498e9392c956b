"""Plain statement of the Purusun decoder: one function per mechanism, sequential loops, no cache.

TEST INFRASTRUCTURE ONLY (see the package docstring).  Every function takes explicit tensors and computes in the dtype
it is given (the tests use float64); nothing is fused, chunked or shared with ``ajllm_amd``.  Tensor names are those of a
checkpoint: ``embed``, ``l<i>.norm1``, ``l<i>.mix.q``, ``l<i>.hc1.mix`` and so on.
"""

from __future__ import annotations

import math

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """Root of (mean square + eps) over the last dimension, kept as a column."""
    return torch.sqrt((x * x).sum(dim=-1, keepdim=True) / x.shape[-1] + eps)


def centered_rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """The stored weight is the gain's deviation from one."""
    return x / rms(x, eps) * (weight + 1)


def frequency(base: float, dims: int, i: int, scaling: dict | None) -> float:
    """Radians per position of pair i.  With ``scaling``: wavelengths up to original / high stay, those beyond
    original / low grow by ``factor``, and between them the two frequencies are blended linearly in original / wavelength."""
    f = base ** (-2.0 * i / dims)
    if scaling is None:
        return f
    wavelength = 2 * math.pi / f
    if wavelength < scaling["original"] / scaling["high"]:
        return f
    if wavelength > scaling["original"] / scaling["low"]:
        return f / scaling["factor"]
    share = (scaling["original"] / wavelength - scaling["low"]) / (scaling["high"] - scaling["low"])
    return (1 - share) * f / scaling["factor"] + share * f


def rotate(v: torch.Tensor, position: int, rot: dict) -> torch.Tensor:
    """One vector: component i turns against component i + dims / 2, the components from ``dims`` on pass."""
    out, half = v.clone(), rot["dims"] // 2
    for i in range(half):
        a = position * frequency(rot["base"], rot["dims"], i, rot.get("scaling"))
        c, s = math.cos(a), math.sin(a)
        out[..., i] = v[..., i] * c - v[..., i + half] * s
        out[..., i + half] = v[..., i + half] * c + v[..., i] * s
    return out


def rotate_rows(v: torch.Tensor, rot: dict) -> torch.Tensor:
    """``rotate`` of ``v [T, heads, dim]``, row t at position t."""
    return torch.stack([rotate(v[t], t, rot) for t in range(v.shape[0])])


def visible(i: int, j: int, window: int | None, keep_first: int) -> bool:
    """Whether position i reads position j: one of the last ``window`` up to itself, or one of the first ``keep_first``."""
    return j <= i and (window is None or i - j < window or j < keep_first)


def visible_mask(count: int, window: int | None, keep_first: int) -> torch.Tensor:
    i, j = torch.arange(count)[:, None], torch.arange(count)[None, :]
    near = torch.ones(count, count, dtype=torch.bool) if window is None else (i - j < window) | (j < keep_first)
    return (j <= i) & near


def softmax(scores: torch.Tensor) -> torch.Tensor:
    weights = torch.exp(scores - scores.amax(dim=-1, keepdim=True))
    return weights / weights.sum(dim=-1, keepdim=True)


def key_value_attention(h: torch.Tensor, w: dict[str, torch.Tensor], mixer: dict, eps: float) -> torch.Tensor:
    """Grouped-query attention whose values are the projected keys themselves, before their norm and rotation."""
    heads, groups, dim = mixer["heads"], mixer["kv_heads"], mixer["dim"]
    count = h.shape[0]
    q = (h @ w["q"].T).view(count, heads, dim)
    value = (h @ w["k"].T).view(count, groups, dim)
    q = rotate_rows(q / rms(q, eps) * w["q.norm"], mixer["rot"])
    key = rotate_rows(value / rms(value, eps) * w["k.norm"], mixer["rot"])
    mask = mixer.get("mask") or {}
    sees = visible_mask(count, mask.get("size"), mask.get("keep_first", 0))
    joined = []
    for n in range(heads):
        of = n // (heads // groups)
        scores = (q[:, n] @ key[:, of].T) * mixer["scale"]
        joined.append(softmax(scores.masked_fill(~sees, float("-inf"))) @ value[:, of])
    return (torch.cat(joined, dim=1) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def causal_conv(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """Per channel: out[t] = bias + sum_j weight[:, taps - 1 - j] x[t - j], zeros ahead of the sequence."""
    taps = weight.shape[1]
    out = []
    for t in range(x.shape[0]):
        total = bias.clone()
        for j in range(taps):
            if t - j >= 0:
                total = total + weight[:, taps - 1 - j] * x[t - j]
        out.append(total)
    return torch.stack(out)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.where(z > 0, z, torch.zeros_like(z)) + torch.log1p(torch.exp(-z.abs()))


def recurrence(x: torch.Tensor, dt: torch.Tensor, a: torch.Tensor, b: torch.Tensor, c: torch.Tensor, d: torch.Tensor,
               state: torch.Tensor | None = None) -> tuple[torch.Tensor, torch.Tensor]:
    """Token by token: S <- exp(dt A) S + (dt x) B^T per channel, y = S C + D x.  x, dt [T, channels]; a [channels, states];
    b, c [T, states].  Returns y and the last S."""
    s = torch.zeros_like(a) if state is None else state
    out = []
    for t in range(x.shape[0]):
        s = torch.exp(dt[t][:, None] * a) * s + (dt[t] * x[t])[:, None] * b[t][None, :]
        out.append(s @ c[t] + d * x[t])
    return torch.stack(out), s


def selective_scan(h: torch.Tensor, w: dict[str, torch.Tensor], mixer: dict) -> torch.Tensor:
    inner, n, r = mixer["inner"], mixer["state"], mixer["dt_rank"]
    both = h @ w["in"].T
    x, z = both[:, :inner], both[:, inner:]
    x = silu(causal_conv(x, w["conv"], w["conv.b"]))
    low = x @ w["x"].T
    dt = softplus(low[:, :r] @ w["dt"].T + w["dt.b"])
    y, _ = recurrence(x, dt, -torch.exp(w["A_log"]), low[:, r:r + n], low[:, r + n:], w["D"])
    return (y * silu(z)) @ w["o"].T


def squared_relu(h: torch.Tensor, up: torch.Tensor, down: torch.Tensor) -> torch.Tensor:
    return torch.relu(h @ up.T) ** 2 @ down.T


def hyper_sublayer(streams: torch.Tensor, hc: dict[str, torch.Tensor], body) -> torch.Tensor:
    """``streams [S, T, width]``: the sublayer reads one weighted sum of them; its result goes to every stream with a weight of
    its own, beside the streams mixed among themselves (mix[from, to])."""
    count = streams.shape[0]
    u = sum(hc["in"][s] * streams[s] for s in range(count))
    y = body(u)
    return torch.stack([sum(hc["mix"][s, t] * streams[s] for s in range(count)) + hc["out"][t] * y for t in range(count)])


def layer(streams: torch.Tensor, w: dict[str, torch.Tensor], spec: dict, eps: float) -> torch.Tensor:
    def part(prefix: str) -> dict[str, torch.Tensor]:
        return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}

    def mixer(u: torch.Tensor) -> torch.Tensor:
        h, mix = centered_rms_norm(u, w["norm1"], eps), part("mix.")
        y = key_value_attention(h, mix, spec["mixer"], eps) if spec["type"] == "attention" else selective_scan(h, mix, spec["mixer"])
        return y * w["ls1"]

    streams = hyper_sublayer(streams, part("hc1."), mixer)
    if spec.get("mlp") is not None:
        streams = hyper_sublayer(streams, part("hc2."), lambda u: squared_relu(
            centered_rms_norm(u, w["norm2"], eps), w["mlp.up"], w["mlp.down"]) * w["ls2"])
    return streams


def layer_order(layers: int, loop: dict | None) -> list[int]:
    """Layer indices in the order they run."""
    if not loop:
        return list(range(layers))
    inner = list(range(loop["start"], loop["stop"]))
    return list(range(loop["start"])) + inner * loop["times"] + list(range(loop["stop"], layers))


def forward(config: dict, weights: dict[str, torch.Tensor], tokens: list[int], dtype: torch.dtype = torch.float64,
            residuals: list[torch.Tensor] | None = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of a whole sequence; ``residuals`` collects the streams' sum after every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    e = torch.stack([w["embed"][t] for t in tokens])
    streams = torch.stack([e] * config["streams"])
    for index in layer_order(len(config["layers"]), config.get("loop")):
        prefix = f"l{index}."
        streams = layer(streams, {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}, config["layers"][index], eps)
        if residuals is not None:
            residuals.append(streams.sum(dim=0))
    return centered_rms_norm(streams.sum(dim=0), w["final.norm"], eps) @ w["embed"].T
