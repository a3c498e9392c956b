"""What the dense (bf16 / fp32) decoders share: packing helpers, calls of ``libajq_dense.so`` that are not tied to one
mechanism, and ``DenseLM``, whose ``forward(token_ids, cache)`` is the one step function: whole prompts, portions of
prompts and single tokens; ``modeling.greedy_decode``, the decoders of ``decoding`` and ``trace`` call it.

All of it runs on a ROCm device, weights and activations in bf16 or fp32 (plain matrix products of prompts are the vendor
library's).  There is no CPU path.
"""

from __future__ import annotations

import ctypes
import math
from dataclasses import dataclass
from typing import Any

import torch
from torch import nn

from . import _lib
from .modeling import Linear, RMSNorm

GEMV_ROWS = 16    # rows of a prompt up to which the head's product is a matrix-vector kernel of this library
# rows up to which the decode products form the norms themselves (their workgroups each normalise every row: free at one
# row, 7 us of 55 at two, where a norm launch costs 3)
NORM_PROLOGUE_ROWS = 1


@dataclass(frozen=True)
class Loop:
    """Layers ``start .. stop - 1`` run ``times`` times in a row."""

    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class FrequencyScaling:
    """Rotary frequencies for sequences longer than those a model was trained on: wavelengths below ``original / high`` keep
    their frequency, those above ``original / low`` have it divided by ``factor``, and in between the two are blended."""

    factor: float
    low: float
    high: float
    original: float


def rotary_frequencies(base: float, dims: int, scaling: FrequencyScaling | None = None) -> torch.Tensor:
    """Radians per position of the ``dims / 2`` rotated pairs (double, on the host)."""
    f = torch.pow(torch.tensor(base, dtype=torch.float64), -2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
    if scaling is None:
        return f
    turns = scaling.original * f / (2 * math.pi)    # of the original length: original / wavelength
    share = ((turns - scaling.low) / (scaling.high - scaling.low)).clamp(0.0, 1.0) if scaling.high != scaling.low else (turns >= scaling.high).double()
    return (1.0 - share) * (f / scaling.factor) + share * f


def _up(n: int, to: int) -> int:
    return (n + to - 1) // to * to


def _padded(t: torch.Tensor, *sizes: int) -> torch.Tensor:
    """``t`` with zeros appended up to ``sizes``."""
    if tuple(t.shape) == sizes:
        return t.contiguous()
    out = torch.zeros(sizes, dtype=t.dtype, device=t.device)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def _ptr(t: torch.Tensor | None) -> int | None:
    return t.data_ptr() if t is not None else None


def _flag(dtype: torch.dtype) -> int:
    return _lib.AJQD_BF16 if dtype == torch.bfloat16 else _lib.AJQD_F32


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _product(x: torch.Tensor, w: torch.Tensor, out_dtype: torch.dtype) -> torch.Tensor:
    """``x w^T`` of many rows (the vendor library's product, fp32 accumulation)."""
    if x.dtype == out_dtype:
        return torch.mm(x, w.t())
    return torch.mm(x, w.t(), out_dtype=out_dtype)


def _add_norms(x: torch.Tensor, delta: torch.Tensor | None, again: torch.Tensor | None, step: torch.Tensor | None,
               gain1: torch.Tensor | None, gain2: torch.Tensor | None, eps: float, center: int, true_width: int,
               dtype: torch.dtype) -> tuple[torch.Tensor | None, torch.Tensor | None]:
    """``x += delta + again + step`` in place; the normed rows for each gain given."""
    out1 = torch.empty(x.shape, dtype=dtype, device=x.device) if gain1 is not None else None
    out2 = torch.empty(x.shape, dtype=dtype, device=x.device) if gain2 is not None else None
    _lib.check_dense(_lib.load_dense().ajqd_add_norms(
        _ptr(x), _ptr(delta), _flag(delta.dtype) if delta is not None else _lib.AJQD_F32, _ptr(again), _ptr(step), _ptr(gain1),
        _ptr(gain2), eps, center, _ptr(out1), _ptr(out2), x.shape[0], true_width, x.shape[1], _flag(dtype), _stream()), "add_norms")
    return out1, out2


def _matvec(w: torch.Tensor, groups: int, x: torch.Tensor, x_batch: int, x_group: int, y: torch.Tensor, y_batch: int,
            y_group: int, batch: int) -> None:
    """``y[b, g] = w[g] x[b, g]`` for ``w [groups * n, k]``; strides in elements."""
    _lib.check_dense(_lib.load_dense().ajqd_matvec(
        _ptr(w), _ptr(x), x_batch, x_group, _ptr(y), y_batch, y_group, groups, w.shape[0] // groups, w.shape[1], batch,
        _flag(w.dtype), _flag(y.dtype), _stream()), "matvec")


class DenseLM(nn.Module):
    """A decoder on the dense operators.  A subclass has ``vocab_size``, ``context_length``, ``d_model``, ``loop``,
    ``token_embeddings``, ``layers``, ``final_norm``, and fills in ``_pack`` (the weights as the kernels read them, with
    ``_head [vocab, width]`` and ``_final_gain [width]``, both padded), ``_prompt`` and ``_token`` (the residual rows behind the
    last layer run and what is still to be added to them), ``new_cache``, ``checkpoint_names`` and ``ignored_names``."""

    loop: Loop | None

    def _check_loop(self, layers: int) -> None:
        loop = self.loop
        if loop is not None and not (0 <= loop.start < loop.stop <= layers and loop.times >= 1):
            raise ValueError(f"the loop {loop} does not fit {layers} layers")

    # ---- structure
    @property
    def runs(self) -> list[tuple[int, int | None]]:
        """``(layer, pass)`` in running order; the pass is given on the layer run that begins it."""
        if self.loop is None:
            return [(i, None) for i in range(len(self.layers))]
        lo, hi = self.loop.start, self.loop.stop
        inner = [(i, t if i == lo else None) for t in range(self.loop.times) for i in range(lo, hi)]
        return [(i, None) for i in range(lo)] + inner + [(i, None) for i in range(hi, len(self.layers))]

    # ---- weights as the kernels read them
    def prepare(self) -> None:
        """(Re)build the packed weights from the parameters; done by itself at the first call.  Call it again after
        changing parameters in place."""
        name, weight = type(self).__name__, self.token_embeddings.weight
        if weight.dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("the model must be bfloat16 or float32")
        if weight.device.type != "cuda":
            raise ValueError(f"{name} runs on a ROCm device (there is no CPU path)")
        if any(not isinstance(m, Linear) for layer in self.layers for m in layer.modules() if hasattr(m, "in_features")):
            raise ValueError(f"{name} runs on dense weights (its linears have been replaced)")
        if any(p.dtype != weight.dtype or p.device != weight.device for p in self.parameters()):
            raise ValueError("all parameters must share one dtype and device")
        with torch.no_grad():
            self._pack()
        self._packed = (weight.data_ptr(), weight.dtype, weight.device)

    def _pack(self) -> None:
        raise NotImplementedError

    def _ready(self) -> None:
        weight = self.token_embeddings.weight
        if getattr(self, "_packed", None) != (weight.data_ptr(), weight.dtype, weight.device):
            self.prepare()

    def _prompt(self, token_ids: torch.Tensor, cache, start: int, residuals: list | None) -> tuple[torch.Tensor, torch.Tensor | None]:
        raise NotImplementedError

    def _token(self, token_ids: torch.Tensor, cache) -> tuple[torch.Tensor, torch.Tensor | None]:
        raise NotImplementedError

    # ---- the step
    @torch.no_grad()
    def forward(self, token_ids: torch.Tensor, cache: Any | None = None, last_token_only: bool = False,
                want: torch.Tensor | None = None, residuals: list | None = None) -> torch.Tensor:
        """Logits (fp32) ``[B, n, V]`` of the new tokens ``token_ids [B, T]``, which continue at ``cache.length``
        (``cache.position`` for a static cache).  ``last_token_only``, or ``want`` (a list of places among the T tokens,
        possibly empty) selects the places whose logits are formed.  ``residuals`` collects copies of the residual
        stream after every layer run (prompts only)."""
        batch, seq = token_ids.shape
        self._ready()
        if not token_ids.is_cuda:
            raise ValueError("the model takes token ids on the model's device")
        token_ids = token_ids.contiguous()
        static = cache is not None and cache.static
        if static and seq != 1:
            raise ValueError("a static cache takes one token per call")
        if cache is not None and cache.batch != batch:
            raise ValueError(f"the cache holds {cache.batch} sequences, {batch} given")
        start = cache.length if cache is not None and not static else 0
        if not static and start + seq > self.context_length:
            raise ValueError(f"Input length {start + seq} exceeds context length {self.context_length}")
        if not static and cache is not None and start + seq > cache.max_len:
            raise ValueError(f"the cache holds {cache.max_len} positions, {start + seq} needed")
        single = cache is not None and seq == 1 and residuals is None
        if single:
            if not static:
                cache.position.fill_(start)
            x, delta = self._token(token_ids, cache)
        else:
            x, delta = self._prompt(token_ids, cache, start, residuals)
        if cache is not None and not static:
            cache.length = start + seq
        if last_token_only:
            want = [seq - 1]
        if want is not None:
            picks = list(want)
            if not picks:
                return torch.empty((batch, 0, self.vocab_size), dtype=torch.float32, device=x.device)
            if not (seq == 1 and len(picks) == 1):
                rows = torch.tensor([b * seq + t for b in range(batch) for t in picks], device=x.device)
                x = x.index_select(0, rows)
                delta = delta.index_select(0, rows) if delta is not None else None
        return self._logits(x, delta, single).view(batch, -1, self._head.shape[0])[:, :, : self.vocab_size]

    def _logits(self, x: torch.Tensor, delta: torch.Tensor | None, single: bool) -> torch.Tensor:
        """``head norm(x + delta)``, fp32, columns padded to a multiple of 16.  ``single``: a decode step (its products are
        this library's for any number of sequences: library kernels stay out of recorded graphs)."""
        rows, dtype = x.shape[0], self._head.dtype
        if not single and rows > GEMV_ROWS:
            normed, _ = _add_norms(x, delta, None, None, self._final_gain, None, self.final_norm.epsilon,
                                   0 if isinstance(self.final_norm, RMSNorm) else 1, self.d_model, dtype)
            return _product(normed, self._head, torch.float32)
        center = 0 if isinstance(self.final_norm, RMSNorm) else 1
        eps, gain = self.final_norm.epsilon, self._final_gain
        y = torch.empty((rows, self._head.shape[0]), dtype=torch.float32, device=x.device)
        if dtype == torch.bfloat16:
            if delta is None and rows <= NORM_PROLOGUE_ROWS:
                self._dense_in(x, None, None, gain, None, eps, center, self._head, None, y, None, 0, 0)
                return y
            normed, _ = _add_norms(x, delta, None, None, gain, None, eps, center, self.d_model, dtype)
            self._dense_in(None, normed, None, None, None, eps, center, self._head, None, y, None, 0, 0)
            return y
        normed, _ = _add_norms(x, delta, None, None, gain, None, eps, center, self.d_model, dtype)
        _matvec(self._head, 1, normed, normed.shape[1], 0, y, y.shape[1], 0, rows)
        return y

    def _dense_in(self, x, n1, n2, gain1, gain2, eps, center, w1, w2, y1, gated, gated_ld, act, pairs: bool = True) -> None:
        """``y1 = norm1(x) w1^T`` and the activated ``norm2(x) w2^T`` of one decode step in one launch; either matrix may be None."""
        rows, w = next(t for t in (x, n1, n2) if t is not None), w1 if w1 is not None else w2
        batch = rows.shape[0]
        args = _lib.DenseInArgs(
            x=_ptr(x), n1=_ptr(n1), n2=_ptr(n2), gain1=_ptr(gain1), gain2=_ptr(gain2), w1=_ptr(w1), w2=_ptr(w2), y1=_ptr(y1),
            gated=gated, batch=batch, true_width=self.d_model, width=w.shape[1],
            tiles1=w1.shape[0] // 16 if w1 is not None else 0,
            tiles2=w2.shape[0] // 16 if w2 is not None else 0, gated_ld=gated_ld, act=act, center=center,
            pairs=int(pairs), eps=eps)
        _lib.check_dense(_lib.load_dense().ajqd_dense_in(ctypes.byref(args), _stream()), "dense_in")
