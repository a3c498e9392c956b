"""Dense decoder whose layers mix attention and selective-scan mixers on hyper-connected residual streams.

One architecture is registered here, ``Purusun``; its mechanisms are modules of their own with their constants as
arguments:

* ``KeyValueAttention``  grouped-query attention whose values are the projected keys; query and key norms, rotary positions
                         on the first dimensions of a head (with frequency scaling), a sliding window beside first tokens
                         that stay visible, a sigmoid gate per output column
* ``SelectiveScan``      a Mamba mixer: short causal convolution, then a diagonal recurrence whose step size, input and output
                         weights depend on the token
* ``HyperConnection``    how one sublayer reads from and writes to several residual streams
* ``HybridBlock``        mixer and feed-forward, each between a norm of its own and a scale per column
* ``HybridLM``           the decoder (``dense.DenseLM``); a ``dense.Loop`` gives every pass rings and states of its own

Whatever the dtype, fp32: residual streams, norms, angles, attention scores and sums, gates, step sizes, decays and states.

A prompt runs on the vendor library's products with this library's kernels between them.  A single token runs on matrix-
vector kernels with what surrounds them folded in: the product that ends a sublayer updates all streams and forms the next
sublayer's input; attention treats a key / value head as a sequence of its own for the latent decode kernel (a cache row is
value and key at once); the scan's projection convolves its own operands.
"""

from __future__ import annotations

import ctypes
import math
from typing import Any

import torch
from torch import nn

from . import _lib
from .dense import (NORM_PROLOGUE_ROWS, DenseLM, FrequencyScaling, Loop, _add_norms, _flag, _matvec, _padded, _product, _ptr,
                    _stream, _up, rotary_frequencies)
from .modeling import Embedding, Linear, PlainFeedForward, RingCache, RMSNorm, build_feed_forward, build_norm, register_architecture

UNBOUNDED = 1 << 30   # context length of a model without a position table


class KeyValueAttention(nn.Module):
    def __init__(self, d_model: int, num_heads: int, num_kv_heads: int, dim: int, scale: float, rot_dim: int, rot_base: float,
                 scaling: FrequencyScaling | None = None, window: int | None = None, keep_first: int = 0, epsilon: float = 1e-5) -> None:
        super().__init__()
        if num_heads % num_kv_heads != 0:
            raise ValueError("num_heads must be divisible by num_kv_heads")
        if rot_dim % 2 != 0 or not 0 <= rot_dim <= dim:
            raise ValueError("the rotated width must be even and at most the head's")
        if window is not None and window < 1:
            raise ValueError("the window must hold at least the token itself")
        if keep_first < 0:
            raise ValueError("keep_first must not be negative")
        self.num_heads, self.num_kv_heads, self.dim = num_heads, num_kv_heads, dim
        self.scale, self.rot_dim, self.rot_base, self.scaling = float(scale), rot_dim, float(rot_base), scaling
        self.window, self.keep_first = window, keep_first if window is not None else 0
        self.q_proj = Linear(d_model, num_heads * dim)
        self.k_proj = Linear(d_model, num_kv_heads * dim)    # keys, and before their norm the values
        self.q_norm = RMSNorm(dim, epsilon)
        self.k_norm = RMSNorm(dim, epsilon)
        self.gate_proj = Linear(d_model, num_heads * dim)
        self.output_proj = Linear(num_heads * dim, d_model)


class SelectiveScan(nn.Module):
    def __init__(self, d_model: int, inner: int, state: int, dt_rank: int, conv: int) -> None:
        super().__init__()
        if min(inner, state, dt_rank, conv) < 1:
            raise ValueError("the sizes of a selective scan must be positive")
        self.inner, self.state, self.dt_rank, self.conv = inner, state, dt_rank, conv
        self.in_proj = Linear(d_model, 2 * inner)             # convolved half, gate half
        self.conv_weight = nn.Parameter(torch.randn(inner, conv) * conv ** -0.5)   # last column: the current token's
        self.conv_bias = nn.Parameter(torch.zeros(inner))
        self.x_proj = Linear(inner, dt_rank + 2 * state)      # step size, input weights, output weights
        self.dt_proj = Linear(dt_rank, inner)
        self.dt_bias = nn.Parameter(torch.full((inner,), -4.6))   # softplus: steps of about 0.01
        self.a_log = nn.Parameter(torch.log(torch.arange(1, state + 1, dtype=torch.float32)).repeat(inner, 1))
        self.skip = nn.Parameter(torch.ones(inner))
        self.output_proj = Linear(inner, d_model)


class HyperConnection(nn.Module):
    """A sublayer reads sum_s reads[s] x_s; with its result y, x_t becomes sum_s mix[s, t] x_s + writes[t] y."""

    def __init__(self, streams: int) -> None:
        super().__init__()
        self.reads = nn.Parameter(torch.full((streams,), 1.0 / streams))
        self.writes = nn.Parameter(torch.ones(streams))
        self.mix = nn.Parameter(torch.eye(streams))


class HybridBlock(nn.Module):
    def __init__(self, d_model: int, mixer: nn.Module, feed_forward: PlainFeedForward | None, streams: int, norm: str, epsilon: float) -> None:
        super().__init__()
        self.norm1 = build_norm(norm, d_model, epsilon)
        self.mixer = mixer
        self.scale1 = nn.Parameter(torch.ones(d_model))
        self.hyper1 = HyperConnection(streams)
        self.feed_forward = feed_forward
        has = feed_forward is not None
        self.norm2 = build_norm(norm, d_model, epsilon) if has else None
        self.scale2 = nn.Parameter(torch.ones(d_model)) if has else None
        self.hyper2 = HyperConnection(streams) if has else None


def _f32(t: torch.Tensor, *sizes: int) -> torch.Tensor:
    return _padded(t.detach().float(), *sizes)


def _gain(norm: RMSNorm, width: int) -> torch.Tensor:
    """The factors a norm applies, fp32, padded."""
    return _f32(norm.weight.detach().float() + (1.0 if norm.zero_centered else 0.0), width)


def state_planes(t: torch.Tensor) -> torch.Tensor:
    """``[.., channels, states]`` -> ``[.., states / 4, channels, 4]``, as the scan kernels read states and decays."""
    *lead, channels, states = t.shape
    return t.view(*lead, channels, states // 4, 4).transpose(-3, -2).contiguous()


class PackedSublayer:
    """What the stream kernels need of one sublayer: its norm's gain, its column scale, its coefficients (fp32)."""

    def __init__(self, norm: RMSNorm, scale: torch.Tensor, hyper: HyperConnection, width: int) -> None:
        self.gain, self.eps = _gain(norm, width), norm.epsilon
        self.scale = _f32(scale, width)
        self.reads, self.writes, self.mix = (_f32(t, *t.shape) for t in (hyper.reads, hyper.writes, hyper.mix))


class PackedAttention:
    """Projections that share the input stacked into one matrix (queries, keys, gates), heads padded to 16 columns."""

    def __init__(self, mix: KeyValueAttention, width: int) -> None:
        heads, groups, dim = mix.num_heads, mix.num_kv_heads, mix.dim
        d = mix.q_proj.weight.shape[1]
        self.heads, self.groups, self.dim, self.dimp = heads, groups, dim, _up(dim, 16)
        self.share, self.rot, self.scale = heads // groups, mix.rot_dim, mix.scale
        self.window, self.keep, self.row = mix.window, mix.keep_first, 2 * self.dimp

        def stacked(linear: Linear, count: int) -> torch.Tensor:
            return _padded(linear.weight.detach().view(count, dim, d), count, self.dimp, width).view(-1, width)

        self.w_in = torch.cat((stacked(mix.q_proj, heads), stacked(mix.k_proj, groups), stacked(mix.gate_proj, heads)), dim=0).contiguous()
        self.gate_column = (heads + groups) * self.dimp
        out = mix.output_proj.weight.detach()
        self.w_out = _padded(out.view(d, heads, dim), width, heads, self.dimp).view(width, -1)
        self.q_gain, self.k_gain, self.eps = _gain(mix.q_norm, self.dimp), _gain(mix.k_norm, self.dimp), mix.q_norm.epsilon
        self.half_turns = (rotary_frequencies(mix.rot_base, mix.rot_dim, mix.scaling) / math.pi).to(out.device)


class PackedScan:
    """Widths padded to 16 channels, 8 columns of the step size's rank, 4 states; see ``state_planes``."""

    def __init__(self, mix: SelectiveScan, width: int) -> None:
        inner, n, r = mix.inner, mix.state, mix.dt_rank
        d = mix.in_proj.weight.shape[1]
        self.inner, self.states, self.rank, self.taps = _up(inner, 16), _up(n, 4), _up(r, 8), mix.conv
        self.w_in = _padded(mix.in_proj.weight.detach().view(2, inner, d), 2, self.inner, width).view(-1, width)
        self.conv = _f32(mix.conv_weight.detach().t(), self.taps, self.inner)
        self.conv_bias, self.dt_bias, self.skip = (_f32(t, self.inner) for t in (mix.conv_bias, mix.dt_bias, mix.skip))
        low = mix.x_proj.weight.detach()
        parts = [_padded(low[:r], self.rank, self.inner), _padded(low[r:r + n], self.states, self.inner), _padded(low[r + n:], self.states, self.inner)]
        self.low_rows = _up(self.rank + 2 * self.states, 16)
        self.w_low = _padded(torch.cat(parts, dim=0), self.low_rows, self.inner)
        self.w_dt = _padded(mix.dt_proj.weight.detach(), self.inner, self.rank)
        decay = -torch.exp(mix.a_log.detach().double()) * math.log2(math.e)
        self.a2 = state_planes(_f32(decay, self.inner, self.states))
        self.w_out = _padded(mix.output_proj.weight.detach(), width, self.inner)


class PackedFeedForward:
    def __init__(self, ff: PlainFeedForward, width: int) -> None:
        self.width = _up(ff.w1.weight.shape[0], 16)
        self.act = _lib.AJQD_ACTIVATIONS[ff.activation]
        self.w_in = _padded(ff.w1.weight.detach(), self.width, width)
        self.w_out = _padded(ff.w2.weight.detach(), width, self.width)


class HybridLM(DenseLM):
    """The decoder.  ``blocks``: one ``(mixer kind, its arguments, feed-forward (width, kind) or None)`` per layer; kinds as in
    ``MIXERS`` and ``modeling.build_feed_forward``.  The head is the embedding table."""

    MIXERS = {"attention": KeyValueAttention, "mamba1": SelectiveScan}

    def __init__(self, vocab_size: int, d_model: int, streams: int, blocks: list[tuple[str, dict[str, Any], tuple[int, str] | None]],
                 loop: Loop | None = None, norm: str = "zero_centered_rmsnorm", epsilon: float = 1e-5, context_length: int = UNBOUNDED) -> None:
        super().__init__()
        self.vocab_size, self.context_length, self.d_model, self.streams, self.loop = vocab_size, context_length, d_model, streams, loop
        self._check_loop(len(blocks))
        self.token_embeddings = Embedding(vocab_size, d_model)
        self.layers = nn.ModuleList()
        for kind, mixer, ff in blocks:
            if kind == "attention":
                mixer = {"epsilon": epsilon, **mixer}
            self.layers.append(HybridBlock(d_model, self.MIXERS[kind](d_model, **mixer),
                                           build_feed_forward(ff[1], d_model, ff[0]) if ff is not None else None, streams, norm, epsilon))
        self.final_norm = build_norm(norm, d_model, epsilon)

    # ---- structure
    def checkpoint_names(self) -> dict[str, str]:
        """State-dict key -> tensor name in a checkpoint file."""
        names = {"token_embeddings.weight": "embed", "final_norm.weight": "final.norm"}
        parts = {"norm1.weight": "norm1", "norm2.weight": "norm2", "scale1": "ls1", "scale2": "ls2", "feed_forward.w1.weight": "mlp.up",
                 "feed_forward.w2.weight": "mlp.down", "mixer.q_proj.weight": "mix.q", "mixer.k_proj.weight": "mix.k",
                 "mixer.q_norm.weight": "mix.q.norm", "mixer.k_norm.weight": "mix.k.norm", "mixer.gate_proj.weight": "mix.g",
                 "mixer.output_proj.weight": "mix.o", "mixer.in_proj.weight": "mix.in", "mixer.conv_weight": "mix.conv",
                 "mixer.conv_bias": "mix.conv.b", "mixer.x_proj.weight": "mix.x", "mixer.dt_proj.weight": "mix.dt", "mixer.dt_bias": "mix.dt.b",
                 "mixer.a_log": "mix.A_log", "mixer.skip": "mix.D"}
        for q in ("1", "2"):
            parts.update({f"hyper{q}.reads": f"hc{q}.in", f"hyper{q}.writes": f"hc{q}.out", f"hyper{q}.mix": f"hc{q}.mix"})
        for key in self.state_dict():
            if key.startswith("layers."):
                _, index, part = key.split(".", 2)
                names[key] = f"l{index}.{parts[part]}"
        return names

    def ignored_names(self) -> set[str]:
        """Tensors a checkpoint may hold that no layer reads: what belongs to the second sublayer of a layer without one."""
        return {f"l{i}.{name}" for i, layer in enumerate(self.layers) if layer.feed_forward is None
                for name in ("norm2", "ls2", "hc2.in", "hc2.out", "hc2.mix")}

    def new_cache(self, batch: int, max_len: int | None = None, dtype: torch.dtype | None = None) -> RingCache:
        """An empty cache: rows of keys and values in the activations' dtype for attention (a ring per key / value head), the last
        columns of the convolution and the fp32 states for a scan."""
        weight = self.token_embeddings.weight
        if dtype is not None and dtype != weight.dtype:
            raise ValueError("the cache has the model's own dtype")
        max_len = max_len or self.context_length
        if max_len >= UNBOUNDED:
            raise ValueError("this model has no longest sequence of its own: give max_len")
        capacities, widths, groups, kept, states = [], [], [], [], []
        for i, _ in self.runs:
            m = self.layers[i].mixer
            if isinstance(m, KeyValueAttention):
                reach = max_len if m.window is None else min(m.window + m.keep_first, max_len)
                capacities.append(reach)
                widths.append(2 * _up(m.dim, 16))
                groups.append(m.num_kv_heads)
                kept.append(m.keep_first if reach > m.keep_first else 0)   # (a shorter cache never wraps)
                states.append(None)
            else:
                capacities.append(m.conv - 1)
                widths.append(_up(m.inner, 16))
                groups.append(None)
                kept.append(0)
                states.append((_up(m.state, 4) // 4, _up(m.inner, 16), 4))
        return RingCache(capacities, widths, batch, max_len, weight.device, weight.dtype, groups, kept, states)

    def _pack(self) -> None:
        dp = _up(self.d_model, 16)
        self._embed = self._head = _padded(self.token_embeddings.weight.detach(), _up(self.vocab_size, 16), dp)
        self._final_gain = _gain(self.final_norm, dp)
        self._mixers, self._forwards, self._subs = [], [], []
        for layer in self.layers:
            packed = PackedAttention if isinstance(layer.mixer, KeyValueAttention) else PackedScan
            self._mixers.append(packed(layer.mixer, dp))
            self._subs.append([PackedSublayer(layer.norm1, layer.scale1, layer.hyper1, dp)])
            self._forwards.append(None)
            if layer.feed_forward is not None:
                self._forwards[-1] = PackedFeedForward(layer.feed_forward, dp)
                self._subs[-1].append(PackedSublayer(layer.norm2, layer.scale2, layer.hyper2, dp))

    def _sublayers(self) -> list[tuple[int, Any, PackedSublayer]]:
        """``(run, packed mixer or feed-forward, sublayer)`` in running order."""
        order = []
        for run, (i, _) in enumerate(self.runs):
            order.append((run, self._mixers[i], self._subs[i][0]))
            if self._forwards[i] is not None:
                order.append((run, self._forwards[i], self._subs[i][1]))
        return order

    # ---- residual streams
    def _start(self, token_ids: torch.Tensor, first: PackedSublayer, want_u: bool) -> tuple[torch.Tensor, torch.Tensor | None]:
        """Streams ``[rows, streams, width]`` holding the embedding, and the first sublayer's input where it is asked for."""
        rows, dp = token_ids.numel(), self._embed.shape[1]
        x = torch.empty((rows, self.streams, dp), dtype=torch.float32, device=self._embed.device)
        u = torch.empty((rows, dp), dtype=torch.float32, device=x.device) if want_u else None
        _lib.check_dense(_lib.load_dense().ajqd_embed_streams(
            _ptr(token_ids), rows, _ptr(self._embed), self.vocab_size, _ptr(first.reads), _ptr(x), _ptr(u), self.streams, dp,
            _flag(self._embed.dtype), _stream()), "embed_streams")
        return x, u

    def _streams_norm(self, x: torch.Tensor, delta: torch.Tensor | None, done: PackedSublayer | None,
                      sub: PackedSublayer | None) -> torch.Tensor:
        """The result ``delta`` of sublayer ``done`` joins the streams; then the normed input of ``sub``, or (None) the streams'
        sum in fp32."""
        rows, streams, dp = x.shape
        out = torch.empty((rows, dp), dtype=self._embed.dtype if sub is not None else torch.float32, device=x.device)
        _lib.check_dense(_lib.load_dense().ajqd_streams_norm(
            _ptr(x), _ptr(delta), *((_ptr(done.scale), _ptr(done.writes), _ptr(done.mix)) if delta is not None else (None,) * 3),
            *((_ptr(sub.reads), _ptr(sub.gain), sub.eps, _ptr(out), None) if sub is not None else (None, None, 0.0, None, _ptr(out))),
            streams, rows, self.d_model, dp, _flag(self._embed.dtype), _stream()), "streams_norm")
        return out

    # ---- many tokens per sequence
    def _prompt(self, token_ids: torch.Tensor, cache: RingCache | None, start: int, residuals: list | None) -> tuple[torch.Tensor, None]:
        batch, seq = token_ids.shape
        order = self._sublayers()
        x, _ = self._start(token_ids, order[0][2], False)
        delta, done = None, None
        for k, (run, w, sub) in enumerate(order):
            h = self._streams_norm(x, delta, done, sub)
            if isinstance(w, PackedAttention):
                mixed = self._attend(h, w, cache, run, batch, seq, start)
            elif isinstance(w, PackedScan):
                mixed = self._scan(h, w, cache, run, batch, seq, start)
            else:
                mixed = self._activated(_product(h, w.w_in, h.dtype), w.act)
            delta, done = _product(mixed, w.w_out, torch.float32), sub
            if residuals is not None and (k + 1 == len(order) or order[k + 1][0] != run):
                total = (sub.mix.sum(dim=1)[:, None] * x).sum(dim=1) + sub.writes.sum() * (sub.scale * delta)
                residuals.append(total[:, : self.d_model].view(batch, seq, -1))
        return self._streams_norm(x, delta, done, None), None

    def _activated(self, y: torch.Tensor, act: int) -> torch.Tensor:
        _lib.check_dense(_lib.load_dense().ajqd_activation(_ptr(y), _ptr(y), y.numel(), act, _flag(y.dtype), _stream()), "activation")
        return y

    def _split(self, y: torch.Tensor, w: PackedAttention, q: torch.Tensor, q_at: int, rows: torch.Tensor, seq: int, start: int,
               pos: torch.Tensor | None, prior: int, kept: int) -> None:
        """Queries into ``q [.., heads, columns]``; keys and values into ``rows [B, groups, slots, row]``."""
        args = _lib.KeyValueSplitArgs(
            y=_ptr(y), q_gain=_ptr(w.q_gain), k_gain=_ptr(w.k_gain), half_turns=_ptr(w.half_turns), pos=_ptr(pos), q=_ptr(q), rows=_ptr(rows),
            rows_batch=rows.stride(0), rows_head=rows.stride(1), tokens=y.shape[0], seq=seq, start=start, ldy=y.shape[1], heads=w.heads,
            groups=w.groups, dim=w.dim, dimp=w.dimp, rot=w.rot, q_ld=q.shape[-1], q_at=q_at, prior=prior, cap=rows.shape[2], kept=kept, eps=w.eps)
        _lib.check_dense(_lib.load_dense().ajqd_key_value_split(ctypes.byref(args), _flag(y.dtype), _flag(q.dtype), _stream()), "key_value_split")

    def _windowed(self, w: PackedAttention, q: torch.Tensor, rows: torch.Tensor, y: torch.Tensor, seq: int, prior: int,
                  pos: torch.Tensor | None) -> torch.Tensor:
        """Attention of ``q`` on key / value ``rows``, gated by the gate columns of ``y``."""
        size, lib = rows.element_size(), _lib.load_dense()
        out = torch.empty((q.shape[0], w.heads * w.dimp), dtype=q.dtype, device=q.device)
        window = 0 if w.window is None or pos is not None else w.window
        args = _lib.WindowedAttentionArgs(
            q=_ptr(q), k1=rows.data_ptr() + w.dimp * size, v=_ptr(rows), column_gates=y.data_ptr() + w.gate_column * size, pos=_ptr(pos),
            out=_ptr(out), k1_batch=rows.stride(0), v_batch=rows.stride(0), k1_head=rows.stride(1), v_head=rows.stride(1), k1_row=w.row,
            v_row=w.row, d1=w.dimp, d2=0, dv=w.dimp, batch=rows.shape[0], heads=w.heads, share=w.share, seq=seq, rows=rows.shape[2],
            prior=prior, window=window, keep=w.keep if window else 0, gate_ld=y.shape[1], out_ld=out.shape[1], scale=w.scale)
        if pos is None and q.dtype == torch.bfloat16 and lib.ajqd_windowed_prefill_supported(w.dimp, 0, w.dimp):
            _lib.check_dense(lib.ajqd_windowed_prefill(ctypes.byref(args), _stream()), "windowed_prefill")
        else:
            _lib.check_dense(lib.ajqd_windowed_attention(ctypes.byref(args), _flag(q.dtype), _flag(q.dtype), _stream()), "windowed_attention")
        return out

    def _attend(self, h: torch.Tensor, w: PackedAttention, cache: RingCache | None, run: int, batch: int, seq: int, start: int) -> torch.Tensor:
        lib, st, dtype, dev = _lib.load_dense(), _stream(), h.dtype, h.device
        y = _product(h, w.w_in, dtype)
        # rows in reach of the first new token: the first ones that stay (as far as the window does not reach them), the
        # window's, then the new ones; a row below `keep` is a position below `keep` either way
        reach = start if w.window is None else min(start, w.window - 1)
        stay = min(w.keep, start - reach)
        prior = stay + reach
        rows = torch.empty((batch, w.groups, prior + seq, w.row), dtype=dtype, device=dev)
        ring = cache.rings[run] if cache is not None else None
        row_bytes = w.row * rows.element_size()

        def copy(first_row: int, position: int, count: int, to_ring: int) -> None:
            if count > 0:
                _lib.check_dense(lib.ajqd_ring_copy(_ptr(ring), ring.shape[2], cache.kept[run], _ptr(rows), prior + seq, row_bytes, first_row,
                                                    position, count, row_bytes, batch * w.groups, to_ring, st), "ring_copy")

        copy(0, 0, stay, 0)
        copy(stay, start - reach, reach, 0)
        q = torch.empty((batch * seq, w.heads, w.dimp), dtype=dtype, device=dev)
        self._split(y, w, q, 0, rows, seq, start, None, prior, 0)
        out = self._windowed(w, q, rows, y, seq, prior, None)
        if ring is not None:
            end, kept = start + seq, cache.kept[run]
            copy(prior, start, min(kept, end) - start, 1)                      # first positions that stay
            from_ = max(start, kept, end - (ring.shape[2] - kept))             # the last ones of the others
            copy(prior + from_ - start, from_, end - from_, 1)
        return out

    def _scan(self, h: torch.Tensor, w: PackedScan, cache: RingCache | None, run: int, batch: int, seq: int, start: int) -> torch.Tensor:
        y = _product(h, w.w_in, h.dtype)
        ring, state = (cache.rings[run], cache.states[run]) if cache is not None else (None, None)
        x = self._convolved(y, w, ring, start, None, seq)
        low = _product(x, w.w_low, h.dtype)
        raw = torch.mm(low[:, : w.rank], w.w_dt.t())
        out = self._recur(x, raw, low, y, w, state, batch, seq, start, None)
        keep = min(seq, w.taps - 1)
        if ring is not None and keep > 0:
            size = y.element_size()
            _lib.check_dense(_lib.load_dense().ajqd_ring_copy(
                _ptr(ring), ring.shape[1], 0, _ptr(y), seq, y.shape[1] * size, seq - keep, start + seq - keep, keep, w.inner * size, batch, 1,
                _stream()), "ring_copy")
        return out

    def _convolved(self, y: torch.Tensor, w: PackedScan, ring: torch.Tensor | None, start: int, pos: torch.Tensor | None, seq: int) -> torch.Tensor:
        x = torch.empty((y.shape[0], w.inner), dtype=y.dtype, device=y.device)
        _lib.check_dense(_lib.load_dense().ajqd_conv_silu(
            _ptr(y), y.shape[1], _ptr(ring) if w.taps > 1 else None, _ptr(w.conv), _ptr(w.conv_bias), start, _ptr(pos), y.shape[0], seq, w.inner,
            w.taps, _ptr(x), _flag(y.dtype), _stream()), "conv_silu")
        return x

    def _recur(self, x: torch.Tensor, raw: torch.Tensor, low: torch.Tensor, y: torch.Tensor, w: PackedScan, state: torch.Tensor | None,
               batch: int, seq: int, start: int, pos: torch.Tensor | None) -> torch.Tensor:
        out = torch.empty_like(x)
        args = _lib.ScanArgs(
            x=_ptr(x), dt=_ptr(raw), low=_ptr(low), z=y.data_ptr() + w.inner * y.element_size(), a2=_ptr(w.a2), d=_ptr(w.skip),
            dt_bias=_ptr(w.dt_bias), state=_ptr(state), pos=_ptr(pos), out=_ptr(out), batch=batch, seq=seq, start=start, inner=w.inner,
            states=w.states, dt_ld=raw.shape[1], low_ld=low.shape[1], b_col=w.rank, c_col=w.rank + w.states, z_ld=y.shape[1], out_ld=out.shape[1])
        _lib.check_dense(_lib.load_dense().ajqd_scan(ctypes.byref(args), _flag(x.dtype), _stream()), "scan")
        return out

    # ---- one token per sequence, at the device-side position ``cache.position``
    def _token(self, token_ids: torch.Tensor, cache: RingCache) -> tuple[torch.Tensor, None]:
        if self._embed.dtype == torch.bfloat16:
            return self._token_fused(token_ids, cache), None
        order = self._sublayers()
        x, _ = self._start(token_ids, order[0][2], False)
        delta, done = None, None
        for run, w, sub in order:
            h = self._streams_norm(x, delta, done, sub)
            y = self._times(w.w_in, h)
            if isinstance(w, PackedAttention):
                mixed = self._attend_token(y, w, cache, run)
            elif isinstance(w, PackedScan):
                mixed = self._scan_token(y, w, cache, run)
            else:
                mixed = self._activated(y, w.act)
            delta, done = torch.empty((h.shape[0], h.shape[1]), dtype=torch.float32, device=h.device), sub
            _matvec(w.w_out, 1, mixed, mixed.shape[1], 0, delta, delta.shape[1], 0, h.shape[0])
        return self._streams_norm(x, delta, done, None), None

    def _times(self, w: torch.Tensor, x: torch.Tensor, stride: int | None = None) -> torch.Tensor:
        y = torch.empty((x.shape[0], w.shape[0]), dtype=x.dtype, device=x.device)
        _matvec(w, 1, x, stride or x.shape[1], 0, y, y.shape[1], 0, x.shape[0])
        return y

    def _attend_token(self, y: torch.Tensor, w: PackedAttention, cache: RingCache, run: int) -> torch.Tensor:
        ring = cache.rings[run]
        q = torch.empty((y.shape[0], w.heads, w.dimp), dtype=y.dtype, device=y.device)
        self._split(y, w, q, 0, ring, 1, 0, cache.position, 0, cache.kept[run])
        return self._windowed(w, q, ring, y, 1, 0, cache.position)

    def _scan_token(self, y: torch.Tensor, w: PackedScan, cache: RingCache, run: int) -> torch.Tensor:
        x = self._convolved(y, w, cache.rings[run], 0, cache.position, 1)
        low = self._times(w.w_low, x)
        raw = self._times(w.w_dt, low, low.shape[1])
        return self._recur(x, raw, low, y, w, cache.states[run], y.shape[0], 1, 0, cache.position)

    def _token_fused(self, token_ids: torch.Tensor, cache: RingCache) -> torch.Tensor:
        """The bf16 step: a product in front of a sublayer (with the norm where that is free), what the sublayer is, a product
        behind it that updates the streams and leaves the next sublayer's input."""
        lib, st, dev = _lib.load_dense(), _stream(), self._embed.device
        batch, dp = token_ids.shape[0], self._embed.shape[1]
        order = self._sublayers()
        x, u = self._start(token_ids, order[0][2], True)
        for k, (run, w, sub) in enumerate(order):
            ff = isinstance(w, PackedFeedForward)
            y = torch.empty((batch, w.w_in.shape[0]), dtype=torch.bfloat16 if ff else torch.float32, device=dev)
            rows, n = (u, None) if batch <= NORM_PROLOGUE_ROWS else (None, _add_norms(u, None, None, None, sub.gain, None, sub.eps, 0, self.d_model,
                                                                                     torch.bfloat16)[0])
            if ff:
                self._dense_in(rows, None, n, None, sub.gain, sub.eps, 0, None, w.w_in, None, _ptr(y), w.width, w.act, pairs=False)
                mixed = y
            else:
                self._dense_in(rows, n, None, sub.gain, None, sub.eps, 0, w.w_in, None, y, None, 0, 0)
                mixed = (self._attend_fused if isinstance(w, PackedAttention) else self._scan_fused)(y, w, cache, run)
            following = order[k + 1][2].reads if k + 1 < len(order) else None
            u = torch.empty_like(u)
            _lib.check_dense(lib.ajqd_dense_out_streams(
                _ptr(mixed), _ptr(w.w_out), _ptr(x), _ptr(sub.scale), _ptr(sub.writes), _ptr(sub.mix), _ptr(following), _ptr(u), self.streams,
                batch, mixed.shape[1], dp, st), "dense_out_streams")
        return u

    def _attend_fused(self, y: torch.Tensor, w: PackedAttention, cache: RingCache, run: int) -> torch.Tensor:
        lib, st, ring, batch = _lib.load_dense(), _stream(), cache.rings[run], y.shape[0]
        cap = ring.shape[2]
        chunks = lib.ajqd_latent_decode_chunks(batch * w.groups, w.share, w.dimp, w.dimp, cap)
        if chunks == 0:   # heads wider than the kernel takes
            return self._attend_token(y.to(torch.bfloat16), w, cache, run)
        q = torch.empty((batch, w.heads, w.row), dtype=torch.bfloat16, device=y.device)
        self._split(y, w, q, w.dimp, ring, 1, 0, cache.position, 0, cache.kept[run])
        units = batch * w.groups
        partial = torch.empty(lib.ajqd_latent_decode_workspace(units, w.share, w.dimp, chunks), dtype=torch.uint8, device=y.device)
        _lib.check_dense(lib.ajqd_latent_decode(_ptr(q), _ptr(ring), _ptr(cache.position), _ptr(partial), units, w.share, w.dimp, w.dimp, cap,
                                                chunks, w.dimp, w.scale, st), "latent_decode")
        out = torch.empty((batch, w.heads * w.dimp), dtype=torch.bfloat16, device=y.device)
        _lib.check_dense(lib.ajqd_group_merge(_ptr(partial), y.data_ptr() + 4 * w.gate_column, y.shape[1], _ptr(out), out.shape[1], batch,
                                              w.groups, w.share, chunks, w.dimp, st), "group_merge")
        return out

    def _scan_fused(self, y: torch.Tensor, w: PackedScan, cache: RingCache, run: int) -> torch.Tensor:
        lib, st, ring, batch = _lib.load_dense(), _stream(), cache.rings[run], y.shape[0]
        splits = lib.ajqd_scan_splits(batch, w.inner)
        partial = torch.empty((splits, batch, w.low_rows), dtype=torch.float32, device=y.device)
        held = _ptr(ring) if w.taps > 1 else None
        _lib.check_dense(lib.ajqd_scan_project(_ptr(y), y.shape[1], held, _ptr(w.conv), _ptr(w.conv_bias), _ptr(cache.position), _ptr(w.w_low),
                                               _ptr(partial), batch, w.inner, w.taps, w.low_rows, splits, st), "scan_project")
        out = torch.empty((batch, w.inner), dtype=torch.bfloat16, device=y.device)
        args = _lib.ScanStepArgs(
            y=_ptr(y), ring=held, weight=_ptr(w.conv), bias=_ptr(w.conv_bias), pos=_ptr(cache.position), partial=_ptr(partial), w_dt=_ptr(w.w_dt),
            dt_bias=_ptr(w.dt_bias), a2=_ptr(w.a2), d=_ptr(w.skip), state=_ptr(cache.states[run]), out=_ptr(out), batch=batch, ldy=y.shape[1],
            inner=w.inner, taps=w.taps, rows=w.low_rows, splits=splits, rank=w.rank, states=w.states, out_ld=w.inner)
        _lib.check_dense(lib.ajqd_scan_step(ctypes.byref(args), st), "scan_step")
        return out


@register_architecture("Purusun")
def build_purusun(config: dict[str, Any]) -> HybridLM:
    """The model a ``config.json`` of this architecture describes: ``vocab``, ``width``, ``streams``, ``norm.eps``, ``layers`` (each
    ``type``, ``mixer``, ``mlp`` or null) and ``loop`` (optional)."""
    blocks: list[tuple[str, dict[str, Any], tuple[int, str] | None]] = []
    for i, layer in enumerate(config["layers"]):
        m, mlp = layer["mixer"], layer.get("mlp")
        if layer["type"] == "attention":
            if m.get("vdim", m["dim"]) != m["dim"]:
                raise ValueError(f"layer {i}: vdim must equal dim (the values are the keys)")
            mask, rot = m.get("mask") or {}, m.get("rot") or {"dims": 0, "base": 1.0}
            s = rot.get("scaling")
            mixer = dict(num_heads=int(m["heads"]), num_kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), scale=float(m["scale"]),
                         rot_dim=int(rot["dims"]), rot_base=float(rot["base"]),
                         scaling=FrequencyScaling(float(s["factor"]), float(s["low"]), float(s["high"]), float(s["original"])) if s else None,
                         window=int(mask["size"]) if mask.get("size") else None, keep_first=int(mask.get("keep_first") or 0))
        elif layer["type"] == "mamba1":
            mixer = {name: int(m[name]) for name in ("inner", "state", "dt_rank", "conv")}
        else:
            raise ValueError(f"layer {i}: unsupported mixer {layer['type']!r}")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: unsupported feed-forward {mlp['kind']!r}")
        blocks.append((layer["type"], mixer, (int(mlp["ff"]), "squared_relu") if mlp is not None else None))
    loop = config.get("loop")
    return HybridLM(int(config["vocab"]), int(config["width"]), int(config["streams"]), blocks,
                    Loop(int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else None, epsilon=float(config["norm"]["eps"]))
