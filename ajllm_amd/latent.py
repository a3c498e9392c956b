"""Dense decoder with latent attention: parallel layers, sliding window, attention sink, gated heads, looped layers.

One architecture is registered here, ``Dorutar``; its mechanisms are modules of their own with their constants as
arguments:

* ``LatentAttention``    keys and values expanded per head from a low-rank latent, one rotated key part shared by all
                         heads, so that a position costs ``kv_rank + rot_dim`` cache elements; a sliding window (or
                         none), a learned sink per head in the softmax denominator, a sigmoid gate per head
* ``ParallelBlock``      mixer and feed-forward side by side on two norms of the incoming stream, one sum at the end
* ``Loop``               a span of layers traversed several times; every traversal has rings of its own in the cache and a
                         learned offset for the stream it starts from, the later ones take the embedding in again as well
* ``LatentLM``           the decoder (``dense.DenseLM``)

All of it runs on the operators of ``libajq_dense.so`` on a ROCm device, weights and activations in bf16 or fp32 (plain
matrix products of prompts are the vendor library's).  There is no CPU path.  The residual stream, norms, angles,
attention scores and sums, gates and logits are fp32 in both.

A prompt expands keys and values per head (two products per position, then attention at the head width); a single token
moves its query into the latent space instead and attends to the cached latents themselves, which all heads share.
"""

from __future__ import annotations

import ctypes
from typing import Any

import torch
from torch import nn

from . import _lib
from .dense import (NORM_PROLOGUE_ROWS, DenseLM, Loop, _add_norms, _flag, _matvec, _padded, _product, _ptr, _stream, _up,
                    rotary_frequencies)
from .modeling import Embedding, GatedFeedForward, Linear, RingCache, RMSNorm, build_norm, register_architecture


class LatentAttention(nn.Module):
    def __init__(self, d_model: int, num_heads: int, dim: int, rot_dim: int, value_dim: int, kv_rank: int, scale: float,
                 rot_base: float, window: int | None = None, epsilon: float = 1e-5, sink: bool = True, gate: bool = True) -> None:
        super().__init__()
        if rot_dim < 2 or rot_dim % 2 != 0:
            raise ValueError("the rotated width must be even and positive")
        if window is not None and window < 1:
            raise ValueError("the window must hold at least the token itself")
        self.num_heads, self.dim, self.rot_dim, self.value_dim, self.kv_rank = num_heads, dim, rot_dim, value_dim, kv_rank
        self.scale, self.rot_base, self.window = float(scale), float(rot_base), window
        self.q_proj = Linear(d_model, num_heads * (dim + rot_dim))    # per head: unrotated, rotated
        self.dkv_proj = Linear(d_model, kv_rank + rot_dim)            # latent, shared rotated key part
        self.dkv_norm = RMSNorm(kv_rank, epsilon)
        self.uk_proj = Linear(kv_rank, num_heads * dim)
        self.uv_proj = Linear(kv_rank, num_heads * value_dim)
        self.sink = nn.Parameter(torch.zeros(num_heads)) if sink else None
        self.gate_proj = Linear(d_model, num_heads) if gate else None
        self.output_proj = Linear(num_heads * value_dim, d_model)


class ParallelBlock(nn.Module):
    def __init__(self, d_model: int, mixer: LatentAttention, feed_forward: GatedFeedForward | None, norm: str, epsilon: float) -> None:
        super().__init__()
        self.norm1 = build_norm(norm, d_model, epsilon)
        self.mixer = mixer
        self.norm2 = build_norm(norm, d_model, epsilon) if feed_forward is not None else None
        self.feed_forward = feed_forward


def rotary_tables(base: float, dims: int, length: int) -> tuple[torch.Tensor, torch.Tensor]:
    """cos and sin of p * base^(-2 i / dims), ``[length, dims / 2]`` fp32 (angles formed in double on the host)."""
    angles = torch.arange(length, dtype=torch.float64)[:, None] * rotary_frequencies(base, dims)
    return torch.cos(angles).float(), torch.sin(angles).float()


def interleave_gate(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """Rows of two matrices in alternating blocks of 8 (``rows % 8 == 0``): a 16-row tile holds both factors of 8 outputs."""
    blocks = torch.stack((gate.reshape(-1, 8, gate.shape[1]), up.reshape(-1, 8, up.shape[1])), dim=1)
    return blocks.reshape(2 * gate.shape[0], gate.shape[1]).contiguous()


class PackedBlock:
    """One block's weights as the kernels read them: projections that share an input stacked into one matrix, widths
    padded with zeros (rows of 8 or 16), the two products of a layer's end side by side (one product over the
    concatenated heads and feed-forward columns), the key expansion a second time transposed per head."""

    def __init__(self, block: ParallelBlock, tables: tuple[torch.Tensor, torch.Tensor]) -> None:
        mix, ff = block.mixer, block.feed_forward
        weight = mix.q_proj.weight.detach()
        dtype, dev, d = weight.dtype, weight.device, weight.shape[1]
        heads = mix.num_heads
        self.heads, self.scale, self.window = heads, mix.scale, mix.window
        self.dimp, self.rotp = _up(mix.dim, 8), _up(mix.rot_dim, 8)
        self.vdimp, self.rankp, dp = _up(mix.value_dim, 16), _up(mix.kv_rank, 16), _up(d, 16)
        self.width = self.rankp + self.rotp
        q = weight.view(heads, mix.dim + mix.rot_dim, d)
        q = torch.cat((_padded(q[:, :mix.dim], heads, self.dimp, dp), _padded(q[:, mix.dim:], heads, self.rotp, dp)), dim=1)
        down = mix.dkv_proj.weight.detach()
        rows = [q.reshape(-1, dp), _padded(down[:mix.kv_rank], self.rankp, dp), _padded(down[mix.kv_rank:], self.rotp, dp)]
        gate = mix.gate_proj.weight.detach() if mix.gate_proj is not None else torch.zeros(heads, d, dtype=dtype, device=dev)
        rows.append(_padded(gate, heads, dp))
        w1 = torch.cat(rows, dim=0)
        self.gate_column = w1.shape[0] - heads
        self.w1 = _padded(w1, _up(w1.shape[0], 16), dp)
        uk = _padded(mix.uk_proj.weight.detach().view(heads, mix.dim, mix.kv_rank), heads, self.dimp, self.rankp)
        uv = _padded(mix.uv_proj.weight.detach().view(heads, mix.value_dim, mix.kv_rank), heads, self.vdimp, self.rankp)
        self.ukv = torch.cat((uk.reshape(-1, self.rankp), uv.reshape(-1, self.rankp)), dim=0).contiguous()
        self.uv = self.ukv[heads * self.dimp:]
        self.ukt = uk.transpose(1, 2).contiguous()
        out = _padded(mix.output_proj.weight.detach().view(d, heads, mix.value_dim), dp, heads, self.vdimp).view(dp, -1)
        self.w2, self.ff, self.act = None, 0, 0
        if ff is not None:
            f = ff.w1.weight.shape[0]
            self.ff = _up(f, 8)
            self.act = _lib.AJQD_ACTIVATIONS[ff.activation]
            self.w2 = interleave_gate(_padded(ff.w1.weight.detach(), self.ff, dp), _padded(ff.w3.weight.detach(), self.ff, dp))
            out = torch.cat((out, _padded(ff.w2.weight.detach(), dp, self.ff)), dim=1)
        self.wo = out.contiguous()
        self.joined = self.wo.shape[1]           # columns of (heads | feed-forward)

        def gain(norm: nn.Module | None, width: int) -> torch.Tensor | None:
            return _padded(norm.weight.detach().float(), width) if norm is not None else None

        self.center = 0 if isinstance(block.norm1, RMSNorm) else 1
        self.eps = block.norm1.epsilon
        self.gain1, self.gain2 = gain(block.norm1, dp), gain(block.norm2, dp)
        self.latent_gain = gain(mix.dkv_norm, self.rankp)
        self.gated_heads = mix.gate_proj is not None
        self.sink = mix.sink.detach().float().contiguous() if mix.sink is not None else None
        self.cosine, self.sine = tables
        self.shape = _lib.LatentShape(heads, self.dimp, mix.rot_dim, self.rotp, mix.kv_rank, self.rankp, mix.dkv_norm.epsilon)


class LatentLM(DenseLM):
    """The decoder.  ``blocks``: one ``(mixer arguments, feed-forward (width, activation) or None)`` per layer."""

    def __init__(self, vocab_size: int, context_length: int, d_model: int, blocks: list[tuple[dict[str, Any], tuple[int, str] | None]],
                 loop: Loop | None = None, norm: str = "layernorm", epsilon: float = 1e-5) -> None:
        super().__init__()
        self.vocab_size, self.context_length, self.d_model, self.loop = vocab_size, context_length, d_model, loop
        self._check_loop(len(blocks))
        self.token_embeddings = Embedding(vocab_size, d_model)
        self.position_embeddings = Embedding(context_length, d_model)
        self.layers = nn.ModuleList([
            ParallelBlock(d_model, LatentAttention(d_model, epsilon=epsilon, **mixer),
                          GatedFeedForward(d_model, ff[0], ff[1]) if ff is not None else None, norm, epsilon)
            for mixer, ff in blocks
        ])
        self.loop_step = nn.Parameter(torch.zeros(loop.times, d_model)) if loop is not None else None
        self.final_norm = build_norm(norm, d_model, epsilon)
        self.lm_head = Linear(d_model, vocab_size)

    def checkpoint_names(self) -> dict[str, str]:
        """State-dict key -> tensor name in a checkpoint file."""
        names = {"token_embeddings.weight": "embed", "position_embeddings.weight": "pos", "final_norm.weight": "final.norm",
                 "lm_head.weight": "head"}
        if self.loop is not None:
            names["loop_step"] = "loop.step"
        parts = {"norm1.weight": "norm1", "norm2.weight": "norm2", "mixer.q_proj.weight": "mix.q",
                 "mixer.dkv_proj.weight": "mix.dkv", "mixer.dkv_norm.weight": "mix.dkv.norm", "mixer.uk_proj.weight": "mix.uk",
                 "mixer.uv_proj.weight": "mix.uv", "mixer.sink": "mix.sink", "mixer.gate_proj.weight": "mix.g",
                 "mixer.output_proj.weight": "mix.o", "feed_forward.w1.weight": "mlp.gate",
                 "feed_forward.w3.weight": "mlp.up", "feed_forward.w2.weight": "mlp.down"}
        for key in self.state_dict():
            if key.startswith("layers."):
                _, index, part = key.split(".", 2)
                names[key] = f"l{index}.{parts[part]}"
        return names

    def ignored_names(self) -> set[str]:
        """Tensors a checkpoint may hold that no layer reads: the second norm of a layer without a feed-forward."""
        return {f"l{i}.norm2" for i, layer in enumerate(self.layers) if layer.feed_forward is None}

    def new_cache(self, batch: int, max_len: int | None = None, dtype: torch.dtype | None = None) -> RingCache:
        """An empty cache.  Rows are kept in the activations' dtype."""
        weight = self.token_embeddings.weight
        if dtype is not None and dtype != weight.dtype:
            raise ValueError("the latent cache has the model's own dtype")
        max_len = max_len or self.context_length
        mixers = [self.layers[i].mixer for i, _ in self.runs]
        return RingCache([min(m.window or max_len, max_len) for m in mixers],
                         [_up(m.kv_rank, 16) + _up(m.rot_dim, 8) for m in mixers], batch, max_len, weight.device, weight.dtype)

    def _pack(self) -> None:
        weight = self.token_embeddings.weight
        tables: dict = {}
        blocks = []
        for layer in self.layers:
            key = (layer.mixer.rot_base, layer.mixer.rot_dim)
            if key not in tables:
                tables[key] = tuple(t.to(weight.device) for t in rotary_tables(*key, self.context_length))
            blocks.append(PackedBlock(layer, tables[key]))
        dp = _up(self.d_model, 16)
        self._blocks = blocks
        self._embed = _padded(weight.detach(), self.vocab_size, dp)
        self._pos = _padded(self.position_embeddings.weight.detach(), self.context_length, dp)
        self._steps = _padded(self.loop_step.detach().float(), self.loop.times, dp) if self.loop is not None else None
        self._final_gain = _padded(self.final_norm.weight.detach().float(), dp)
        self._head = _padded(self.lm_head.weight.detach(), _up(self.vocab_size, 16), dp)

    def _begins(self, run: int) -> tuple[bool, torch.Tensor | None]:
        """What is added to x ahead of a layer run: whether the embedding output is, and the pass's vector."""
        t = self.runs[run][1] if run < len(self.runs) else None
        return (t is not None and t > 0), (self._steps[t] if t is not None else None)

    def _embedded(self, token_ids: torch.Tensor, start: int, pos: torch.Tensor | None) -> tuple[torch.Tensor, torch.Tensor | None]:
        """The residual stream in front of the first layer run, and the embedding output where a loop needs it again."""
        batch, seq = token_ids.shape
        dp = self._embed.shape[1]
        x = torch.empty((batch * seq, dp), dtype=torch.float32, device=self._embed.device)
        embedded = torch.empty_like(x) if self.loop is not None and self.loop.times > 1 else None
        _lib.check_dense(_lib.load_dense().ajqd_embed(
            _ptr(token_ids), batch * seq, seq, _ptr(self._embed), self.vocab_size, _ptr(self._pos), self.context_length, start,
            _ptr(pos), _ptr(self._begins(0)[1]), _ptr(x), _ptr(embedded), dp, _flag(self._embed.dtype), _stream()), "embed")
        return x, embedded

    # ---- many tokens per sequence
    def _prompt(self, token_ids: torch.Tensor, cache: RingCache | None, start: int,
                residuals: list | None) -> tuple[torch.Tensor, torch.Tensor]:
        lib, st, dtype = _lib.load_dense(), _stream(), self._embed.dtype
        batch, seq = token_ids.shape
        m, dev = batch * seq, self._embed.device
        x, embedded = self._embedded(token_ids, start, None)
        delta = None
        for run, (index, _) in enumerate(self.runs):
            w = self._blocks[index]
            again, step = self._begins(run) if run > 0 else (False, None)
            n1, n2 = _add_norms(x, delta, embedded if again else None, step, w.gain1, w.gain2, w.eps, w.center, self.d_model, dtype)
            y = _product(n1, w.w1, torch.float32)
            # rows of the keys' latents: those still in the window of the first new token, then the new ones
            reach = start if w.window is None else min(start, w.window - 1)
            rows = torch.empty((batch, reach + seq, w.width), dtype=dtype, device=dev)
            ring = cache.rings[run] if cache is not None else None
            row_bytes = w.width * rows.element_size()
            if reach > 0:
                _lib.check_dense(lib.ajqd_ring_copy(_ptr(ring), ring.shape[1], 0, _ptr(rows), reach + seq, row_bytes, 0,
                                                    start - reach, reach, row_bytes, batch, 0, st), "ring_copy")
            q = torch.empty((m, w.heads, w.dimp + w.rotp), dtype=dtype, device=dev)
            gates = torch.empty((m, w.heads), dtype=torch.float32, device=dev)
            _lib.check_dense(lib.ajqd_latent_split(
                _ptr(y), _lib.AJQD_F32, y.shape[1], ctypes.byref(w.shape), _ptr(w.latent_gain), _ptr(w.cosine), _ptr(w.sine),
                self.context_length, m, seq, start, None, reach, 0, _ptr(q), q.shape[2], q.data_ptr() + w.dimp * q.element_size(),
                q.shape[2], _ptr(rows), rows.stride(0), _ptr(gates), _flag(dtype), st), "latent_split")
            del y
            kv = _product(rows.view(-1, w.width)[:, : w.rankp], w.ukv, dtype)
            joined = torch.empty((m, w.joined), dtype=dtype, device=dev)
            size, per_seq, columns = kv.element_size(), reach + seq, kv.shape[1]
            args = _lib.WindowedAttentionArgs(
                q=_ptr(q), k1=_ptr(kv), k2=rows.data_ptr() + w.rankp * size, v=kv.data_ptr() + w.heads * w.dimp * size, sink=_ptr(w.sink),
                gates=_ptr(gates) if w.gated_heads else None, pos=None, out=_ptr(joined), k1_batch=per_seq * columns,
                k2_batch=per_seq * w.width, v_batch=per_seq * columns, k1_row=columns, k1_head=w.dimp, k2_row=w.width,
                v_row=columns, v_head=w.vdimp, d1=w.dimp, d2=w.rotp, dv=w.vdimp, batch=batch, heads=w.heads, seq=seq,
                rows=per_seq, prior=reach, window=w.window or 0, out_ld=w.joined, scale=w.scale)
            if dtype == torch.bfloat16 and lib.ajqd_windowed_prefill_supported(w.dimp, w.rotp, w.vdimp):
                _lib.check_dense(lib.ajqd_windowed_prefill(ctypes.byref(args), st), "windowed_prefill")
            else:
                _lib.check_dense(lib.ajqd_windowed_attention(ctypes.byref(args), _flag(dtype), _flag(dtype), st), "windowed_attention")
            del kv, q
            if w.w2 is not None:
                self._gate(_product(n2, w.w2, dtype), joined, w)
            delta = _product(joined, w.wo, torch.float32)
            if ring is not None:
                keep = min(seq, ring.shape[1])
                _lib.check_dense(lib.ajqd_ring_copy(_ptr(ring), ring.shape[1], 0, _ptr(rows), reach + seq, row_bytes, reach + seq - keep,
                                                    start + seq - keep, keep, row_bytes, batch, 1, st), "ring_copy")
            if residuals is not None:
                residuals.append((x + delta)[:, : self.d_model].view(batch, seq, -1))
        return x, delta

    def _gate(self, y: torch.Tensor, joined: torch.Tensor, w: PackedBlock) -> None:
        """The gated activation of ``y`` into the feed-forward columns of ``joined``."""
        at = joined.data_ptr() + w.heads * w.vdimp * joined.element_size()
        _lib.check_dense(_lib.load_dense().ajqd_gated_activation(_ptr(y), _flag(y.dtype), at, w.joined, y.shape[0], w.ff, w.act,
                                                                 _flag(joined.dtype), _stream()), "gated_activation")

    # ---- one token per sequence, at the device-side position ``cache.position``
    def _token(self, token_ids: torch.Tensor, cache: RingCache) -> tuple[torch.Tensor, torch.Tensor | None]:
        x, embedded = self._embedded(token_ids, 0, cache.position)
        delta = None
        for run, (index, _) in enumerate(self.runs):
            w, ring = self._blocks[index], cache.rings[run]
            chunks = 0
            if x.shape[0] and w.w1.dtype == torch.bfloat16:
                chunks = _lib.load_dense().ajqd_latent_decode_chunks(x.shape[0], w.heads, w.rankp, w.rotp, ring.shape[1])
            if chunks > 0:
                delta = self._token_fused(x, delta, embedded, run, w, ring, cache.position, chunks)
            else:
                delta = self._token_plain(x, delta, embedded, run, w, ring, cache.position)
        return x, delta

    def _token_fused(self, x, delta, embedded, run: int, w: PackedBlock, ring, pos, chunks: int) -> None:
        """One layer run in five launches (six for more than one sequence); x is updated in place, with what the next layer run
        adds first included."""
        lib, st, dtype, dev = _lib.load_dense(), _stream(), w.w1.dtype, x.device
        batch = x.shape[0]
        if delta is not None:  # a layer run on the plain operators came before
            again, step = self._begins(run)
            _add_norms(x, delta, embedded if again else None, step, None, None, 0.0, 1, self.d_model, dtype)
        y = torch.empty((batch, w.w1.shape[0]), dtype=torch.float32, device=dev)
        joined = torch.empty((batch, w.joined), dtype=dtype, device=dev)
        gated = joined.data_ptr() + w.heads * w.vdimp * joined.element_size()
        if batch <= NORM_PROLOGUE_ROWS:
            self._dense_in(x, None, None, w.gain1, w.gain2, w.eps, w.center, w.w1, w.w2, y, gated, w.joined, w.act)
        else:
            n1, n2 = _add_norms(x, None, None, None, w.gain1, w.gain2, w.eps, w.center, self.d_model, dtype)
            self._dense_in(None, n1, n2, None, None, w.eps, w.center, w.w1, w.w2, y, gated, w.joined, w.act)
        q = torch.empty((batch, w.heads, w.width), dtype=dtype, device=dev)
        _lib.check_dense(lib.ajqd_latent_absorb(_ptr(y), y.shape[1], ctypes.byref(w.shape), _ptr(w.ukt), _ptr(w.latent_gain),
                                                _ptr(w.cosine), _ptr(w.sine), self.context_length, _ptr(pos), _ptr(q), _ptr(ring),
                                                ring.shape[1], batch, st), "latent_absorb")
        partial = torch.empty(lib.ajqd_latent_decode_workspace(batch, w.heads, w.rankp, chunks), dtype=torch.uint8, device=dev)
        _lib.check_dense(lib.ajqd_latent_decode(_ptr(q), _ptr(ring), _ptr(pos), _ptr(partial), batch, w.heads, w.rankp, w.rotp,
                                                ring.shape[1], chunks, 0, w.scale, st), "latent_decode")
        gate = y.data_ptr() + 4 * w.gate_column if w.gated_heads else None
        _lib.check_dense(lib.ajqd_latent_expand(_ptr(partial), _ptr(w.sink), gate, y.shape[1], _ptr(w.uv), _ptr(joined),
                                                w.joined, batch, w.heads, chunks, w.rankp, w.vdimp, st), "latent_expand")
        again, step = self._begins(run + 1)
        _lib.check_dense(lib.ajqd_dense_out(_ptr(joined), _ptr(w.wo), _ptr(x), _ptr(embedded) if again else None, _ptr(step), batch,
                                            w.joined, x.shape[1], st), "dense_out")

    def _token_plain(self, x, delta, embedded, run: int, w: PackedBlock, ring, pos) -> torch.Tensor:
        """The same layer run on operators of any width, bf16 or fp32; returns what is still to be added to x."""
        lib, st, dtype, dev = _lib.load_dense(), _stream(), w.w1.dtype, x.device
        batch, cap = x.shape[0], ring.shape[1]
        again, step = self._begins(run) if delta is not None else (False, None)  # (else: already in x)
        n1, n2 = _add_norms(x, delta, embedded if again else None, step, w.gain1, w.gain2, w.eps, w.center, self.d_model, dtype)
        y = torch.empty((batch, w.w1.shape[0]), dtype=torch.float32, device=dev)
        _matvec(w.w1, 1, n1, n1.shape[1], 0, y, y.shape[1], 0, batch)
        qu = torch.empty((batch, w.heads, w.dimp), dtype=dtype, device=dev)
        q = torch.empty((batch, w.heads, w.width), dtype=dtype, device=dev)
        gates = torch.empty((batch, w.heads), dtype=torch.float32, device=dev)
        size = q.element_size()
        _lib.check_dense(lib.ajqd_latent_split(
            _ptr(y), _lib.AJQD_F32, y.shape[1], ctypes.byref(w.shape), _ptr(w.latent_gain), _ptr(w.cosine), _ptr(w.sine),
            self.context_length, batch, 1, 0, _ptr(pos), 0, cap, _ptr(qu), w.dimp, q.data_ptr() + w.rankp * size, w.width, _ptr(ring),
            ring.stride(0), _ptr(gates), _flag(dtype), st), "latent_split")
        _matvec(w.ukt.view(-1, w.dimp), w.heads, qu, w.heads * w.dimp, w.dimp, q, w.heads * w.width, w.width, batch)
        summed = torch.empty((batch, w.heads * w.rankp), dtype=dtype, device=dev)
        args = _lib.WindowedAttentionArgs(
            q=_ptr(q), k1=_ptr(ring), k2=ring.data_ptr() + w.rankp * size, v=_ptr(ring), sink=_ptr(w.sink),
            gates=_ptr(gates) if w.gated_heads else None, pos=_ptr(pos), out=_ptr(summed), k1_batch=ring.stride(0),
            k2_batch=ring.stride(0), v_batch=ring.stride(0), k1_row=w.width, k1_head=0, k2_row=w.width, v_row=w.width, v_head=0,
            d1=w.rankp, d2=w.rotp, dv=w.rankp, batch=batch, heads=w.heads, seq=1, rows=cap, prior=0, window=0,
            out_ld=w.heads * w.rankp, scale=w.scale)
        _lib.check_dense(lib.ajqd_windowed_attention(ctypes.byref(args), _flag(dtype), _flag(dtype), st), "windowed_attention")
        joined = torch.empty((batch, w.joined), dtype=dtype, device=dev)
        _matvec(w.uv, w.heads, summed, w.heads * w.rankp, w.rankp, joined, w.joined, w.vdimp, batch)
        if w.w2 is not None:
            y2 = torch.empty((batch, w.w2.shape[0]), dtype=torch.float32, device=dev)
            _matvec(w.w2, 1, n2, n2.shape[1], 0, y2, y2.shape[1], 0, batch)
            self._gate(y2, joined, w)
        delta = torch.empty_like(x)
        _matvec(w.wo, 1, joined, w.joined, 0, delta, x.shape[1], 0, batch)
        return delta


@register_architecture("Dorutar")
def build_dorutar(config: dict[str, Any]) -> LatentLM:
    """The model a ``config.json`` of this architecture describes: ``vocab``, ``width``, ``max_positions``, ``norm.eps``,
    ``layers`` (each ``type``, ``mixer``, ``mlp`` or null) and ``loop`` (optional)."""
    blocks = []
    for i, layer in enumerate(config["layers"]):
        if layer["type"] != "latent_attention":
            raise ValueError(f"layer {i}: unsupported mixer {layer['type']!r}")
        mixer, mlp = layer["mixer"], layer.get("mlp")
        if mixer["rot"]["dims"] != mixer["rot_dim"]:
            raise ValueError(f"layer {i}: rot.dims must equal rot_dim")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: unsupported feed-forward {mlp['kind']!r}")
        mask = mixer.get("mask") or {}
        blocks.append((dict(num_heads=int(mixer["heads"]), dim=int(mixer["dim"]), rot_dim=int(mixer["rot_dim"]),
                            value_dim=int(mixer["vdim"]), kv_rank=int(mixer["kv_rank"]), scale=float(mixer["scale"]),
                            rot_base=float(mixer["rot"]["base"]), window=int(mask["size"]) if mask.get("size") else None),
                       (int(mlp["ff"]), "relu") if mlp is not None else None))
    loop = config.get("loop")
    return LatentLM(int(config["vocab"]), int(config["max_positions"]), int(config["width"]), blocks,
                    Loop(int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else None,
                    epsilon=float(config["norm"]["eps"]))
