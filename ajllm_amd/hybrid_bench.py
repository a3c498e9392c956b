"""Throughput of the decoder with key-value attention and selective scans on several residual streams (``hybrid.HybridLM``) at
layer sizes of real models, random weights, beside the library's closest existing model at equal size: the dense
latent-attention decoder (``latent.LatentLM``), of the same width, heads, window and number of layer runs.

Whole-model figures (prompt of 4 x 2048 tokens, decoding at context 2048 with batch 1, 8 and 32) and, kernel by kernel, the
share of its roofline next to the like kernel of the other model.  Bytes are the algorithmic ones: weights, cache rows, states
and activations once.  The scan of a prompt has two rooflines, HBM bytes and the exponential unit (one exponential per token,
channel and state; a SIMD takes 16 lanes a cycle at a quarter rate); both shares are given.
"""

from __future__ import annotations

import ctypes
import time

import torch

from . import _lib, decoding, hybrid, latent
from .dense import Loop, _add_norms
from .latent_bench import CONTEXT, HBM_PEAK_GBS, MFMA_BF16_PEAK_TFLOPS, PROMPT_ROWS, VOCAB, _graph_us, _hbm, _seconds, _st, build_latent
from .latent_bench import SIZES as LATENT_SIZES

EXP_PEAK_GIGA = 256 * 4 * 4 * 2.4   # exponentials per ns: CUs x SIMDs x lanes per cycle x GHz
SIZES = {
    "width 2048": dict(width=2048, heads=16, kv_heads=4, dim=128, rot=64, window=1024, keep=4, ff=8192, inner=4096, state=16, dt_rank=128,
                       conv=4, streams=2, layers=8, loop=Loop(2, 6, 2)),
    "width 4096": dict(width=4096, heads=32, kv_heads=8, dim=128, rot=64, window=1024, keep=4, ff=16384, inner=8192, state=16, dt_rank=256,
                       conv=4, streams=2, layers=4, loop=Loop(1, 3, 2)),
}


def build_hybrid(size: dict, device, seed: int = 78, dtype: torch.dtype = torch.bfloat16) -> hybrid.HybridLM:
    """Scans and attention layers in turn."""
    torch.manual_seed(seed)
    attention = dict(num_heads=size["heads"], num_kv_heads=size["kv_heads"], dim=size["dim"], scale=size["dim"] ** -0.5, rot_dim=size["rot"],
                     rot_base=10_000.0, window=size["window"], keep_first=size["keep"])
    scan = {name: size[name] for name in ("inner", "state", "dt_rank", "conv")}
    blocks = [("attention", attention, (size["ff"], "squared_relu")) if i % 2 else ("mamba1", scan, (size["ff"], "squared_relu"))
              for i in range(size["layers"])]
    with torch.device(device):
        model = hybrid.HybridLM(VOCAB, size["width"], size["streams"], blocks, size["loop"], context_length=CONTEXT + 512)
    model = model.to(dtype).eval()
    model.prepare()
    return model


def _weights(w) -> list[torch.Tensor]:
    return [t for t in vars(w).values() if isinstance(t, torch.Tensor)]


def _bytes(*tensors: torch.Tensor) -> int:
    return sum(t.numel() * t.element_size() for t in tensors)


@torch.no_grad()
def bench_whole(name: str, device, log=print, batches=(1, 8, 32), steps: int = 64) -> dict:
    """Prompt and decode throughput of both models."""
    prompt = torch.randint(0, VOCAB, (max(batches), CONTEXT), generator=torch.Generator().manual_seed(5)).to(device)
    out: dict = {"prompt": {"tokens": PROMPT_ROWS * CONTEXT}, "decode": [{"batch": b} for b in batches]}
    for kind in ("hybrid", "latent"):
        model = build_hybrid(SIZES[name], device) if kind == "hybrid" else build_latent(LATENT_SIZES[name], device)
        out[f"{kind}_layer_runs"] = len(model.runs)
        if kind == "hybrid":
            weight_bytes = sum(_bytes(*_weights(w), *_weights(sub)) for _, w, sub in model._sublayers())
        else:
            weight_bytes = sum(2 * sum(t.numel() for t in (w.w1, w.w2, w.uv, w.ukt, w.wo)) for i, _ in model.runs for w in [model._blocks[i]])
        cache = model.new_cache(PROMPT_ROWS, CONTEXT)

        def prefill():
            cache.reset()
            model(prompt[:PROMPT_ROWS], cache, last_token_only=True)

        seconds = _seconds(prefill)
        out["prompt"].update({f"{kind}_ms": seconds * 1e3, f"{kind}_tok/s": PROMPT_ROWS * CONTEXT / seconds})
        for row in out["decode"]:
            batch = row["batch"]
            dec = decoding.DenseDecoder(model, batch, CONTEXT + steps + 16)
            dec.prefill(prompt[:batch], rows_per_pass=PROMPT_ROWS)
            dec.generate(12)
            t0 = time.perf_counter()
            dec.generate(12 + steps)
            step = (time.perf_counter() - t0) / steps
            states = [s for s in dec.cache.states if s is not None]
            total = weight_bytes + _bytes(*dec.cache.rings) + 2 * _bytes(*states) + _bytes(model._head)
            row.update({f"{kind}_ms_per_step": step * 1e3, f"{kind}_tok/s": batch / step, f"{kind}_bytes_per_step": total,
                        f"{kind}_frac_hbm_peak": total / step * 1e-9 / HBM_PEAK_GBS})
            del dec
        del model, cache
        torch.cuda.empty_cache()
    log("hybrid whole model", out)
    return out


@torch.no_grad()
def bench_kernels(name: str, device, log=print, batches=(1, 8, 32)) -> list[dict]:
    """Kernel by kernel: microseconds in a graph chain over distinct operands, share of the roofline, and the like kernel."""
    size, near_size, lib = SIZES[name], LATENT_SIZES[name], _lib.load_dense()
    d, heads, groups, window, streams = size["width"], size["heads"], size["kv_heads"], size["window"], size["streams"]
    model = build_hybrid({**size, "layers": 8, "loop": None}, device)
    near = build_latent({**near_size, "layers": 4, "loop": None}, device)
    scans, attends = model._mixers[0::2], model._mixers[1::2]
    forwards, subs, blocks = model._forwards, [pair[0] for pair in model._subs], near._blocks
    a0, s0, f0, b0 = attends[0], scans[0], forwards[0], blocks[0]
    rows: list[dict] = []

    def bf(*shape):
        return torch.randn(shape, device=device).to(torch.bfloat16)

    def add(kernel, batch, ours, like, theirs, **more):
        key = "frac_hbm_peak" if "frac_hbm_peak" in ours else "frac_mfma_peak"
        row = {"kernel": kernel, "batch": batch, **ours, "like_kernel": like, "like": theirs, "like_over_ours": theirs[key] / ours[key], **more}
        log("hybrid kernel", row)
        rows.append(row)

    for batch in batches:
        prologue = batch <= latent.NORM_PROLOGUE_ROWS
        x, normed = torch.randn((batch, d), device=device), bf(batch, d)
        xs, u = torch.randn((batch, streams, d), device=device) * 0.1, torch.empty((batch, d), device=device)
        y = torch.randn((batch, a0.w_in.shape[0]), device=device)
        ys = torch.randn((batch, s0.w_in.shape[0]), device=device)
        mid, joined, near_joined = bf(batch, f0.width), bf(batch, heads * a0.dimp), bf(batch, b0.joined)
        near_y = torch.randn((batch, b0.w1.shape[0]), device=device)
        pos = torch.tensor([CONTEXT + 7], device=device)

        # ---- products in front of a sublayer
        like_in = lambda w: near._dense_in(x if prologue else None, normed, normed, w.gain1, w.gain2, w.eps, 1, w.w1, w.w2, near_y,
                                           near_joined.data_ptr() + 2 * heads * b0.vdimp, b0.joined, w.act)
        like = _hbm(_bytes(b0.w1, b0.w2) + batch * (4 * d + 4 * b0.w1.shape[0] + 2 * near_size["ff"]), _graph_us([lambda w=w: like_in(w) for w in blocks]))
        project = lambda w, to: model._dense_in(x if prologue else None, normed, None, subs[0].gain, None, 1e-5, 0, w.w_in, None, to, None, 0, 0)
        up = lambda w: model._dense_in(x if prologue else None, None, normed, None, subs[0].gain, 1e-5, 0, None, w.w_in, None, mid.data_ptr(), w.width,
                                       w.act, pairs=False)
        for label, ws, run, cols in (("dense_in: queries | keys | gates", attends, lambda w: project(w, y), 4 * y.shape[1]),
                                     ("dense_in: scan input | gate", scans, lambda w: project(w, ys), 4 * ys.shape[1]),
                                     ("dense_in: feed-forward up, squared relu", forwards, up, 2 * f0.width)):
            add(label, batch, _hbm(_bytes(ws[0].w_in) + batch * (4 * d + cols), _graph_us([lambda w=w: run(w) for w in ws])),
                "dense_in (both matrices of a latent layer)", like)
        # ---- products behind it
        like_out = lambda w: _lib.check_dense(lib.ajqd_dense_out(near_joined.data_ptr(), w.wo.data_ptr(), x.data_ptr(), None, None, batch, w.joined, d,
                                                                 _st()), "dense_out")
        like = _hbm(_bytes(b0.wo) + batch * (2 * b0.joined + 8 * d), _graph_us([lambda w=w: like_out(w) for w in blocks]))
        back = lambda w, a, sub: _lib.check_dense(lib.ajqd_dense_out_streams(
            a.data_ptr(), w.w_out.data_ptr(), xs.data_ptr(), sub.scale.data_ptr(), sub.writes.data_ptr(), sub.mix.data_ptr(), sub.reads.data_ptr(),
            u.data_ptr(), streams, batch, w.w_out.shape[1], d, _st()), "dense_out_streams")
        for label, ws, a in (("dense_out_streams: heads back, streams mixed", attends, joined), ("dense_out_streams: feed-forward back, streams mixed", forwards, mid)):
            add(label, batch, _hbm(_bytes(ws[0].w_out) + batch * (2 * a.shape[1] + 8 * streams * d + 4 * d),
                                   _graph_us([lambda w=w: back(w, a, subs[0]) for w in ws])), "dense_out (latent layer)", like)
        # ---- attention of one token
        rings = [bf(batch, groups, window + size["keep"], a0.row) for _ in range(max(2, min(32, int(4e8 / (2 * batch * groups * window * a0.row)))))]
        cap, units = rings[0].shape[2], batch * groups
        q = torch.empty((batch, heads, a0.row), dtype=torch.bfloat16, device=device)
        split = lambda r: model._split(y, a0, q, a0.dimp, r, 1, 0, pos, 0, size["keep"])
        latents = [bf(batch, near_size["window"], b0.width) for _ in range(max(2, min(32, int(4e8 / (2 * batch * near_size["window"] * b0.width)))))]
        near_q = torch.empty((batch, heads, b0.width), dtype=torch.bfloat16, device=device)
        absorb = lambda w: _lib.check_dense(lib.ajqd_latent_absorb(
            near_y.data_ptr(), near_y.shape[1], ctypes.byref(w.shape), w.ukt.data_ptr(), w.latent_gain.data_ptr(), w.cosine.data_ptr(),
            w.sine.data_ptr(), CONTEXT + 512, pos.data_ptr(), near_q.data_ptr(), latents[0].data_ptr(), near_size["window"], batch, _st()), "latent_absorb")
        add("key_value_split: norms, rotation, cache rows", batch,
            _hbm(batch * (4 * (heads + groups) * a0.dimp + 2 * heads * a0.row + 2 * groups * a0.row), _graph_us([lambda r=r: split(r) for r in rings])),
            "latent_absorb", _hbm(_bytes(b0.ukt) + batch * (4 * near_y.shape[1] + 2 * heads * b0.width), _graph_us([lambda w=w: absorb(w) for w in blocks])))
        chunks = lib.ajqd_latent_decode_chunks(units, a0.share, a0.dimp, a0.dimp, cap)
        partial = torch.empty(lib.ajqd_latent_decode_workspace(units, a0.share, a0.dimp, chunks), dtype=torch.uint8, device=device)
        attend = lambda r: _lib.check_dense(lib.ajqd_latent_decode(q.data_ptr(), r.data_ptr(), pos.data_ptr(), partial.data_ptr(), units, a0.share, a0.dimp,
                                                                   a0.dimp, cap, chunks, a0.dimp, a0.scale, _st()), "latent_decode")
        near_chunks = lib.ajqd_latent_decode_chunks(batch, heads, b0.rankp, b0.rotp, near_size["window"])
        near_partial = torch.empty(lib.ajqd_latent_decode_workspace(batch, heads, b0.rankp, near_chunks), dtype=torch.uint8, device=device)
        near_attend = lambda r: _lib.check_dense(lib.ajqd_latent_decode(near_q.data_ptr(), r.data_ptr(), pos.data_ptr(), near_partial.data_ptr(), batch, heads,
                                                                        b0.rankp, b0.rotp, near_size["window"], near_chunks, 0, b0.scale, _st()), "latent_decode")
        add(f"latent_decode on (value | key) rows, {cap} per head", batch, _hbm(_bytes(rings[0]), _graph_us([lambda r=r: attend(r) for r in rings])),
            f"latent_decode on {near_size['window']} latents", _hbm(_bytes(latents[0]), _graph_us([lambda r=r: near_attend(r) for r in latents])))
        merge = lambda: _lib.check_dense(lib.ajqd_group_merge(partial.data_ptr(), y.data_ptr() + 4 * a0.gate_column, y.shape[1], joined.data_ptr(),
                                                              joined.shape[1], batch, groups, a0.share, chunks, a0.dimp, _st()), "group_merge")
        expand = lambda w: _lib.check_dense(lib.ajqd_latent_expand(near_partial.data_ptr(), w.sink.data_ptr(), near_y.data_ptr() + 4 * b0.gate_column,
                                                                   near_y.shape[1], w.uv.data_ptr(), near_joined.data_ptr(), b0.joined, batch, heads,
                                                                   near_chunks, w.rankp, w.vdimp, _st()), "latent_expand")
        heads_read = 4 * batch * heads * chunks * a0.dimp
        add("group_merge: chunks merged, gated", batch, _hbm(heads_read + 6 * batch * heads * a0.dimp, _graph_us([merge] * 4)), "latent_expand",
            _hbm(_bytes(b0.uv, near_partial) + 2 * batch * heads * b0.vdimp, _graph_us([lambda w=w: expand(w) for w in blocks])))
        del rings, latents
        # ---- scan of one token: beside a product of as many bytes
        columns = [bf(batch, s0.taps - 1, s0.inner) for _ in scans]
        states = [torch.zeros((batch, s0.states // 4, s0.inner, 4), device=device) for _ in range(max(len(scans), min(32, int(4e8 / (4 * batch * s0.states * s0.inner)))))]
        splits = lib.ajqd_scan_splits(batch, s0.inner)
        parts = torch.empty((splits, batch, s0.low_rows), dtype=torch.float32, device=device)
        gated = torch.empty((batch, s0.inner), dtype=torch.bfloat16, device=device)

        def project_low(i):
            w = scans[i]
            _lib.check_dense(lib.ajqd_scan_project(ys.data_ptr(), ys.shape[1], columns[i].data_ptr(), w.conv.data_ptr(), w.conv_bias.data_ptr(), pos.data_ptr(),
                                                   w.w_low.data_ptr(), parts.data_ptr(), batch, w.inner, w.taps, w.low_rows, splits, _st()), "scan_project")

        def step(i):
            w = scans[i % len(scans)]
            args = _lib.ScanStepArgs(
                y=ys.data_ptr(), ring=columns[i % len(scans)].data_ptr(), weight=w.conv.data_ptr(), bias=w.conv_bias.data_ptr(), pos=pos.data_ptr(),
                partial=parts.data_ptr(), w_dt=w.w_dt.data_ptr(), dt_bias=w.dt_bias.data_ptr(), a2=w.a2.data_ptr(), d=w.skip.data_ptr(),
                state=states[i].data_ptr(), out=gated.data_ptr(), batch=batch, ldy=ys.shape[1], inner=w.inner, taps=w.taps, rows=w.low_rows,
                splits=splits, rank=w.rank, states=w.states, out_ld=w.inner)
            _lib.check_dense(lib.ajqd_scan_step(ctypes.byref(args), _st()), "scan_step")

        def equal_product(nbytes):
            n = max(16, nbytes // (2 * d) // 16 * 16)
            ws = [bf(n, d) * 0.02 for _ in range(max(2, min(32, int(4e8 / (2 * n * d)))))]
            to = torch.empty((batch, n), device=device)
            us = _graph_us([lambda w=w: near._dense_in(None, normed, None, None, None, 1e-5, 1, w, None, to, None, 0, 0) for w in ws])
            return f"dense_in {n} x {d} (equal bytes)", _hbm(2 * n * d + batch * (2 * d + 4 * n), us)

        nbytes = _bytes(s0.w_low, s0.conv, s0.conv_bias, columns[0]) + batch * (4 * s0.inner + 4 * splits * s0.low_rows)
        add("scan_project: convolution, step size | B | C", batch, _hbm(nbytes, _graph_us([lambda i=i: project_low(i) for i in range(len(scans))])), *equal_product(nbytes))
        nbytes = _bytes(s0.w_dt, s0.a2, s0.conv, s0.dt_bias, s0.skip, parts, columns[0]) + 2 * _bytes(states[0]) + batch * 10 * s0.inner
        add("scan_step: step sizes, states, gated output", batch, _hbm(nbytes, _graph_us([lambda i=i: step(i) for i in range(len(states))])), *equal_product(nbytes))
        del states, columns
        torch.cuda.empty_cache()

    # ---- prompts
    t, m = CONTEXT, PROMPT_ROWS * CONTEXT
    y = bf(m, a0.w_in.shape[0])
    kv = bf(PROMPT_ROWS, groups, t, a0.row)
    qp = bf(m, heads, a0.dimp)
    out = torch.empty((m, heads * a0.dimp), dtype=torch.bfloat16, device=device)
    near_cols = heads * (b0.dimp + b0.vdimp)
    near_q, near_kv, near_lat = bf(m, heads, b0.dimp + b0.rotp), bf(m, near_cols), bf(m, b0.width)
    gates = torch.rand((m, heads), device=device)
    near_out = torch.empty((m, b0.joined), dtype=torch.bfloat16, device=device)
    for reach in (window, t):
        pairs = sum(min(i + 1, reach) for i in range(t)) * PROMPT_ROWS * heads
        args = _lib.WindowedAttentionArgs(
            q=qp.data_ptr(), k1=kv.data_ptr() + 2 * a0.dimp, v=kv.data_ptr(), column_gates=y.data_ptr() + 2 * a0.gate_column, out=out.data_ptr(),
            k1_batch=kv.stride(0), v_batch=kv.stride(0), k1_head=kv.stride(1), v_head=kv.stride(1), k1_row=a0.row, v_row=a0.row, d1=a0.dimp, d2=0,
            dv=a0.dimp, batch=PROMPT_ROWS, heads=heads, share=a0.share, seq=t, rows=t, prior=0, window=reach, keep=size["keep"], gate_ld=y.shape[1],
            out_ld=out.shape[1], scale=a0.scale)
        near_args = _lib.WindowedAttentionArgs(
            q=near_q.data_ptr(), k1=near_kv.data_ptr(), k2=near_lat.data_ptr() + 2 * b0.rankp, v=near_kv.data_ptr() + 2 * heads * b0.dimp, sink=b0.sink.data_ptr(),
            gates=gates.data_ptr(), out=near_out.data_ptr(), k1_batch=t * near_cols, k2_batch=t * b0.width, v_batch=t * near_cols, k1_row=near_cols,
            k1_head=b0.dimp, k2_row=b0.width, v_row=near_cols, v_head=b0.vdimp, d1=b0.dimp, d2=b0.rotp, dv=b0.vdimp, batch=PROMPT_ROWS, heads=heads,
            seq=t, rows=t, prior=0, window=reach, out_ld=b0.joined, scale=b0.scale)
        measured = []
        for a, flops in ((args, 4.0 * pairs * size["dim"]), (near_args, 2.0 * pairs * (near_size["dim"] + near_size["rot"] + near_size["vdim"]))):
            us = _graph_us([lambda: _lib.check_dense(lib.ajqd_windowed_prefill(ctypes.byref(a), _st()), "windowed_prefill")] * 4)
            measured.append({"us": us, "TFLOP/s": flops / us * 1e-6, "frac_mfma_peak": flops / us * 1e-6 / MFMA_BF16_PEAK_TFLOPS})
        add(f"windowed_prefill, window {reach} of {t}, kept rows, column gates", PROMPT_ROWS, measured[0], "windowed_prefill (latent layer)", measured[1])
    del near_kv, near_q
    xs, delta, near_x = (torch.randn(shape, device=device) for shape in ((m, streams, d), (m, d), (m, d)))
    sub = subs[0]
    like = _hbm(m * d * 16, _graph_us([lambda: _add_norms(near_x, delta, None, None, b0.gain1, b0.gain2, 1e-5, 1, d,
                                                         torch.bfloat16)] * 3))
    add("streams_norm: update of the streams, next input, norm", m, _hbm(m * d * (8 * streams + 4 + 2), _graph_us([lambda: model._streams_norm(xs, delta, sub, sub)] * 3)),
        "add_norms (residual add, two norms)", like)
    del xs, delta, near_x
    near_yf = torch.randn((m, b0.w1.shape[0]), device=device)
    near_q = bf(m, heads, b0.dimp + b0.rotp)
    latent_split = lambda: _lib.check_dense(lib.ajqd_latent_split(
        near_yf.data_ptr(), _lib.AJQD_F32, near_yf.shape[1], ctypes.byref(b0.shape), b0.latent_gain.data_ptr(), b0.cosine.data_ptr(), b0.sine.data_ptr(),
        CONTEXT + 512, m, t, 0, None, 0, 0, near_q.data_ptr(), near_q.shape[2], near_q.data_ptr() + 2 * b0.dimp, near_q.shape[2], near_lat.data_ptr(),
        t * b0.width, gates.data_ptr(), _lib.AJQD_BF16, _st()), "latent_split")
    like = _hbm(m * (4 * near_yf.shape[1] + 2 * heads * near_q.shape[2] + 2 * b0.width), _graph_us([latent_split] * 3))
    add("key_value_split: norms, rotation, key / value rows", m, _hbm(m * 2 * a0.dimp * (2 * heads + 3 * groups),
                                                                      _graph_us([lambda: model._split(y, a0, qp, 0, kv, t, 0, None, 0, 0)] * 3)), "latent_split", like)
    del near_yf, near_q, near_lat, y, kv, qp
    yb = bf(m, 2 * near_size["ff"])
    like = _hbm(m * near_size["ff"] * 6, _graph_us([lambda: near._gate(yb, near_out, b0)] * 3))
    del yb
    mid = bf(m, f0.width)
    add("activation: squared relu in place", m, _hbm(4 * mid.numel(), _graph_us([lambda: model._activated(mid, f0.act)] * 3)), "gated_activation", like)
    ys = bf(m, 2 * s0.inner)
    add("conv_silu", m, _hbm(4 * m * s0.inner, _graph_us([lambda: model._convolved(ys, s0, None, 0, None, t)] * 3)), "gated_activation", like)
    x, raw, low = bf(m, s0.inner), bf(m, s0.inner), bf(m, s0.low_rows)
    for rows_of in (PROMPT_ROWS, 1):
        n = rows_of * t
        us = _graph_us([lambda: model._recur(x[:n], raw[:n], low[:n], ys[:n], s0, None, rows_of, t, 0, None)] * 2, reps=5)
        exps = n * s0.inner * size["state"]
        add("scan: recurrence, gated output", n, _hbm(n * (8 * s0.inner + 4 * s0.states), us), "gated_activation", like,
            frac_exp_peak=exps / us * 1e-3 / EXP_PEAK_GIGA)
    del model, near
    torch.cuda.empty_cache()
    return rows


def bench_hybrid(device, log=print) -> dict:
    out = {}
    for name, size in SIZES.items():
        out[name] = {"config": {k: (v if not isinstance(v, Loop) else vars(v)) for k, v in size.items()},
                     "model": bench_whole(name, device, log), "kernels": bench_kernels(name, device, log)}
    return out
