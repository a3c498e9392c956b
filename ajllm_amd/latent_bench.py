"""Throughput of the dense latent-attention decoder (``latent.LatentLM``) at layer sizes of real models, random weights,
beside the library's closest existing model at equal size: the quantized Transformer with W8A16 linears and a bf16
KV cache (``decoding.FusedDecoder``), with as many layers as the latent model has layer runs.

Whole-model figures (prompt of 4 x 2048 tokens, decoding at context 2048 with batch 1, 8 and 32) and, kernel by kernel, the
share of its roofline (HBM bytes or bf16 MFMA flops against the vendor peaks) next to the like kernel of the other model.
Bytes are the algorithmic ones: weights, cache rows and activations once.
"""

from __future__ import annotations

import ctypes
import time

import torch

from . import _lib, decoding, latent
from .attention import flash_prefill
from .e2e_bench import build_quantized_model
from .quant import quantize_w8, repack_w8, w8a16_matmul

HBM_PEAK_GBS = 8000.0
MFMA_BF16_PEAK_TFLOPS = 2500.0
CONTEXT = 2048
PROMPT_ROWS = 4
SIZES = {
    "width 2048": dict(width=2048, heads=16, dim=128, rot=64, vdim=128, rank=512, ff=5632, window=1024, layers=8,
                       loop=latent.Loop(2, 6, 2), kv_heads=16),
    "width 4096": dict(width=4096, heads=32, dim=128, rot=64, vdim=128, rank=512, ff=14336, window=1024, layers=4,
                       loop=latent.Loop(1, 3, 2), kv_heads=8),
}
VOCAB = 32000


def build_latent(size: dict, device, seed: int = 77, dtype: torch.dtype = torch.bfloat16) -> latent.LatentLM:
    torch.manual_seed(seed)
    mixer = dict(num_heads=size["heads"], dim=size["dim"], rot_dim=size["rot"], value_dim=size["vdim"], kv_rank=size["rank"],
                 scale=(size["dim"] + size["rot"]) ** -0.5, rot_base=10_000.0, window=size["window"])
    with torch.device(device):
        model = latent.LatentLM(VOCAB, CONTEXT + 512, size["width"], [(mixer, (size["ff"], "relu"))] * size["layers"], size["loop"])
    model = model.to(dtype).eval()
    model.prepare()
    return model


def _graph_us(launches, reps: int = 20) -> float:
    """Microseconds per launch of ``launches`` (a list of zero-argument calls), chained in a HIP graph of at least 48."""
    launches = launches * max(1, 48 // len(launches))
    stream = torch.cuda.Stream()
    torch.cuda.synchronize()
    with torch.cuda.stream(stream):
        for fn in launches:
            fn()
        stream.synchronize()
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph, stream=stream):
            for fn in launches:
                fn()
        graph.replay()
        stream.synchronize()
        start, stop = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        start.record(stream)
        for _ in range(reps):
            graph.replay()
        stop.record(stream)
        stop.synchronize()
    return start.elapsed_time(stop) * 1e3 / reps / len(launches)


def _st() -> int:
    return torch.cuda.current_stream().cuda_stream


def _hbm(nbytes: float, us: float) -> dict:
    return {"us": us, "GB/s": nbytes / us * 1e-3, "frac_hbm_peak": nbytes / us * 1e-3 / HBM_PEAK_GBS}


def _seconds(fn, reps: int = 5) -> float:
    fn()
    torch.cuda.synchronize()
    times = []
    for _ in range(reps):
        t0 = time.perf_counter()
        fn()
        torch.cuda.synchronize()
        times.append(time.perf_counter() - t0)
    return sorted(times)[len(times) // 2]


@torch.no_grad()
def bench_whole(size: dict, device, log=print, batches=(1, 8, 32), steps: int = 64) -> dict:
    """Prompt and decode throughput of both models."""
    g = torch.Generator().manual_seed(5)
    prompt = torch.randint(0, VOCAB, (max(batches), CONTEXT), generator=g).to(device)
    model = build_latent(size, device)
    runs = len(model.runs)
    weight_bytes = sum(2 * sum(t.numel() for t in (w.w1, w.w2, w.uv, w.ukt, w.wo)) for i, _ in model.runs for w in [model._blocks[i]])
    cache = model.new_cache(PROMPT_ROWS, CONTEXT)

    def prefill():
        cache.reset()
        model(prompt[:PROMPT_ROWS], cache, last_token_only=True)

    seconds = _seconds(prefill)
    out: dict = {"layer_runs": runs, "prompt": {"tokens": PROMPT_ROWS * CONTEXT, "latent_ms": seconds * 1e3,
                                                "latent_tok/s": PROMPT_ROWS * CONTEXT / seconds}, "decode": []}
    for batch in batches:
        dec = decoding.DenseDecoder(model, batch, CONTEXT + steps + 16)
        dec.prefill(prompt[:batch], rows_per_pass=PROMPT_ROWS)
        dec.generate(12)
        t0 = time.perf_counter()
        dec.generate(12 + steps)
        step = (time.perf_counter() - t0) / steps
        cache_bytes = 2 * batch * sum(ring.shape[1] * ring.shape[2] for ring in dec.cache.rings)
        total = weight_bytes + cache_bytes + 2 * model._head.numel()
        out["decode"].append({"batch": batch, "latent_ms_per_step": step * 1e3, "latent_tok/s": batch / step,
                              "latent_bytes_per_step": total, "latent_frac_hbm_peak": total / step * 1e-9 / HBM_PEAK_GBS})
        del dec
    del model, cache
    torch.cuda.empty_cache()
    near = build_quantized_model(device, "w8a16", config=dict(
        vocab_size=VOCAB, context_length=CONTEXT + 512, d_model=size["width"], num_layers=runs, num_heads=size["heads"],
        num_kv_heads=size["kv_heads"], d_ff=size["ff"]))
    dec = decoding.FusedDecoder(near, PROMPT_ROWS, CONTEXT + 8, torch.bfloat16)
    seconds = _seconds(lambda: dec.prefill(prompt[:PROMPT_ROWS], fused=True))
    out["prompt"].update({"w8a16_transformer_ms": seconds * 1e3, "w8a16_transformer_tok/s": PROMPT_ROWS * CONTEXT / seconds})
    del dec
    packed = sum(m.wq.numel() * 4 + m.meta.numel() * m.meta.element_size() for m in near.modules() if hasattr(m, "wq"))
    for row in out["decode"]:
        batch = row["batch"]
        dec = decoding.FusedDecoder(near, batch, CONTEXT + steps + 16, torch.bfloat16)
        dec.prefill(prompt[:batch], rows_per_pass=PROMPT_ROWS, fused=True)
        dec.generate(12)
        t0 = time.perf_counter()
        dec.generate(12 + steps)
        step = (time.perf_counter() - t0) / steps
        total = packed + 2 * 2 * batch * runs * size["kv_heads"] * CONTEXT * (size["width"] // size["heads"])
        row.update({"w8a16_transformer_ms_per_step": step * 1e3, "w8a16_transformer_tok/s": batch / step,
                    "w8a16_transformer_frac_hbm_peak": total / step * 1e-9 / HBM_PEAK_GBS})
        del dec
    del near
    torch.cuda.empty_cache()
    log("latent whole model", out)
    return out


@torch.no_grad()
def bench_kernels(size: dict, device, log=print, batches=(1, 8, 32)) -> list[dict]:
    """Kernel by kernel: microseconds in a graph chain over distinct operands, share of the roofline, and the like kernel."""
    lib, quant = _lib.load_dense(), _lib.load()
    d, heads, ff, window = size["width"], size["heads"], size["ff"], size["window"]
    model = build_latent({**size, "layers": max(4, size["layers"]), "loop": None}, device)
    blocks = model._blocks
    w0 = blocks[0]
    copies = range(len(blocks))
    rows: list[dict] = []

    def add(name, batch, ours, like, theirs):
        key = "frac_hbm_peak" if "frac_hbm_peak" in ours else "frac_mfma_peak"
        row = {"kernel": name, "batch": batch, **ours, "like_kernel": like, "like": theirs, "like_over_ours": theirs[key] / ours[key]}
        log("latent kernel", row)
        rows.append(row)

    def w8(batch, n, k):
        """The W8A16 product of that shape (GEMV up to 16 rows, weight-streaming kernel above)."""
        made = []
        for _ in range(max(2, int(3e8 / (n * k)) + 1)):
            q, s = quantize_w8(torch.randn((n, k), device=device) * 0.02)
            made.append((repack_w8(q), s))
        x = torch.randn((batch, k), device=device).to(torch.bfloat16)
        us = _graph_us([lambda a=a, s=s: w8a16_matmul(x, a, s, torch.float32) for a, s in made])
        return _hbm(n * k + 2 * n + 2 * batch * k + 4 * batch * n, us)

    for batch in batches:
        x = torch.randn((batch, d), device=device)
        normed = torch.randn((batch, d), device=device).to(torch.bfloat16)
        y = torch.randn((batch, w0.w1.shape[0]), device=device)
        joined = torch.randn((batch, w0.joined), device=device).to(torch.bfloat16)
        gated = joined.data_ptr() + 2 * heads * w0.vdimp
        prologue = batch <= latent.NORM_PROLOGUE_ROWS

        def project(w):
            model._dense_in(x if prologue else None, normed, normed, w.gain1, w.gain2, w.eps, 1, w.w1, w.w2, y, gated, w.joined, w.act)

        nbytes = 2 * (w0.w1.numel() + w0.w2.numel()) + batch * (4 * d + 4 * w0.w1.shape[0] + 2 * ff)
        add("dense_in: queries | latent | gates and gate | up", batch, _hbm(nbytes, _graph_us([lambda i=i: project(blocks[i]) for i in copies])),
            f"W8A16 product {2 * ff} x {d} (w1|w3)", w8(batch, 2 * ff, d))
        out = lambda w: _lib.check_dense(lib.ajqd_dense_out(joined.data_ptr(), w.wo.data_ptr(), x.data_ptr(), None, None, batch,
                                                            w.joined, d, _st()), "dense_out")
        add("dense_out: heads and feed-forward back, residual added", batch,
            _hbm(2 * w0.wo.numel() + batch * (2 * w0.joined + 8 * d), _graph_us([lambda i=i: out(blocks[i]) for i in copies])),
            f"W8A16 product {d} x {ff} (w2)", w8(batch, d, ff))
        small_n = w0.ukt.numel() * 2 // 2048   # a W8A16 product of as many bytes
        small = w8(batch, small_n, 2048)
        pos = torch.tensor([CONTEXT + 7], device=device)
        q = torch.empty((batch, heads, w0.width), dtype=torch.bfloat16, device=device)
        ring_bytes = 2 * batch * window * w0.width
        rings = [torch.randn((batch, window, w0.width), device=device).to(torch.bfloat16) for _ in range(min(32, int(4e8 / ring_bytes) + 1))]
        absorb = lambda w: _lib.check_dense(lib.ajqd_latent_absorb(
            y.data_ptr(), y.shape[1], ctypes.byref(w.shape), w.ukt.data_ptr(), w.latent_gain.data_ptr(), w.cosine.data_ptr(),
            w.sine.data_ptr(), CONTEXT + 512, pos.data_ptr(), q.data_ptr(), rings[0].data_ptr(), window, batch, _st()), "latent_absorb")
        add("latent_absorb: queries into the latent space, cache row", batch,
            _hbm(2 * w0.ukt.numel() + batch * (4 * y.shape[1] + 2 * heads * w0.width), _graph_us([lambda i=i: absorb(blocks[i]) for i in copies])),
            f"W8A16 product {small_n} x 2048 (equal bytes)", small)
        chunks = lib.ajqd_latent_decode_chunks(batch, heads, w0.rankp, w0.rotp, window)
        partial = torch.empty(lib.ajqd_latent_decode_workspace(batch, heads, w0.rankp, chunks), dtype=torch.uint8, device=device)
        attend = lambda r: _lib.check_dense(lib.ajqd_latent_decode(q.data_ptr(), r.data_ptr(), pos.data_ptr(), partial.data_ptr(), batch, heads,
                                                                   w0.rankp, w0.rotp, window, chunks, 0, w0.scale, _st()), "latent_decode")
        # the other model's decode attention over a bf16 cache of about as many bytes
        hd, hkv = d // heads, size["kv_heads"]
        context = max(16, ring_bytes // (4 * batch * hkv * hd))
        qkv = torch.randn((batch, (heads + 2 * hkv) * hd), device=device)
        caches = [torch.randn((2, batch, hkv, context, hd), device=device).to(torch.bfloat16) for _ in rings]
        cos = torch.ones((context, hd // 2), device=device)
        at = torch.tensor([context - 1], device=device)
        done = torch.empty((batch, d), dtype=torch.bfloat16, device=device)
        need = int(quant.ajq_attn_step_workspace_bytes(batch, heads))
        ws = torch.empty(max(need, 16), dtype=torch.uint8, device=device)
        step = lambda c: _lib.check(quant.ajq_attn_step(qkv.data_ptr(), cos.data_ptr(), cos.data_ptr(), at.data_ptr(), c[0].data_ptr(),
                                                        c[1].data_ptr(), _lib.AJQ_KV_BF16, batch, heads, hkv, hd, context, done.data_ptr(),
                                                        ws.data_ptr(), need, _st()), "attn_step")
        add(f"latent_decode: attention over {window} cached rows", batch, _hbm(ring_bytes, _graph_us([lambda r=r: attend(r) for r in rings])),
            f"attn_step (bf16 cache, {context} positions: equal bytes)",
            _hbm(4 * batch * hkv * hd * context, _graph_us([lambda c=c: step(c) for c in caches])))
        gate = y.data_ptr() + 4 * w0.gate_column
        expand = lambda w: _lib.check_dense(lib.ajqd_latent_expand(partial.data_ptr(), w.sink.data_ptr(), gate, y.shape[1], w.uv.data_ptr(),
                                                                   joined.data_ptr(), w.joined, batch, heads, chunks, w.rankp, w.vdimp, _st()), "latent_expand")
        add("latent_expand: chunks merged, values expanded, gated", batch,
            _hbm(2 * w0.uv.numel() + partial.numel() + 2 * batch * heads * w0.vdimp, _graph_us([lambda i=i: expand(blocks[i]) for i in copies])),
            f"W8A16 product {small_n} x 2048 (equal bytes)", small)
        del rings, caches
        torch.cuda.empty_cache()

    # ---- prompts: attention on MFMA, and the row operators
    t = CONTEXT
    kv_cols = heads * (w0.dimp + w0.vdimp)
    qp = torch.randn((PROMPT_ROWS * t, heads, w0.dimp + w0.rotp), device=device).to(torch.bfloat16)
    kv = torch.randn((PROMPT_ROWS * t, kv_cols), device=device).to(torch.bfloat16)
    lat = torch.randn((PROMPT_ROWS * t, w0.width), device=device).to(torch.bfloat16)
    gates = torch.rand((PROMPT_ROWS * t, heads), device=device)
    joined = torch.empty((PROMPT_ROWS * t, w0.joined), dtype=torch.bfloat16, device=device)
    hd, hkv = d // heads, size["kv_heads"]
    fq = torch.randn((PROMPT_ROWS, heads, t, hd), device=device)
    fk, fv = (torch.randn((PROMPT_ROWS, hkv, t, hd), device=device).to(torch.bfloat16) for _ in range(2))
    us = _graph_us([lambda: flash_prefill(fq, fk, fv, 0, torch.bfloat16)] * 4)
    flops = 4.0 * PROMPT_ROWS * heads * hd * t * (t + 1) / 2
    theirs = {"us": us, "TFLOP/s": flops / us * 1e-6, "frac_mfma_peak": flops / us * 1e-6 / MFMA_BF16_PEAK_TFLOPS}
    for reach in (window, t):
        args = _lib.WindowedAttentionArgs(
            q=qp.data_ptr(), k1=kv.data_ptr(), k2=lat.data_ptr() + 2 * w0.rankp, v=kv.data_ptr() + 2 * heads * w0.dimp, sink=w0.sink.data_ptr(),
            gates=gates.data_ptr(), out=joined.data_ptr(), k1_batch=t * kv_cols, k2_batch=t * w0.width, v_batch=t * kv_cols, k1_row=kv_cols,
            k1_head=w0.dimp, k2_row=w0.width, v_row=kv_cols, v_head=w0.vdimp, d1=w0.dimp, d2=w0.rotp, dv=w0.vdimp, batch=PROMPT_ROWS,
            heads=heads, seq=t, rows=t, prior=0, window=reach, out_ld=w0.joined, scale=w0.scale)
        us = _graph_us([lambda: _lib.check_dense(lib.ajqd_windowed_prefill(ctypes.byref(args), _st()), "windowed_prefill")] * 4)
        pairs = sum(min(i + 1, reach) for i in range(t)) * PROMPT_ROWS * heads
        flops = 2.0 * pairs * (size["dim"] + size["rot"] + size["vdim"])
        add(f"windowed_prefill, window {reach} of {t}", PROMPT_ROWS,
            {"us": us, "TFLOP/s": flops / us * 1e-6, "frac_mfma_peak": flops / us * 1e-6 / MFMA_BF16_PEAK_TFLOPS},
            f"attn_prefill (causal, bf16 cache, head_dim {hd})", theirs)
    m = PROMPT_ROWS * t
    xs, delta = torch.randn((m, d), device=device), torch.randn((m, d), device=device)
    both = _graph_us([lambda: latent._add_norms(xs, delta, None, None, w0.gain1, w0.gain2, 1e-5, 1, d, torch.bfloat16)] * 3)
    one = torch.empty((m, d), dtype=torch.bfloat16, device=device)
    like = _graph_us([lambda: _lib.check(quant.ajq_add_rmsnorm(xs.data_ptr(), delta.data_ptr(), w0.gain1.data_ptr(), 1e-5, one.data_ptr(), m, d,
                                                               _st()), "add_rmsnorm")] * 3)
    add("add_norms: residual add and two norms", m, _hbm(m * d * (4 + 4 + 4 + 2 + 2), both), "add_rmsnorm (one norm)", _hbm(m * d * (4 + 4 + 4 + 2), like))
    yb = torch.randn((m, 2 * ff), device=device).to(torch.bfloat16)
    ours = _graph_us([lambda: model._gate(yb, joined, w0)] * 3)
    ab, go = torch.randn((m, 2 * ff), device=device), torch.empty((m, ff), dtype=torch.bfloat16, device=device)
    like = _graph_us([lambda: _lib.check(quant.ajq_swiglu(ab.data_ptr(), go.data_ptr(), m, ff, _st()), "swiglu")] * 3)
    add("gated_activation (bf16 in)", m, _hbm(m * ff * 6, ours), "swiglu (fp32 in)", _hbm(m * ff * 10, like))
    del ab, yb
    yf = torch.randn((m, w0.w1.shape[0]), device=device)
    split = lambda: _lib.check_dense(lib.ajqd_latent_split(
        yf.data_ptr(), _lib.AJQD_F32, yf.shape[1], ctypes.byref(w0.shape), w0.latent_gain.data_ptr(), w0.cosine.data_ptr(), w0.sine.data_ptr(),
        CONTEXT + 512, m, t, 0, None, 0, 0, qp.data_ptr(), qp.shape[2], qp.data_ptr() + 2 * w0.dimp, qp.shape[2], lat.data_ptr(),
        t * w0.width, gates.data_ptr(), _lib.AJQD_BF16, _st()), "latent_split")
    qkv = torch.randn((m, (heads + 2 * hkv) * hd), device=device)
    cos = torch.ones((t, hd // 2), device=device)
    like = _graph_us([lambda: _lib.check(quant.ajq_rope_prefill(qkv.data_ptr(), cos.data_ptr(), cos.data_ptr(), fq.data_ptr(), fk.data_ptr(), fv.data_ptr(),
                                                                _lib.AJQ_KV_BF16, PROMPT_ROWS, t, heads, hkv, hd, 0, t, _st()), "rope_prefill")] * 3)
    add("latent_split: rotation, latent norm, cache rows", m, _hbm(m * (4 * yf.shape[1] + 2 * heads * qp.shape[2] + 2 * w0.width), _graph_us([split] * 3)),
        "rope_prefill", _hbm(m * hd * (4 * (heads + 2 * hkv) + 4 * heads + 4 * hkv), like))
    del model
    torch.cuda.empty_cache()
    return rows


def bench_latent(device, log=print) -> dict:
    out = {}
    for name, size in SIZES.items():
        out[name] = {"config": {k: (v if not isinstance(v, latent.Loop) else vars(v)) for k, v in size.items()},
                     "model": bench_whole(size, device, log), "kernels": bench_kernels(size, device, log)}
    return out
