"""Key-value attention, the selective scan and hyper-connected streams on the GPU: every operator alone and the whole Purusun
decoder against the plain implementation (oracle/purusun.py, float64 on the host), in fp32 (where the comparison is sharp) and in
bf16."""

import ctypes
import json
import math

import pytest
import torch
from safetensors.torch import save_file

from ajllm_amd import _lib, checkpoint, decoding, dense, hybrid, modeling
from oracle import purusun as O
from tests.hybrid_models import SCALING, attention, config, random_weights, scan

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
# relative rms error of logits against the float64 implementation on the same (bf16-representable) weights
LOGIT_TOL = {torch.float32: 2e-5, torch.bfloat16: 2.5e-2}


def _rel(got: torch.Tensor, want: torch.Tensor) -> float:
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    assert torch.isfinite(got).all()
    return float((got - want).norm() / want.norm())


def _ok(status: int) -> None:
    _lib.check_dense(status, "test")


def _st() -> int:
    return torch.cuda.current_stream().cuda_stream


def _p(t):
    return t.data_ptr()


def _bf(g, *shape, std=1.0):
    return (torch.randn(shape, generator=g) * std).to(torch.bfloat16)


def _padded(t: torch.Tensor, *sizes: int) -> torch.Tensor:
    out = torch.zeros(sizes, dtype=t.dtype)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def _up(n, to):
    return (n + to - 1) // to * to


def _build(cfg, weights, device, dtype):
    with torch.device("meta"):
        model = modeling.build_model(cfg)
    model.load_state_dict({k: weights[n].to(device=device, dtype=dtype) for k, n in model.checkpoint_names().items()}, assign=True)
    return model.eval()


def _tokens(cfg, count, seed):
    return torch.randint(0, cfg["vocab"], (count,), generator=torch.Generator().manual_seed(seed)).tolist()


def _ids(tokens, device):
    return torch.tensor([tokens], device=device)


# ------------------------------------------------------------------ residual streams
def _coefficients(g, s):
    return {"in": torch.randn(s, generator=g), "out": torch.randn(s, generator=g), "mix": torch.randn((s, s), generator=g)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("streams", [1, 2, 3, 5, 16])
@pytest.mark.parametrize("true_width", [16, 52, 2048, 9000])
def test_streams_norm(cuda, dtype, streams, true_width):
    g, rows, width = torch.Generator().manual_seed(true_width + streams), 5, _up(true_width, 16)
    x = _padded(torch.randn((rows, streams, true_width), generator=g), rows, streams, width)
    delta, scale = (_padded(torch.randn(n, generator=g), *n[:-1], width) for n in ((rows, true_width), (true_width,)))
    gain = _padded(torch.randn(true_width, generator=g), width)
    hc, following = _coefficients(g, streams), torch.randn(streams, generator=g)
    want = O.hyper_sublayer(x.double().transpose(0, 1), {k: v.double() for k, v in hc.items()}, lambda u: delta.double() * scale.double())
    d = {k: v.to(cuda) for k, v in dict(x=x, delta=delta, scale=scale, gain=gain, following=following, **hc).items()}
    normed, u = torch.full((rows, width), 9.0, dtype=dtype, device=cuda), torch.full((rows, width), 9.0, device=cuda)
    lib = _lib.load_dense()
    _ok(lib.ajqd_streams_norm(_p(d["x"]), _p(d["delta"]), _p(d["scale"]), _p(d["out"]), _p(d["mix"]), _p(d["following"]), _p(d["gain"]), 1e-3,
                              _p(normed), _p(u), streams, rows, true_width, width, dense._flag(dtype), _st()))
    assert _rel(d["x"].transpose(0, 1), want) < 1e-6
    reads = (following.double()[:, None, None] * want).sum(0)
    assert _rel(u, reads) < 2e-6
    plain = O.centered_rms_norm(reads[:, :true_width], gain[:true_width].double() - 1, 1e-3)
    assert _rel(normed[:, :true_width], plain) < (2e-6 if dtype == torch.float32 else 4e-3) and (normed[:, true_width:] == 0).all()
    before = d["x"].clone()   # without an update: the plain sum, nothing written
    _ok(lib.ajqd_streams_norm(_p(d["x"]), None, None, None, None, None, None, 0.0, None, _p(u), streams, rows, true_width, width,
                              dense._flag(dtype), _st()))
    assert torch.equal(before, d["x"]) and _rel(u, want.sum(0)) < 2e-6


@pytest.mark.parametrize("dtype", DTYPES)
def test_embed_streams(cuda, dtype):
    table, tokens, reads = torch.randn(19, 32).to(dtype), torch.tensor([3, 18, 0, 7, 7, 2]), torch.randn(3)
    x, u = torch.empty((6, 3, 32), device=cuda), torch.empty((6, 32), device=cuda)
    dt, ids, dr = table.to(cuda), tokens.to(cuda), reads.to(cuda)
    _ok(_lib.load_dense().ajqd_embed_streams(_p(ids), 6, _p(dt), 19, _p(dr), _p(x), _p(u), 3, 32, dense._flag(dtype), _st()))
    for s in range(3):
        assert torch.equal(x[:, s].cpu(), table.float()[tokens])
    assert _rel(u, table.double()[tokens] * reads.double().sum()) < 1e-6


@pytest.mark.parametrize("batch", [1, 3, 17, 40])
@pytest.mark.parametrize("shape", [(2, 40, 16), (1, 264, 64), (3, 2056, 96), (16, 72, 48), (2, 48, 8192), (4, 512, 8192)])
def test_dense_out_streams(cuda, batch, shape):
    streams, k, width = shape
    g = torch.Generator().manual_seed(sum(shape) + batch)
    a, w = _bf(g, batch, k), _bf(g, width, k, std=k ** -0.5)
    x, scale, hc, following = torch.randn((batch, streams, width), generator=g), torch.randn(width, generator=g), _coefficients(g, streams), torch.randn(streams, generator=g)
    y = (a.double() @ w.double().T) * scale.double()
    want = O.hyper_sublayer(x.double().transpose(0, 1), {n: v.double() for n, v in hc.items()}, lambda u: y)
    d = {n: v.to(cuda) for n, v in dict(a=a, w=w, x=x, scale=scale, following=following, **hc).items()}
    for reader in (following, None):
        u = torch.full((batch, width), 9.0, device=cuda)
        d["x"].copy_(x)
        _ok(_lib.load_dense().ajqd_dense_out_streams(_p(d["a"]), _p(d["w"]), _p(d["x"]), _p(d["scale"]), _p(d["out"]), _p(d["mix"]),
                                                     _p(d["following"]) if reader is not None else None, _p(u), streams, batch, k, width, _st()))
        assert _rel(d["x"].transpose(0, 1), want) < 2e-6
        weights = reader.double() if reader is not None else torch.ones(streams).double()
        assert _rel(u, (weights[:, None, None] * want).sum(0)) < 4e-6


@pytest.mark.parametrize("dtype", DTYPES)
def test_squared_relu(cuda, dtype):
    y = torch.randn(7, 40).to(dtype)
    dy = y.to(cuda)
    _ok(_lib.load_dense().ajqd_activation(_p(dy), _p(dy), 280, _lib.AJQD_ACTIVATIONS["squared_relu"], dense._flag(dtype), _st()))
    assert _rel(dy, torch.relu(y.double()) ** 2) < (1e-6 if dtype == torch.float32 else 4e-3)


# ------------------------------------------------------------------ key-value attention
SPLITS = [  # heads, groups, dim, rot
    (4, 2, 16, 8), (3, 1, 12, 6), (6, 3, 40, 40), (5, 5, 64, 16), (4, 1, 128, 32), (2, 2, 200, 120), (9, 3, 72, 0), (1, 1, 20, 2), (2, 1, 300, 300),
]


def _split_weights(g, shape):
    heads, groups, dim, rot = shape
    return {"q": torch.randn(dim, generator=g), "k": torch.randn(dim, generator=g), "rot": {"base": 700.0, "dims": rot, "scaling": SCALING}}


def _split_plain(y, w, shape, dimp, position):
    """Queries, rotated keys, values of one projection row."""
    heads, groups, dim, _ = shape
    parts = y[: (heads + groups) * dimp].view(heads + groups, dimp)[:, :dim].double()
    turned = [O.rotate(v / O.rms(v, 1e-4) * w[n].double(), position, w["rot"]) for v, n in ((parts[:heads], "q"), (parts[heads:], "k"))]
    return turned[0], turned[1], parts[heads:]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SPLITS)
@pytest.mark.parametrize("static", [False, True])
def test_key_value_split(cuda, dtype, shape, static):
    """Rows of two sequences at far positions, in a linear buffer or each in its slot of a ring."""
    heads, groups, dim, rot = shape
    g, dimp, batch = torch.Generator().manual_seed(sum(shape)), _up(dim, 16), 2
    seq, start, prior = (1, 100_007, 0) if static else (5, 70_001, 2)
    cap, kept = (11, 3) if static else (prior + seq, 0)
    w = _split_weights(g, shape)
    ld = (heads + groups) * dimp + 16
    y = torch.randn((batch * seq, ld), generator=g).to(dtype)
    y[:, : (heads + groups) * dimp].view(-1, heads + groups, dimp)[:, :, dim:] = 0
    turns = (dense.rotary_frequencies(700.0, rot, dense.FrequencyScaling(**{k: float(v) for k, v in SCALING.items()})) / math.pi).to(cuda)
    d = {k: v.to(cuda) for k, v in dict(y=y, qg=_padded(w["q"], dimp), kg=_padded(w["k"], dimp), pos=torch.tensor([start])).items()}
    q = torch.full((batch * seq, heads, 16 + dimp), 9.0, dtype=dtype, device=cuda)
    rows = torch.full((batch, groups, cap, 2 * dimp), 9.0, dtype=dtype, device=cuda)
    args = _lib.KeyValueSplitArgs(
        y=_p(d["y"]), q_gain=_p(d["qg"]), k_gain=_p(d["kg"]), half_turns=_p(turns), pos=_p(d["pos"]) if static else None, q=_p(q), rows=_p(rows),
        rows_batch=rows.stride(0), rows_head=rows.stride(1), tokens=batch * seq, seq=seq, start=0 if static else start, ldy=ld, heads=heads,
        groups=groups, dim=dim, dimp=dimp, rot=rot, q_ld=16 + dimp, q_at=16, prior=prior, cap=cap, kept=kept, eps=1e-4)
    _ok(_lib.load_dense().ajqd_key_value_split(ctypes.byref(args), dense._flag(dtype), dense._flag(dtype), _st()))
    tol = 1e-6 if dtype == torch.float32 else 4e-3
    assert (q[:, :, :16] == 0).all() and (q[:, :, 16 + dim:] == 0).all()
    written = set()
    for m in range(batch * seq):
        b, t = divmod(m, seq)
        slot = kept + (start - kept) % (cap - kept) if static else prior + t
        written.add(slot)
        wq, wk, wv = _split_plain(y[m], w, shape, dimp, start + t)
        assert _rel(q[m, :, 16:16 + dim], wq) < tol
        row = rows[b, :, slot]
        assert _rel(row[:, dimp:dimp + dim], wk) < tol and torch.equal(row[:, :dim].double().cpu(), wv)
        assert (row[:, dim:dimp] == 0).all() and (row[:, dimp + dim:] == 0).all()
    for slot in set(range(cap)) - written:
        assert (rows[:, :, slot] == 9.0).all()


def _attention_case(b, heads, groups, t, prior, d, seed):
    g = torch.Generator().manual_seed(seed)
    return dict(q=_bf(g, b, t, heads, d), rows=_bf(g, b, groups, prior + t, 2 * d), gate=_bf(g, b * t, heads * d))


def _attention_plain(c, prior, window, keep, scale):
    q, rows = c["q"].double(), c["rows"].double()
    b, t, heads, d = q.shape
    groups, n = rows.shape[1:3]
    mask = O.visible_mask(n, window or None, keep)[prior:]
    out = torch.empty(b, t, heads, d, dtype=torch.float64)
    for i in range(b):
        for h in range(heads):
            r = rows[i, h // (heads // groups)]
            out[i, :, h] = O.softmax(((q[i, :, h] @ r[:, d:].T) * scale).masked_fill(~mask, float("-inf"))) @ r[:, :d]
    return out.reshape(b * t, heads * d) * torch.sigmoid(c["gate"].double())


def _attention_gpu(c, prior, window, keep, scale, cuda, form):
    dtype = torch.float32 if form == "plain-f32" else torch.bfloat16
    dv = {k: v.to(cuda).to(dtype) for k, v in c.items()}
    b, t, heads, d = dv["q"].shape
    groups, n = dv["rows"].shape[1:3]
    out = torch.full((b * t, heads * d + 16), 7.0, dtype=dtype, device=cuda)
    args = _lib.WindowedAttentionArgs(
        q=_p(dv["q"]), k1=_p(dv["rows"]) + d * dv["rows"].element_size(), v=_p(dv["rows"]), column_gates=_p(dv["gate"]), out=_p(out),
        k1_batch=groups * n * 2 * d, v_batch=groups * n * 2 * d, k1_head=n * 2 * d, v_head=n * 2 * d, k1_row=2 * d, v_row=2 * d, d1=d, d2=0, dv=d,
        batch=b, heads=heads, share=heads // groups, seq=t, rows=n, prior=prior, window=window, keep=keep, gate_ld=heads * d, out_ld=heads * d + 16,
        scale=scale)
    lib = _lib.load_dense()
    if form == "mfma":
        assert lib.ajqd_windowed_prefill_supported(d, 0, d)
        _ok(lib.ajqd_windowed_prefill(ctypes.byref(args), _st()))
    else:
        _ok(lib.ajqd_windowed_attention(ctypes.byref(args), dense._flag(dtype), dense._flag(dtype), _st()))
    assert (out[:, heads * d:] == 7.0).all()
    return out[:, : heads * d]


ATTENTION_SHAPES = [  # b, heads, groups, t, prior, dim, window, keep
    (1, 4, 2, 150, 0, 16, 17, 3),
    (2, 6, 2, 70, 31, 48, 30, 2),       # the window's rows and the kept ones ahead of the new ones
    (1, 8, 8, 300, 0, 64, 64, 64),      # as many kept as one block of keys
    (1, 8, 1, 260, 9, 128, 100, 5),
    (1, 2, 1, 200, 0, 96, 33, 70),      # kept rows reach into a second block of keys
    (1, 4, 2, 2, 66, 32, 64, 3),        # two tokens
    (2, 3, 1, 65, 0, 32, 1, 1),         # every token sees itself and the first
    (1, 4, 4, 129, 0, 256, 0, 0),       # no window
    (1, 16, 2, 500, 0, 64, 70, 1),
    (1, 2, 2, 90, 0, 80, 1000, 4),      # a window longer than the sequence
]


@pytest.mark.parametrize("shape", ATTENTION_SHAPES)
@pytest.mark.parametrize("form", ["mfma", "plain-bf16", "plain-f32"])
def test_windowed_attention_with_kept_rows(cuda, shape, form):
    b, heads, groups, t, prior, d, window, keep = shape
    c = _attention_case(b, heads, groups, t, prior, d, sum(shape))
    got = _attention_gpu(c, prior, window, keep, 1.1 * d ** -0.5, cuda, form)
    assert _rel(got, _attention_plain(c, prior, window, keep, 1.1 * d ** -0.5)) < (2e-6 if form == "plain-f32" else 6e-3)


@pytest.mark.parametrize("form", ["mfma", "plain-bf16", "plain-f32"])
@pytest.mark.parametrize("keep", [1, 4, 64, 67])
def test_a_standing_out_key_at_every_edge(cuda, form, keep):
    """One query and one key whose score dominates: a key takes all the weight where it is just inside the window or the last one
    that is kept, and leaves no trace one token beyond either."""
    window, t, d = 70, 300, 32
    cases = [(at, at + window - 1 + out, out == 0) for at in (keep + 1, 100, 127, 128, 190) for out in (0, 1)]
    cases += [(keep - 1, q, True) for q in (keep + window, 255, 299)] + [(keep, q, False) for q in (keep + window, 255, 299)] + [(0, 299, True)]
    for at, query, dominates in cases:
        if query >= t:
            continue
        c = _attention_case(1, 4, 2, t, 0, d, at + query)
        c["rows"][0, :, at, d:] = 3.0
        c["q"][0, query] = 3.0
        c["gate"].fill_(20.0)
        got = _attention_gpu(c, 0, window, keep, 0.2, cuda, form).cpu()
        assert _rel(got, _attention_plain(c, 0, window, keep, 0.2)) < 8e-3
        value = c["rows"][0, :, at, :d].float().repeat_interleave(2, 0).reshape(-1)
        assert (_rel(got[query].float(), value) < 2e-2) == dominates, (at, query)


DECODE_SHAPES = [  # batch, groups, share, dim, rows of the ring, position
    (1, 2, 3, 16, 45, 500), (3, 1, 16, 48, 64, 63), (1, 4, 2, 128, 65, 64), (2, 2, 17, 64, 200, 130), (1, 1, 40, 128, 300, 1000),
    (5, 8, 4, 128, 1000, 5000), (2, 3, 1, 96, 70, 0), (1, 8, 1, 256, 130, 4000),
]


@pytest.mark.parametrize("shape", DECODE_SHAPES)
def test_decode_attention_and_merge(cuda, shape):
    """Chunked attention of one token on (value | key) rows, for every number of chunks, with one standing-out row."""
    batch, groups, share, d, cap, position = shape
    lib, g = _lib.load_dense(), torch.Generator().manual_seed(sum(shape))
    heads, units, scale = groups * share, batch * groups, 0.8 * d ** -0.5
    assert lib.ajqd_latent_decode_chunks(units, share, d, d, cap) >= 1
    q, ring, gate = _bf(g, units, share, 2 * d), _bf(g, units, cap, 2 * d), torch.randn((batch, heads * d), generator=g)
    q[:, :, :d] = 0
    valid = min(position, cap - 1) + 1
    ring[:, valid - 1, d:] *= 3
    ring[:, valid:] = float("nan")   # rows that were never written must not be read
    scores = torch.matmul(q[..., d:].double(), ring[:, :valid, d:].double().transpose(1, 2)) * scale
    want = torch.matmul(O.softmax(scores), ring[:, :valid, :d].double()).reshape(batch, heads * d)
    dev = {k: v.to(cuda) for k, v in dict(q=q, ring=ring, gate=gate, pos=torch.tensor([position])).items()}
    for chunks in sorted({1, 2, 3, 7, 32, lib.ajqd_latent_decode_chunks(units, share, d, d, cap)}):
        partial = torch.full((lib.ajqd_latent_decode_workspace(units, share, d, chunks),), 255, dtype=torch.uint8, device=cuda)
        _ok(lib.ajqd_latent_decode(_p(dev["q"]), _p(dev["ring"]), _p(dev["pos"]), _p(partial), units, share, d, d, cap, chunks, d, scale, _st()))
        for gated in (True, False):
            out = torch.full((batch, heads * d + 8), 5.0, dtype=torch.bfloat16, device=cuda)
            _ok(lib.ajqd_group_merge(_p(partial), _p(dev["gate"]) if gated else None, heads * d, _p(out), heads * d + 8, batch, groups, share, chunks,
                                     d, _st()))
            plain = want * torch.sigmoid(gate.double()) if gated else want
            assert _rel(out[:, : heads * d], plain) < 8e-3, chunks
            assert (out[:, heads * d:] == 5.0).all()


def test_ring_copy_keeps_the_first_rows(cuda):
    lib, kept, cap = _lib.load_dense(), 3, 8
    line = torch.arange(20 * 4, dtype=torch.float32, device=cuda).view(1, 20, 4)
    ring = torch.full((1, cap, 4), -1.0, device=cuda)
    for first, count in ((0, 3), (3, 4), (7, 5), (12, 2)):
        _ok(lib.ajqd_ring_copy(_p(ring), cap, kept, _p(line), 20, 16, first, first, count, 16, 1, 1, _st()))
    for p in (0, 1, 2, 9, 10, 11, 12, 13):
        assert torch.equal(ring[0, p if p < kept else kept + (p - kept) % (cap - kept)], line[0, p])


# ------------------------------------------------------------------ selective scan
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
def test_convolution_in_portions_and_token_by_token(cuda, dtype, taps):
    lib, inner, total, batch = _lib.load_dense(), 40, 19, 2
    g = torch.Generator().manual_seed(taps)
    y = torch.randn((batch, total, inner + 8), generator=g).to(dtype)
    weight, bias = torch.randn((inner, taps), generator=g), torch.randn(inner, generator=g)
    want = torch.stack([O.silu(O.causal_conv(y[b, :, :inner].double(), weight.double(), bias.double())) for b in range(batch)])
    dw, db, size = weight.T.contiguous().to(cuda), bias.to(cuda), torch.finfo(dtype).bits // 8
    for cuts in ([19], [1, 2, 2, 5, 9], [2] * 9 + [1], [0] + [1] * 19, [7] + [1] * 12):
        ring = torch.full((batch, taps - 1, inner), float("nan"), dtype=dtype, device=cuda)
        held, got, at, static = _p(ring) if taps > 1 else None, [], 0, cuts[0] == 0
        for n in cuts[1:] if static else cuts:
            part = y[:, at:at + n].contiguous().to(cuda).view(batch * n, inner + 8)
            out = torch.empty((batch * n, inner), dtype=dtype, device=cuda)
            pos = torch.tensor([at], device=cuda)
            _ok(lib.ajqd_conv_silu(_p(part), inner + 8, held, _p(dw), _p(db), 0 if static else at, _p(pos) if static else None, batch * n, n, inner,
                                   taps, _p(out), dense._flag(dtype), _st()))
            last = min(n, taps - 1)
            if not static and last > 0:
                _ok(lib.ajqd_ring_copy(_p(ring), taps - 1, 0, _p(part), n, (inner + 8) * size, n - last, at + n - last, last, inner * size, batch, 1, _st()))
            got.append(out.view(batch, n, inner))
            at += n
        assert _rel(torch.cat(got, dim=1), want) < (1e-6 if dtype == torch.float32 else 4e-3), cuts


SCANS = [  # batch, tokens, inner, states
    (2, 300, 40, 16), (1, 130, 2048, 4), (8, 5, 2560, 16), (16, 37, 2560, 12), (1, 150, 72, 24), (8, 33, 2560, 32), (16, 40, 2560, 24),
    (16, 9, 2560, 28), (1, 70, 96, 40), (16, 18, 2560, 64), (2, 35, 48, 100), (1, 21, 24, 256), (3, 2, 16, 8), (2, 1, 64, 20),
]


def _scan_case(batch, seq, inner, states, seed):
    g = torch.Generator().manual_seed(seed)
    rank = 8
    c = dict(x=_bf(g, batch, seq, inner), raw=_bf(g, batch, seq, inner), z=_bf(g, batch, seq, inner), low=_bf(g, batch, seq, rank + 2 * states),
             bias=torch.randn(inner, generator=g) - 2, a_log=torch.randn((inner, states), generator=g), d=torch.randn(inner, generator=g),
             state=torch.randn((batch, inner, states), generator=g))
    return c, rank


def _scan_plain(c, rank, states, carried):
    out, ends = [], []
    for b in range(c["x"].shape[0]):
        x, low = c["x"][b].double(), c["low"][b].double()
        dt = O.softplus(c["raw"][b].double() + c["bias"].double())
        y, end = O.recurrence(x, dt, -torch.exp(c["a_log"].double()), low[:, rank:rank + states], low[:, rank + states:], c["d"].double(),
                              c["state"][b].double() if carried else None)
        out.append(y * O.silu(c["z"][b].double()))
        ends.append(end)
    return torch.stack(out), torch.stack(ends)


def _scan_gpu(c, rank, states, start, cuda, dtype, state, span=slice(None), static=False):
    d = {k: c[k][:, span].contiguous().to(cuda).to(dtype) for k in ("x", "raw", "z", "low")}
    batch, seq, inner = d["x"].shape
    a2 = hybrid.state_planes(-torch.exp(c["a_log"].double()) * math.log2(math.e)).float().to(cuda)
    skip, bias, pos = c["d"].to(cuda), c["bias"].to(cuda), torch.tensor([start], device=cuda)
    out = torch.empty((batch, seq, inner), dtype=dtype, device=cuda)
    args = _lib.ScanArgs(x=_p(d["x"]), dt=_p(d["raw"]), low=_p(d["low"]), z=_p(d["z"]), a2=_p(a2), d=_p(skip), dt_bias=_p(bias), state=_p(state),
                         pos=_p(pos) if static else None, out=_p(out), batch=batch, seq=seq, start=0 if static else start, inner=inner, states=states,
                         dt_ld=inner, low_ld=rank + 2 * states, b_col=rank, c_col=rank + states, z_ld=inner, out_ld=inner)
    _ok(_lib.load_dense().ajqd_scan(ctypes.byref(args), dense._flag(dtype), _st()))
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SCANS)
def test_scan_against_the_sequential_recurrence(cuda, dtype, shape):
    """From zeros whatever the state buffer holds, and from a state; outputs and the state left behind."""
    batch, seq, inner, states = shape
    c, rank = _scan_case(*shape, sum(shape))
    tol = 4e-6 if dtype == torch.float32 else 4e-3
    for carried in (False, True):
        state = hybrid.state_planes(c["state"] if carried else torch.full_like(c["state"], float("nan"))).to(cuda)
        got = _scan_gpu(c, rank, states, 7 if carried else 0, cuda, dtype, state)
        want, end = _scan_plain(c, rank, states, carried)
        assert _rel(got, want) < tol
        assert _rel(state, hybrid.state_planes(end)) < 4e-6


@pytest.mark.parametrize("dtype", DTYPES)
def test_scan_portions_equal_the_whole(cuda, dtype):
    batch, seq, inner, states = 2, 150, 48, 20
    c, rank = _scan_case(batch, seq, inner, states, 5)
    state = torch.full((batch, states // 4, inner, 4), float("nan"), device=cuda)
    whole = _scan_gpu(c, rank, states, 0, cuda, dtype, state)
    for cuts in ([2] * 75, [64, 64, 22], [128, 1, 1, 20], [0] + [1] * 150):
        part, got, at, static = torch.full_like(state, float("nan")), [], 0, cuts[0] == 0
        for n in cuts[1:] if static else cuts:
            got.append(_scan_gpu(c, rank, states, at, cuda, dtype, part, slice(at, at + n), static))
            at += n
        assert torch.equal(torch.cat(got, dim=1), whole) and torch.equal(part, state)


STEPS = [  # batch, inner, states, rank, taps
    (1, 48, 8, 8, 4), (3, 400, 28, 16, 4), (1, 1552, 16, 40, 2), (5, 80, 40, 8, 1), (17, 640, 16, 24, 3), (20, 2048, 4, 128, 4), (33, 32, 64, 8, 7),
]


@pytest.mark.parametrize("shape", STEPS)
def test_decode_step_of_the_scan(cuda, shape):
    """scan_project and scan_step from the first token on: convolution columns and states carried in buffers that start as NaN."""
    batch, inner, states, rank, taps = shape
    lib, g, tokens = _lib.load_dense(), torch.Generator().manual_seed(sum(shape)), taps + 3
    rows = _up(rank + 2 * states, 16)
    conv, bias, dt_bias, skip = torch.randn((inner, taps), generator=g), torch.randn(inner, generator=g), torch.randn(inner, generator=g) - 2, torch.randn(inner, generator=g)
    a_log, w_low, w_dt = torch.randn((inner, states), generator=g), _bf(g, rows, inner, std=inner ** -0.5), _bf(g, inner, rank, std=rank ** -0.5)
    y = _bf(g, tokens, batch, 2 * inner).float()
    d = {k: v.to(cuda) for k, v in dict(conv=conv.T.contiguous(), bias=bias, dt_bias=dt_bias, skip=skip, w_low=w_low, w_dt=w_dt,
                                        a2=hybrid.state_planes(-torch.exp(a_log.double()) * math.log2(math.e)).float()).items()}
    ring = torch.full((batch, taps - 1, inner), float("nan"), dtype=torch.bfloat16, device=cuda)
    held = _p(ring) if taps > 1 else None
    state = torch.full((batch, states // 4, inner, 4), float("nan"), device=cuda)
    pos, splits, got = torch.zeros(1, dtype=torch.long, device=cuda), lib.ajqd_scan_splits(batch, inner), []
    for t in range(tokens):
        pos.fill_(t)
        row, out = y[t].to(cuda), torch.empty((batch, inner), dtype=torch.bfloat16, device=cuda)
        partial = torch.full((splits, batch, rows), float("nan"), device=cuda)
        _ok(lib.ajqd_scan_project(_p(row), 2 * inner, held, _p(d["conv"]), _p(d["bias"]), _p(pos), _p(d["w_low"]), _p(partial), batch, inner, taps, rows,
                                  splits, _st()))
        args = _lib.ScanStepArgs(y=_p(row), ring=held, weight=_p(d["conv"]), bias=_p(d["bias"]), pos=_p(pos), partial=_p(partial), w_dt=_p(d["w_dt"]),
                                 dt_bias=_p(d["dt_bias"]), a2=_p(d["a2"]), d=_p(d["skip"]), state=_p(state), out=_p(out), batch=batch, ldy=2 * inner,
                                 inner=inner, taps=taps, rows=rows, splits=splits, rank=rank, states=states, out_ld=inner)
        _ok(lib.ajqd_scan_step(ctypes.byref(args), _st()))
        got.append(out)
    for b in range(batch):
        x = O.silu(O.causal_conv(y[:, b, :inner].double(), conv.double(), bias.double()))
        low = x @ w_low.double().T
        dt = O.softplus(low[:, :rank] @ w_dt.double().T + dt_bias.double())
        want, end = O.recurrence(x, dt, -torch.exp(a_log.double()), low[:, rank:rank + states], low[:, rank + states:rank + 2 * states], skip.double())
        want = want * O.silu(y[:, b, inner:].double())
        assert _rel(torch.stack([o[b] for o in got]), want) < 2e-2 and _rel(state[b], hybrid.state_planes(end)) < 2e-2


# ------------------------------------------------------------------ the decoder against the plain implementation
SHAPES = {
    "plain": dict(),
    # every width off the kernels' grids
    "ragged": dict(layers=[attention(heads=3, kv_heads=1, dim=12, rot=6, window=7, keep=1, ff=28), scan(inner=44, state=5, rank=3, conv=2, ff=36)],
                   width=52, vocab=61, streams=2, loop={"start": 0, "stop": 2, "times": 2}),
    # one stream, no loop, sublayers missing, a convolution of one tap, no window, plain multi-head attention, whole heads rotated
    "single": dict(layers=[scan(conv=1, ff=None), attention(heads=4, kv_heads=4, dim=24, rot=24, window=None, ff=None), scan(inner=16, state=1, rank=1, ff=None)],
                   streams=1, loop=None),
    # many query heads on one key head, more streams than most, the loop at the end
    "shared": dict(layers=[scan(inner=64, state=20, rank=9, conv=5), attention(heads=18, kv_heads=1, dim=16, rot=4, window=33, keep=5),
                           attention(heads=6, kv_heads=2, dim=40, rot=16, scaling=SCALING, window=64, keep=70)],
                   width=96, streams=5, loop={"start": 2, "stop": 3, "times": 3}),
    # constants far from the usual: an eps that dominates, fast rotations, a large score scale, windows of one and two
    "constants": dict(layers=[attention(base=3.0, scale=0.9, window=1, keep=2), attention(base=3.0, scale=0.02, window=2, keep=0), scan(conv=7)], eps=0.4,
                      loop={"start": 0, "stop": 1, "times": 1}),
    # sizes of a larger model's heads and channels
    "wide": dict(layers=[attention(heads=4, kv_heads=2, dim=128, rot=32, scaling=SCALING, window=70, keep=4, ff=520), scan(inner=640, state=24, rank=20, ff=264)],
                 width=320, streams=2, loop={"start": 0, "stop": 1, "times": 2}),
    # heads wider than the MFMA kernels take, many states per channel
    "beyond": dict(layers=[attention(heads=2, kv_heads=1, dim=304, rot=60, window=20, keep=3), scan(inner=32, state=70, rank=12)], loop=None),
}


@pytest.mark.parametrize("name", list(SHAPES))
@pytest.mark.parametrize("dtype", DTYPES)
def test_prompt_portions_and_decoding_match_plain(cuda, name, dtype):
    """Whole prompt, token by token from the first on, and portions of several sizes: all against one plain run."""
    cfg = config(**SHAPES[name])
    weights = random_weights(cfg, 7, spread=1.5)
    model = _build(cfg, weights, cuda, dtype)
    tokens = _tokens(cfg, 90, 1)
    seen: list[torch.Tensor] = []
    want = O.forward(cfg, weights, tokens, residuals=seen)
    ids = _ids(tokens, cuda)
    got_seen: list[torch.Tensor] = []
    whole = model(ids, residuals=got_seen)[0]
    tol = LOGIT_TOL[dtype]
    assert len(got_seen) == len(seen) == len(model.runs)
    for a, b in zip(got_seen, seen):
        assert _rel(a[0], b) < tol
    assert _rel(whole, want) < tol
    cache = model.new_cache(1, 90)
    assert _rel(model(ids, cache)[0], want) < tol
    for cuts in ([1] * 90, [2] * 45, [50] + [1] * 40, [3, 2, 17, 1, 1, 33, 2, 31], [64, 26], [5] * 18):
        cache.reset()
        parts, at = [], 0
        for n in cuts:
            parts.append(model(ids[:, at:at + n], cache)[0])
            at += n
        got = torch.cat(parts)
        assert _rel(got, want) < tol
        worst = (got.double().cpu() - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
        assert float(worst.max()) < 3 * tol, (cuts[:4], int(worst.argmax()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", ["whole", "decoded", "portions"])
@pytest.mark.parametrize("keep", [0, 2, 20])
def test_reach_by_dependence(cuda, dtype, cuts, keep):
    """In a model of one attention layer, changing a token changes the logits of window positions from it on, of all later ones if
    it is kept, and of no other, in prompts and in decoding, wherever the ring wraps."""
    window, count = 13, 80
    cfg = config([attention(window=window, keep=keep)], loop=None)
    model = _build(cfg, random_weights(cfg, 11, spread=2.0), cuda, dtype)
    base = _tokens(cfg, count, 3)
    sizes = {"whole": [count], "decoded": [1] * count, "portions": [2, 3, 13, 1, 14, 12, 2, 27, 1, 1, 4]}[cuts]

    def run(tokens):
        cache, parts, at = model.new_cache(1, count), [], 0
        for n in sizes:
            parts.append(model(_ids(tokens[at:at + n], cuda), cache)[0])
            at += n
        return torch.cat(parts)

    first = run(base)
    for at in (0, 1, 2, 12, 13, 19, 20, 25, 26, 52, 63, 64):
        other = list(base)
        other[at] = (other[at] + 1) % cfg["vocab"]
        moved = (run(other) - first).abs().amax(dim=1).cpu()
        assert (moved[:at] == 0).all()
        end = count if at < keep else min(count, at + window)
        assert (moved[at:end] > 0).all() and (moved[end:] == 0).all(), at


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_token_shows_through_the_state(cuda, dtype):
    """Slow decays: the first token is still read hundreds of positions on, across portions and decoded tokens."""
    cfg = config([scan(inner=32, state=4, rank=2)], loop=None)
    weights = random_weights(cfg, 12)
    weights["l0.mix.A_log"].fill_(-9.0)
    weights["l0.mix.dt.b"].fill_(-1.0)
    weights["embed"][:, 7] = 0        # a column that tells token 0, which comes first and nowhere else, from the others
    weights["embed"][0] = 0
    weights["embed"][0, 7] = 30
    weights["l0.mix.in"][:32, 7] = 3  # its input and B are large
    tokens = [0] + [t or 2 for t in _tokens(cfg, 299, 4)]
    want = O.forward(cfg, weights, tokens)
    assert _rel(O.forward(cfg, weights, [1] + tokens[1:])[250:], want[250:]) > 2 * LOGIT_TOL[torch.bfloat16]
    model = _build(cfg, weights, cuda, dtype)
    cache, parts, at = model.new_cache(1, 300), [], 0
    for n in (1, 99, 2, 150, 1, 1, 40, 6):
        parts.append(model(_ids(tokens[at:at + n], cuda), cache)[0])
        at += n
    assert _rel(torch.cat(parts)[250:], want[250:]) < LOGIT_TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_kept_token_shows_far_away(cuda, dtype):
    """Queries that look for the first token (its key and their own queries share one direction): hundreds of positions on it still
    takes most of the weight, and with one token kept less it takes none."""
    cfg = config([attention(heads=2, kv_heads=1, dim=16, rot=0, window=20, keep=2, scale=1.0)], loop=None, streams=2)
    weights = random_weights(cfg, 13)
    weights["l0.mix.q.norm"].fill_(1.0)
    weights["l0.mix.k.norm"].fill_(1.0)
    weights["l0.hc1.in"].fill_(0.5)
    tokens = [1, 0] + [t or 2 for t in _tokens(cfg, 399, 5)]   # position 1 is the last one kept; token 0 occurs nowhere else
    unit = torch.zeros(16)
    unit[5] = 1.0
    axis = torch.zeros(cfg["width"])
    axis[7] = 1.0
    weights["embed"][:, 7] = -3.0     # a column that tells token 0 from the others
    weights["embed"][0] = 30 * axis
    weights["l0.mix.k"] = weights["l0.mix.k"] * 0.3 + 2.0 * torch.outer(unit, axis)
    weights["l0.mix.q"] = weights["l0.mix.q"] * 0.3 - 2.0 * torch.outer(unit.repeat(2), axis)
    weights = {k: v.to(torch.bfloat16).float() for k, v in weights.items()}
    want = O.forward(cfg, weights, tokens)
    less = {**cfg, "layers": [attention(heads=2, kv_heads=1, dim=16, rot=0, window=20, keep=1, scale=1.0)]}
    assert _rel(O.forward(less, weights, tokens)[300:], want[300:]) > 3 * LOGIT_TOL[torch.bfloat16]
    model = _build(cfg, weights, cuda, dtype)
    whole = model(_ids(tokens, cuda))[0]
    cache = model.new_cache(1, 401)
    parts = [model(_ids(tokens[:330], cuda), cache)[0]] + [model(_ids([t], cuda), cache)[0] for t in tokens[330:]]
    for got in (whole, torch.cat(parts)):
        assert _rel(got[300:], want[300:]) < LOGIT_TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_cache_that_is_used_again_equals_a_fresh_one(cuda, dtype):
    cfg = config()
    model = _build(cfg, random_weights(cfg, 15), cuda, dtype)
    cache = model.new_cache(1, 100)
    model(_ids(_tokens(cfg, 95, 5), cuda), cache)
    for buffer in cache.rings + [s for s in cache.states if s is not None]:
        buffer.fill_(float("nan"))   # whatever an earlier sequence left must not be read
    for lengths in ((3, 4, 6, 39, 40), (1, 2, 3, 4, 30)):
        cache.reset()
        tokens, fresh, at = _tokens(cfg, 40, 6), model.new_cache(1, 100), 0
        for end in lengths:
            assert torch.equal(model(_ids(tokens[at:end], cuda), cache), model(_ids(tokens[at:end], cuda), fresh))
            at = end


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("batch", [2, 5, 17, 37])
def test_batch_rows_equal_sequences_alone(cuda, dtype, batch):
    """One, up to 16, up to 32 and more rows take different kernels; every row is its sequence's own."""
    cfg = config()
    weights = random_weights(cfg, 17)
    model = _build(cfg, weights, cuda, dtype)
    prompts = torch.tensor([_tokens(cfg, 31, 20 + i) for i in range(batch)], device=cuda)
    cache = model.new_cache(batch, 31)
    got = torch.cat([model(prompts[:, :23], cache)] + [model(prompts[:, t:t + 1], cache) for t in range(23, 31)], dim=1)
    for i in range(batch):
        want = O.forward(cfg, weights, prompts[i].tolist())
        assert _rel(got[i], want) < LOGIT_TOL[dtype], i


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(cuda, dtype):
    """Several hundred decoded tokens: rings wrap many times, states and angles run on."""
    cfg = config([attention(scaling=SCALING, window=24, keep=3), scan()], loop={"start": 0, "stop": 2, "times": 2})
    weights = random_weights(cfg, 18)
    model = _build(cfg, weights, cuda, dtype)
    tokens = _tokens(cfg, 400, 8)
    want = O.forward(cfg, weights, tokens)
    cache = model.new_cache(1, 400)
    got = torch.cat([model(_ids(tokens[:2], cuda), cache)[0]] + [model(_ids([t], cuda), cache)[0] for t in tokens[2:]])
    assert _rel(got, want) < LOGIT_TOL[dtype] and _rel(got[-50:], want[-50:]) < LOGIT_TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_wanted_places_and_lengths(cuda, dtype):
    cfg = config()
    model = _build(cfg, random_weights(cfg, 19), cuda, dtype)
    tokens = _tokens(cfg, 60, 7)
    full = model(_ids(tokens, cuda))[0]
    for want in ([0], [59, 3, 3], list(range(20)), []):
        got = model(_ids(tokens, cuda), want=want)[0]
        assert got.shape == (len(want), cfg["vocab"])
        if want:
            assert _rel(got, full[want]) < (1e-6 if dtype == torch.float32 else 5e-3)
    with pytest.raises(ValueError, match="holds"):
        model(_ids(tokens, cuda), model.new_cache(1, 30))
    with pytest.raises(ValueError, match="sequences"):
        model(_ids(tokens, cuda), model.new_cache(2, 64))


# ------------------------------------------------------------------ generation
def _margins(cfg, weights, prompt, follow):
    """How far every chosen token is below the plain implementation's maximum, given the tokens before it."""
    rows = O.forward(cfg, weights, prompt + follow)[len(prompt) - 1:-1]
    return rows.max(dim=-1).values - rows.gather(1, torch.tensor(follow).view(-1, 1)).squeeze(1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("batch", [1, 3, 6])
def test_greedy_generation_through_the_decoders(cuda, dtype, batch):
    """Graph-replayed decoding over several times the window: every chosen token is the plain implementation's maximum up to
    rounding, and the eager loop and portioned prompts agree with it the same way."""
    cfg = config()
    weights = random_weights(cfg, 21)
    model = _build(cfg, weights, cuda, dtype)
    prompts = torch.tensor([_tokens(cfg, 37, 40 + i) for i in range(batch)], device=cuda)
    scale = float(O.forward(cfg, weights, prompts[0].tolist()).pow(2).mean().sqrt())
    noise, new = 4 * LOGIT_TOL[dtype] * scale, 75
    graph = decoding.greedy_decode_graph(model, prompts, new)
    eager = modeling.greedy_decode(model, prompts, new)
    dec = decoding.decoder_for(model)(model, batch, 37 + new)
    dec.prefill(prompts, tokens_per_pass=8)
    portions = dec.generate(new)
    for i in range(batch):
        for tokens in (graph[i, 37:], eager[i, 37:], portions[i]):
            assert float(_margins(cfg, weights, prompts[i].tolist(), tokens.tolist()).max()) <= noise
    assert graph.shape == eager.shape == (batch, 37 + new)


def test_graph_replays_equal_the_eager_step(cuda):
    """The same decoder used for three prompts (the later ones from a used cache), with other work between the replays."""
    cfg = config()
    model = _build(cfg, random_weights(cfg, 23), cuda, torch.bfloat16)
    dec = decoding.DenseDecoder(model, 2, 120)
    for seed in (1, 2, 3):
        prompts = torch.tensor([_tokens(cfg, 20, seed), _tokens(cfg, 20, seed + 9)], device=cuda)
        dec.prefill(prompts)
        steps = []
        for count in (2, 3, 20, 60):
            steps = dec.generate(count)
            torch.randn(256, 256, device=cuda) @ torch.randn(256, 256, device=cuda)
            torch.cuda.synchronize()
        cache = model.new_cache(2, 120)
        token = model(prompts, cache, last_token_only=True)[:, -1].argmax(-1, keepdim=True)
        want = [token]
        for _ in range(59):
            token = model(token, cache)[:, -1].argmax(-1, keepdim=True)
            want.append(token)
        assert torch.equal(steps, torch.cat(want, dim=1))


def test_sampling_and_stop_token(cuda):
    cfg = config()
    model = _build(cfg, random_weights(cfg, 25), cuda, torch.bfloat16)
    prompts = torch.tensor([_tokens(cfg, 12, 3)], device=cuda)

    def generate(seed=None, **kw):
        dec = decoding.DenseDecoder(model, 1, 80)
        if seed is not None:
            dec.set_sampling(1.5, 0.95, seed)
        dec.prefill(prompts)
        return dec.generate(60, **kw)[0].tolist()

    assert generate(1) == generate(1) and generate(1) != generate(2)
    tokens = generate()
    assert generate(eos_token_id=tokens[30]) == tokens[: tokens.index(tokens[30]) + 1]


def test_checkpoint_trace_and_command_line(cuda, tmp_path, capsys):
    """A folder is loaded, replayed step by step through the trace session, and continued from the command line."""
    from ajllm_amd.__main__ import main as command
    from ajllm_amd.trace import Session

    cfg = config()
    weights = random_weights(cfg, 27)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in weights.items()}, str(tmp_path / "model.safetensors"))
    for dtype in DTYPES:
        session = Session(checkpoint.load_model(tmp_path, cuda, dtype), 64)
        for name, seed in (("a", 1), ("b", 2)):   # the second request gets the first one's cache
            tokens = _tokens(cfg, 40, seed)
            want = O.forward(cfg, weights, tokens)
            parts = [session.step([{"id": name, "tokens": tokens[:25], "want": [3, 24]}], [])]
            assert session.step([{"id": name, "tokens": tokens[25:27], "want": []}], []) is None
            parts.append(session.step([{"id": name, "tokens": tokens[27:28], "want": [0]}], []))
            parts.append(session.step([{"id": name, "tokens": tokens[28:], "want": [0, 11]}], [name]))
            assert _rel(torch.cat(parts), want[[3, 24, 27, 28, 39]]) < LOGIT_TOL[dtype]
        assert len(session.free) == 1 and not session.live
    prompt = _tokens(cfg, 9, 3)
    assert command(["generate", "--model", str(tmp_path), "--dtype", "float32", "--tokens", ",".join(map(str, prompt)),
                    "--max-new-tokens", "12"]) == 0
    new = [int(t) for t in capsys.readouterr().out.strip().splitlines()[-1].split(",")]
    assert len(new) == 12 and float(_margins(cfg, weights, prompt, new).max()) < 1e-3
