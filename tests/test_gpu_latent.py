"""The dense model family on the GPU: every operator of libajq_dense.so and the whole Dorutar decoder against the plain
implementation (oracle/dorutar.py, float64 on the host), in fp32 (where the comparison is sharp) and in bf16."""

import ctypes
import json

import pytest
import torch
from safetensors.torch import save_file

from ajllm_amd import _lib, checkpoint, decoding, latent, modeling
from oracle import dorutar as O
from tests.latent_models import config, random_weights

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


def _build(cfg, weights, device, dtype):
    with torch.device("meta"):
        model = modeling.build_model(cfg)
    names = model.checkpoint_names()
    model.load_state_dict({k: weights[n].to(device=device, dtype=dtype) for k, n in names.items()}, assign=True)
    return model.eval()


def _tokens(cfg, count, seed):
    return torch.randint(0, cfg["vocab"], (count,), generator=torch.Generator().manual_seed(seed)).tolist()


def _ids(tokens, device):
    return torch.tensor([tokens], device=device)


# ------------------------------------------------------------------ operators alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("true_width", [16, 52, 200, 2048, 9000])
def test_add_norms(cuda, dtype, true_width):
    width = (true_width + 15) // 16 * 16
    g = torch.Generator().manual_seed(true_width)

    def padded(*shape):
        t = torch.zeros(*shape[:-1], width)
        t[..., : shape[-1]] = torch.randn(shape, generator=g)
        return t

    rows = 5
    x, again, step = padded(rows, true_width) + 0, padded(rows, true_width), padded(true_width)
    x[:, :true_width] += 3.0  # a mean worth removing
    delta, g1, g2 = padded(rows, true_width), padded(true_width), padded(true_width)
    dx = x.to(cuda)
    o1, o2 = torch.empty((rows, width), dtype=dtype, device=cuda), torch.empty((rows, width), dtype=dtype, device=cuda)
    args = [t.to(cuda) for t in (again, step, g1, g2)]
    dd = delta.to(cuda)
    for center in (1, 0):
        dx.copy_(x)
        _ok(_lib.load_dense().ajqd_add_norms(dx.data_ptr(), dd.data_ptr(), _lib.AJQD_F32, args[0].data_ptr(), args[1].data_ptr(),
                                             args[2].data_ptr(), args[3].data_ptr(), 1e-5, center, o1.data_ptr(), o2.data_ptr(), rows,
                                             true_width, width, latent._flag(dtype), _st()))
        total = (x + delta + again + step).double()
        assert _rel(dx, total) < 1e-6
        norm = O.layer_norm if center else O.rms_norm
        for out, gain in ((o1, g1), (o2, g2)):
            want = norm(total[:, :true_width], gain[:true_width].double(), 1e-5)
            assert _rel(out[:, :true_width].float(), want) < (1e-6 if dtype == torch.float32 else 4e-3)
            assert (out[:, true_width:] == 0).all()


@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_and_device_side_position(cuda, dtype):
    table, pos = torch.randn(19, 32).to(dtype), torch.randn(40, 32).to(dtype)
    tokens = torch.tensor([3, 18, 0, 7, 7, 2])
    x, kept = torch.empty((6, 32), device=cuda), torch.empty((6, 32), device=cuda)
    extra = torch.randn(32)
    dt, dp, ids, de = table.to(cuda), pos.to(cuda), tokens.to(cuda), extra.to(cuda)
    _ok(_lib.load_dense().ajqd_embed(ids.data_ptr(), 6, 3, dt.data_ptr(), 19, dp.data_ptr(), 40, 11, None, de.data_ptr(),
                                     x.data_ptr(), kept.data_ptr(), 32, latent._flag(dtype), _st()))
    want = torch.cat([O.embedding(tokens[:3].tolist(), table.float(), pos.float(), 11),
                      O.embedding(tokens[3:].tolist(), table.float(), pos.float(), 11)])
    assert torch.equal(kept.cpu(), want) and torch.equal(x.cpu(), want + extra)
    where = torch.tensor([17], device=cuda)
    _ok(_lib.load_dense().ajqd_embed(ids.data_ptr(), 6, 1, dt.data_ptr(), 19, dp.data_ptr(), 40, 0, where.data_ptr(), None,
                                     x.data_ptr(), None, 32, latent._flag(dtype), _st()))
    assert torch.equal(x.cpu(), table.float()[tokens] + pos.float()[17])


@pytest.mark.parametrize("act", ["relu", "silu", "gelu_tanh"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_gated_activation(cuda, dtype, act):
    gate, up = torch.randn(40, 7), torch.randn(40, 7)
    y = latent.interleave_gate(gate, up).T.contiguous().to(cuda)
    out = torch.full((7, 48), 9.0, dtype=dtype, device=cuda)
    _ok(_lib.load_dense().ajqd_gated_activation(y.data_ptr(), _lib.AJQD_F32, out.data_ptr() + 8 * out.element_size(), 48, 7, 40,
                                                _lib.AJQD_ACTIVATIONS[act], latent._flag(dtype), _st()))
    want = (modeling.ACTIVATIONS[act](gate.double()) * up.double()).T
    assert _rel(out[:, 8:], want) < (1e-6 if dtype == torch.float32 else 4e-3)
    assert (out[:, :8] == 9.0).all()


@pytest.mark.parametrize("k", [8, 40, 264, 1040])
def test_matvec(cuda, k):
    w, x = torch.randn(3, 13, k), torch.randn(2, 3, k)
    y = torch.zeros((2, 3, 16), device=cuda)
    dw, dx = w.to(cuda), x.to(cuda)
    _ok(_lib.load_dense().ajqd_matvec(dw.data_ptr(), dx.data_ptr(), 3 * k, k, y.data_ptr(), 48, 16, 3, 13, k, 2, 1, 1, _st()))
    want = (w.double().unsqueeze(0) * x.double().unsqueeze(2)).sum(-1)
    assert _rel(y[:, :, :13], want) < 1e-6 and (y[:, :, 13:] == 0).all()


def test_ring_copy_both_ways(cuda):
    ring = torch.zeros((2, 7, 16), device=cuda)
    line = torch.arange(2 * 9 * 16, dtype=torch.float32, device=cuda).view(2, 9, 16)
    _ok(_lib.load_dense().ajqd_ring_copy(ring.data_ptr(), 7, 0, line.data_ptr(), 9, 64, 3, 12, 6, 64, 2, 1, _st()))
    back = torch.zeros_like(line)
    _ok(_lib.load_dense().ajqd_ring_copy(ring.data_ptr(), 7, 0, back.data_ptr(), 9, 64, 1, 12, 6, 64, 2, 0, _st()))
    for i in range(6):
        assert torch.equal(ring[:, (12 + i) % 7], line[:, 3 + i])
    assert (ring[:, (12 + 6) % 7] == 0).all()
    assert torch.equal(back[:, 1:7], line[:, 3:9]) and (back[:, 0] == 0).all() and (back[:, 7:] == 0).all()


def _attention_case(b, h, t, prior, d1, d2, dv, seed):
    g = torch.Generator().manual_seed(seed)
    rows = prior + t

    def bf(*shape):
        return torch.randn(shape, generator=g).to(torch.bfloat16)

    return dict(q=bf(b, t, h, d1 + d2), k1=bf(b, rows, h, d1), k2=bf(b, rows, d2), v=bf(b, rows, h, dv),
                sink=torch.randn(h, generator=g) * 2, gates=torch.rand((b * t, h), generator=g))


def _attention_plain(c, prior, window, scale, sink=True, gates=True):
    q, k1, k2, v = (c[n].double() for n in ("q", "k1", "k2", "v"))
    b, t, h, _ = q.shape
    d1 = k1.shape[-1]
    rows = k1.shape[1]
    mask = O.window_mask(rows, window if window > 0 else rows)[prior:]
    out = torch.empty(b, t, h, v.shape[-1], dtype=torch.float64)
    for i in range(b):
        for n in range(h):
            scores = (q[i, :, n, :d1] @ k1[i, :, n].T + q[i, :, n, d1:] @ k2[i].T) * scale
            weights = O.softmax_with_sink(scores.masked_fill(~mask, float("-inf")), c["sink"][n].double() if sink else float("-inf"))
            out[i, :, n] = weights @ v[i, :, n]
    if gates:
        out *= c["gates"].double().view(b, t, h, 1)
    return out.reshape(b * t, h * v.shape[-1])


def _attention_gpu(c, prior, window, scale, cuda, dtype, mfma, sink=True, gates=True):
    d = {k: v.to(cuda).to(dtype) if k in ("q", "k1", "k2", "v") else v.to(cuda) for k, v in c.items()}
    b, t, h, _ = d["q"].shape
    rows, d1, d2, dv = d["k1"].shape[1], d["k1"].shape[3], d["k2"].shape[2], d["v"].shape[3]
    out = torch.full((b * t, h * dv + 16), 7.0, dtype=dtype, device=cuda)
    args = _lib.WindowedAttentionArgs(
        q=d["q"].data_ptr(), k1=d["k1"].data_ptr(), k2=d["k2"].data_ptr(), v=d["v"].data_ptr(),
        sink=d["sink"].data_ptr() if sink else None, gates=d["gates"].data_ptr() if gates else None, out=out.data_ptr(),
        k1_batch=rows * h * d1, k2_batch=rows * d2, v_batch=rows * h * dv, k1_row=h * d1, k1_head=d1, k2_row=d2, v_row=h * dv,
        v_head=dv, d1=d1, d2=d2, dv=dv, batch=b, heads=h, seq=t, rows=rows, prior=prior, window=window, out_ld=h * dv + 16, scale=scale)
    lib = _lib.load_dense()
    if mfma:
        _ok(lib.ajqd_windowed_prefill(ctypes.byref(args), _st()))
    else:
        _ok(lib.ajqd_windowed_attention(ctypes.byref(args), latent._flag(dtype), latent._flag(dtype), _st()))
    assert (out[:, h * dv:] == 7.0).all()
    return out[:, : h * dv]


ATTENTION_SHAPES = [  # b, h, t, prior, d1, d2, dv, window
    (1, 3, 150, 0, 16, 8, 32, 17),        # 1 key step
    (2, 4, 70, 31, 40, 8, 48, 32),        # 2 key steps, window exactly reached by the prior rows
    (1, 8, 300, 0, 72, 24, 96, 64),       # 3
    (1, 2, 129, 99, 96, 32, 112, 100),    # 4
    (1, 2, 260, 0, 128, 64, 128, 130),    # 6
    (1, 1, 90, 5, 192, 64, 256, 0),       # 8, no window
    (1, 5, 2, 63, 16, 16, 16, 64),        # two tokens
    (1, 2, 65, 0, 24, 8, 16, 1),          # every token sees itself only
    (1, 2, 200, 0, 32, 16, 64, 1000),     # a window longer than the sequence
]


@pytest.mark.parametrize("shape", ATTENTION_SHAPES)
@pytest.mark.parametrize("form", ["mfma", "plain-bf16", "plain-f32"])
def test_windowed_attention_against_plain(cuda, shape, form):
    b, h, t, prior, d1, d2, dv, window = shape
    c = _attention_case(b, h, t, prior, d1, d2, dv, sum(shape))
    scale = 0.9 * (d1 + d2) ** -0.5
    dtype = torch.float32 if form == "plain-f32" else torch.bfloat16
    got = _attention_gpu(c, prior, window, scale, cuda, dtype, form == "mfma")
    assert _rel(got, _attention_plain(c, prior, window, scale)) < (2e-6 if dtype == torch.float32 else 6e-3)
    bare = _attention_gpu(c, prior, window, scale, cuda, dtype, form == "mfma", sink=False, gates=False)
    assert _rel(bare, _attention_plain(c, prior, window, scale, sink=False, gates=False)) < (2e-6 if dtype == torch.float32 else 6e-3)


@pytest.mark.parametrize("mfma", [True, False])
@pytest.mark.parametrize("distance_to_edge", [0, 1])
def test_a_standing_out_key_at_the_window_edge(cuda, mfma, distance_to_edge):
    """One query and one key scaled so that their score dominates: just inside the window it takes all the weight, one
    token further out it leaves no trace.  Every query row of a block and both sides of key blocks are tried."""
    window, t = 70, 300
    for at in (63, 64, 65, 127, 128, 190):   # the key's row; the query that just sees / just misses it
        c = _attention_case(1, 2, t, 0, 32, 16, 32, at)
        query = at + window - 1 + distance_to_edge
        c["k1"][0, at] = 3.0
        c["q"][0, query, :, :32] = 3.0
        got = _attention_gpu(c, 0, window, 0.2, cuda, torch.bfloat16, mfma).cpu()
        want = _attention_plain(c, 0, window, 0.2)
        assert _rel(got, want) < 8e-3
        row = got[query].float() / c["gates"][query].repeat_interleave(32)
        dominated = _rel(row, c["v"][0, at].float().reshape(-1)) < 2e-2
        assert dominated == (distance_to_edge == 0)


@pytest.mark.parametrize("mfma", [True, False])
def test_sinks_of_any_size(cuda, mfma):
    c = _attention_case(1, 4, 80, 0, 16, 16, 32, 5)
    for sink in (-300.0, -20.0, 0.0, 20.0, 300.0):
        c["sink"] = torch.tensor([sink, 0.0, -sink, 1.0])
        got = _attention_gpu(c, 0, 30, 0.3, cuda, torch.bfloat16, mfma).double().cpu()
        want = _attention_plain(c, 0, 30, 0.3)
        assert torch.isfinite(got).all() and float((got - want).abs().max()) < 2e-2


DECODE_SHAPES = [  # batch, heads, rank, rot, vdim, rows of the ring, position
    (1, 6, 112, 24, 48, 45, 500),      # a full ring, smaller than a block of rows
    (3, 16, 48, 8, 32, 64, 63),        # exactly one block
    (1, 5, 32, 16, 16, 65, 64),        # one row in the second block
    (2, 33, 128, 24, 48, 200, 130),    # three head tiles, a ring that is partly filled
    (5, 20, 272, 64, 64, 300, 1000),
    (9, 32, 512, 64, 128, 1000, 5000),
    (1, 128, 512, 64, 128, 129, 128),
    (2, 4, 176, 8, 144, 70, 0),        # the very first token
]


@pytest.mark.parametrize("shape", DECODE_SHAPES)
def test_latent_decode_and_expand_against_plain(cuda, shape):
    """Attention in the latent space and the merge of its chunks, for every number of chunks, with one standing-out row."""
    batch, heads, rank, rot, vdim, cap, position = shape
    lib = _lib.load_dense()
    g = torch.Generator().manual_seed(sum(shape))
    bf = lambda *s: torch.randn(s, generator=g).to(torch.bfloat16)
    q, ring, uv = bf(batch, heads, rank + rot), bf(batch, cap, rank + rot), bf(heads, vdim, rank)
    sink, gate = torch.randn(heads, generator=g), torch.randn((batch, heads), generator=g)
    valid = min(position, cap - 1) + 1
    strong = valid - 1
    ring[:, strong] *= 3
    ring[:, valid:] = float("nan")   # never written rows must not be read
    scale = 0.8 * (rank + rot) ** -0.5
    scores = torch.matmul(q.double(), ring[:, :valid].double().transpose(1, 2)) * scale
    weights = O.softmax_with_sink(scores, sink.double()[None, :].expand(batch, heads))
    latents = torch.matmul(weights, ring[:, :valid, :rank].double())
    want = (uv.double()[None] * latents[:, :, None, :]).sum(-1) * torch.sigmoid(gate.double())[:, :, None]
    d = {k: v.to(cuda) for k, v in dict(q=q, ring=ring, uv=uv, sink=sink, gate=gate).items()}
    pos = torch.tensor([position], device=cuda)
    suggested = lib.ajqd_latent_decode_chunks(batch, heads, rank, rot, cap)
    assert suggested >= 1
    for chunks in sorted({1, 2, 3, 7, 32, suggested}):
        partial = torch.full((lib.ajqd_latent_decode_workspace(batch, heads, rank, chunks),), 255, dtype=torch.uint8, device=cuda)
        _ok(lib.ajqd_latent_decode(d["q"].data_ptr(), d["ring"].data_ptr(), pos.data_ptr(), partial.data_ptr(), batch, heads, rank, rot,
                                   cap, chunks, 0, scale, _st()))
        out = torch.full((batch, heads * vdim + 8), 5.0, dtype=torch.bfloat16, device=cuda)
        _ok(lib.ajqd_latent_expand(partial.data_ptr(), d["sink"].data_ptr(), d["gate"].data_ptr(), heads, d["uv"].data_ptr(),
                                   out.data_ptr(), heads * vdim + 8, batch, heads, chunks, rank, vdim, _st()))
        assert _rel(out[:, : heads * vdim], want.reshape(batch, -1)) < 8e-3, chunks
        assert (out[:, heads * vdim:] == 5.0).all()


# ------------------------------------------------------------------ the decoder against the plain implementation
SHAPES = {
    "plain": {},
    # every width off the kernels' grids, an odd head count, value width unlike the key width
    "ragged": dict(width=52, heads=3, dim=12, rot=6, vdim=10, rank=20, ff=28, vocab=61, window=7),
    # more heads than a tile, another window per layer, a layer without a feed-forward, the loop at the start
    "heads": dict(width=96, heads=18, dim=24, rot=16, vdim=40, rank=72, ff=64, window=[5, 33, 64], mlp_missing=(1,),
                  loop={"start": 0, "stop": 3, "times": 2}),
    # constants far from the usual: an eps that dominates, fast rotations, a large score scale
    "constants": dict(layers=2, eps=0.4, base=3.0, scale=0.9, loop={"start": 0, "stop": 2, "times": 2}, window=[19, 20]),
    "no loop": dict(loop=None, layers=2, window=[1, 2]),
    # one pass only (its vector is still added), the loop at the end, one head, a window no sequence here fills
    "one pass": dict(loop={"start": 2, "stop": 3, "times": 1}, heads=1, window=400),
    # widths beyond the MFMA prompt kernel: operators of any width, also in bf16
    "beyond": dict(layers=2, heads=2, dim=256, rot=16, vdim=272, loop=None, window=9),
    # wide: value tiles and key steps of a large model's layer, latents of several tiles per wave
    "wide": dict(layers=2, width=320, heads=2, dim=128, rot=64, vdim=128, rank=272, ff=520, window=70, loop={"start": 0, "stop": 1, "times": 2}),
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
def test_decode_on_plain_operators_where_widths_are_not_built(cuda, dtype, monkeypatch):
    """A latent wider than the decode kernel takes goes through the operators of any width, in bf16 as well."""
    cfg = config(layers=2, rank=544, dim=16, loop={"start": 1, "stop": 2, "times": 2})
    weights = random_weights(cfg, 9)
    model = _build(cfg, weights, cuda, dtype)
    assert _lib.load_dense().ajqd_latent_decode_chunks(1, 4, 544, 8, 11) == 0
    tokens = _tokens(cfg, 30, 2)
    want = O.forward(cfg, weights, tokens)
    cache = model.new_cache(1, 30)
    got = torch.cat([model(_ids([t], cuda), cache)[0] for t in tokens])
    assert _rel(got, want) < LOGIT_TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
def test_window_edge_by_dependence(cuda, dtype, decoded):
    """In a one-layer model a token reaches exactly window - 1 positions ahead, in prompts and in decoding, wherever the
    ring wraps: changing it changes the logits there and nothing one position further."""
    window = 13
    cfg = config(layers=1, window=window, loop=None)
    model = _build(cfg, random_weights(cfg, 11, spread=2.0), cuda, dtype)
    base = _tokens(cfg, 80, 3)

    def run(tokens):
        cache = model.new_cache(1, 80)
        if not decoded:
            return model(_ids(tokens, cuda), cache)[0]
        return torch.cat([model(_ids([t], cuda), cache)[0] for t in tokens])

    first = run(base)
    for at in (0, 1, 12, 13, 25, 26, 52, 63, 64):
        other = list(base)
        other[at] = (other[at] + 1) % cfg["vocab"]
        moved = (run(other) - first).abs().amax(dim=1).cpu()
        assert (moved[:at] == 0).all() and (moved[at + window:] == 0).all()
        assert (moved[at:min(80, at + window)] > 0).all()


@pytest.mark.parametrize("dtype", DTYPES)
def test_sinks_and_gates_show_in_the_logits(cuda, dtype):
    """Sinks far above the scores silence the heads: the plain run says how much, and it is not little."""
    cfg = config(layers=2, loop=None)
    weights = random_weights(cfg, 13)
    without = O.forward(cfg, weights, _tokens(cfg, 20, 4))
    for i in range(2):
        weights[f"l{i}.mix.sink"] = torch.tensor([9.0, -9.0, 4.0, 0.5])
        weights[f"l{i}.mix.g"] = weights[f"l{i}.mix.g"] * 4
    want = O.forward(cfg, weights, _tokens(cfg, 20, 4))
    assert _rel(without, want) > 0.05
    model = _build(cfg, weights, cuda, dtype)
    assert _rel(model(_ids(_tokens(cfg, 20, 4), cuda))[0], want) < LOGIT_TOL[dtype]
    cache = model.new_cache(1, 20)
    got = torch.cat([model(_ids([t], cuda), cache)[0] for t in _tokens(cfg, 20, 4)])
    assert _rel(got, want) < LOGIT_TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_cache_that_is_used_again_equals_a_fresh_one(cuda, dtype):
    cfg = config(window=[9, 30, 17])
    model = _build(cfg, random_weights(cfg, 15), cuda, dtype)
    cache = model.new_cache(1, 100)
    model(_ids(_tokens(cfg, 95, 5), cuda), cache)
    for ring in cache.rings:
        ring.fill_(float("nan"))   # whatever an earlier sequence left must not be read
    cache.reset()
    tokens = _tokens(cfg, 40, 6)
    fresh = model.new_cache(1, 100)
    for a, b in ((0, 3), (3, 4), (4, 6), (6, 39), (39, 40)):
        got, want = model(_ids(tokens[a:b], cuda), cache), model(_ids(tokens[a:b], cuda), fresh)
        assert torch.equal(got, want)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("batch", [2, 5, 17, 37])
def test_batch_rows_equal_sequences_alone(cuda, dtype, batch):
    """One, up to 16, up to 32 and more rows take different kernels; every row is its sequence's own."""
    cfg = config(heads=3, window=[6, 20, 11])
    weights = random_weights(cfg, 17)
    model = _build(cfg, weights, cuda, dtype)
    prompts = torch.tensor([_tokens(cfg, 31, 20 + i) for i in range(batch)], device=cuda)
    cache = model.new_cache(batch, 31)
    got = torch.cat([model(prompts[:, :23], cache)] + [model(prompts[:, t:t + 1], cache) for t in range(23, 31)], dim=1)
    for i in range(batch):
        want = O.forward(cfg, weights, prompts[i].tolist())
        assert _rel(got[i], want) < LOGIT_TOL[dtype], i


@pytest.mark.parametrize("dtype", DTYPES)
def test_wanted_places_and_lengths(cuda, dtype):
    cfg = config(positions=64)
    model = _build(cfg, random_weights(cfg, 19), cuda, dtype)
    tokens = _tokens(cfg, 60, 7)
    full = model(_ids(tokens, cuda))[0]
    for want in ([0], [59, 3, 3], list(range(20)), []):
        got = model(_ids(tokens, cuda), want=want)[0]
        assert got.shape == (len(want), cfg["vocab"])
        if want:
            assert _rel(got, full[want]) < (1e-6 if dtype == torch.float32 else 5e-3)
    assert torch.equal(model(_ids(tokens, cuda), last_token_only=True)[0, 0], model(_ids(tokens, cuda), want=[59])[0, 0])
    cache = model.new_cache(1, 64)
    model(_ids(tokens, cuda), cache)
    with pytest.raises(ValueError, match="context"):
        model(_ids(tokens[:5], cuda), cache)
    with pytest.raises(ValueError, match="holds"):
        model(_ids(tokens, cuda), model.new_cache(1, 30))
    with pytest.raises(ValueError, match="sequences"):
        model(_ids(tokens, cuda), model.new_cache(2, 64))


# ------------------------------------------------------------------ generation
def _plain_greedy(cfg, weights, prompt, count, follow):
    """Teacher-forced check of a greedy continuation: margins of every chosen token under the plain implementation."""
    logits = O.forward(cfg, weights, prompt + follow)
    rows = logits[len(prompt) - 1:len(prompt) - 1 + count]
    return rows.max(dim=-1).values - rows.gather(1, torch.tensor(follow[:count]).view(-1, 1)).squeeze(1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("batch", [1, 3, 6])
def test_greedy_generation_through_the_decoders(cuda, dtype, batch):
    """Graph-replayed decoding over several times the window: every chosen token is the plain implementation's maximum
    up to rounding, and the eager loop and portioned prompts agree with it the same way."""
    cfg = config(window=[9, 14, 30], positions=256)
    weights = random_weights(cfg, 21)
    model = _build(cfg, weights, cuda, dtype)
    prompts = torch.tensor([_tokens(cfg, 37, 40 + i) for i in range(batch)], device=cuda)
    noise = 4 * LOGIT_TOL[dtype]
    new = 75
    graph = decoding.greedy_decode_graph(model, prompts, new)
    eager = modeling.greedy_decode(model, prompts, new)
    dec = decoding.DenseDecoder(model, batch, 37 + new)
    dec.prefill(prompts, tokens_per_pass=8)
    portions = dec.generate(new)
    for i in range(batch):
        for tokens in (graph[i, 37:], eager[i, 37:], portions[i]):
            assert float(_plain_greedy(cfg, weights, prompts[i].tolist(), new, tokens.tolist()).max()) <= noise
    assert graph.shape == eager.shape == (batch, 37 + new)


def test_graph_replays_equal_the_eager_step(cuda):
    """The same decoder used for two prompts (the second from a used cache), with other work between the replays."""
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

    def draw(seed):
        dec = decoding.DenseDecoder(model, 1, 80)
        dec.set_sampling(1.0, 0.9, seed)
        dec.prefill(prompts)
        return dec.generate(60)

    assert torch.equal(draw(1), draw(1)) and not torch.equal(draw(1), draw(2))
    dec = decoding.DenseDecoder(model, 1, 80)
    dec.prefill(prompts)
    tokens = dec.generate(60)[0].tolist()
    dec = decoding.DenseDecoder(model, 1, 80)
    dec.prefill(prompts)
    stop = tokens[30]
    assert dec.generate(60, eos_token_id=stop)[0].tolist() == tokens[: tokens.index(stop) + 1]


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
    assert len(new) == 12 and float(_plain_greedy(cfg, weights, prompt, 12, new).max()) < 1e-3
