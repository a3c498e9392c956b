"""Dorutar on the host: the plain implementation (oracle/dorutar.py) against itself and against closed forms, the
registry and the checkpoint reader, the packed weights, the ring cache's bookkeeping and the dense library's ABI."""

import json
import math
import re
from pathlib import Path

import pytest
import torch
from safetensors.torch import save_file

from ajllm_amd import _lib, checkpoint, latent, modeling
from tests.latent_models import config, random_weights
from oracle import dorutar as O

HEADER = Path(__file__).resolve().parents[1] / "include" / "ajq_dense.h"


# ------------------------------------------------------------------ the plain implementation
def test_rotation_is_the_closed_form_and_relative():
    v = torch.randn(10, dtype=torch.float64)
    out = O.rotate_halves(v, 7, 1000.0, 8)
    for i in range(4):
        angle = 7 * 1000.0 ** (-2 * i / 8)
        assert out[i] == pytest.approx(float(v[i]) * math.cos(angle) - float(v[i + 4]) * math.sin(angle))
        assert out[i + 4] == pytest.approx(float(v[i + 4]) * math.cos(angle) + float(v[i]) * math.sin(angle))
    assert torch.equal(out[8:], v[8:])
    a, b = torch.randn(8, dtype=torch.float64), torch.randn(8, dtype=torch.float64)
    near = O.rotate_halves(a, 5, 1000.0, 8) @ O.rotate_halves(b, 3, 1000.0, 8)
    far = O.rotate_halves(a, 105, 1000.0, 8) @ O.rotate_halves(b, 103, 1000.0, 8)
    assert near == pytest.approx(float(far))
    rows = torch.randn(6, 3, 10, dtype=torch.float64)
    whole = O.rotate_sequence(rows, 1000.0, 8)
    for t in range(6):
        for h in range(3):
            assert torch.allclose(whole[t, h], O.rotate_halves(rows[t, h], t, 1000.0, 8))


def test_norms_match_the_library():
    x, w = torch.randn(5, 12, dtype=torch.float64), torch.rand(12, dtype=torch.float64)
    assert torch.allclose(O.layer_norm(x, w, 1e-5), torch.nn.functional.layer_norm(x, (12,), w, None, 1e-5))
    assert torch.allclose(O.rms_norm(x, w, 1e-5), torch.nn.functional.rms_norm(x, (12,), w, 1e-5))
    norm = modeling.build_norm("layernorm", 12, 1e-3)
    assert torch.allclose(norm(x.float()), torch.nn.functional.layer_norm(x.float(), (12,), eps=1e-3), atol=1e-6)


def test_sink_counts_once_without_a_value():
    scores = torch.tensor([[0.3, -1.0, 2.0]], dtype=torch.float64)
    got = O.softmax_with_sink(scores, torch.tensor([0.7], dtype=torch.float64))
    exps = scores.exp()
    assert torch.allclose(got, exps / (exps.sum() + math.exp(0.7)))
    assert float(got.sum()) < 1.0


def test_window_holds_exactly_its_size():
    mask = O.window_mask(9, 4)
    for i in range(9):
        assert [j for j in range(9) if mask[i, j]] == [j for j in range(9) if O.visible(i, j, 4)] == list(range(max(0, i - 3), i + 1))


def test_later_tokens_do_not_change_earlier_logits_and_distant_ones_leave_one_layer():
    cfg = config(layers=1, window=5, loop=None)
    w = random_weights(cfg, 3)
    tokens = list(range(12))
    full = O.forward(cfg, w, tokens)
    assert torch.allclose(O.forward(cfg, w, tokens[:7]), full[:7])
    changed = [5] + tokens[1:]
    other = O.forward(cfg, w, changed)
    assert torch.allclose(other[5:], full[5:]) and not torch.allclose(other[4], full[4])  # position 5 no longer sees 0


def test_loop_runs_and_what_is_added_before_each_pass():
    assert O.layer_runs(4, {"start": 1, "stop": 3, "times": 2}) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert O.layer_runs(2, None) == [(0, None), (1, None)]
    cfg = config(layers=1, loop={"start": 0, "stop": 1, "times": 2})
    w = random_weights(cfg, 4)
    for name in list(w):  # layers that add nothing leave x = embedded + step0, then + embedded + step1
        if name.endswith((".mix.o", ".mlp.down")):
            w[name] = torch.zeros_like(w[name])
    seen: list[torch.Tensor] = []
    O.forward(cfg, w, [1, 2, 3], residuals=seen)
    e = O.embedding([1, 2, 3], w["embed"].double(), w["pos"].double())
    step = w["loop.step"].double()
    assert torch.allclose(seen[0], e + step[0]) and torch.allclose(seen[1], 2 * e + step[0] + step[1])


# ------------------------------------------------------------------ registry, configuration, weights
def test_registry_builds_the_architecture_and_refuses_others():
    cfg = config()
    with torch.device("meta"):
        model = modeling.build_model(cfg)
    assert isinstance(model, latent.LatentLM) and model.runs == O.layer_runs(len(cfg["layers"]), cfg["loop"])
    assert set(model.checkpoint_names().values()) == set(random_weights(cfg, 0))
    with pytest.raises(ValueError, match="architecture"):
        modeling.build_model({**cfg, "architecture": "Nothing"})
    with pytest.raises(ValueError):
        modeling.build_model({"d_model": 8})
    bad = config()
    bad["layers"][0]["type"] = "other"
    with pytest.raises(ValueError, match="mixer"):
        modeling.build_model(bad)
    bad = config()
    bad["layers"][0]["mlp"] = {"kind": "sparse", "ff": 8}
    with pytest.raises(ValueError, match="feed-forward"):
        modeling.build_model(bad)
    bad = config()
    bad["loop"] = {"start": 1, "stop": 9, "times": 2}
    with pytest.raises(ValueError, match="loop"):
        modeling.build_model(bad)


def _folder(tmp_path, cfg, weights):
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in weights.items()}, str(tmp_path / "model.safetensors"))
    return tmp_path


def test_checkpoint_folder_loads_strictly(tmp_path):
    cfg = config(mlp_missing=(0,))
    w = random_weights(cfg, 1)
    model = checkpoint.load_model(_folder(tmp_path, cfg, w), "cpu", torch.float32)
    state, names = model.state_dict(), model.checkpoint_names()
    assert model.layers[0].feed_forward is None and model.layers[0].norm2 is None
    for key, name in names.items():
        assert torch.equal(state[key], w[name].to(torch.bfloat16).float())
    extra = {**w, "l0.norm2": torch.ones(cfg["width"])}   # a norm no layer reads may be there
    checkpoint.load_model(_folder(tmp_path, cfg, extra), "cpu")
    with pytest.raises(ValueError, match="unexpected"):
        checkpoint.load_model(_folder(tmp_path, cfg, {**w, "l0.bias": torch.ones(3)}), "cpu")
    with pytest.raises(ValueError, match="missing"):
        checkpoint.load_model(_folder(tmp_path, cfg, {k: v for k, v in w.items() if k != "l1.mix.sink"}), "cpu")


def test_the_model_has_no_cpu_path(tmp_path):
    cfg = config()
    model = checkpoint.load_model(_folder(tmp_path, cfg, random_weights(cfg, 1)), "cpu")
    with pytest.raises(ValueError, match="ROCm"):
        model(torch.zeros((1, 3), dtype=torch.long))


def test_packed_weights_compute_the_same_projections():
    """Every padded, stacked or transposed weight gives the product its parts give (host tensors: packing is plain torch)."""
    cfg = config(width=52, heads=3, dim=12, rot=6, vdim=10, rank=20, ff=28)
    model = modeling.build_model(cfg)
    block = model.layers[0]
    with torch.no_grad():
        for p in block.parameters():
            p.normal_()
        w = latent.PackedBlock(block, latent.rotary_tables(100.0, 6, 8))
        mix, ff = block.mixer, block.feed_forward
        h = torch.randn(52)
        hp = torch.zeros(w.w1.shape[1])
        hp[:52] = h
        y = w.w1 @ hp
        q = y[: 3 * (w.dimp + w.rotp)].view(3, -1)
        want = (mix.q_proj.weight @ h).view(3, 18)
        assert torch.allclose(q[:, :12], want[:, :12], atol=1e-4) and torch.allclose(q[:, w.dimp:w.dimp + 6], want[:, 12:], atol=1e-4)
        assert (q[:, 12:w.dimp] == 0).all() and (q[:, w.dimp + 6:] == 0).all()
        at = 3 * (w.dimp + w.rotp)
        down = mix.dkv_proj.weight @ h
        assert torch.allclose(y[at:at + 20], down[:20], atol=1e-4)
        assert torch.allclose(y[at + w.rankp:at + w.rankp + 6], down[20:], atol=1e-4)
        assert torch.allclose(y[w.gate_column:w.gate_column + 3], mix.gate_proj.weight @ h, atol=1e-4)
        c = torch.randn(20)
        cp = torch.zeros(w.rankp)
        cp[:20] = c
        kv = w.ukv @ cp
        assert torch.allclose(kv[: 3 * w.dimp].view(3, -1)[:, :12], (mix.uk_proj.weight @ c).view(3, 12), atol=1e-4)
        assert torch.allclose(kv[3 * w.dimp:].view(3, -1)[:, :10], (mix.uv_proj.weight @ c).view(3, 10), atol=1e-4)
        assert torch.equal(w.ukt[1, :20, :12], mix.uk_proj.weight.view(3, 12, 20)[1].T)
        gu = (w.w2 @ hp).view(-1, 2, 8)
        assert torch.allclose(gu[:, 0].reshape(-1)[:28], ff.w1.weight @ h, atol=1e-4)
        assert torch.allclose(gu[:, 1].reshape(-1)[:28], ff.w3.weight @ h, atol=1e-4)
        heads, mid = torch.randn(3, 10), torch.randn(28)
        joined = torch.zeros(w.joined)
        joined[: 3 * w.vdimp].view(3, -1)[:, :10] = heads
        joined[3 * w.vdimp:3 * w.vdimp + 28] = mid
        want = mix.output_proj.weight @ heads.reshape(-1) + ff.w2.weight @ mid
        assert torch.allclose((w.wo @ joined)[:52], want, atol=1e-4)


def test_rotary_tables():
    cos, sin = latent.rotary_tables(50.0, 6, 2000)
    for p in (0, 1, 1999):
        for i in range(3):
            angle = p * 50.0 ** (-2 * i / 6)
            assert float(cos[p, i]) == pytest.approx(math.cos(angle), abs=1e-7)
            assert float(sin[p, i]) == pytest.approx(math.sin(angle), abs=1e-7)


def test_ring_cache_holds_a_window_per_run():
    cfg = config(layers=3, window=[5, 9, 7], loop={"start": 0, "stop": 2, "times": 2})
    model = modeling.build_model(cfg)
    cache = model.new_cache(2, 8)
    assert [tuple(r.shape[:2]) for r in cache.rings] == [(2, 5), (2, 8), (2, 5), (2, 8), (2, 7)]
    part = cache.rows(1, 2)
    assert part.batch == 1 and part.rings[0].data_ptr() == cache.rings[0][1].data_ptr()
    cache.length, cache.static = 4, True
    cache.reset()
    assert cache.length == 0 and not cache.static
    with pytest.raises(ValueError):
        model.new_cache(1, 8, torch.float16)


def test_gated_feed_forward_activations():
    ff = modeling.build_feed_forward("reglu", 6, 10)
    x = torch.randn(3, 6)
    with torch.no_grad():
        assert torch.allclose(ff(x), O.gated_relu(x, ff.w1.weight, ff.w3.weight, ff.w2.weight), atol=1e-6)
        assert torch.allclose(modeling.ACTIVATIONS["gelu_tanh"](x), torch.nn.functional.gelu(x, approximate="tanh"), atol=1e-6)
    with pytest.raises(ValueError):
        modeling.GatedFeedForward(6, 10, "none")


# ------------------------------------------------------------------ the library
def test_dense_library_exports_what_its_header_declares():
    text = re.sub(r"/\*.*?\*/", "", HEADER.read_text(), flags=re.S)
    names = sorted(set(re.findall(r"\b(ajqd_[a-z0-9_]+)\s*\(", text)))
    lib = _lib.load_dense()
    assert names == sorted(_lib.DENSE_SIGNATURES) and len(names) >= 14
    for name in names:
        assert hasattr(lib, name)


def test_dense_library_refuses_bad_arguments_before_any_launch():
    import ctypes

    lib = _lib.load_dense()
    buf = ctypes.create_string_buffer(4096)
    p = ctypes.c_void_p((ctypes.addressof(buf) + 15) & ~15)
    assert lib.ajqd_embed(None, 1, 1, None, 4, None, 0, 0, None, None, None, None, 16, 0, None) == -1
    assert b"null" in lib.ajqd_last_error()
    assert lib.ajqd_embed(p, 3, 3, p, 4, p, 8, 6, None, None, p, None, 16, 0, None) == -2      # positions 6 .. 8 of 8
    assert lib.ajqd_embed(p, 1, 1, p, 4, p, 8, 0, None, None, p, None, 16, 7, None) == -4      # unknown dtype
    assert lib.ajqd_add_norms(p, None, 1, None, None, p, None, 1e-5, 1, p, None, 1, 12, 12, 0, None) == -2
    assert lib.ajqd_ring_copy(p, 4, 0, p, 8, 32, 0, 0, 5, 32, 1, 1, None) == -2                        # more rows than the ring has
    assert lib.ajqd_matvec(p, p, 8, 0, p, 4, 0, 1, 4, 12, 1, 0, 1, None) == -2
    assert lib.ajqd_dense_out(p, p, p, None, None, 1, 8, 24, None) == -2
    args = _lib.WindowedAttentionArgs(q=p, k1=p, k2=p, v=p, out=p, k1_row=16, k1_head=8, k2_row=8, v_row=16, v_head=16, d1=8,
                                      d2=8, dv=16, batch=1, heads=1, seq=4, rows=4, prior=1, out_ld=16, scale=1.0)
    assert lib.ajqd_windowed_attention(ctypes.byref(args), 0, 0, None) == -2 and b"do not fit" in lib.ajqd_last_error()
    args.prior, args.scale = 0, 0.0
    assert lib.ajqd_windowed_prefill(ctypes.byref(args), None) == -2
    assert lib.ajqd_windowed_prefill_supported(128, 64, 128) == 1 and lib.ajqd_windowed_prefill_supported(256, 64, 128) == 0
    assert lib.ajqd_latent_decode_chunks(1, 32, 512, 64, 1024) == 16 and lib.ajqd_latent_decode_chunks(1, 32, 528, 64, 1024) == 0
    dense_in = _lib.DenseInArgs(x=p, gain1=p, w1=p, y1=p, batch=5, true_width=16, width=16, tiles1=1)
    assert lib.ajqd_dense_in(ctypes.byref(dense_in), None) == -4                                # norm prologue: at most 4 rows


def test_trace_replay_refuses_bad_steps():
    from ajllm_amd.trace import Session

    class Fake:
        vocab_size, context_length = 8, 16

    session = Session(Fake(), 64)
    assert session.max_len == 16
    for entry in ({"id": "a", "tokens": [9], "want": []}, {"id": "a", "tokens": [], "want": []},
                  {"id": "a", "tokens": [1, 2], "want": [2]}):
        with pytest.raises(ValueError):
            session.step([entry], [])
