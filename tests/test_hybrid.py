"""Purusun on the host: the plain implementation (oracle/purusun.py) against closed forms and torch's own functions, the registry
and the checkpoint reader, the packed weights, the cache's shapes and the dense library's argument checks."""

import ctypes
import json
import math

import pytest
import torch
from safetensors.torch import save_file

from ajllm_amd import _lib, checkpoint, dense, hybrid, modeling
from oracle import purusun as O
from tests.hybrid_models import SCALING, attention, config, random_weights, scan

F = torch.nn.functional


# ------------------------------------------------------------------ the plain implementation
def test_norms_and_activations_match_torch():
    x, w = torch.randn(5, 12, dtype=torch.float64), torch.randn(12, dtype=torch.float64)
    assert torch.allclose(O.centered_rms_norm(x, w, 1e-3), F.rms_norm(x, (12,), 1 + w, 1e-3))
    norm = modeling.build_norm("zero_centered_rmsnorm", 12, 1e-3)
    assert (norm.weight == 0).all()
    with torch.no_grad():
        norm.weight.copy_(w)
        assert torch.allclose(norm(x.float()), F.rms_norm(x.float(), (12,), 1 + w.float(), 1e-3), atol=1e-5)
    z = torch.cat((torch.linspace(-60, 60, 41, dtype=torch.float64), torch.zeros(1, dtype=torch.float64)))
    assert torch.allclose(O.softplus(z), F.softplus(z, threshold=1000)) and torch.allclose(O.silu(z), F.silu(z))
    h, up, down = torch.randn(3, 6), torch.randn(10, 6), torch.randn(6, 10)
    ff = modeling.build_feed_forward("squared_relu", 6, 10)
    with torch.no_grad():
        ff.w1.weight.copy_(up)
        ff.w2.weight.copy_(down)
        assert torch.allclose(ff(h), O.squared_relu(h, up, down), atol=1e-5)


def test_frequency_scaling_keeps_blends_and_divides():
    dims, base = 64, 500.0
    plain = [O.frequency(base, dims, i, None) for i in range(dims // 2)]
    scaled = [O.frequency(base, dims, i, SCALING) for i in range(dims // 2)]
    kinds = set()
    for f, s in zip(plain, scaled):
        wavelength = 2 * math.pi / f
        if wavelength < SCALING["original"] / SCALING["high"]:
            kinds.add("kept")
            assert s == f
        elif wavelength > SCALING["original"] / SCALING["low"]:
            kinds.add("divided")
            assert s == f / SCALING["factor"]
        else:
            kinds.add("between")
            assert f / SCALING["factor"] <= s <= f
    assert kinds == {"kept", "between", "divided"}
    assert all(a >= b for a, b in zip(scaled, scaled[1:]))   # the blend meets both ends: no jump upwards
    for scaling in (None, SCALING):
        held = dense.FrequencyScaling(**{k: float(v) for k, v in scaling.items()}) if scaling else None
        got = dense.rotary_frequencies(base, dims, held)
        want = torch.tensor([O.frequency(base, dims, i, scaling) for i in range(dims // 2)], dtype=torch.float64)
        assert torch.allclose(got, want, rtol=1e-14, atol=0)


def test_rotation_turns_halves_and_is_relative():
    rot = {"dims": 8, "base": 50.0, "scaling": None}
    v = torch.randn(11, dtype=torch.float64)
    out = O.rotate(v, 9, rot)
    for i in range(4):
        turned = torch.view_as_complex(torch.stack((v[i], v[i + 4]))) * torch.polar(torch.tensor(1.0).double(), torch.tensor(9 * 50.0 ** (-i / 4)).double())
        assert torch.allclose(torch.view_as_real(turned), torch.stack((out[i], out[i + 4])))
    assert torch.equal(out[8:], v[8:])
    a, b = torch.randn(8, dtype=torch.float64), torch.randn(8, dtype=torch.float64)
    assert torch.allclose(O.rotate(a, 5, rot) @ O.rotate(b, 3, rot), O.rotate(a, 2005, rot) @ O.rotate(b, 2003, rot))


def test_window_beside_kept_first_tokens():
    for window, keep in ((4, 0), (4, 2), (1, 1), (3, 9), (None, 0)):
        mask = O.visible_mask(12, window, keep)
        for i in range(12):
            near = range(0 if window is None else max(0, i - window + 1), i + 1)
            want = sorted(set(near) | set(range(min(keep, i + 1))))
            assert [j for j in range(12) if mask[i, j]] == want == [j for j in range(12) if O.visible(i, j, window, keep)]


def test_attention_is_torchs_with_keys_as_values():
    spec = attention(heads=6, kv_heads=2, dim=10, rot=4, window=5, keep=2)
    w = {k[len("l0.mix."):]: v.double() for k, v in random_weights(config([spec], loop=None), 3).items() if k.startswith("l0.mix.")}
    h = torch.randn(20, 48, dtype=torch.float64)
    raw = (h @ w["k"].T).view(20, 2, 10)
    q = O.rotate_rows(F.rms_norm((h @ w["q"].T).view(20, 6, 10), (10,), w["q.norm"], 1e-5), spec["mixer"]["rot"])
    k = O.rotate_rows(F.rms_norm(raw, (10,), w["k.norm"], 1e-5), spec["mixer"]["rot"])
    got = F.scaled_dot_product_attention(q.transpose(0, 1), k.transpose(0, 1).repeat_interleave(3, 0), raw.transpose(0, 1).repeat_interleave(3, 0),
                                         attn_mask=O.visible_mask(20, 5, 2), scale=spec["mixer"]["scale"])
    want = (got.transpose(0, 1).reshape(20, 60) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T
    assert torch.allclose(O.key_value_attention(h, w, spec["mixer"], 1e-5), want)


def test_convolution_is_torchs():
    x, w, b = torch.randn(9, 5, dtype=torch.float64), torch.randn(5, 4, dtype=torch.float64), torch.randn(5, dtype=torch.float64)
    want = F.conv1d(F.pad(x.T[None], (3, 0)), w[:, None], b, groups=5)[0].T
    assert torch.allclose(O.causal_conv(x, w, b), want)


def test_recurrence_in_closed_form_and_from_a_state():
    t, ch, n = 7, 3, 2
    x, dt = torch.randn(t, ch, dtype=torch.float64), torch.rand(t, ch, dtype=torch.float64)
    a, d = -torch.rand(ch, n, dtype=torch.float64), torch.randn(ch, dtype=torch.float64)
    b, c = torch.randn(t, n, dtype=torch.float64), torch.randn(t, n, dtype=torch.float64)
    y, last = O.recurrence(x, dt, a, b, c, d)
    for i in range(t):
        for k in range(ch):
            want = float(d[k] * x[i, k])
            for j in range(i + 1):
                for m in range(n):
                    decay = math.exp(float(a[k, m]) * float(dt[j + 1:i + 1, k].sum()))
                    want += decay * float(dt[j, k] * x[j, k] * b[j, m] * c[i, m])
            assert float(y[i, k]) == pytest.approx(want)
    head, state = O.recurrence(x[:3], dt[:3], a, b[:3], c[:3], d)
    tail, end = O.recurrence(x[3:], dt[3:], a, b[3:], c[3:], d, state)
    assert torch.allclose(torch.cat((head, tail)), y) and torch.allclose(end, last)


def test_hyper_connection_reads_mixes_and_writes():
    """One stream with neutral coefficients is the plain residual sum; the mix is indexed [from, to], all from the old streams."""
    x = torch.randn(1, 4, 6, dtype=torch.float64)
    one = {"in": torch.ones(1).double(), "out": torch.ones(1).double(), "mix": torch.ones(1, 1).double()}
    assert torch.allclose(O.hyper_sublayer(x, one, torch.sin), x + torch.sin(x))
    x = torch.randn(2, 4, 6, dtype=torch.float64)
    hc = {"in": torch.tensor([2.0, -1.0]).double(), "out": torch.tensor([0.5, 3.0]).double(), "mix": torch.tensor([[1.0, 10.0], [0.0, 1.0]]).double()}
    got = O.hyper_sublayer(x, hc, torch.sin)
    y = torch.sin(2 * x[0] - x[1])
    assert torch.allclose(got[0], x[0] + 0.5 * y) and torch.allclose(got[1], 10 * x[0] + x[1] + 3 * y)


def test_loop_order():
    assert O.layer_order(4, {"start": 1, "stop": 3, "times": 2}) == [0, 1, 2, 1, 2, 3]
    assert O.layer_order(2, None) == [0, 1] and O.layer_order(2, {"start": 0, "stop": 2, "times": 1}) == [0, 1]


def test_later_tokens_do_not_change_earlier_logits():
    cfg = config()
    w = random_weights(cfg, 3)
    tokens = list(range(14))
    full = O.forward(cfg, w, tokens)
    assert torch.allclose(O.forward(cfg, w, tokens[:8]), full[:8])
    other = O.forward(cfg, w, [5] + tokens[1:])
    assert not torch.allclose(other[-1], full[-1])


# ------------------------------------------------------------------ registry, configuration, weights
def test_registry_builds_the_architecture_and_refuses_others():
    cfg = config()
    with torch.device("meta"):
        model = modeling.build_model(cfg)
    assert isinstance(model, hybrid.HybridLM) and [i for i, _ in model.runs] == O.layer_order(4, cfg["loop"])
    assert set(model.checkpoint_names().values()) == set(random_weights(cfg, 0))
    bare = attention(window=None)
    bare["mixer"].update(rot=None, mask=None)
    with torch.device("meta"):
        mix = modeling.build_model(config([bare], loop=None)).layers[0].mixer
    assert mix.window is None and mix.rot_dim == 0
    for change, message in (({"type": "other"}, "mixer"), ({"mlp": {"kind": "sparse", "ff": 8}}, "feed-forward")):
        with pytest.raises(ValueError, match=message):
            modeling.build_model(config([{**scan(), **change}], loop=None))
    for bad, message in ((attention(heads=5, kv_heads=2), "divisible"), (attention(rot=18), "rotated"), (attention(rot=7), "rotated")):
        with pytest.raises(ValueError, match=message):
            modeling.build_model(config([bad], loop=None))
    odd = attention()
    odd["mixer"]["vdim"] = 8
    with pytest.raises(ValueError, match="vdim"):
        modeling.build_model(config([odd], loop=None))
    with pytest.raises(ValueError, match="loop"):
        modeling.build_model(config(loop={"start": 2, "stop": 9, "times": 2}))


def _folder(tmp_path, cfg, weights):
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in weights.items()}, str(tmp_path / "model.safetensors"))
    return tmp_path


def test_checkpoint_folder_loads_strictly(tmp_path):
    cfg = config([scan(ff=None), attention()], loop=None)
    w = random_weights(cfg, 1)
    model = checkpoint.load_model(_folder(tmp_path, cfg, w), "cpu", torch.float32)
    state = model.state_dict()
    for key, name in model.checkpoint_names().items():
        assert torch.equal(state[key], w[name])
    assert model.layers[0].feed_forward is None and model.layers[0].hyper2 is None
    extra = {**w, "l0.norm2": torch.ones(cfg["width"]), "l0.hc2.in": torch.ones(3)}   # of a sublayer that is not there
    checkpoint.load_model(_folder(tmp_path, cfg, extra), "cpu")
    with pytest.raises(ValueError, match="unexpected"):
        checkpoint.load_model(_folder(tmp_path, cfg, {**w, "l1.mix.v": torch.ones(3)}), "cpu")
    with pytest.raises(ValueError, match="missing"):
        checkpoint.load_model(_folder(tmp_path, cfg, {k: v for k, v in w.items() if k != "l0.mix.D"}), "cpu")


def test_the_model_has_no_cpu_path(tmp_path):
    cfg = config()
    model = checkpoint.load_model(_folder(tmp_path, cfg, random_weights(cfg, 1)), "cpu")
    with pytest.raises(ValueError, match="ROCm"):
        model(torch.zeros((1, 3), dtype=torch.long))


def test_packed_attention_computes_the_same_projections():
    cfg = config([attention(heads=3, kv_heads=1, dim=12, rot=6)], width=52, loop=None)
    model = modeling.build_model(cfg)
    mix = model.layers[0].mixer
    with torch.no_grad():
        for p in model.parameters():
            p.normal_()
        w = hybrid.PackedAttention(mix, 64)
        h, joined = torch.randn(52), torch.randn(3, 12)
        y = w.w_in @ F.pad(h, (0, 12))
        parts = y.view(7, 16)
        want = torch.cat((mix.q_proj.weight, mix.k_proj.weight, mix.gate_proj.weight)) @ h
        assert torch.allclose(parts[:, :12].reshape(-1), want, atol=1e-4) and (parts[:, 12:] == 0).all()
        assert torch.allclose(y[w.gate_column:].view(3, 16)[:, :12].reshape(-1), mix.gate_proj.weight @ h, atol=1e-4)
        out = w.w_out @ F.pad(joined, (0, 4)).reshape(-1)
        assert torch.allclose(out[:52], mix.output_proj.weight @ joined.reshape(-1), atol=1e-4) and (out[52:] == 0).all()
        assert torch.equal(w.q_gain[:12], mix.q_norm.weight) and (w.q_gain[12:] == 0).all()
        assert torch.allclose(w.half_turns * math.pi, dense.rotary_frequencies(300.0, 6), rtol=1e-15)


def test_packed_scan_computes_the_same_projections():
    cfg = config([scan(inner=20, state=5, rank=3, conv=2)], width=44, loop=None)
    model = modeling.build_model(cfg)
    mix = model.layers[0].mixer
    with torch.no_grad():
        for p in model.parameters():
            p.normal_()
        w = hybrid.PackedScan(mix, 48)
        assert (w.inner, w.states, w.rank, w.taps, w.low_rows) == (32, 8, 8, 2, 32)
        h, x, dt = torch.randn(44), torch.randn(20), torch.randn(3)
        y = (w.w_in @ F.pad(h, (0, 4))).view(2, 32)
        assert torch.allclose(y[:, :20].reshape(-1), mix.in_proj.weight @ h, atol=1e-4) and (y[:, 20:] == 0).all()
        low, want = w.w_low @ F.pad(x, (0, 12)), mix.x_proj.weight @ x
        assert torch.allclose(low[:3], want[:3], atol=1e-4) and torch.allclose(low[8:13], want[3:8], atol=1e-4)
        assert torch.allclose(low[16:21], want[8:], atol=1e-4) and (low[[3, 7, 13, 15, 21]] == 0).all()
        assert torch.allclose((w.w_dt @ F.pad(dt, (0, 5)))[:20], mix.dt_proj.weight @ dt, atol=1e-5)
        planes = w.a2.permute(1, 0, 2).reshape(32, 8)    # [channels, states]
        assert torch.allclose(planes[:20, :5] * math.log(2), -torch.exp(mix.a_log), rtol=1e-6) and (planes[20:] == 0).all() and (planes[:, 5:] == 0).all()
        assert torch.equal(w.conv[1, :20], mix.conv_weight[:, 1])   # the last row meets the token itself


def test_cache_holds_windows_kept_rows_columns_and_states():
    cfg = config([attention(window=5, keep=2), attention(window=9, keep=0), attention(window=None), scan(conv=1, state=6), scan(inner=20)],
                 loop={"start": 0, "stop": 1, "times": 2})
    model = modeling.build_model(cfg)
    cache = model.new_cache(2, 8)
    assert [tuple(r.shape) for r in cache.rings] == [(2, 2, 7, 32), (2, 2, 7, 32), (2, 2, 8, 32), (2, 2, 8, 32), (2, 0, 48), (2, 3, 32)]
    assert cache.kept == [2, 2, 0, 0, 0, 0]
    assert [None if s is None else tuple(s.shape) for s in cache.states] == [None] * 4 + [(2, 2, 48, 4), (2, 2, 32, 4)]
    assert all(s.dtype == torch.float32 for s in cache.states[4:])
    part = cache.rows(1, 2)
    assert part.rings[0].data_ptr() == cache.rings[0][1].data_ptr() and part.states[4].data_ptr() == cache.states[4][1].data_ptr()
    with pytest.raises(ValueError, match="max_len"):
        model.new_cache(1)
    with pytest.raises(ValueError):
        model.new_cache(1, 8, torch.float16)


# ------------------------------------------------------------------ the library
def test_dense_library_refuses_bad_arguments_before_any_launch():
    lib = _lib.load_dense()
    buf = ctypes.create_string_buffer(4096)
    p = ctypes.c_void_p((ctypes.addressof(buf) + 15) & ~15)
    assert lib.ajqd_embed_streams(p, 1, p, 4, p, p, p, 17, 16, 0, None) == -4                            # streams
    assert lib.ajqd_streams_norm(p, p, None, None, None, p, p, 1e-5, p, None, 2, 1, 16, 16, 0, None) == -1
    assert lib.ajqd_streams_norm(p, None, None, None, None, p, p, 1e-5, p, None, 2, 1, 24, 16, 0, None) == -2
    assert lib.ajqd_dense_out_streams(p, p, p, p, p, p, None, p, 2, 1, 12, 16, None) == -2
    assert lib.ajqd_activation(p, p, 12, 0, 0, None) == -2 and lib.ajqd_activation(p, p, 16, 9, 0, None) == -4
    split = _lib.KeyValueSplitArgs(y=p, q_gain=p, k_gain=p, half_turns=p, q=p, rows=p, tokens=4, seq=4, ldy=48, heads=1, groups=1, dim=16, dimp=16,
                                   rot=18, q_ld=16, rows_batch=128, rows_head=128)
    assert lib.ajqd_key_value_split(ctypes.byref(split), 0, 0, None) == -2                               # rotates more than a head has
    split.rot, split.groups, split.rows_head = 8, 2, 64
    assert lib.ajqd_key_value_split(ctypes.byref(split), 0, 0, None) == -2 and b"overlap" in lib.ajqd_last_error()
    split.pos, split.cap, split.kept = p, 4, 4
    assert lib.ajqd_key_value_split(ctypes.byref(split), 0, 0, None) == -2                               # no slot beside the kept ones
    assert lib.ajqd_ring_copy(p, 6, 2, p, 8, 32, 0, 2, 5, 32, 1, 1, None) == -2                          # 5 positions for 4 moving slots
    assert lib.ajqd_group_merge(p, None, 0, p, 16, 1, 1, 1, 40, 16, None) == -2
    assert lib.ajqd_conv_silu(p, 16, None, p, p, 3, None, 2, 2, 16, 4, p, 0, None) == -1                 # no columns from before
    args = _lib.ScanArgs(x=p, dt=p, low=p, z=p, a2=p, d=p, dt_bias=p, out=p, batch=1, seq=2, inner=16, states=6, dt_ld=16, low_ld=16, z_ld=16, out_ld=16)
    assert lib.ajqd_scan(ctypes.byref(args), 0, None) == -2
    args.states, args.low_ld, args.start = 4, 16, 5
    assert lib.ajqd_scan(ctypes.byref(args), 0, None) == -1                                              # no state to start from
    args.start, args.states, args.low_ld, args.c_col = 0, 260, 600, 260
    assert lib.ajqd_scan(ctypes.byref(args), 0, None) == -4
    assert lib.ajqd_scan_project(p, 16, p, p, p, p, p, p, 1, 16, 4, 16, 1, None) == -2                   # y holds both halves
    step = _lib.ScanStepArgs(y=p, ring=p, weight=p, bias=p, pos=p, partial=p, w_dt=p, dt_bias=p, a2=p, d=p, state=p, out=p, batch=1, ldy=32, inner=16,
                             taps=4, rows=16, splits=1, rank=8, states=8, out_ld=16)
    assert lib.ajqd_scan_step(ctypes.byref(step), None) == -2                                            # 8 + 16 rows in 16
