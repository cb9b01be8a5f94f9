"""Hybrid designs on the CPU: configuration, weight layout, registry, state pool, row packing,
trace replay, and the plain reference checked against independent formulations."""
import json
import math
from types import SimpleNamespace

import hybrid_oracle as O
import pytest
import torch
from hybrid_cases import CASES, attention, delta, model, tokens, weights_of

from cake_amd.models.base import StepEntry
from cake_amd.models.hybrid.config import Run, from_config
from cake_amd.models.hybrid.state import StatePool
from cake_amd.models.hybrid.weights import LayerWeights, ModelWeights, tensor_shapes
from cake_amd.models.registry import HYBRID, LLAMA, check_placement, family_of
from cake_amd.ops.mixers import AttnShape, DeltaShape, Rows


# ---------------------------------------------------------------------------- configuration
def test_run_order():
    cfg = from_config(CASES["mixed"])
    assert [(r.layer, r.enter) for r in cfg.runs()] == \
        [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert cfg.runs()[3] == Run(3, 1, 1)
    for d in CASES.values():
        cfg = from_config(d)
        assert [(r.layer) for r in cfg.runs()] == [i for i, _ in O.run_order(d)]
    assert from_config(CASES["no_loop"]).loop is None


def test_config_reads_every_size_and_constant():
    d = model([attention(heads=6, kv_heads=2, dim=10, vdim=14, rot=6, base=77.0, scale=0.3, ff=5),
               delta(heads=3, kv_heads=1, dim=12, vdim=9, conv=5, ff=0)], width=18, vocab=11,
              loop=(0, 1, 4), mult=0.25, eps=3e-4, eos_token_id=[3, 4])
    c = from_config(d)
    a, b = c.layers[0].mixer, c.layers[1].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.rot.dims, a.rot.base) == \
        (6, 2, 10, 14, 0.3, 6, 77.0)
    assert a.sink and a.gated and a.qk_norm
    assert (b.heads, b.kv_heads, b.dim, b.vdim, b.taps) == (3, 1, 12, 9, 5)
    assert c.layers[0].mlp.ff == 5 and c.layers[1].mlp is None
    assert (c.eps, c.residual_mult, c.norm_offset, c.hidden_size, c.vocab_size) == \
        (3e-4, 0.25, 1.0, 18, 11)
    assert (c.loop.start, c.loop.stop, c.loop.times) == (0, 1, 4) and c.eos_token_id == [3, 4]
    assert c.width_padded == 24


@pytest.mark.parametrize("bad", [
    {"architecture": "Other"}, model([]), model([attention()], loop=(1, 1, 2)),
    model([attention()], loop=(0, 2, 2)), model([attention()], loop=(0, 1, 0)),
    model([{**attention(), "type": "conv"}]),
    model([{**attention(), "mlp": {"kind": "experts", "ff": 8}}])])
def test_bad_configs_are_refused(bad):
    with pytest.raises(ValueError):
        from_config(bad)


def test_bad_shapes_are_refused():
    for kw in (dict(heads=3, kv_heads=2, dim=8, vdim=8), dict(heads=2, kv_heads=1, dim=300, vdim=8),
               dict(heads=2, kv_heads=1, dim=8, vdim=0)):
        with pytest.raises(ValueError):
            AttnShape(**kw)
        with pytest.raises(ValueError):
            DeltaShape(**kw, taps=4)
    with pytest.raises(ValueError):
        DeltaShape(2, 1, 8, 8, 0)


# ---------------------------------------------------------------------------- weights
@pytest.mark.parametrize("name", list(CASES))
def test_weight_layout(name):
    """x through the two packed matrices equals x through the named tensors."""
    cfg, get, w = weights_of(CASES[name])
    f64 = torch.float64
    for i, L in enumerate(cfg.layers):
        lw = LayerWeights.load(get, i, cfg, "cpu", torch.float32)
        m = L.mixer
        names = ["q", "k", "v", "g"] + (["a", "b"] if m.kind == "delta" else [])
        h = torch.zeros(cfg.width_padded)
        h[:cfg.hidden_size] = torch.randn(cfg.hidden_size)
        want = [w[f"l{i}.mix.{n}"].float() @ h[:cfg.hidden_size] for n in names]
        got = lw.w_in @ h
        torch.testing.assert_close(got[:lw.n_raw], torch.cat(want), atol=1e-4, rtol=1e-4)
        assert lw.n_raw == lw.n_main + lw.n_ab and lw.n_ab == (2 * m.heads if len(names) > 4 else 0)
        ao, af = torch.randn(m.heads * m.vdim), torch.randn(lw.ff)
        a = torch.zeros(lw.out_cols)
        a[:len(ao)] = ao
        a[lw.mix_cols:lw.mix_cols + lw.ff] = af
        y = w[f"l{i}.mix.o"].to(f64) @ ao.to(f64)
        if lw.ff:
            y += w[f"l{i}.mlp.down"].to(f64) @ af.to(f64)
            torch.testing.assert_close(got[lw.n_raw:], w[f"l{i}.mlp.up"].float() @
                                       h[:cfg.hidden_size], atol=1e-4, rtol=1e-4)
        torch.testing.assert_close((lw.w_out @ a).to(f64), y, atol=1e-4, rtol=1e-4)
        assert lw.mix_cols % 8 == 0 and lw.out_cols % 8 == 0
        if m.kind == "delta":
            cat = torch.cat([w[f"l{i}.mix.{n}.conv"].float() for n in "qkv"])
            assert torch.equal(lw.consts["conv"].t(), cat)
    mw = ModelWeights.load(get, cfg, "cpu", torch.float32)
    assert mw.embed.shape == (cfg.vocab_size, cfg.width_padded)
    assert not mw.embed[:, cfg.hidden_size:].any() and not mw.lm_head[:, cfg.hidden_size:].any()
    assert (mw.loop_in is None) == (cfg.loop is None)


def test_wrong_tensor_shape_is_refused():
    cfg, get, w = weights_of(CASES["mixed"])
    with pytest.raises(ValueError, match="l0.mix.k"):
        LayerWeights.load(lambda n: w[n][:-1] if n == "l0.mix.k" else w[n], 0, cfg, "cpu",
                          torch.float32)


def test_random_tensors_do_not_depend_on_order():
    cfg, get, w = weights_of(CASES["mixed"])
    for n in reversed(list(tensor_shapes(cfg))):
        assert torch.equal(get(n), w[n])


# ---------------------------------------------------------------------------- registry, roles
def _write(tmp_path, d):
    (tmp_path / "config.json").write_text(json.dumps(d))
    return tmp_path


def test_registry_follows_config(tmp_path):
    assert family_of(_write(tmp_path, CASES["mixed"])) is HYBRID
    assert family_of(_write(tmp_path, {"hidden_size": 8, "model_type": "llama"})) is LLAMA
    with pytest.raises(ValueError, match="Nothing"):
        family_of(_write(tmp_path, {"architecture": "Nothing"}))


def test_placement_is_refused_for_looped_designs(tmp_path):
    _write(tmp_path, CASES["mixed"])

    def ctx(mode="master", transport="tcp", nodes=()):
        return SimpleNamespace(model_path=tmp_path, mode=mode, topology=SimpleNamespace(nodes=nodes),
                               args=SimpleNamespace(transport=transport))
    check_placement(ctx())
    for bad in (ctx(mode="worker"), ctx(transport="rccl"), ctx(transport="loopback"),
                ctx(nodes=("w1",))):
        with pytest.raises(ValueError, match="one GPU"):
            check_placement(bad)
    _write(tmp_path, {"hidden_size": 8})
    check_placement(ctx(mode="worker"))


def test_model_refuses_the_cpu():
    from cake_amd.models.hybrid.model import HybridModel
    cfg, get, _ = weights_of(CASES["no_loop"])
    with pytest.raises(ValueError, match="GPU"):
        HybridModel.build(cfg, get, "cpu", torch.float32, 64)


# ---------------------------------------------------------------------------- state, rows
def test_state_pool_slots():
    cfg = from_config(CASES["mixed"])
    p = StatePool(cfg, "cpu", torch.float32, 2, 100)
    assert p.S == 128 and len(p.bufs) == len(cfg.runs())
    a, b = p.open(), p.open()
    assert {a, b} == {0, 1} and p.reserve(a, 60) == 0 and p.reserve(a, 40) == 60
    with pytest.raises(ValueError):
        p.reserve(a, 1)
    p.bufs[1][0][b].fill_(3.0)
    old = p.bufs[1][0]
    c = p.open()  # grows: contents move with their slots, the old buffers stay alive
    assert c == 2 and p.slots == 4 and p.version == 1 and p.bufs[1][0] is not old
    assert bool((p.bufs[1][0][b] == 3.0).all()) and p._old[0][1][0] is old
    p.close(a)
    assert p.open() == a and p.length[a] == 0
    assert len(p.recurrent(b)) == 2 * sum(L.mixer.kind == "delta" for L in
                                          [cfg.layers[r.layer] for r in cfg.runs()])


def test_rows_pack():
    r = Rows.pack([(3, 0, [5, 6, 7]), (1, 10, [9])], "cpu")
    assert (r.N, r.B, r.max_len) == (4, 2, 3)
    assert r.tok.tolist() == [5, 6, 7, 9] and r.pos.tolist() == [0, 1, 2, 10]
    assert r.slot.tolist() == [3, 3, 3, 1] and r.first.tolist() == [0, 0, 0, 3]
    assert r.seq.tolist() == [[0, 3, 0, 3], [3, 1, 10, 1]]
    r = Rows.pack([(0, 0, [1] * 33), (1, 0, [1] * 16), (2, 5, [1])], "cpu")
    assert r.chunk.tolist() == [[0, 16], [16, 16], [32, 1], [33, 16], [49, 1]]
    assert r.chunk0.tolist() == [0, 3, 4]
    assert all(t.data_ptr() % 16 == 0 for t in (r.seq, r.chunk))
    with pytest.raises(ValueError):
        Rows.pack([(0, 0, [])], "cpu")


# ---------------------------------------------------------------------------- steps and replay
def test_replay_names_sequences_and_returns_their_slots():
    from cake_amd.trace_run import Replay
    calls = []

    class Fake:
        free = [0, 1, 2]

        def open_sequence(self):
            return self.free.pop(0)

        def close_sequence(self, s):
            self.free.insert(0, s)

        def step(self, batch):
            calls.append([(e.seq, e.tokens, e.want) for e in batch])
            return [torch.full((len(e.want), 2), float(e.seq)) for e in batch]
    r = Replay(Fake())
    out = r.step([{"id": "x", "tokens": [1, 2], "want": [1]}, {"id": "y", "tokens": [3], "want": []}],
                 ["y"])
    assert out.tolist() == [[0.0, 0.0]] and calls[0] == [(0, [1, 2], [1]), (1, [3], [])]
    assert r.step([{"id": "z", "tokens": [4], "want": []}], ["x", "z"]) is None
    assert calls[1][0][0] == 1 and r.seqs == {}


def test_llama_model_steps_like_its_forward():
    """The same step interface on the Llama family: interleaved sequences against each alone."""
    from cake_amd.models.llama3.config import preset
    from cake_amd.models.llama3.factory import random_model
    m = random_model(preset("tiny"), "cpu", torch.float32, max_seq=64, backend="torch")
    a, b = tokens(9, 512, 1), tokens(5, 512, 2)
    ref = []
    for t in (a, b):
        m.reset()
        ref.append(m.forward(t, 0))
    sa, sb = m.open_sequence(), m.open_sequence()
    m.step([StepEntry(sa, a[:7], []), StepEntry(sb, b[:3], [0])])
    ya, yb = m.step([StepEntry(sa, a[7:], [1]), StepEntry(sb, b[3:], [1])])
    torch.testing.assert_close(ya[0], ref[0], atol=1e-4, rtol=1e-4)
    torch.testing.assert_close(yb[0], ref[1], atol=1e-4, rtol=1e-4)
    m.close_sequence(sa)
    assert m.open_sequence() == sa


# ---------------------------------------------------------------------------- the reference
def test_reference_delta_rule_is_the_closed_form():
    """With decay 1 and orthonormal keys the rule stores v exactly (beta 1)."""
    d, e, T = 8, 5, 8
    k = torch.linalg.qr(torch.randn(d, d, dtype=torch.float64))[0][:, None]
    v = torch.randn(T, 1, e, dtype=torch.float64)
    one = torch.ones(T, 1, dtype=torch.float64)
    out = O.delta_rule(k, k, v, one, one, 1, 1)
    torch.testing.assert_close(out, v)
    # a second write under the same key replaces the first
    k2, v2 = torch.cat([k, k[:1]]), torch.cat([v, 9 * v[:1]])
    one = torch.ones(T + 1, 1, dtype=torch.float64)
    torch.testing.assert_close(O.delta_rule(k2, k2, v2, one, one, 1, 1)[-1], 9 * v[0])


def test_reference_sink_and_rotation():
    T, d = 6, 8
    q = torch.zeros(T, 1, d, dtype=torch.float64)
    v = torch.ones(T, 1, 3, dtype=torch.float64)
    out = O.attend_with_sink(q, q, v, 1.0, 1, 1)  # equal scores 0: i + 1 keys and the sink
    want = torch.tensor([(i + 1) / (i + 2) for i in range(T)], dtype=torch.float64)
    torch.testing.assert_close(out[:, 0, 0], want)
    x = torch.randn(T, 2, d, dtype=torch.float64)
    r = O.rotate_pairs(x, 4, 100.0)
    z = torch.view_as_complex(x[..., :4].reshape(T, 2, 2, 2).contiguous())
    f = torch.tensor([1.0, 0.1], dtype=torch.float64)
    ang = torch.arange(T, dtype=torch.float64)[:, None, None] * f
    want = torch.view_as_real(z * torch.exp(1j * ang)).reshape(T, 2, 4)
    torch.testing.assert_close(r[..., :4], want)
    assert torch.equal(r[..., 4:], x[..., 4:])


def test_reference_gelu_and_conv():
    x = torch.linspace(-4, 4, 33, dtype=torch.float64)
    torch.testing.assert_close(O.gelu_exact(x), torch.nn.functional.gelu(x))
    T, C, taps = 7, 3, 4
    x, w = torch.randn(T, C, dtype=torch.float64), torch.randn(C, taps, dtype=torch.float64)
    y = torch.nn.functional.conv1d(torch.nn.functional.pad(x.t()[None], (taps - 1, 0)),
                                   w[:, None], groups=C)[0].t()
    torch.testing.assert_close(O.short_conv_silu(x, w), torch.nn.functional.silu(y))
    assert math.isclose(float(O.softplus(torch.tensor(0.0))), math.log(2.0), rel_tol=1e-6)
