"""Hybrid designs on the GPU against the plain reference (hybrid_oracle.py): each mechanism
alone, whole models, portions of prompts, ragged batches, slots used again, key distances at
every tile and split border, long decoding, and generation through the master."""
import json

import hybrid_oracle as O
import pytest
import torch
from hybrid_cases import CASES, attention, delta, model, rel_rms, tokens, weights_of

pytestmark = pytest.mark.gpu

F64 = torch.float64
DTYPES = [torch.float32, torch.bfloat16, torch.float16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 2e-2, torch.float16: 4e-3}
LOGIT_TOL = {torch.float32: 5e-5, torch.bfloat16: 6e-2, torch.float16: 1e-2}


def _rand(*shape, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g) * scale


# ---------------------------------------------------------------------------- row kernels
@pytest.mark.parametrize("dt", DTYPES, ids=str)
@pytest.mark.parametrize("W", [8, 61, 256, 1000, 9000])
def test_norm_rows(cuda, dt, W):
    from cake_amd.ops import mixers as M
    Wp = M.pad_to(W, 8)
    x = torch.zeros(5, Wp)
    x[:, :W] = _rand(5, W, scale=3.0)
    w = torch.zeros(Wp)
    w[:W] = _rand(W, seed=1, scale=0.2)
    want = O.norm_around_one(x[:, :W].to(F64), w[:W].to(F64), 1e-5)
    for rows in (None, [3, 0, 4]):
        r = None if rows is None else torch.tensor(rows, dtype=torch.int32, device=cuda)
        out = torch.full((5 if rows is None else 3, Wp), 7.0, device=cuda, dtype=dt)
        M.norm(x.to(cuda), w.to(cuda), 1.0, 1e-5, W, out, rows=r)
        got = out.cpu()
        assert rel_rms(got[:, :W], want if rows is None else want[rows]) < TOL[dt]
        assert not got[:, W:].any()


@pytest.mark.parametrize("dt", DTYPES, ids=str)
@pytest.mark.parametrize("W", [24, 61])
def test_embed_and_loop_rows(cuda, dt, W):
    from cake_amd.ops import mixers as M
    Wp = M.pad_to(W, 8)
    table = torch.zeros(11, Wp)
    table[:, :W] = _rand(11, W)
    table = table.to(dt)
    tok = torch.tensor([4, 0, 10], dtype=torch.int32)
    x, x0 = (torch.empty(3, Wp, device=cuda) for _ in range(2))
    M.embed(table.to(cuda), tok.to(cuda), x, x0)
    assert torch.equal(x.cpu(), table[tok.long()].float()) and torch.equal(x, x0)
    step = _rand(W, seed=2)
    y = torch.empty(3, Wp, device=cuda)
    a = torch.empty(3, M.pad_to(2 * W, 8), device=cuda, dtype=dt)
    M.loop_rows(x * 2, x0, step.to(cuda), W, a, y)
    e = table[tok.long()].float()[:, :W]
    assert torch.equal(a.cpu()[:, :2 * W], torch.cat([2 * e, e], 1).to(dt))
    assert not a.cpu()[:, 2 * W:].any()
    assert torch.equal(y.cpu()[:, :W], step.expand(3, W)) and not y.cpu()[:, W:].any()


@pytest.mark.parametrize("dt", DTYPES[1:], ids=str)
@pytest.mark.parametrize("W,n_raw,ff", [(61, 37, 51), (256, 130, 0), (2048, 9, 300),
                                        (4096, 300, 77), (5000, 64, 64), (9216, 40, 8)])
def test_decode_projections(cuda, dt, W, n_raw, ff):
    """layer_in (norm + projections + GELU), layer_out (scaled residual), loop_in."""
    from cake_amd.ops import mixers as M
    Wp = M.pad_to(W, 8)

    def mat(n, k, kp, seed):
        t = torch.zeros(n, kp)
        t[:, :k] = _rand(n, k, seed=seed, scale=k ** -0.5)
        return t.to(dt)
    x, nw = torch.zeros(Wp), torch.zeros(Wp)
    x[:W] = _rand(W, scale=2.0)
    nw[:W] = _rand(W, seed=1, scale=0.2)
    nw = nw.to(dt)
    w_in = mat(n_raw + ff, W, Wp, 2)
    out = torch.empty(n_raw, device=cuda)
    act = torch.empty(max(ff, 1), device=cuda, dtype=dt)
    M.layer_in(x.to(cuda), nw.to(cuda), 1e-5, 1.0, W, w_in.to(cuda), n_raw, out, act[:ff])
    h = w_in.to(F64) @ torch.nn.functional.pad(
        O.norm_around_one(x[:W].to(F64), nw[:W].to(F64), 1e-5), (0, Wp - W))
    assert rel_rms(out[None], h[None, :n_raw]) < 1e-5
    if ff:
        assert rel_rms(act[None, :ff], O.gelu_exact(h[n_raw:])[None]) < TOL[dt]
    K = M.pad_to(n_raw, 8) + M.pad_to(ff, 8)
    a = _rand(K, seed=4).to(dt)
    w_out = mat(W, K, K, 5)
    y = torch.empty(Wp, device=cuda)
    M.layer_out(a.to(cuda), w_out.to(cuda), 0.37, x.to(cuda), y)
    want = x[:W].to(F64) + 0.37 * (w_out.to(F64) @ a.to(F64))
    assert rel_rms(y[None, :W], want[None]) < 1e-5
    x2 = x.to(cuda)
    M.layer_out(a.to(cuda), w_out.to(cuda), 0.37, x2, x2)  # in place
    assert torch.equal(x2[:W], y[:W])
    w_l = mat(W, 2 * W, M.pad_to(2 * W, 8), 6)
    x0, step = torch.zeros(Wp), _rand(W, seed=8)
    x0[:W] = _rand(W, seed=7)
    M.loop_in(x.to(cuda), x0.to(cuda), step.to(cuda), w_l.to(cuda), W, y)
    want = O.enter_pass(x[None, :W].to(F64), x0[None, :W].to(F64),
                        {"loop.in": w_l[:, :2 * W].to(F64), "loop.step": step[None].to(F64)}, 0)
    assert rel_rms(y[None, :W], want) < 1e-5


@pytest.mark.parametrize("alpha", [1.0, -0.3])
@pytest.mark.parametrize("M_,N,K", [(3, 61, 64), (70, 130, 104), (300, 512, 1024)])
def test_gemm_alpha(cuda, alpha, M_, N, K):
    """The scaled f32 epilogues of the shared GEMM, split-K included."""
    from cake_amd.ops import gemm as G
    x, w, r = _rand(M_, K).bfloat16(), _rand(N, K, seed=1).bfloat16(), _rand(M_, N, seed=2)
    want = x.to(F64) @ w.to(F64).t()
    for splits in (1, 4):
        y = r.to(cuda)
        G.linear(x.to(cuda), w.to(cuda), epi="resid32", resid=y, alpha=alpha, splits=splits)
        assert rel_rms(y, r.to(F64) + alpha * want) < 1e-5
        G.linear(x.to(cuda), w.to(cuda), epi="store32", resid=y, alpha=alpha, splits=splits)
        assert rel_rms(y, alpha * want) < 1e-5
    with pytest.raises(ValueError):
        G.linear(x.to(cuda), w.to(cuda), alpha=2.0)


# ---------------------------------------------------------------------------- attention
# heads, kv_heads, dim, vdim, rotated dims
ATTN = [(4, 2, 64, 56, 24), (2, 2, 20, 20, 0), (3, 1, 66, 30, 66), (8, 2, 128, 128, 64),
        (20, 1, 64, 64, 64), (2, 1, 200, 72, 10), (2, 1, 40, 256, 40)]


class AttnBench:
    """One attention layer's kernels over a cache of `slots` x S."""

    def __init__(self, dev, shape, dt, S=512, slots=3, base=50.0, eps=1e-5):
        from cake_amd.ops import mixers as M
        self.M, self.dev, self.dt, self.eps = M, dev, dt, eps
        H, G, d, e, rd = shape
        self.sh = M.AttnShape(H, G, d, e, rd // 2)
        n = rd // 2
        ang = torch.arange(S, dtype=F64)[:, None] * base ** (-2 * torch.arange(n, dtype=F64) /
                                                             max(rd, 1))
        self.cs = torch.stack([ang.cos(), ang.sin()], -1).reshape(S, 2 * n).float().to(dev)
        if n == 0:
            self.cs = torch.zeros(2, device=dev)
        self.base, self.rd = base, rd
        self.kc = torch.zeros(slots, G, S, self.sh.DP, device=dev, dtype=dt)
        self.vc = torch.zeros(slots, G, self.sh.DVP, S, device=dev, dtype=dt)

    def project(self, T, seed=0):
        """[T, q|k|v|gate] random rows in the storage type (CPU)."""
        return _rand(T, self.sh.qkv_cols + self.sh.out_cols, seed=seed).to(self.dt)

    def prompt(self, seqs, scale, sink=True, gated=True):
        """seqs: [(slot, pos0, rows)] -> [rows, H e] per sequence."""
        M, sh = self.M, self.sh
        rows = M.Rows.pack([(s, p0, [0] * r.shape[0]) for s, p0, r in seqs], self.dev)
        proj = torch.cat([r for _, _, r in seqs]).to(self.dev)
        qn = torch.empty(rows.N, sh.heads, sh.DP, device=self.dev, dtype=self.dt)
        out = torch.empty(rows.N, sh.out_cols, device=self.dev, dtype=self.dt)
        M.attn_prep(sh, proj, rows, self.cs, True, self.eps, qn, self.kc, self.vc)
        M.attn_prompt(sh, qn, self.kc, self.vc, rows, proj[:, sh.qkv_cols:] if gated else None,
                      out, scale, sink)
        return list(out.cpu().split([r.shape[0] for _, _, r in seqs]))

    def decode(self, seqs, scale, nsplit, sink=True, gated=True):
        """seqs: [(slot, pos, row)] -> [B, H e]."""
        M, sh, B = self.M, self.sh, len(seqs)
        i32 = dict(dtype=torch.int32, device=self.dev)
        out = torch.empty(B, sh.out_cols, device=self.dev, dtype=self.dt)
        part = torch.zeros(sh.part_floats(B, nsplit), device=self.dev)
        tick = torch.zeros(B * sh.tiles, **i32)
        for _ in range(2):  # a second launch: the tickets were re-armed, the append repeats
            M.attn_decode(sh, torch.stack([r for _, _, r in seqs]).float().to(self.dev),
                          torch.tensor([p for _, p, _ in seqs], **i32),
                          torch.tensor([s for s, _, _ in seqs], **i32), self.cs, True, sink,
                          gated, self.eps, scale, self.kc, self.vc, out, nsplit, part, tick)
        assert not tick.any()
        return out.cpu()

    def reference(self, rows, scale, sink=True, gated=True):
        H, G, d, e = self.sh.heads, self.sh.kv_heads, self.sh.dim, self.sh.vdim
        T, x = rows.shape[0], rows.to(F64)
        q, k, v, g = x.split([H * d, G * d, G * e, H * e], 1)
        rot = [O.rms(O.rotate_pairs(t.reshape(T, n, d), self.rd, self.base), self.eps)
               for t, n in ((q, H), (k, G))]
        v = v.reshape(T, G, e)
        if sink:
            o = O.attend_with_sink(*rot, v, scale, H, G)
        else:  # a sink-free softmax through a value column of ones
            one = torch.ones(T, G, 1, dtype=F64)
            o = O.attend_with_sink(*rot, torch.cat([v, one], -1), scale, H, G)
            o = o[..., :-1] / o[..., -1:]
        o = o.reshape(T, H * e)
        return o * torch.sigmoid(g) if gated else o


@pytest.mark.parametrize("dt", DTYPES, ids=str)
@pytest.mark.parametrize("shape", ATTN, ids=str)
def test_attention_prompt(cuda, shape, dt):
    """Ragged prompts around the tile sizes, in one launch; every variant of the mechanism."""
    b = AttnBench(cuda, shape, dt, slots=8)
    scale = 3.0 / shape[2] ** 0.5
    lens = [1, 33, 64, 65, 127, 129, 200]
    seqs = [(7 - i, 0, b.project(n, seed=i)) for i, n in enumerate(lens)]
    for sink, gated in ((True, True), (False, True), (True, False)):
        for (_, _, r), got in zip(seqs, b.prompt(seqs, scale, sink, gated)):
            assert rel_rms(got, b.reference(r, scale, sink, gated)) < TOL[dt], (sink, gated, len(r))
    got = b.prompt(seqs[3:5], -scale)  # a negative scale turns the order of the scores round
    assert rel_rms(got[0], b.reference(seqs[3][2], -scale)) < TOL[dt]


@pytest.mark.parametrize("dt", DTYPES, ids=str)
@pytest.mark.parametrize("shape", ATTN, ids=str)
def test_attention_decode(cuda, shape, dt):
    """Token after token at positions around the block and split borders, as a batch."""
    b = AttnBench(cuda, shape, dt, slots=10)
    scale = 3.0 / shape[2] ** 0.5
    at = [0, 1, 31, 32, 33, 127, 128, 129, 256, 300]
    rows = [b.project(p + 1, seed=p) for p in at]
    for i, r in enumerate(rows):
        if at[i]:
            b.prompt([(i, 0, r[:-1])], scale)
    for nsplit in (1, 3, 16):
        for sink, gated in ((True, True), (False, False)):
            got = b.decode([(i, p, rows[i][-1]) for i, p in enumerate(at)], scale, nsplit, sink,
                           gated)
            for i in range(len(at)):
                want = b.reference(rows[i], scale, sink, gated)[-1:]
                assert rel_rms(got[i:i + 1], want) < TOL[dt], (nsplit, at[i])


@pytest.mark.parametrize("dt", DTYPES[:2], ids=str)
def test_one_standing_out_key(cuda, dt):
    """A query that matches exactly one key — first, last, on either side of every block and
    split border, and the query's own — returns that key's value; without it, the sink takes
    nearly everything."""
    H, G, d, e = 2, 1, 64, 32
    b = AttnBench(cuda, (H, G, d, e, 0), dt, S=768)
    T, scale = 641, 0.5  # a match scores 32, an orthogonal or opposite key 0 or less
    keys = [0, 1, 15, 16, 31, 32, 63, 64, 65, 127, 128, 255, 256, 257, 511, 512, 639, 640]
    rows = torch.zeros(T, b.sh.qkv_cols + b.sh.out_cols)
    rows[:, H * d] = 1.0                                # every key along axis 0 ...
    for i, j in enumerate(keys):
        rows[j, H * d:H * d + d] = torch.eye(d)[i + 1]  # ... the listed ones on axes of their own
    rows[:, (H + G) * d:(H + G) * d + e] = _rand(T, e)  # values
    rows[:, b.sh.qkv_cols:] = 30.0                      # gates open
    v = rows[:, (H + G) * d:(H + G) * d + e].to(dt).float()

    def ask(head_axes):
        q = torch.zeros(H * d)
        for h, (axis, sign) in enumerate(head_axes):
            q[h * d + axis] = sign
        r = rows.clone()
        r[-1, :H * d] = q
        return r.to(dt)
    tol = dict(atol=2e-2 if dt != torch.float32 else 1e-5, rtol=1e-2)
    for i, j in enumerate(keys):
        r = ask([(i + 1, 1.0), (0, -1.0)])  # head 0: key j; head 1: opposite to most keys
        got = [b.prompt([(0, 0, r)], scale)[0][-1].float()]
        got += [b.decode([(0, T - 1, r[-1])], scale, n)[0].float() for n in (1, 5, 32)]
        for y in got:
            torch.testing.assert_close(y[:e], v[j], **tol)
            # keys of axis 0 score -32, the listed ones 0 like the sink: a plain mean
            torch.testing.assert_close(y[e:], v[keys].sum(0) / (len(keys) + 1), **tol)


def test_attention_portions_and_used_slots(cuda):
    """A prompt cut into portions (two tokens up) on slots that held something longer."""
    dt = torch.float32
    b = AttnBench(cuda, (4, 2, 48, 40, 16), dt)
    b.prompt([(s, 0, b.project(400, seed=9 + s)) for s in range(3)], 0.4)
    r = b.project(333, seed=1)
    want = b.reference(r, 0.4)
    for cuts in ([2, 4, 66, 67, 195, 331], [64, 128, 256], [1, 130]):
        got, at = [], 0
        for c in cuts + [333]:
            got += b.prompt([(2, at, r[at:c])], 0.4)
            at = c
        assert rel_rms(torch.cat(got), want) < TOL[dt]


# ---------------------------------------------------------------------------- delta rule
# heads, kv_heads, dim, vdim, taps
DELTA = [(2, 2, 40, 40, 4), (4, 2, 24, 40, 3), (3, 1, 20, 12, 1), (2, 1, 128, 128, 4),
         (2, 2, 200, 72, 2), (1, 1, 64, 250, 7), (2, 1, 256, 256, 4)]


class DeltaBench:
    def __init__(self, dev, shape, dt, slots=4, eps=1e-5, seed=0):
        from cake_amd.ops import mixers as M
        self.M, self.dev, self.dt, self.eps = M, dev, dt, eps
        H, G, d, e, taps = shape
        sh = self.sh = M.DeltaShape(H, G, d, e, taps)
        self.w = {".A_log": torch.linspace(-4.0, 2.0, H), ".dt_bias": _rand(H, seed=seed + 1),
                  ".norm": 1 + _rand(e, seed=seed + 2, scale=0.2)}
        self.conv = _rand(sh.channels, taps, seed=seed + 3, scale=taps ** -0.5)
        self.state = torch.full((slots, H, d, sh.EP), 5.0, device=dev)   # as if used before
        self.ring = torch.full((slots, taps, sh.channels), -3.0, device=dev)
        self.const = [self.conv.t().contiguous().to(dev)] + \
            [self.w[k].to(dev) for k in (".A_log", ".dt_bias", ".norm")]

    def project(self, T, seed=0):
        """([T, q|k|v|gate] storage type, [T, a|b] f32), CPU."""
        return (_rand(T, self.sh.channels + self.sh.out_cols, seed=seed).to(self.dt),
                _rand(T, 2 * self.sh.heads, seed=seed + 50))

    def prompt(self, seqs):
        M, sh = self.M, self.sh
        rows = M.Rows.pack([(s, p0, [0] * x.shape[0]) for s, p0, x, _ in seqs], self.dev)
        out = torch.empty(rows.N, sh.out_cols, device=self.dev, dtype=self.dt)
        M.delta_prompt(sh, torch.cat([s[2] for s in seqs]).to(self.dev),
                       torch.cat([s[3] for s in seqs]).to(self.dev), rows, self.eps, *self.const,
                       self.state, self.ring, out)
        return list(out.cpu().split([s[2].shape[0] for s in seqs]))

    def decode(self, seqs):
        M, sh = self.M, self.sh
        i32 = dict(dtype=torch.int32, device=self.dev)
        out = torch.empty(len(seqs), sh.out_cols, device=self.dev, dtype=self.dt)
        M.delta_decode(sh, torch.stack([s[2] for s in seqs]).float().to(self.dev),
                       torch.stack([s[3] for s in seqs]).to(self.dev),
                       torch.tensor([s[1] for s in seqs], **i32),
                       torch.tensor([s[0] for s in seqs], **i32), self.eps, *self.const,
                       self.state, self.ring, out)
        return out.cpu()

    def reference(self, x, ab):
        sh, T = self.sh, x.shape[0]
        H, G, d, e = sh.heads, sh.kv_heads, sh.dim, sh.vdim
        x, ab = x.to(F64), ab.to(F64)
        y = O.short_conv_silu(x[:, :sh.channels], self.conv.to(F64))
        q, k, v = y.split([G * d, G * d, H * e], 1)
        q = O.unit(q.reshape(T, G, d)) * d ** -0.5
        k, v = O.unit(k.reshape(T, G, d)), v.reshape(T, H, e)
        w = {n: t.to(F64) for n, t in self.w.items()}
        dec = torch.exp(-torch.exp(w[".A_log"]) * O.softplus(ab[:, :H] + w[".dt_bias"]))
        o = O.delta_rule(q, k, v, torch.sigmoid(ab[:, H:]), dec, H, G)
        z = x[:, sh.channels:].reshape(T, H, e)
        return (O.rms(o, self.eps) * w[".norm"] * z * torch.sigmoid(z)).reshape(T, H * e)


@pytest.mark.parametrize("dt", DTYPES, ids=str)
@pytest.mark.parametrize("shape", DELTA, ids=str)
def test_delta_prompt_and_decode(cuda, shape, dt):
    """Ragged prompts on used slots, then token by token, against the whole sequence."""
    b = DeltaBench(cuda, shape, dt)
    lens, more = [1, 15, 17, 70], 6
    data = [b.project(n + more, seed=i) for i, n in enumerate(lens)]
    want = [b.reference(*d) for d in data]
    got = b.prompt([(3 - i, 0, x[:n], ab[:n]) for i, (n, (x, ab)) in enumerate(zip(lens, data))])
    for g, w, n in zip(got, want, lens):
        assert rel_rms(g, w[:n]) < TOL[dt], n
    for t in range(more):
        y = b.decode([(3 - i, n + t, x[n + t], ab[n + t])
                      for i, (n, (x, ab)) in enumerate(zip(lens, data))])
        for i, (w, n) in enumerate(zip(want, lens)):
            assert rel_rms(y[i:i + 1], w[n + t:n + t + 1]) < TOL[dt], (n, t)


@pytest.mark.parametrize("taps", [1, 2, 4, 6])
def test_delta_portions(cuda, taps):
    """Portions down to one token: the state and the convolution's tail carry over."""
    b = DeltaBench(cuda, (2, 1, 36, 28, taps), torch.float32)
    x, ab = b.project(90)
    want = b.reference(x, ab)
    for cuts in ([2, 4, 5, 21, 53, 88], [1, 2, 3, 4, 5, 6, 7, 8], [16, 32, 64]):
        got, at = [], 0
        for c in cuts + [90]:
            got += b.prompt([(1, at, x[at:c], ab[at:c])])
            at = c
        assert rel_rms(torch.cat(got), want) < TOL[torch.float32]
    y = torch.cat([b.decode([(2, t, x[t], ab[t])]) for t in range(90)])
    assert rel_rms(y, want) < TOL[torch.float32]


def test_delta_long_memory(cuda):
    """Decay near one: what the first token wrote is read back 1500 tokens later."""
    b = DeltaBench(cuda, (1, 1, 64, 32, 1), torch.float32)
    b.w[".A_log"].fill_(-12.0)
    b.const[1].fill_(-12.0)
    b.conv.fill_(1.0)
    b.const[0].fill_(1.0)
    T, d = 1500, 64
    x, ab = b.project(T)
    x[:, d:2 * d] = 0.0
    x[1:, d] = 20.0            # later keys along axis 0
    x[0, d + 5] = 20.0         # the first along axis 5
    x[-1, :d] = 0.0
    x[-1, 5] = 20.0            # the last query asks for it
    ab[:, 1] = 9.0             # step size near one
    got, want = b.prompt([(0, 0, x, ab)])[0], b.reference(x, ab)
    assert rel_rms(got[-1:], want[-1:]) < 1e-4
    b.prompt([(0, 0, x[:700], ab[:700])])
    for t in range(700, T):
        y = b.decode([(0, t, x[t], ab[t])])
    assert rel_rms(y, want[-1:]) < 1e-4


# ---------------------------------------------------------------------------- whole models
def _build(cuda, name_or_dict, dt, max_seq=400, seed=0, slots=2):
    from cake_amd.models.hybrid.model import HybridModel
    d = CASES[name_or_dict] if isinstance(name_or_dict, str) else name_or_dict
    cfg, get, w = weights_of(d, seed)
    return HybridModel.build(cfg, get, cuda, dt, max_seq, slots), d, w


def _feed(m, seq, toks, cuts=()):
    """Logits [len(toks), V] of one sequence fed in the given portions."""
    from cake_amd.models.base import StepEntry
    out, at = [], 0
    for c in [*cuts, len(toks)]:
        out += m.step([StepEntry(seq, toks[at:c], list(range(c - at)))])
        at = c
    return torch.cat(out).cpu()


def _alone(m, toks, cuts=()):
    s = m.open_sequence()
    try:
        return _feed(m, s, toks, cuts)
    finally:
        m.close_sequence(s)


@pytest.mark.parametrize("dt", DTYPES, ids=str)
@pytest.mark.parametrize("name", list(CASES))
def test_model_matches_reference(cuda, name, dt):
    """Residual after every layer run, and the logits: prompt, prompt + decode, token by token."""
    from cake_amd.models.base import StepEntry
    m, d, w = _build(cuda, name, dt)
    toks = tokens(70, d["vocab"])
    layers, seen = [], []
    want = O.forward(d, w, toks, layers_out=layers)
    s = m.open_sequence()
    m.step([StepEntry(s, toks, [])], observe=lambda x: seen.append(x.cpu().clone()))
    m.close_sequence(s)
    assert len(seen) == len(layers) == len(m.runs)
    for got, ref in zip(seen, layers):
        assert rel_rms(got, ref) < LOGIT_TOL[dt]
    for cuts in ((), (40, *range(41, 70)), range(1, 70)):
        assert rel_rms(_alone(m, toks, cuts), want) < LOGIT_TOL[dt], list(cuts)[:2]


@pytest.mark.parametrize("seed", [1, 2])
def test_portions(cuda, seed):
    m, d, w = _build(cuda, "mixed", torch.float32, seed=seed)
    toks = tokens(300, d["vocab"], seed)
    want = O.forward(d, w, toks)
    for cuts in (range(2, 300, 2), range(63, 300, 63), (1, 2, 130, 131, 299), (128, 256)):
        assert rel_rms(_alone(m, toks, cuts), want) < LOGIT_TOL[torch.float32]


@pytest.mark.parametrize("dt", DTYPES[:2], ids=str)
def test_batches_of_unequal_requests(cuda, dt):
    """Prompts together, then decoded together while shorter ones end and their slots go to
    new requests; the pool grows on the way.  Each sequence against the reference."""
    from cake_amd.models.base import StepEntry
    m, d, w = _build(cuda, "mixed", dt)
    reqs = [tokens(n, d["vocab"], n) for n in (1, 2, 65, 130, 40)]
    want = [O.forward(d, w, t + tokens(12, d["vocab"], 7)) for t in reqs]
    full = [t + tokens(12, d["vocab"], 7) for t in reqs]
    steps = [12, 3, 12, 5, 8]  # how many tokens each decodes
    seq = [m.open_sequence() for _ in reqs]
    assert m.pool.version > 0
    got = [[x] for x in m.step([StepEntry(s, t, list(range(len(t)))) for s, t in zip(seq, reqs)])]
    for k in range(12):
        live = [i for i in range(len(reqs)) if k < steps[i]]
        out = m.step([StepEntry(seq[i], [full[i][len(reqs[i]) + k]], [0]) for i in live])
        for i, y in zip(live, out):
            got[i].append(y)
        for i in live:
            if k + 1 == steps[i]:
                m.close_sequence(seq[i])
        if k == 6:  # a new request on a used slot, next to sequences that go on
            y = _alone(m, reqs[2], (60,))
            assert rel_rms(y, want[2][:65]) < LOGIT_TOL[dt]
    for i, t in enumerate(reqs):
        y = torch.cat(got[i])
        assert rel_rms(y, want[i][:len(y)]) < LOGIT_TOL[dt], i
    # mixed: one sequence prefills while another decodes
    a, b = m.open_sequence(), m.open_sequence()
    y0 = m.step([StepEntry(a, full[3][:100], [99])])
    y1 = m.step([StepEntry(a, full[3][100:101], [0]), StepEntry(b, full[4], [len(full[4]) - 1])])
    assert rel_rms(y0[0], want[3][99:100]) < LOGIT_TOL[dt]
    assert rel_rms(y1[0], want[3][100:101]) < LOGIT_TOL[dt]
    assert rel_rms(y1[1], want[4][-1:]) < LOGIT_TOL[dt]


@pytest.mark.parametrize("dt", DTYPES[:2], ids=str)
def test_long_decode(cuda, dt):
    """1300 positions, most of them decoded, over the split-count changes of decode attention."""
    d = model([attention(heads=2, kv_heads=1, dim=32, vdim=32, rot=32, base=1e4), delta()],
              width=64, vocab=67, loop=(0, 2, 2))
    m, d, w = _build(cuda, d, dt, max_seq=1300)
    toks = tokens(1300, d["vocab"])
    a = _alone(m, toks)
    b = _alone(m, toks, range(200, 1300))
    assert rel_rms(b, a.double()) < LOGIT_TOL[dt]
    assert rel_rms(a[:260], O.forward(d, w, toks[:260])) < LOGIT_TOL[dt]


def test_step_refuses_bad_input(cuda):
    from cake_amd.models.base import StepEntry
    m, d, _ = _build(cuda, "no_loop", torch.bfloat16, max_seq=16)
    s = m.open_sequence()
    for bad in ([StepEntry(s, [], [])], [StepEntry(s, [d["vocab"]], [])], [StepEntry(s, [1], [1])],
                [StepEntry(s, [1] * 17, [])], [StepEntry(s, [1], []), StepEntry(s, [2], [])]):
        with pytest.raises(ValueError):
            m.step(bad)
    assert m.pool.length[s] == 0


# ---------------------------------------------------------------------------- generation
GEN = model([attention(ff=96), delta(), attention(heads=2, kv_heads=1), delta(ff=0)], width=96,
            vocab=300, loop=(1, 3, 2), eos_token_id=260)


@pytest.fixture(scope="module")
def checkpoint(tmp_path_factory):
    from cake_amd.utils.synth import write_hybrid_checkpoint
    return write_hybrid_checkpoint(tmp_path_factory.mktemp("hybrid"), GEN, seed=3)


def _master(path, dtype, *flags):
    from cake_amd.cli import build_parser
    from cake_amd.context import Context
    from cake_amd.master import Master
    a = build_parser().parse_args(["--model", str(path), "--topology", "/nonexistent", "--dtype",
                                   dtype, "--max-seq-len", "512", *flags])
    return Master(Context.from_args(a))


def _prompt_ids(llm, text):
    from cake_amd.models.chat import Message
    llm.add_message(Message.user(text))
    return llm.tokenizer.encode(llm.history.encode_dialog_to_prompt(), add_special_tokens=False).ids


@pytest.mark.parametrize("dtype,flags", [("bf16", ()), ("f16", ()), ("bf16", ("--no-graph",)),
                                         ("f32", ())], ids=str)
def test_greedy_generation(cuda, checkpoint, dtype, flags):
    """Master -> generator -> captured decode loop: every token is the reference's choice under
    teacher forcing (repeat penalty included), or within rounding of it."""
    m = _master(checkpoint, dtype, "--temperature", "0", "--repeat-penalty", "1.1",
                "--repeat-last-n", "16", *flags)
    assert m.llm.MODEL_NAME == "fonapel"
    _, _, w = weights_of(GEN, 3)
    tol = 1e-3 if dtype == "f32" else 0.15
    for text in ("one two", "a longer request than the first one"):
        m.reset()
        ids = _prompt_ids(m.llm, text)
        m.llm.history.clear()
        from cake_amd.models.chat import Message
        m.llm.add_message(Message.user(text))
        out = []
        m.llm.stream(40, lambda t: out.append(t.id), stop_at_eos=False)
        assert len(out) == 40
        ref = O.forward(GEN, w, ids + out)
        for i, t in enumerate(out):
            lg = ref[len(ids) + i - 1].clone()
            for p in set((ids + out[:i])[-16:]):
                lg[p] = lg[p] / 1.1 if lg[p] >= 0 else lg[p] * 1.1
            assert float(lg.max() - lg[t]) <= tol * float(ref.std()), (i, t)


def test_generation_stops_and_samples(cuda, checkpoint):
    from cake_amd.models.sampling import SamplingConfig
    m = _master(checkpoint, "bf16", "--temperature", "0")
    got = []
    stats = m.generate_text(got.append, max_tokens=5)
    assert stats["generated"] <= 5
    m.reset()
    m.llm.set_sampling(SamplingConfig(temperature=0.8, top_k=20, seed=5))
    ids = []
    for _ in range(2):
        m.reset()
        out = []
        _prompt_ids(m.llm, "sample")
        m.llm.stream(12, lambda t: out.append(t.id), stop_at_eos=False)
        ids.append(out)
    assert ids[0] == ids[1] and len(ids[0]) == 12


def test_metrics_leave_the_state_alone(cuda, checkpoint):
    """Per-layer timing between two tokens replays layers; the recurrent state comes back."""
    m = _master(checkpoint, "bf16", "--temperature", "0")

    def run(measure):
        m.reset()
        _prompt_ids(m.llm, "timing")
        out = [m.llm.next_token(0).id]
        for i in range(1, 16):
            if measure and i == 8:
                d = m.llm.metrics()
                assert len(d["layer_ms"]) == len(m.llm.model.runs) and d["layers_ms_total"] > 0
            out.append(m.llm.next_token(i).id)
        return out
    assert run(False) == run(True)


def test_rest_api(cuda, checkpoint):
    from fastapi.testclient import TestClient

    from cake_amd.api.server import create_app
    m = _master(checkpoint, "bf16", "--temperature", "0")
    body = {"messages": [{"role": "user", "content": "hello"}], "max_tokens": 6}
    with TestClient(create_app(m)) as c:
        a, b = (c.post("/api/v1/chat/completions", json=body).json() for _ in range(2))
    assert a["model"] == "fonapel" and a["choices"] == b["choices"]
    assert 0 < a["usage"]["completion_tokens"] <= 6


def test_cli_executable(cuda, checkpoint):
    """The cake-cli executable hands the design to the embedded runtime and generates what the
    master does."""
    import os
    import subprocess
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([os.path.join(root, "cake_amd", "lib", "cake-cli"), "--model",
                        str(checkpoint), "--topology", "/nonexistent", "--dtype", "bf16",
                        "--temperature", "0", "--prompt", "hi", "-n", "8", "--max-seq-len", "512"],
                       capture_output=True, timeout=110, cwd=root)
    assert r.returncode == 0, r.stderr.decode(errors="replace")[-2000:]
    m = _master(checkpoint, "bf16", "--temperature", "0", "--prompt", "hi", "-n", "8")
    from cake_amd.models.chat import Message
    m.llm.add_message(Message.system(m.ctx.args.system_prompt))
    m.llm.add_message(Message.user("hi"))
    out = []
    m.generate_text(out.append)
    assert r.stdout.decode(errors="replace").strip("\n") == "".join(out).strip("\n")


def test_graph_survives_pool_growth(cuda, checkpoint):
    """Steps of other sequences between two generations, with the pool moving: the decoder
    captures again and generates the same tokens."""
    m = _master(checkpoint, "bf16", "--temperature", "0")

    def run():
        m.reset()
        out = []
        _prompt_ids(m.llm, "grow")
        m.llm.stream(20, lambda t: out.append(t.id), stop_at_eos=False)
        return out
    first = run()
    model_ = m.llm.model
    seqs = [model_.open_sequence() for _ in range(5)]
    assert model_.pool.version > 0
    assert run() == first
    for s in seqs:
        model_.close_sequence(s)
    assert run() == first


def test_graph_replay_equals_eager(cuda):
    """Captured steps replayed with eager steps of another sequence in between."""
    from cake_amd.models.base import StepEntry
    from cake_amd.models.decoder import DeviceDecoder
    m, d, w = _build(cuda, "mixed", torch.bfloat16)
    prompt = tokens(30, d["vocab"])
    dec = DeviceDecoder(m, repeat_penalty=1.0)
    toks = [dec.start(prompt)]
    dec.capture()
    other = m.open_sequence()
    for k in range(25):
        dec.launch()
        toks.append(int(dec.bufs.tok.item()))
        m.step([StepEntry(other, [k], [0])])
    y = _alone(m, prompt + toks)
    for i, t in enumerate(toks):
        row = y[29 + i]
        assert float(row.max() - row[t]) <= 0.1 * float(row.std())


def test_trace_replay(cuda, checkpoint, tmp_path, monkeypatch, capsys):
    """bin/trace_run's program on a written checkpoint: files, 'done' lines and logits."""
    import io

    from cake_amd import trace_run
    toks = tokens(20, 300)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:18], "want": [3, 17]},
                                     {"id": "b", "tokens": toks[:5], "want": []}], "end": ["b"]},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[18:19], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[19:], "want": [0]}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    rc = trace_run.main(["--model", str(checkpoint), "--dtype", "float32", "--out", str(tmp_path),
                         "--max-tokens", "32"])
    assert rc == 0
    assert [x for x in capsys.readouterr().out.split("\n") if x] == ["done 0", "done 1", "done 2"]
    import numpy as np
    _, _, w = weights_of(GEN, 3)
    want = O.forward(GEN, w, toks)
    got = [torch.from_numpy(np.fromfile(tmp_path / f"{s}.f32", "<f4").reshape(-1, 300).copy())
           for s in (0, 2)]
    assert not (tmp_path / "1.f32").exists()
    assert rel_rms(got[0], want[[3, 17]]) < 5e-5 and rel_rms(got[1], want[[19]]) < 5e-5
