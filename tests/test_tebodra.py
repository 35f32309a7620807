"""Tebodra (attention whose values are its convolved keys, with capped scores; chunked attention with norms over whole
projections, sinks and borrowed keys; an exponentially gated matrix memory; plain gelu feed-forwards under one residual
factor) on the engine against the plain float64 oracle of tests/oracle_tebodra.py: every mechanism alone, whole prompts,
token-by-token decoding, prompt portions down to two tokens, unequal batches, reuse of freed blocks and state slots, keys
far back / at page borders / just inside and outside a chunk with peaked softmax weights, odd sizes, long decoding, greedy
generation through the scheduler, graph replays, and the trace runner's command line.

Each engine test runs on the CPU plumbing path (fp32) and, marked gpu, on the HIP kernels in fp32 and bf16."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

import oracle_tebodra as O
from localai_tfp_amd.engine.engine import EngineConfig, LLMEngine
from localai_tfp_amd.engine.sequence import Request
from localai_tfp_amd.models import tebodra as TE
from localai_tfp_amd.ops import hybrid as HY
from localai_tfp_amd.ops.sampling import SamplingParams
from localai_tfp_amd.tokenizer import ByteTokenizer
from test_vugotar import _FB, close, engine, run_cuts, steps_of, toks

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.param("cuda", marks=pytest.mark.gpu)
DEVS = ["cpu", GPU]
RUNS = [("cpu", "float32", 2e-4), pytest.param("cuda", "float32", 2e-4, marks=pytest.mark.gpu),
        pytest.param("cuda", "bfloat16", 6e-2, marks=pytest.mark.gpu)]
F64 = torch.float64
BANDS = (3.0, 1.0, 5.0, 60.0)  # (factor, low, high, original): kept, blended and divided pairs among these small heads'

SHAPES = {
    # all mixers, a layer that borrows keys under a chunk of its own, both kinds of scaled rotation, a layer without a
    # feed-forward
    "plain": dict(hidden=64, vocab=97, pattern=("attention_2", "mlstm", "attention", "attention_2", "mlstm"), kv_from={3: 0},
                  heads=4, kv_heads=2, dim=16, vdim=24, chunk={0: 24, 3: 11}, rot_dims=12, rot_base=500.0, rot_factor=3.0,
                  t_heads=6, t_kv_heads=3, t_dim=20, t_rot_dims=16, t_rot_base=300.0, t_scaling=BANDS, conv=4, softcap=2.0,
                  m_heads=3, m_dim=12, m_vdim=20, gate_cap=6.0, mlps=("dense", "dense", "dense", None, "dense"), ff=96,
                  residual_mult=0.6),
    # the whole head rotated without scaling, as many key heads as heads, two taps, chunks shorter than a page, memories
    # wider than a lane keeps alone, a feed-forward of odd width, a large eps
    "odd": dict(hidden=40, vocab=61, pattern=("attention", "attention_2", "mlstm"), heads=3, kv_heads=3, dim=24, vdim=8,
                chunk=7, rot_base=300.0, scale=0.4, t_heads=2, t_kv_heads=2, t_dim=12, t_scale=0.7, conv=2, softcap=0.9,
                m_heads=2, m_dim=40, m_vdim=9, gate_cap=15.0, ff=51, residual_mult=1.0, eps=1e-3),
    # one key head for all, no rotation in one kind and a partial one in the other, seven taps, chunks of 33, a memory of 160
    # numbers per column, one memory head, no feed-forward anywhere
    "wide": dict(hidden=48, vocab=53, pattern=("mlstm", "attention", "attention_2", "attention_2"), kv_from={3: 2}, heads=4,
                 kv_heads=1, dim=72, vdim=8, chunk={2: 33, 3: 50}, rot_dims=0, scale=0.2, t_heads=5, t_kv_heads=1, t_dim=40,
                 t_rot_dims=10, t_scaling=(8.0, 0.5, 2.0, 40.0), conv=7, softcap=25.0, m_heads=1, m_dim=160, m_vdim=72,
                 gate_cap=3.0, mlps=(None,), residual_mult=0.4),
    # nothing a multiple of eight, one tap, no cap, chunks of one token, plain causal among the "chunked" ones
    "ragged": dict(hidden=44, vocab=101, pattern=("attention_2", "attention", "attention_2", "mlstm"), heads=5, kv_heads=5,
                   dim=20, vdim=12, chunk={0: 1, 2: 0}, rot_dims=10, rot_factor=7.0, scale=0.3, t_heads=3, t_kv_heads=1,
                   t_dim=14, t_rot_dims=14, conv=1, softcap=0.0, m_heads=5, m_dim=6, m_vdim=10, gate_cap=20.0, ff=30,
                   residual_mult=0.8),
}


def build(device="cpu", dtype="float32", seed=0, **kw):
    cfg = TE.make_config(**kw)
    get = TE.synthetic_source(cfg, seed)
    model = TE.TebodraModel.load(cfg, get, torch.device(device), getattr(torch, dtype))
    return cfg, {k: get(k) for k in get.names}, model


def oracle(cfg, tensors, tokens, layers=None):
    return O.forward(cfg.to_json(), tensors.get, tokens, layers).float()


def greedy(cfg, tensors, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(oracle(cfg, tensors, seq)[-1].argmax()))
    return seq[len(prompt):]


def batches(lens, plan):
    """The ragged steps of several sequences: `plan` lists per step the (sequence, rows) pairs; single tokens after a
    sequence's start are decode rows and come first. Yields (n_dec, chunks, [(sequence, first position, rows)])."""
    at = [0] * len(lens)
    for step in plan:
        seg = [(s, at[s], n) for s, n in step]
        for s, n in step:
            at[s] += n
        dec = [x for x in seg if x[2] == 1 and x[1] > 0]
        pf = [x for x in seg if not (x[2] == 1 and x[1] > 0)]
        yield len(dec), [x[2] for x in pf], dec + pf
    assert at == list(lens)


# ------------------------------------------------------------------------------------------------ mechanisms alone
def test_frequencies_with_and_without_scaling():
    bands = dict(zip(("factor", "low", "high", "original"), BANDS))
    for rot in ({"dims": 32, "base": 10000.0}, {"dims": 24, "base": 700.0, "scaling": {"factor": 5.0}},
                {"dims": 24, "base": 700.0, "scaling": bands}, {"dims": 16, "base": 50.0, "scaling": {"factor": 1.0}},
                {"dims": 64, "base": 5e5, "scaling": dict(factor=8.0, low=1.0, high=4.0, original=8192)},
                {"dims": 8, "base": 1e4, "scaling": dict(factor=3.0, low=0.5, high=32.0, original=100)}):
        close(TE.RotCfg.from_json(rot).table("cpu"), O.frequencies(rot), 1e-6)
        assert TE.RotCfg.from_json(TE.RotCfg.from_json(rot).to_json()) == TE.RotCfg.from_json(rot)
    plain = O.frequencies({"dims": 24, "base": 700.0})
    banded = O.frequencies({"dims": 24, "base": 700.0, "scaling": bands})
    assert banded[0] == plain[0] and banded[-1] == plain[-1] / 3.0  # short waves kept, long ones divided, a blend between
    assert ((banded < plain) & (banded > plain / 3.0)).sum() > 0
    assert TE.RotCfg().table("cpu").numel() == 0


@pytest.mark.parametrize("dev", DEVS)
def test_gelu_unit_and_residual_factor(dev):
    g = torch.Generator().manual_seed(3)
    for F in (33, 700):
        x = torch.randn(5, F + 2, generator=g) * 3
        x[0, 2:6] = torch.tensor([0.0, -30.0, 30.0, -0.5])
        want = O.gelu(x[:, 2:].double())
        for md, tol in ((torch.float32, 1e-6), (torch.bfloat16, 1e-2)):
            out = torch.empty(5, F, device=dev, dtype=md)
            HY.glu(x.to(dev)[:, 2:], None, None, None, out, act="gelu")
            close(out.float(), want, tol)
        # the tanh form differs visibly, so the two are not mixed up
        assert (torch.nn.functional.gelu(x[:, 2:].double(), approximate="tanh") - want).abs().max() > 1e-4
    rw = torch.rand(5, 3, generator=g)
    out = torch.empty(5, 33, device=dev)
    a = torch.randn(5, 33, generator=g)
    HY.glu(a.to(dev), None, None, None, out, scale=rw.to(dev), group=11, act="gelu")
    close(out, O.gelu(a.double()) * rw.double().repeat_interleave(11, 1), 1e-6)
    with pytest.raises(ValueError):
        HY.glu(a.to(dev), a.to(dev), None, None, out, act="gelu")
    eps = 0.3  # a large eps shows whether it sits inside the root
    for C in (40, 1000, 2300, 9000):
        y, x = torch.randn(3, C + 3, generator=g) * 2, torch.randn(3, C, generator=g)
        b, s, w = (torch.randn(C, generator=g) for _ in range(3))
        for bias, scale in ((None, None), (b, s)):
            up = lambda v: None if v is None else v.to(dev)  # noqa: E731
            xd, h32 = x.clone().to(dev), torch.empty(3, C, device=dev)
            HY.scale_add_norm(y.to(dev)[:, 3:], up(bias), up(scale), xd, w.to(dev), eps, h32, offset=1.0, mult=0.37)
            z = y[:, 3:].double() if bias is None else (y[:, 3:].double() + b.double()) * s.double()
            want = x.double() + 0.37 * z
            close(xd, want, 1e-6)
            close(h32, O.offset_norm(want, w, eps), 1e-5)


ROW_CASES = [  # H, G, dk, dv (None: values are keys), rot, taps, norm, half
    (4, 2, 16, None, 12, 4, False, True), (3, 1, 10, None, 10, 2, False, True), (5, 5, 24, None, 0, 7, False, True),
    (2, 1, 8, None, 6, 1, False, False), (3, 3, 12, None, 8, 16, False, False), (4, 2, 16, 24, 16, 0, True, True),
    (6, 3, 20, 8, 6, 0, True, False), (2, 2, 40, None, 8, 3, True, True), (40, 10, 128, None, 128, 4, False, True),
    (72, 8, 128, 64, 64, 0, True, True), (72, 72, 72, None, 2, 3, True, True), (3, 0, 16, None, 8, 4, False, True),
    (40, 0, 64, None, 64, 0, True, True), (7, 7, 9, 5, 2, 5, True, True)]


@pytest.mark.parametrize("dev,dt,tol", RUNS)
@pytest.mark.parametrize("H,G,dk,dv,rot,taps,norm,half", ROW_CASES)
def test_convolution_or_norm_rotation_and_append(dev, dt, tol, H, G, dk, dv, rot, taps, norm, half):
    """The fused step over three sequences in mixed steps (single tokens beside portions of 1 to 30 rows), slots that held
    another sequence's inputs, rows that are not stored, rows wider than the kernel keeps in registers."""
    tol = 1e-2 if dt == "bfloat16" else 1e-5
    md, bs = getattr(torch, dt), 4
    g = torch.Generator().manual_seed(H * 100 + dk)
    lens = (37, 9, 20)
    plan = [[(0, 5), (1, 1)], [(1, 2), (0, 1)], [(0, 1), (2, 17), (1, 1)], [(2, 1), (0, 30), (1, 5)], [(2, 1)], [(2, 1)]]
    own, tied = G > 0, dv is None
    dv = dk if tied else dv
    f = O.frequencies({"dims": rot, "base": 50.0}) if rot else torch.empty(0, dtype=F64)
    eps = 0.2
    n_ch = (H + G) * dk
    cw = torch.randn(n_ch, taps, generator=g) if taps else None
    qw, kw = 1 + 0.3 * torch.randn(H * dk, generator=g), 1 + 0.3 * torch.randn(max(G, 1) * dk, generator=g)
    x = [torch.randn(n, n_ch + (0 if tied else G * dv), generator=g) * 2 for n in lens]

    def expected(s):
        u = x[s][:, :n_ch].double()
        if taps:
            u = O.short_conv(u, cw)
        q, k = u[:, :H * dk], u[:, H * dk:]
        if norm:
            q, k = O.plain_norm(q, qw, eps), O.plain_norm(k, kw, eps) if own else k
        v = k if tied else x[s][:, n_ch:].double()

        def turn(z, n):
            z = z.reshape(-1, n, dk)
            if not rot:
                return z.reshape(len(z), -1)
            if not half:  # the oracle turns (i, i + rot / 2): bring the neighbours there and back
                perm = list(range(0, rot, 2)) + list(range(1, rot, 2)) + list(range(rot, dk))
                back = sorted(range(dk), key=lambda i: perm[i])
                return O.rotate(z[:, :, perm], {"dims": rot, "base": 50.0})[:, :, back].reshape(len(z), -1)
            return O.rotate(z, {"dims": rot, "base": 50.0}).reshape(len(z), -1)
        return turn(q, H), turn(k, G) if own else None, v
    want = [expected(s) for s in range(3)]
    nb = [-(-n // bs) for n in lens]
    order = torch.randperm(sum(nb) + 2, generator=g).tolist()
    tables = [order[sum(nb[:s]):sum(nb[:s + 1])] for s in range(3)]
    kc = torch.full((len(order), bs, max(G, 1) * dk), 7.0, dtype=md, device=dev)
    vc = torch.full((len(order), bs, max(G, 1) * dv), -5.0, dtype=md, device=dev)
    tails = torch.full((4, max(1, taps - 1), n_ch), 3.0, device=dev) if taps else None  # (stale inputs of earlier owners)
    slot_of = [2, 0, 3]
    up = lambda t_: None if t_ is None else t_.to(dev)  # noqa: E731
    conv_w = up(cw.t().contiguous()) if taps else None
    for n_dec, chunks, seg in batches(lens, plan):
        rows = torch.cat([torch.randn(sum(n for _, _, n in seg), 3, generator=g),
                          torch.cat([x[s][a:a + n] for s, a, n in seg])], 1).to(dev)
        pos = [p for _, a, n in seg for p in range(a, a + n)]
        slots = [tables[s][p // bs] * bs + p % bs for s, a, n in seg for p in range(a, a + n)]
        if pos[0] == 35:
            slots[0] = -1
        fb = _FB(n_dec, chunks, pos, [slot_of[s] for s, _, _ in seg], dev, slots)
        T = len(pos)
        qo = torch.empty(T, H * dk + 8, dtype=md, device=dev)[:, :H * dk]
        c1, c2 = 3 + H * dk, 3 + n_ch
        HY.row_rope_append(rows[:, 3:c1], rows[:, c1:c2] if own else None, rows[:, c2:] if own and not tied else None,
                           HY.Ragged(fb), H, G, dk, dv, f.float().to(dev), 1.0, qo, kc if own else None, vc if own else None,
                           up(qw) if norm else None, up(kw) if norm and own else None, eps, conv_w, tails, half=half)
        close(qo.float(), torch.cat([want[s][0][a:a + n] for s, a, n in seg]), tol)
    if taps > 1:  # the newest inputs, for the next step
        for s in range(3):
            w = torch.cat([torch.zeros(taps - 1, n_ch), x[s][:, :n_ch]])[-(taps - 1):]
            assert torch.equal(tails[slot_of[s]].cpu(), w)
        assert (tails[1] == 3.0).all()
    if own:
        for s in range(3):
            at = [(tables[s][p // bs], p % bs) for p in range(lens[s])]
            close(torch.stack([kc[b, o] for b, o in at]).float(), want[s][1], tol)
            close(torch.stack([vc[b, o] for b, o in at]).float(), want[s][2], tol)


@pytest.mark.parametrize("dev", DEVS)
def test_padding_rows_touch_nothing(dev):
    """Rows of a padded batch: no page slot, no state slot."""
    g = torch.Generator().manual_seed(1)
    x = torch.randn(3, 4 * 8, generator=g).to(dev)
    kc, vc = torch.zeros(2, 4, 16, device=dev), torch.zeros(2, 4, 16, device=dev)
    tails = torch.full((2, 3, 32), 5.0, device=dev)
    fb = _FB(3, [], [6, 0, 0], [1, -1, -1], dev, [2, -1, -1])
    q = torch.empty(3, 16, device=dev)
    HY.row_rope_append(x[:, :16], x[:, 16:], None, HY.Ragged(fb), 2, 2, 8, 8, torch.ones(4, device=dev), 1.0, q, kc, vc,
                       conv_w=torch.ones(4, 32, device=dev), tails=tails)
    assert (tails[0] == 5.0).all() and torch.equal(tails[1, 2], x[0]) and (tails[1, :2] == 5.0).all()
    assert int((vc != 0).sum()) == 16 and (q[1:].abs() > 0).any()
    peak, st = torch.full((2, 2), 1.5, device=dev), torch.full((2, 2, 4, 8), 2.0, device=dev)
    z = torch.randn(3, 4, generator=g).to(dev)
    outs = [torch.empty(3, 2, device=dev) for _ in range(4)]
    HY.mlstm_gates(z[:, :2], z[:, 2:], None, None, 4.0, peak, HY.Ragged(fb), *outs[:3])
    HY.state_scan(x[:, :16], x[:, 16:], x[:, :6], outs[0], outs[1], None, st, HY.Ragged(fb), torch.empty(3, 6, device=dev),
                  2, 2, 8, 3, delta=False, norm_out=outs[3])
    assert (peak[0] == 1.5).all() and (peak[1] != 1.5).all() and (st[0] == 2.0).all() and (st[1] != 2.0).any()


def _attn_case(dev, dt, H, G, dk, dv, n, cuts, bs, scale, chunk=0, softcap=0.0, sink=True, gate=1, plant=(), mistake=None):
    """Attention in portions through shuffled pages whose unused slots hold stale numbers. `plant` = [(query, key)]: the query
    becomes a large multiple of the key, so that one score stands out wherever the mask lets it. `gate`: 0 none, 1 per
    number, 2 per head. `mistake` changes the expected values only."""
    g = torch.Generator().manual_seed(11)
    md = getattr(torch, dt)
    q, k, v = torch.randn(n, H, dk, generator=g), torch.randn(n, G, dk, generator=g), torch.randn(n, G, dv, generator=g)
    for qi, kj in plant:
        for h in range(H):
            kk = k[kj, h // (H // G)]
            q[qi, h] = kk * (9.0 / (scale * float((kk * kk).sum())))
    q, k, v = (t_.to(md).double() for t_ in (q, k, v))
    sk = torch.randn(H, generator=g) * 2
    gw = (0, H * dv, H)[gate]
    gt = torch.randn(n, gw + 1, generator=g) * 2
    kw = dict(softcap=softcap or None, chunk=chunk or None, sink=sk.double() if sink else None)
    kw.update(mistake or {})
    want = O.grouped_attention(q, k, v, scale, **kw)
    if gate:
        gg = torch.sigmoid(gt[:, 1:].double()).reshape(n, H, -1)
        want = want * gg
    nb = -(-n // bs)
    table = torch.randperm(nb + 3, generator=g)[:nb].tolist()
    kc = torch.full((nb + 3, bs, G * dk), 7.0, dtype=md, device=dev)
    vc = torch.full((nb + 3, bs, G * dv), -5.0, dtype=md, device=dev)
    for p in range(n):
        kc[table[p // bs], p % bs] = k[p].reshape(-1).to(dev).to(md)
        vc[table[p // bs], p % bs] = v[p].reshape(-1).to(dev).to(md)
    got = torch.empty(n, H * dv + 8, device=dev, dtype=md)
    part = (torch.empty(H * 8, 2, device=dev), torch.empty(H * 8, dv, device=dev))
    qd, gd = q.reshape(n, -1).to(dev).to(md), gt.to(dev)
    for n_dec, chunks, at in steps_of(n, cuts):
        c = 1 if n_dec else chunks[0]
        fb = _FB(n_dec, chunks, list(range(at, at + c)), [0], dev, dec_bt=[table] if n_dec else None,
                 dec_lens=[at + 1] if n_dec else None, pf_bt=None if n_dec else [table], pf_ctx=None if n_dec else [at + c])
        HY.masked_attention(qd[at:at + c], kc, vc, HY.Ragged(fb), H, G, dk, dv, scale, got[at:at + c, 8:], chunk=chunk,
                            sink=sk.to(dev) if sink else False, softcap=softcap, gate=gd[at:at + c, 1:] if gate else None,
                            workspace=part)
    return got[:, 8:].float().reshape(n, H, dv), want


@pytest.mark.parametrize("dev,dt,tol", RUNS)
@pytest.mark.parametrize("H,G,dk,dv", [(4, 2, 24, 40), (8, 2, 64, 128), (4, 4, 96, 96), (3, 1, 128, 64), (6, 3, 128, 128),
                                       (5, 1, 20, 12)])
@pytest.mark.parametrize("gemm_rows", [64, 8])
def test_chunks_caps_sinks_and_gates_on_every_route(dev, dt, tol, H, G, dk, dv, gemm_rows, monkeypatch):
    """Planted keys carry nearly all of a row's weight where the mask lets them: at a chunk's first position and just before
    it, at page borders, far back, the row itself; in portions and in rows decoded alone (split into partitions), on the
    row, matrix-core and library-GEMM routes, with gates per number, per head and none."""
    monkeypatch.setattr(HY, "GEMM_MIN_ROWS", gemm_rows)
    monkeypatch.setattr(HY, "DECODE_WAVES", 16)  # decode rows split into partitions of 64 keys
    tol = 2e-2 if dt == "bfloat16" else 2e-4
    n = 230
    cuts = [97, 2, 60, 3, 40, 20] + [1] * 8
    plant = [(99, 99), (100, 90), (101, 89), (150, 90), (151, 89), (179, 179), (180, 180), (181, 179), (200, 180), (201, 179),
             (222, 180), (223, 179), (224, 0), (225, 224), (226, 15), (227, 16), (228, 63), (229, 64), (60, 0), (61, 60)]
    scale = dk ** -0.5
    for kw in (dict(chunk=90), dict(softcap=5.0, sink=False), dict(chunk=90, softcap=4.0, gate=2), dict(gate=0),
               dict(chunk=16, sink=False, gate=0), dict(softcap=50.0, gate=1)):
        got, want = _attn_case(dev, dt, H, G, dk, dv, n, cuts, 16, scale, plant=plant, **kw)
        close(got, want, tol)


@pytest.mark.parametrize("mistake", [dict(chunk=91), dict(chunk=89), dict(chunk=None), dict(sink=None), dict(softcap=None),
                                     dict(softcap=8.0)])
def test_planted_keys_show_mistakes(mistake):
    """The same planted case, expected with a chunk one token off, without the sink, without the cap: far from the result."""
    plant = [(100, 90), (101, 89), (181, 179), (222, 180), (223, 179)]
    got, want = _attn_case("cpu", "float32", 4, 2, 24, 40, 230, [230], 16, 0.2, 90, 4.0, plant=plant, mistake=mistake)
    assert (got - want).abs().max() > 0.1 * want.abs().max()


def test_a_score_cap_is_positive():
    q = torch.zeros(1, 16)
    with pytest.raises(ValueError):
        HY.masked_attention(q, q.view(1, 1, 16), q.view(1, 1, 16), HY.Ragged(_FB(0, [1], [0], [0], "cpu")), 1, 1, 16, 16, 1.0,
                            q.clone(), softcap=-1.0)


def _memory_inputs(n, H, d, e, kind, g):
    """q (unscaled), k, v and gate pre-activations of one sequence that exercise one end of the recurrence."""
    q, k, v = torch.randn(n, H, d, generator=g), torch.randn(n, H, d, generator=g), torch.randn(n, H, e, generator=g)
    zi, zf = torch.randn(n, H, generator=g) * 3, torch.randn(n, H, generator=g) * 3
    if kind == "bound":  # small keys and input gates: |n . q| below its bound, the division by one
        k, zi = k * 0.01, zi - 6.0
    elif kind == "peaks":  # gates at their caps: the running maximum jumps up and decays slowly or at once
        zi[::17] = 100.0
        zf = torch.where(torch.rand(n, H, generator=g) < 0.1, -100.0, 100.0)
    elif kind == "far":  # nothing forgotten, one early write that the last queries ask for
        zi, zf = zi * 0 - 4.0, zf * 0 + 100.0
        zi[3] = 100.0
        q[-20:] = k[3] * 2.0
    return q, k, v, zi, zf


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("H,d,e", [(3, 12, 20), (2, 32, 64), (2, 64, 15), (1, 100, 16), (2, 160, 33), (1, 256, 8)])
@pytest.mark.parametrize("kind", ["plain", "bound", "peaks", "far"])
def test_matrix_memory(dev, H, d, e, kind):
    """Gates, scan with the normaliser column, division and head norm over three sequences in mixed steps against the plain
    recurrence without a running maximum; slots start with another sequence's state."""
    g = torch.Generator().manual_seed(d + e)
    lens = (340, 9, 70)
    plan = [[(0, 5), (1, 1)], [(1, 2), (0, 1)], [(0, 1), (2, 60), (1, 1)], [(2, 1), (0, 300), (1, 5)], [(0, 2), (2, 8)],
            [(0, 1), (2, 1)]] + [[(0, 1)]] * 30
    cap, eps, bi, bf = 7.0, 0.01, torch.randn(H, generator=g), torch.randn(H, generator=g) + 1.0
    x = [_memory_inputs(n, H, d, e, kind, g) for n in lens]
    gate, w = [torch.randn(n, H * e, generator=g) for n in lens], 1 + 0.2 * torch.randn(H * e, generator=g)
    want = []
    for s, (q, k, v, zi, zf) in enumerate(x):
        i, f = O.mlstm_gates(zi.double() + bi.double(), zf.double() + bf.double(), cap)
        a = (q.double() * d ** -0.5, k.double(), v.double(), i, f)
        o = torch.stack([O.mlstm_plain(a[0][:, h], a[1][:, h], a[2][:, h], i[:, h], f[:, h]) for h in range(H)], 1)
        if s != 0:  # the form with the running maximum is the same function
            o2 = torch.stack([O.mlstm_stabilised(a[0][:, h], a[1][:, h], a[2][:, h], i[:, h], f[:, h]) for h in range(H)], 1)
            close(o2, o, 1e-9)
        o = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps)
        want.append(o.reshape(len(o), -1) * w.double() * torch.sigmoid(gate[s].double()))
    state, peak = torch.full((4, H, e + 1, d), 3.0, device=dev), torch.full((4, H), 50.0, device=dev)
    slot_of = [2, 0, 3]
    up = lambda t_: t_.to(dev)  # noqa: E731
    got = [[] for _ in lens]
    for n_dec, chunks, seg in batches(lens, plan):
        cat = lambda j: torch.cat([x[s][j][a:a + n].reshape(n, -1) for s, a, n in seg])  # noqa: E731
        pos = [p for _, a, n in seg for p in range(a, a + n)]
        T = len(pos)
        y = up(torch.cat([cat(0), cat(1), cat(2), torch.cat([gate[s][a:a + n] for s, a, n in seg]), cat(3), cat(4)], 1))
        cols = np.cumsum([0, H * d, H * d, H * e, H * e, H, H])
        part = [y[:, cols[j]:cols[j + 1]] for j in range(6)]
        rag = HY.Ragged(_FB(n_dec, chunks, pos, [slot_of[s] for s, _, _ in seg], dev))
        decay, coef, floor, nq = (torch.empty(T, H, device=dev) for _ in range(4))
        HY.mlstm_gates(part[4], part[5], up(bi), up(bf), cap, peak, rag, decay, coef, floor)
        o = torch.empty(T, H * e, device=dev)
        HY.state_scan(part[1], part[0], part[2], decay, coef, None, state, rag, o, H, H, d, e, delta=False,
                      q_scale=d ** -0.5, norm_out=nq)
        out = torch.empty(T, H * e, device=dev)
        HY.gated_group_norm(o, part[3], up(w), eps, e, out, gate_first=False, act="sigmoid", den=nq, den_min=floor,
                            den_eps=1e-6)
        r = 0
        for s, _, n in seg:
            got[s].append(out[r:r + n].cpu())
            r += n
    for s in range(3):
        a, b = torch.cat(got[s]).double(), want[s]
        # a row whose divisor |n . q| passes through zero far above its bound amplifies rounding: judged row by row
        err = (a - b).pow(2).mean(1).sqrt() / b.pow(2).mean(1).sqrt().clamp(min=1e-3)
        assert err.median() < 2e-5 and err.sort().values[int(0.99 * (len(err) - 1))] < 2e-3, (s, err.max())
    assert (state[1] == 3.0).all() and (peak[1] == 50.0).all()
    assert (peak[[0, 2, 3]].abs() <= cap + 1e-4).all()


@pytest.mark.parametrize("dev", DEVS)
def test_divided_group_norm_on_wide_groups(dev):
    g = torch.Generator().manual_seed(5)
    for C, group in ((96, 24), (600, 300), (5000, 2500), (20000, 10000), (64 * 40, 40)):
        T, n = 3, C // group
        y, gate, w = torch.randn(T, C, generator=g), torch.randn(T, C, generator=g), torch.randn(C, generator=g)
        den, low = torch.randn(T, n, generator=g) * 2, torch.rand(T, n, generator=g)
        z = (y.double().reshape(T, n, group) / (torch.maximum(den.abs(), low).double() + 0.25)[:, :, None])
        z = (z / torch.sqrt((z * z).mean(-1, keepdim=True) + 0.1)).reshape(T, C) * w.double()
        for act, ga in (("sigmoid", torch.sigmoid(gate.double())), ("silu", torch.nn.functional.silu(gate.double()))):
            out = torch.empty(T, C, device=dev)
            HY.gated_group_norm(y.to(dev), gate.to(dev), w.to(dev), 0.1, group, out, gate_first=False, act=act,
                                den=den.to(dev), den_min=low.to(dev), den_eps=0.25)
            close(out, z * ga, 1e-5)
    with pytest.raises(ValueError):
        HY.gated_group_norm(y.to(dev), gate.to(dev), w.to(dev), 0.1, group, out, gate_first=False, den=den.to(dev))


# ------------------------------------------------------------------------------------------------ whole models
@pytest.mark.parametrize("dev,dt,tol", RUNS)
@pytest.mark.parametrize("shape", list(SHAPES))
def test_prompt_portions_and_decoding(dev, dt, tol, shape):
    cfg, tensors, model = build(dev, dt, seed=5, **SHAPES[shape])
    t = toks(75, cfg.vocab, 1)
    want = oracle(cfg, tensors, t)
    eng = engine(model, 80)
    b16 = dt == "bfloat16"
    if b16 and shape in ("odd", "ragged"):  # some 40 numbers wide: single rows carry several times the typical rounding
        tol *= 2
    close(run_cuts(eng, "whole", t, [75]), want, tol, b16)
    close(run_cuts(eng, "decode", t, [40] + [1] * 35), want, tol, b16)
    close(run_cuts(eng, "cuts", t, [3, 2, 19, 2, 1, 1, 30, 2, 7, 1, 1, 1, 5]), want, tol, b16)
    close(run_cuts(eng, "first", t[:9], [1] * 9), want[:9], tol, b16)  # the first tokens, one by one from position 0
    assert eng.bm.num_free == eng.bm.num_blocks - 1 and len(eng.state_slots.free) == 4


@pytest.mark.parametrize("dev,dt,tol", RUNS)
@pytest.mark.parametrize("kind", ["attention", "attention_2", "mlstm"])
def test_models_of_one_kind_of_layer(dev, dt, tol, kind):
    kw = dict(SHAPES["plain"], pattern=(kind,) * 3, kv_from=None if kind == "mlstm" else {1: 0, 2: 0}, chunk=13)
    cfg, tensors, model = build(dev, dt, seed=13, **kw)
    assert len(model.cache_ranks()) == (0 if kind == "mlstm" else 1)
    assert model.pages_only == (kind == "attention_2")
    t = toks(60, cfg.vocab, 3)
    want = oracle(cfg, tensors, t)
    eng = engine(model, 64, seqs=2)
    b16 = dt == "bfloat16"
    close(run_cuts(eng, "a", t, [60]), want, tol, b16)
    close(run_cuts(eng, "b", t, [7, 2, 30] + [1] * 21), want, tol, b16)


@pytest.mark.parametrize("dev,dt,tol", RUNS)
def test_residual_after_every_layer(dev, dt, tol):
    cfg, tensors, model = build(dev, dt, seed=9, **SHAPES["plain"])
    t = toks(30, cfg.vocab, 2)
    layers = []
    oracle(cfg, tensors, t, layers)
    eng = engine(model, 32)
    for r in range(1, len(layers) + 1):
        orig = eng._build_fb  # the engine's own planner builds the step; stop_layer cuts the forward short

        def fb_cut(plan, tt=None, _r=r):
            fb = orig(plan, tt)
            fb.stop_layer = _r
            return fb
        eng._build_fb = fb_cut
        try:
            eng.replay_step([("k%d" % r, t, [0])], ["k%d" % r])
        finally:
            eng._build_fb = orig
        close(eng.ws.x[:len(t)].float(), layers[r - 1].float(), tol, dt == "bfloat16")


@pytest.mark.parametrize("dev,dt,tol", RUNS)
def test_unequal_batches_reuse_blocks_and_slots(dev, dt, tol):
    """Five requests of unequal length through an engine with three slots and a pool smaller than their sum: portions of
    some beside single tokens of others; finished requests hand their pages and slots on. Every request's logits equal
    those it gets alone."""
    cfg, tensors, model = build(dev, dt, seed=11, **SHAPES["plain"])
    reqs = {k: toks(n, cfg.vocab, 40 + n) for k, n in (("a", 61), ("b", 9), ("c", 33), ("d", 50), ("e", 2))}
    want = {k: oracle(cfg, tensors, v) for k, v in reqs.items()}
    eng = engine(model, max_tokens=160, seqs=3, blocks=11)  # 10 usable pages of 16 tokens
    plan = [[("a", 17), ("b", 2)], [("a", 2), ("b", 1), ("c", 30)], [("a", 1), ("b", 1), ("c", 1)],
            [("a", 30), ("b", 5), ("c", 2)], [("a", 11), ("d", 20)], [("d", 1), ("e", 2)], [("d", 29)]]
    at = {k: 0 for k in reqs}
    got = {k: [] for k in reqs}
    for step in plan:
        entries, end = [], []
        for k, n in step:
            tk = reqs[k][at[k]:at[k] + n]
            entries.append((k, tk, list(range(n))))
            at[k] += n
            if at[k] == len(reqs[k]):
                end.append(k)
        out = eng.replay_step(entries, end)
        r = 0
        for k, tk, _ in entries:
            got[k].append(out[r:r + len(tk)])
            r += len(tk)
    for k in reqs:
        assert at[k] == len(reqs[k])
        close(torch.cat(got[k]), want[k], tol, dt == "bfloat16")
        alone = run_cuts(eng, "alone-" + k, reqs[k], [len(reqs[k])])  # and the same request alone, in the same number format
        close(torch.cat(got[k]), alone, 2e-4 if dt == "float32" else 2e-2)
    assert eng.bm.num_free == eng.bm.num_blocks - 1 and len(eng.state_slots.free) == 3


@pytest.mark.parametrize("dev,dt,tol", RUNS)
def test_peaked_attention_far_keys_and_long_decode(dev, dt, tol):
    """Large score scales make single keys dominate, so a lost or shifted key anywhere in a long prompt (page borders, chunk
    edges, position 0) moves the logits; then 120 tokens decoded one by one, so that two chunks begin and end over decoded
    tokens only."""
    kw = dict(SHAPES["plain"], scale=1.5, t_scale=1.0, softcap=12.0, chunk={0: 50, 3: 90})
    cfg, tensors, model = build(dev, dt, seed=21, **kw)
    t = toks(310, cfg.vocab, 8)
    want = oracle(cfg, tensors, t)
    eng = engine(model, max_tokens=320, seqs=2)
    got = run_cuts(eng, "x", t, [187, 3] + [1] * 120)
    close(got, want, tol * 2, rms=dt == "bfloat16")


@pytest.mark.parametrize("dev,dt,tol", RUNS)
@pytest.mark.parametrize("dim,vdim,heads,kv,tdim", [(64, 128, 8, 2, 96), (128, 64, 3, 1, 64), (96, 96, 4, 4, 128)])
def test_matrix_core_sizes_through_the_engine(dev, dt, tol, dim, vdim, heads, kv, tdim):
    """Head sizes of the matrix-core kernels: a prompt in portions that end inside 16-row tiles, decoded rows behind enough
    keys to be split into partitions."""
    kw = dict(hidden=128, vocab=211, pattern=("attention_2", "attention", "attention_2", "mlstm"), kv_from={2: 0}, heads=heads,
              kv_heads=kv, dim=dim, vdim=vdim, scale=1.5 * dim ** -0.5, chunk={0: 100, 2: 250}, rot_dims=dim // 2,
              rot_factor=2.0, t_heads=6, t_kv_heads=2, t_dim=tdim, t_rot_dims=tdim // 4, t_scaling=(2.0, 1.0, 4.0, 128.0),
              softcap=8.0, m_heads=2, m_dim=64, m_vdim=48, ff=256, residual_mult=0.5)
    cfg, tensors, model = build(dev, dt, seed=17, **kw)
    t = toks(330, cfg.vocab, 9)
    want = oracle(cfg, tensors, t)
    eng = engine(model, max_tokens=336, seqs=2)
    b16 = dt == "bfloat16"
    close(run_cuts(eng, "x", t, [203, 17, 2, 41, 1, 1, 1, 33] + [1] * 31), want, tol, b16)
    close(run_cuts(eng, "y", t[:100], [100]), want[:100], tol, b16)


def _random_shape(rng):
    nl = rng.randint(2, 5)
    pattern, kv_from, owners = [], {}, []
    for i in range(nl):
        kind = rng.choice(["attention", "attention_2", "attention_2", "mlstm"])
        pattern.append(kind)
        if kind == "attention_2":
            if owners and rng.random() < 0.4:
                kv_from[i] = rng.choice(owners)
            else:
                owners.append(i)
    kv, tkv, dim, tdim = rng.choice([1, 2, 3]), rng.choice([1, 2]), rng.choice([16, 24, 32, 64]), rng.choice([8, 20, 48])
    return dict(hidden=rng.choice([64, 96, 160]), vocab=rng.choice([97, 256, 1000]), pattern=tuple(pattern), kv_from=kv_from,
                heads=kv * rng.choice([1, 2, 3]), kv_heads=kv, dim=dim, vdim=rng.choice([16, 32, 64, 128]),
                scale=rng.choice([0.05, 0.1, 0.3]), chunk={i: rng.choice([0, 1, 5, 16, 40, 64, 130]) for i in range(nl)},
                rot_dims=rng.choice([0, 8, dim]), rot_base=rng.choice([100.0, 1e4, 1e6]),
                rot_factor=rng.choice([None, 2.0, 10.0]), t_heads=tkv * rng.choice([1, 2, 4]), t_kv_heads=tkv, t_dim=tdim,
                t_scale=rng.choice([0.1, 0.4]), t_rot_dims=rng.choice([0, 4, tdim]),
                t_scaling=rng.choice([None, (2.0, 1.0, 4.0, 64.0), (16.0, 0.5, 3.0, 500.0)]), conv=rng.choice([1, 2, 3, 4, 6]),
                softcap=rng.choice([0.0, 1.0, 20.0]), m_heads=rng.choice([1, 2, 5]), m_dim=rng.choice([8, 24, 48, 80]),
                m_vdim=rng.choice([8, 33, 64]), gate_cap=rng.choice([2.0, 10.0, 25.0]),
                mlps=tuple(rng.choice(["dense", "dense", None]) for _ in range(rng.randint(1, 3))), ff=rng.choice([40, 99, 256]),
                residual_mult=rng.choice([0.2, 0.7, 1.0]), eps=rng.choice([1e-6, 1e-5]))


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("seed", [1, 2, 3, 4])
def test_random_configurations_and_schedules(dev, seed):
    """Drawn sizes, layer orders, borrowed keys and chunks; five requests fed through four live slots in drawn portions
    (single tokens beside portions of up to 150, requests left out of steps, blocks and slots handed on) in a pool that holds
    the four largest but not all five. fp32 only: every position agrees with the oracle."""
    import random
    rng = random.Random(seed)
    cfg, tensors, model = build(dev, "float32", seed=seed, **_random_shape(rng))
    g = torch.Generator().manual_seed(seed)
    reqs = {"r%d" % i: torch.randint(0, cfg.vocab, (n,), generator=g).tolist()
            for i, n in enumerate(rng.sample([5, 40, 90, 150, 230], 5))}
    want = {k: oracle(cfg, tensors, v) for k, v in reqs.items()}
    eng = engine(model, max_tokens=1024, seqs=4, blocks=34 + 1)  # 16-token pages: 1 + 3 + 6 + 10 + 15 would be 35
    pending, live, at, got = list(reqs), [], {}, {k: [] for k in reqs}
    while pending or live:
        while pending and len(live) < 4 and (not live or rng.random() < 0.5):
            live.append(pending.pop(0))
            at[live[-1]] = 0
        entries, end = [], []
        for k in list(live):
            if rng.random() < 0.15 and len(live) > 1:
                continue  # left out of this step
            n = min(len(reqs[k]) - at[k], rng.choice([1, 1, 1, 2, 3, 16, 37, 64, 150]))
            entries.append((k, reqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(reqs[k]):
                live.remove(k)
                end.append(k)
        if not entries:
            continue
        out = eng.replay_step(entries, end)
        r = 0
        for k, tk, _ in entries:
            got[k].append(out[r:r + len(tk)])
            r += len(tk)
    for k in reqs:
        close(torch.cat(got[k]), want[k], 3e-4)
    assert eng.bm.num_free == eng.bm.num_blocks - 1 and len(eng.state_slots.free) == 4


# ------------------------------------------------------------------------------------------------ serving path
@pytest.mark.parametrize("dev,dt", [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("native", [False, True])
def test_greedy_generation_through_the_scheduler(dev, dt, native):
    """engine.submit: chunked prefill, continuous batching of three requests over two slots, greedy sampling; each request's
    tokens equal the oracle's greedy continuation."""
    cfg, tensors, model = build(dev, dt, seed=4, **SHAPES["plain"])
    ec = EngineConfig(max_num_seqs=2, max_batched_tokens=24, prefill_chunk=10, max_model_len=128, block_size=16,
                      num_blocks=20, use_graphs=False, native_scheduler=native, gemm_autotune=False)
    eng = LLMEngine(model, ByteTokenizer(cfg.vocab), ec)
    if native and not eng.native_sched:
        pytest.skip("native runtime not built")
    prompts = [toks(n, cfg.vocab, 30 + n) for n in (27, 5, 13)]
    hs = [eng.submit(Request(p, SamplingParams(temperature=0.0, ignore_eos=True), 12)) for p in prompts]
    eng.run_until_done()
    for p, h in zip(prompts, hs):
        assert [i for o in h for i in o.token_ids] == greedy(cfg, tensors, p, 12)
    assert len(eng.state_slots.owner) <= 2


@pytest.mark.parametrize("kind", ["attention_2", "mlstm"])
def test_prefix_sharing_only_without_carried_state(kind):
    """A model of chunked layers alone keeps everything in its pages and takes an earlier prompt's full pages over; with a
    memory anywhere every prompt is computed from position 0. Either way the tokens are those of the oracle."""
    kw = dict(SHAPES["plain"], pattern=("attention_2", kind), kv_from=None, chunk=24)
    cfg, tensors, model = build("cpu", "float32", seed=4, **kw)
    ec = EngineConfig(max_num_seqs=2, max_batched_tokens=64, max_model_len=128, block_size=16, num_blocks=24,
                      use_graphs=False, native_scheduler=False, gemm_autotune=False, enable_prefix_cache=True)
    eng = LLMEngine(model, ByteTokenizer(cfg.vocab), ec)
    head = toks(40, cfg.vocab, 5)
    for n in (7, 3):
        p = head + toks(n, cfg.vocab, n)
        h = eng.submit(Request(p, SamplingParams(temperature=0.0, ignore_eos=True), 8))
        eng.run_until_done()
        assert [i for o in h for i in o.token_ids] == greedy(cfg, tensors, p, 8)
    assert eng.stats["cached_tokens_total"] == (32 if kind == "attention_2" else 0)


@pytest.mark.gpu
def test_decode_graphs_replay_like_the_oracle():
    """Decode-only steps replay captured graphs (several buckets as requests come and go, eager prompt chunks between the
    replays); every request still yields the oracle's greedy tokens, also after slots and pages were reused."""
    cfg, tensors, model = build("cuda", "float32", seed=4, **SHAPES["plain"])
    ec = EngineConfig(max_num_seqs=3, max_batched_tokens=32, prefill_chunk=9, max_model_len=128, block_size=16,
                      num_blocks=24, use_graphs=True, gemm_autotune=False, enable_prefix_cache=False)
    eng = LLMEngine(model, ByteTokenizer(cfg.vocab), ec)
    prompts = [toks(n, cfg.vocab, 70 + n) for n in (21, 4, 30, 11, 17)]
    gens = [14, 25, 6, 9, 12]
    hs = [eng.submit(Request(p, SamplingParams(temperature=0.0, ignore_eos=True), g)) for p, g in zip(prompts, gens)]
    eng.run_until_done()
    assert eng.stats["graph_steps"] >= 5
    for p, g, h in zip(prompts, gens, hs):
        assert [i for o in h for i in o.token_ids] == greedy(cfg, tensors, p, g)


@pytest.mark.gpu
def test_decode_graphs_equal_eager_steps_in_bf16():
    """The matrix-core decode kernels inside replayed graphs: many replays with the program's own work between them give the
    tokens of the eager engine (the same kernels, launched one by one)."""
    kw = dict(hidden=128, vocab=211, pattern=("attention_2", "attention", "mlstm", "attention_2"), kv_from={3: 0}, heads=8,
              kv_heads=2, dim=64, vdim=64, chunk=40, t_dim=96, softcap=20.0, m_heads=2, m_dim=64, m_vdim=64, ff=256)
    cfg, _, model = build("cuda", "bfloat16", seed=3, **kw)
    out = []
    for graphs in (False, True):
        ec = EngineConfig(max_num_seqs=2, max_batched_tokens=64, max_model_len=256, block_size=16, num_blocks=40,
                          use_graphs=graphs, gemm_autotune=False, enable_prefix_cache=False)
        eng = LLMEngine(model, ByteTokenizer(cfg.vocab), ec)
        hs = [eng.submit(Request(toks(n, cfg.vocab, n), SamplingParams(temperature=0.0, ignore_eos=True), 60))
              for n in (50, 21)]
        eng.run_until_done()
        out.append([[i for o in h for i in o.token_ids] for h in hs])
        assert (eng.stats["graph_steps"] > 20) == graphs
    # rounding may turn a near tie somewhere: the first tokens, before any such turn could spread, are equal
    assert all(a[:20] == b[:20] for a, b in zip(*out)), out


@pytest.mark.parametrize("native", [False, True])
def test_preempted_request_recomputes_its_state(native):
    """A pool too small for both requests' growth: one is preempted, loses its blocks and its slot and is recomputed from
    position 0 later, in whatever slot it gets. Both still produce the oracle's greedy tokens."""
    cfg, tensors, model = build("cpu", "float32", seed=8, **SHAPES["plain"])
    ec = EngineConfig(max_num_seqs=2, max_batched_tokens=64, max_model_len=128, block_size=16, num_blocks=8,
                      use_graphs=False, native_scheduler=native, gemm_autotune=False)
    eng = LLMEngine(model, ByteTokenizer(cfg.vocab), ec)
    if native and not eng.native_sched:
        pytest.skip("native runtime not built")
    prompts = [toks(30, cfg.vocab, 51), toks(28, cfg.vocab, 52)]
    hs = [eng.submit(Request(p, SamplingParams(temperature=0.0, ignore_eos=True), 40)) for p in prompts]
    eng.run_until_done(max_steps=400)
    assert eng.stats["preemptions"] > 0 and eng.stats["finished"] == 2
    for p, h in zip(prompts, hs):
        assert [i for o in h for i in o.token_ids] == greedy(cfg, tensors, p, 40)


def test_config_reader_and_checkpoint_round_trip(tmp_path):
    cfg = TE.make_config(**SHAPES["odd"])
    get = TE.synthetic_source(cfg, 1)
    TE.save_checkpoint(cfg, get, str(tmp_path))
    assert TE.is_tebodra_dir(str(tmp_path))
    cfg2, get2 = TE.dir_source(str(tmp_path))
    assert cfg2 == TE.TebodraConfig.from_json(cfg.to_json(), cfg2.name) and cfg2.to_json() == cfg.to_json()
    assert cfg2.layers[0].mixer.conv == 2 and cfg2.layers[1].mixer.chunk == 7 and cfg2.layers[0].mixer.rot.scaling is None
    assert torch.equal(get2("l1.mix.q"), get("l1.mix.q")) and get2("l0.mix.v") is None and get2("l0.mix.sink") is None
    from localai_tfp_amd.models.loader import load_llm
    m, _tok, c, _ = load_llm(str(tmp_path), "cpu")
    assert isinstance(m, TE.TebodraModel) and c.layers[1].mixer.scale == 0.4 and c.rms_eps == 1e-3
    assert m.cache_ranks() == [2 * 24, 3 * 32]
    cfg3 = TE.make_config(**SHAPES["plain"])
    j3 = cfg3.to_json()
    assert j3["layers"][3]["mixer"]["kv_from"] == 0 and j3["layers"][3]["mixer"]["mask"] == {"size": 11}
    assert j3["layers"][3]["mlp"] is None and j3["layers"][0]["mixer"]["rot"]["scaling"] == {"factor": 3.0}
    names = TE.tensor_shapes(cfg3)
    assert "l3.mix.k" not in names and "l3.mix.k.norm" not in names and names["l3.mix.q.norm"] == (64,)
    assert names["l2.mix.k.conv"] == (60, 4) and names["l1.mix.norm"] == (60,) and "l3.norm2" not in names
    assert [sorted(e) for e in TE.TebodraModel(cfg3).cache_spec()] == [["kv"], ["peak", "state"], ["kv", "tails"], [],
                                                                      ["peak", "state"]]
    for path, val in ((("layers", 0, "type"), "something_else"), (("layers", 0, "mlp", "kind"), "moe"),
                      (("layers", 3, "mixer", "kv_from"), 3), (("layers", 3, "mixer", "kv_from"), 1),
                      (("layers", 3, "mixer", "vdim"), 8), (("layers", 0, "mixer", "kv_heads"), 3),
                      (("layers", 2, "mixer", "vdim"), 16), (("layers", 2, "mixer", "conv"), 0),
                      (("layers", 2, "mixer", "conv"), 17), (("layers", 1, "mixer", "dim"), 300),
                      (("layers", 1, "mixer", "gate_cap"), 0.0), (("layers", 0, "mixer", "rot", "dims"), 18),
                      (("layers", 0, "mixer", "rot", "dims"), 7)):
        bad = json.loads(json.dumps(j3))
        TE.TebodraConfig.from_json(bad)  # (valid until it is broken)
        node = bad
        for p in path[:-1]:
            node = node[p]
        node[path[-1]] = val
        with pytest.raises(ValueError):
            TE.TebodraConfig.from_json(bad)
    tensors = {k: get(k) for k in get.names}
    tensors["l1.mix.q"] = tensors["l1.mix.q"][:-1]
    with pytest.raises(ValueError):
        TE.TebodraModel.load(cfg, tensors.get, "cpu")
    m, _, c, _ = load_llm("synthetic:tebodra-tiny", "cpu")
    assert isinstance(m, TE.TebodraModel) and c.layers[3].mixer.kv_from == 0


def test_trace_runner_command_line(tmp_path):
    """bin/trace_run on a checkpoint directory: steps on stdin, one logits file per step that wants any."""
    cfg = TE.make_config(**SHAPES["plain"])
    get = TE.synthetic_source(cfg, 6)
    mdir, odir = str(tmp_path / "m"), str(tmp_path / "o")
    TE.save_checkpoint(cfg, get, mdir)
    a, b = toks(21, cfg.vocab, 1), toks(9, cfg.vocab, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:12], "want": [0, 11]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[12:13], "want": []}, {"id": "b", "tokens": b, "want": [8]}],
              "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[13:], "want": [7, 0]}], "end": ["a"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", mdir, "--dtype", "float32", "--out", odir,
                        "--max-tokens", "128", "--device", "cpu"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    tensors = {k: get(k) for k in get.names}
    wa, wb = oracle(cfg, tensors, a), oracle(cfg, tensors, b)
    rd = lambda n: torch.from_numpy(np.fromfile(os.path.join(odir, "%d.f32" % n), dtype="<f4").reshape(-1, cfg.vocab))  # noqa: E731
    close(rd(0), wa[[0, 11]], 2e-4)
    close(rd(1), wb[[8]], 2e-4)
    close(rd(2), wa[[20, 13]], 2e-4)


def test_served_through_the_llm_worker(tmp_path):
    """The gRPC LLM worker loads a Tebodra checkpoint directory like any other model and streams a completion whose tokens
    are the oracle's greedy continuation (byte-level tokenizer: one token per prompt byte after BOS)."""
    from localai_tfp_amd.grpc import pb
    from localai_tfp_amd.grpc.client import BackendClient
    from localai_tfp_amd.grpc.server import AioServer
    from localai_tfp_amd.workers.llm import LLMServicer
    cfg = TE.make_config(**dict(SHAPES["plain"], vocab=300))
    get = TE.synthetic_source(cfg, 12)
    TE.save_checkpoint(cfg, get, str(tmp_path))
    svc = LLMServicer(device="cpu")
    server = AioServer(svc, "127.0.0.1:0", max_workers=4)
    c = BackendClient(f"127.0.0.1:{server.port}")
    try:
        r = c.load_model(pb.ModelOptions(Model=str(tmp_path), ContextSize=256))
        assert r.success, r.message
        assert isinstance(svc.engine.model, TE.TebodraModel)
        o = pb.PredictOptions(Prompt="chunks", Tokens=6, Temperature=0.0, IgnoreEOS=True)
        a = c.predict(o)
        chunks = list(c.predict_stream(o))
        assert a.tokens == 6 and b"".join(x.message for x in chunks) == a.message
        tok = svc.engine.tok
        seq = list(tok.encode("chunks"))
        assert a.prompt_tokens == len(seq)
        want = greedy(cfg, {k: get(k) for k in get.names}, seq, 6)
        assert tok.decode(want).encode(errors="replace") == a.message or a.message == tok.decode(want).encode()
    finally:
        c.close()
        if svc.engine is not None:
            svc.engine.shutdown()
        server.stop()
