"""Zomolix (windowed attention that keeps the first tokens, borrowed keys, latent attention with a rotated key part, sinks
and a gate per number, layer scales, clamped experts behind a group-limited router) on the engine against the plain
float64 oracle of tests/oracle_zomolix.py: every mechanism alone, whole prompts, token-by-token decoding, prompt portions
down to two tokens, unequal batches, reuse of freed blocks, keys far back / at page borders / just inside and outside the
window and the kept tokens with peaked softmax weights, odd sizes, long decoding, greedy generation through the
scheduler, graph replays, shared prefixes, and the trace runner's command line.

Each engine test runs on the CPU plumbing path (fp32) and, marked gpu, on the HIP kernels in fp32 and bf16."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

import oracle_zomolix as O
from localai_tfp_amd.engine.engine import EngineConfig, LLMEngine
from localai_tfp_amd.engine.sequence import Request
from localai_tfp_amd.models import zomolix as ZO
from localai_tfp_amd.ops import hybrid as HY
from localai_tfp_amd.ops import latent as LA
from localai_tfp_amd.ops.sampling import SamplingParams
from localai_tfp_amd.tokenizer import ByteTokenizer
from test_vugotar import _FB, close, engine, run_cuts, steps_of, toks

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.param("cuda", marks=pytest.mark.gpu)
DEVS = ["cpu", GPU]
RUNS = [("cpu", "float32", 2e-4), pytest.param("cuda", "float32", 2e-4, marks=pytest.mark.gpu),
        pytest.param("cuda", "bfloat16", 6e-2, marks=pytest.mark.gpu)]
F64 = torch.float64
YARN = (4.0, 40.0, 4.0, 0.5)  # (factor, original, fast, slow): the ramp lies inside the pairs of these small heads

SHAPES = {
    # both mixers, a layer that borrows keys under a window of its own, both rotations scaled, groups of experts
    "plain": dict(hidden=64, vocab=97, pattern=("attention", "latent_attention", "attention", "latent_attention"),
                  kv_from={2: 0}, heads=4, kv_heads=2, dim=16, vdim=16, window={0: 20, 2: 11}, keep_first={0: 3, 2: 5},
                  rot_dims=8, rot_base=500.0, rot_scaling=YARN, l_heads=3, l_dim=12, l_rot=8, l_vdim=16, kv_rank=40,
                  l_rot_base=300.0, l_rot_scaling=(8.0, 24.0, 3.0, 0.25), experts=8, top=3, groups=(4, 2), expert_ff=24,
                  limit=0.8, shared_ff=32, shared_limit=0.5, emb_scale=2.0),
    # sizes that differ from each other: dim != vdim, the whole head rotated, no scaling, no kept tokens, a window smaller
    # than a page, no window at all, one group, top == experts, no shared expert, a layer without a feed-forward, a large
    # eps, cached rows that are no multiple of eight
    "odd": dict(hidden=40, vocab=61, pattern=("latent_attention", "attention", "attention"), mlps=("moe", None, "moe"),
                heads=6, kv_heads=3, dim=24, vdim=40, window={1: 7, 2: 0}, keep_first={1: 0, 2: 0}, rot_base=300.0, scale=0.4,
                l_heads=2, l_dim=20, l_rot=6, l_vdim=12, kv_rank=21, l_scale=0.3, experts=5, top=5, expert_ff=17,
                limit=0.6, shared_ff=0, emb_scale=1.0, eps=1e-3),
    # one key head, more kept tokens than the window is long, no rotation in the attention layers, one expert of many with
    # one group kept, cached rows of 136 + 24, one latent head
    "wide": dict(hidden=48, vocab=53, pattern=("attention", "attention", "latent_attention"), kv_from={1: 0}, heads=4,
                 kv_heads=1, dim=72, vdim=8, window={0: 9, 1: 30}, keep_first={0: 14, 1: 1}, rot_dims=0, scale=0.2, l_heads=1,
                 l_dim=8, l_rot=24, l_vdim=72, kv_rank=136, l_rot_scaling=(2.0, 64.0, 8.0, 1.0), experts=9, top=1,
                 groups=(3, 1), expert_ff=16, limit=3.0, shared_ff=24, shared_limit=9.0, emb_scale=0.5),
    # nothing a multiple of eight, a window of one token (a row sees itself and the kept ones)
    "ragged": dict(hidden=44, vocab=101, pattern=("attention", "latent_attention", "attention"), heads=5, kv_heads=5, dim=20,
                   vdim=12, window={0: 1, 2: 33}, keep_first={0: 2, 2: 17}, rot_dims=10, rot_scaling=YARN, scale=0.3,
                   l_heads=5, l_dim=6, l_rot=10, l_vdim=10, kv_rank=30, experts=6, top=2, groups=(2, 1), expert_ff=10,
                   limit=1.0, shared_ff=6, emb_scale=3.0),
}


def build(device="cpu", dtype="float32", seed=0, **kw):
    cfg = ZO.make_config(**kw)
    get = ZO.synthetic_source(cfg, seed)
    model = ZO.ZomolixModel.load(cfg, get, torch.device(device), getattr(torch, dtype))
    return cfg, {k: get(k) for k in get.names}, model


def oracle(cfg, tensors, tokens, layers=None):
    return O.forward(cfg.to_json(), tensors.get, tokens, layers).float()


def greedy(cfg, tensors, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(oracle(cfg, tensors, seq)[-1].argmax()))
    return seq[len(prompt):]


# ------------------------------------------------------------------------------------------------ mechanisms alone
def test_frequencies_with_and_without_scaling():
    for rot in ({"dims": 32, "base": 10000.0}, {"dims": 24, "base": 700.0, "scaling": dict(factor=4.0, original=512, fast=32.0,
                                                                                         slow=1.0)},
                {"dims": 64, "base": 5e5, "scaling": dict(factor=32.0, original=8192, fast=16.0, slow=2.0)},
                {"dims": 8, "base": 100.0, "scaling": dict(factor=2.0, original=8, fast=64.0, slow=32.0)},  # hi <= lo
                {"dims": 16, "base": 50.0, "scaling": dict(factor=1.0, original=99, fast=4.0, slow=1.0)}):
        f, mag = ZO.RotCfg.from_json(rot).tables("cpu")
        want, wmag = O.frequencies(rot)
        close(f, want, 1e-6)
        assert abs(mag - wmag) < 1e-9
        assert ZO.RotCfg.from_json(ZO.RotCfg.from_json(rot).to_json()) == ZO.RotCfg.from_json(rot)
    a = O.frequencies({"dims": 16, "base": 10000.0})[0]
    b = O.frequencies({"dims": 16, "base": 10000.0, "scaling": dict(factor=8.0, original=512, fast=32.0, slow=1.0)})[0]
    assert b[0] == a[0] and abs(b[-1] * 8 / a[-1] - 1) < 1e-12 and (b[1:-1] <= a[1:-1]).all()  # fast kept, slow divided


@pytest.mark.parametrize("dev", DEVS)
def test_embedding_scale_and_scaled_add_with_norm(dev):
    g = torch.Generator().manual_seed(2)
    table, ids = torch.randn(17, 40, generator=g), torch.tensor([3, 16, 0, 3], dtype=torch.int32)
    out, o16 = torch.empty(4, 40, device=dev), torch.empty(4, 40, device=dev, dtype=torch.bfloat16)
    HY.embed_rows(table.to(dev), ids.to(dev), out, out16=o16, scale=2.5)
    close(out, table.double()[ids.long()] * 2.5, 1e-6)
    close(o16.float(), out.cpu(), 1e-2)
    eps = 0.3  # a large eps shows whether it sits inside the root
    for C in (40, 300, 1000, 2300, 4100, 9000):
        M = 3
        y, x = torch.randn(M, C + 3, generator=g) * 2, torch.randn(M, C, generator=g)
        b, s, w = (torch.randn(C, generator=g) for _ in range(3))
        want = x.double() + (y[:, 3:].double() + b.double()) * s.double()
        xd, h32 = x.clone().to(dev), torch.empty(M, C, device=dev)
        h16 = torch.empty(M, C, device=dev, dtype=torch.bfloat16)
        HY.scale_add_norm(y.to(dev)[:, 3:], b.to(dev), s.to(dev), xd, w.to(dev), eps, h32, h16)
        close(xd, want, 1e-6)
        close(h32, O.rms_norm(want, w, eps), 1e-5)
        close(h16.float(), O.rms_norm(want, w, eps), 1e-2)
        xd = x.clone().to(dev)  # no bias, an offset norm; then the add alone, without a scale
        HY.scale_add_norm(y.to(dev)[:, 3:], None, s.to(dev), xd, w.to(dev), eps, h32, offset=1.0)
        want = x.double() + y[:, 3:].double() * s.double()
        close(xd, want, 1e-6)
        close(h32, O.rms_norm(want, 1.0 + w.double(), eps), 1e-5)
        xd = x.clone().to(dev)
        HY.scale_add_norm(y.to(dev)[:, 3:], None, None, xd)
        close(xd, x.double() + y[:, 3:].double(), 1e-6)


@pytest.mark.parametrize("dev", DEVS)
def test_clamped_unit_and_group_limited_router(dev):
    g = torch.Generator().manual_seed(4)
    T = 6
    a, b = torch.randn(T, 33, generator=g) * 4, torch.randn(T, 33, generator=g) * 4
    a[0, :3], b[0, :3] = torch.tensor([50.0, -50.0, 0.0]), torch.tensor([-50.0, 50.0, 0.0])
    for limit in (0.7, 2.5, 100.0):
        want = O.clamped_unit(a.double(), b.double(), limit)
        for md, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
            out = torch.empty(T, 33, device=dev, dtype=md)
            HY.glu(a.to(dev), b.to(dev), None, None, out, act="clamped", limit=limit, alpha=1.702)
            close(out.float(), want, tol)
    rw = torch.rand(T, 3, generator=g)
    rw[1, 0] = rw[2, 2] = 0.0
    out = torch.empty(T, 33, device=dev)
    HY.glu(a.to(dev), b.to(dev), None, None, out, scale=rw.to(dev), group=11, act="clamped", limit=1.5, alpha=1.702)
    close(out, O.clamped_unit(a.double(), b.double(), 1.5) * rw.double().repeat_interleave(11, 1), 1e-5)
    for E, top, groups in ((8, 3, (4, 3)), (8, 1, (8, 1)), (12, 4, (3, 1)), (6, 6, (2, 2)), (5, 2, None), (128, 6, (16, 3)),
                           (320, 8, (20, 2)), (9, 3, (9, 5))):
        lg = torch.randn(T, E + 1, generator=g) * 2
        lg[0, 1:] += torch.arange(E).float() * 0.01  # (rows whose best experts crowd together)
        if groups:  # the largest logits all in one group: with few groups kept others than the plain top are chosen
            per = E // groups[0]
            lg[1, 1 + per:1 + 2 * per] += 5.0
            lg[2, 1::per] += 4.0
        want = torch.zeros(T, E, dtype=F64)
        gj = {"count": groups[0], "keep": groups[1]} if groups else None
        for t in range(T):
            for e, wgt in O.route(lg[t, 1:].double(), top, gj):
                want[t, e] = wgt
        out = torch.full((T, E), 7.0, device=dev)
        HY.moe_route(lg.to(dev)[:, 1:], top, 1.0, out, 0.0, mode="scores", groups=groups)
        close(out, want, 1e-5)
        assert int((out > 0).sum()) == T * top
        # the other modes keep their weights and take the same experts
        HY.moe_route(lg.to(dev)[:, 1:], top, 1.5, out, 0.0, groups=groups)
        close(out, want / want.sum(1, keepdim=True) * 1.5, 1e-5)
        HY.moe_route(lg.to(dev)[:, 1:], top, 1.0, out, 0.0, mode="sigmoid", groups=groups)
        close(out, torch.sigmoid(lg[:, 1:].double()) * (want > 0), 1e-5)
    with pytest.raises(ValueError):
        HY.moe_route(torch.zeros(1, 8, device=dev), 4, 1.0, torch.empty(1, 8, device=dev), groups=(4, 1))


def _plant(want_q, rot, positions, bias):
    """Projection outputs whose biased, rotated heads are want_q [n, H, d]: the inverse rotation (by minus the position,
    without the magnitude twice), minus the bias."""
    x = want_q.clone()
    if rot and rot["dims"]:
        mag = O.frequencies(rot)[1]
        y = O.rotate(x, rot, False, [-p for p in positions])
        x = y
        x[:, :, :rot["dims"]] /= mag * mag
    return (x - bias.double().reshape(1, x.shape[1], x.shape[2])).float()


def _window_case(dev, dt, H, G, dk, dv, rot, n, cuts, bs, scale, window, keep, plant=(), share=False, bias_rows=0, sink=False):
    """Biases + rotation + append, then windowed attention with kept first tokens, in portions through shuffled pages whose
    unused slots hold stale numbers. `plant` = [(query position, key position)]: the query is made a large multiple of the
    key, so that one score stands out wherever the mask lets it. `share`: the queries come from a launch without keys."""
    g = torch.Generator().manual_seed(7)
    md = getattr(torch, dt)
    q, k, v = torch.randn(n, H, dk, generator=g), torch.randn(n, G, dk, generator=g), torch.randn(n, G, dv, generator=g)
    qb, kb, vb = (0.5 * torch.randn(x, generator=g) for x in (H * dk, G * dk, G * dv))
    kr = O.rotate((k.double() + kb.double().reshape(G, dk)), rot, False)
    want_q = O.rotate((q.double() + qb.double().reshape(H, dk)), rot, False)
    for qi, kj in plant:
        for h in range(H):
            want_q[qi, h] = kr[kj, h // (H // G)] * 6.0
    q = _plant(want_q, rot, list(range(n)), qb)
    qr = O.rotate(q.double() + qb.double().reshape(H, dk), rot, False)
    vv = v.double() + vb.double().reshape(G, dv)
    if md == torch.bfloat16:  # pools and query operand hold bf16: the oracle reads the same rounded numbers
        qr, kr, vv = qr.float().to(md).double(), kr.float().to(md).double(), vv.float().to(md).double()
    mask = {"size": window, "keep_first": keep} if window else None
    table_b = 3.0 * torch.randn(H, bias_rows, generator=g) if bias_rows else None
    sk = torch.randn(H, generator=g) if sink else None
    if bias_rows or sink:  # with a distance bias and a sink, as other designs combine them
        want = torch.zeros(n, H, dv, dtype=F64)
        for h in range(H):
            for i in range(n):
                js = O.visible(i, mask)
                s = (kr[js, h // (H // G)] @ qr[i, h]) * scale
                if bias_rows:
                    s = s + table_b[h, [min(i - j, bias_rows - 1) for j in js]].double()
                e = torch.exp(s - s.max())
                den = e.sum() + (torch.exp(sk[h].double() - s.max()) if sink else 0.0)
                want[i, h] = (e / den) @ vv[js, h // (H // G)]
    else:
        want = O.grouped_attention(qr, kr, vv, scale, mask)
    nb = -(-n // bs)
    table = torch.randperm(nb + 3, generator=g)[:nb].tolist()
    kc = torch.full((nb + 3, bs, G * dk), 7.0, dtype=md, device=dev)
    vc = torch.full((nb + 3, bs, G * dv), -5.0, dtype=md, device=dev)
    wide = torch.cat([torch.randn(n, 3, generator=g), q.reshape(n, -1), k.reshape(n, -1), v.reshape(n, -1)], 1).to(dev)
    f, mag = ZO.RotCfg.from_json(rot).tables(dev)
    got = torch.empty(n, H * dv + 5, device=dev, dtype=md)
    part = (torch.empty(H * 8, 2, device=dev), torch.empty(H * 8, dv, device=dev))  # room for eight partitions
    c0, c1 = 3 + H * dk, 3 + (H + G) * dk
    dims = rot["dims"] if rot else 0
    for n_dec, chunks, at in steps_of(n, cuts):
        c = 1 if n_dec else chunks[0]
        rws = list(range(at, at + c))
        slots = [table[p // bs] * bs + p % bs for p in rws]
        fb = _FB(n_dec, chunks, rws, [0], dev, slots, dec_bt=[table] if n_dec else None,
                 dec_lens=[at + 1] if n_dec else None, pf_bt=None if n_dec else [table],
                 pf_ctx=None if n_dec else [at + c])
        qo = torch.empty(c, H * dk, device=dev, dtype=md)
        w = wide[at:at + c]
        HY.rope_norm_append(w[:, 3:c0], w[:, c0:c1], w[:, c1:], fb.positions, H, G, dk, dv, dims, 1.0, False, 1e-6, qo, kc,
                            vc, fb.slots, half=True, freqs=f, mag=mag, q_bias=qb.to(dev), k_bias=kb.to(dev),
                            v_bias=vb.to(dev))
        if share:
            q2 = torch.full_like(qo, 3.0)
            HY.rope_norm_append(w[:, 3:c0], None, None, fb.positions, H, G, dk, dv, dims, 1.0, False, 1e-6, q2, None, None,
                                fb.slots, half=True, freqs=f, mag=mag, q_bias=qb.to(dev))
            assert torch.equal(q2, qo)
        HY.masked_attention(qo, kc, vc, HY.Ragged(fb), H, G, dk, dv, scale, got[at:at + c, 5:], window=window, keep=keep,
                            workspace=part, bias=table_b.to(dev) if bias_rows else None, sink=sk.to(dev) if sink else False)
    return got[:, 5:].float().reshape(n, H, dv), want


@pytest.mark.parametrize("dev,dt,tol", RUNS)
@pytest.mark.parametrize("gemm_rows", [64, 8])
def test_window_edges_kept_tokens_pages_and_portions(dev, dt, tol, gemm_rows, monkeypatch):
    """Planted keys carry nearly all of a row's weight where the mask lets them: just inside and just outside the window,
    the last kept token and the next one, page borders, the row itself; in prompt portions and in rows decoded alone
    (split into partitions), on the row, matrix-core and library-GEMM routes."""
    monkeypatch.setattr(HY, "GEMM_MIN_ROWS", gemm_rows)
    monkeypatch.setattr(HY, "DECODE_WAVES", 16)  # decode rows split into partitions of 64 keys
    tol = 2e-2 if dt == "bfloat16" else 2e-4
    rot = {"dims": 16, "base": 500.0, "scaling": dict(zip(("factor", "original", "fast", "slow"), YARN))}
    n, W, K = 290, 90, 5
    plant = [(i, j) for i, j in (
        (200, 200 - W + 1), (201, 201 - W), (202, K - 1), (203, K), (204, 0), (205, 205), (206, 112), (207, 111),
        (30, 29), (92, 2), (93, 3), (94, 4), (95, 5), (96, 6), (97, 7), (150, K - 1), (151, K), (152, 152 - W + 1),
        (153, 153 - W), (284, 284 - W + 1), (285, 285 - W), (286, K - 1), (287, K), (288, 0), (289, 289))]
    cuts = [97, 2, 80, 3, 70, 29] + [1] * 9
    got, want = _window_case(dev, dt, 4, 2, 24, 40, rot, n, cuts, 16, 0.5, W, K, plant, share=True)
    close(got, want, tol)
    # the plants show: a window one token longer or shorter, one kept token more or less moves whole rows
    base = want[[201, 203, 285, 287]].abs().max()
    for dw, dk_ in ((1, 0), (-1, 0), (0, 1), (0, -1)):
        other = _window_case("cpu", "float32", 4, 2, 24, 40, rot, n, [n], 16, 0.5, W + dw, K + dk_, plant)[1]
        assert (other[200:] - want[200:]).abs().max() > 0.3 * base
    # head sizes of the matrix-core kernels; more kept tokens than a tile, a window smaller than a 16-row tile
    plant = [(149, 149 - 9), (148, 148 - 10), (147, 69), (146, 70), (145, 64), (144, 63), (100, 69), (101, 70), (102, 92),
             (103, 94), (79, 69), (78, 69), (77, 72)]
    got, want = _window_case(dev, dt, 8, 2, 64, 128, rot, 150, [75, 40, 2, 20] + [1] * 13, 16, 0.3, 10, 70, plant)
    close(got, want, tol)
    got, want = _window_case(dev, dt, 3, 1, 128, 64, None, 150, [70, 64, 2] + [1] * 14, 16, 0.2, 33, 1,
                             [(149, 0), (148, 148 - 32), (147, 147 - 33), (140, 1), (60, 0), (61, 1), (100, 100 - 32)])
    close(got, want, tol)
    # whole rotation, pages of 4 tokens, as many key heads as heads, no kept tokens, a window of one page
    got, want = _window_case(dev, dt, 2, 2, 16, 16, {"dims": 16, "base": 50.0}, 40, [9, 1, 1, 20, 2, 7], 4, 1.0, 4, 0,
                             [(39, 36), (38, 34), (20, 17), (21, 17)])
    close(got, want, tol)
    got, want = _window_case(dev, dt, 4, 4, 64, 64, rot, 130, [130], 16, 0.4, 1, 3, [(129, 2), (128, 3), (127, 127)])
    close(got, want, tol)
    # beside a distance bias and a sink
    for dk, dv in ((24, 40), (64, 64)):
        got, want = _window_case(dev, dt, 4, 2, dk, dv, rot, 150, [70, 66] + [1] * 14, 16, 0.3, 40, 3,
                                 [(149, 2), (148, 148 - 39), (147, 3), (100, 2)], bias_rows=60, sink=True)
        close(got, want, tol)


def test_kept_tokens_need_a_window():
    q = torch.zeros(1, 16)
    with pytest.raises(ValueError):
        HY.masked_attention(q, q.view(1, 1, 16), q.view(1, 1, 16), HY.Ragged(_FB(0, [1], [0], [0], "cpu")), 1, 1, 16, 16, 1.0,
                            q.clone(), keep=2)


@pytest.mark.parametrize("dev,dt", [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu),
                                    pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("R,rot,H,d", [(40, 8, 3, 12), (21, 6, 2, 20), (104, 24, 4, 40), (512, 64, 16, 24), (512, 64, 20, 8),
                                       (256, 64, 40, 16), (130, 2, 2, 6), (300, 40, 1, 16), (576, 64, 2, 8), (64, 0, 4, 16)])
def test_latent_rows_with_a_rotated_part(dev, dt, R, rot, H, d):
    """Norm + rotation + append of (latent, rotated key part), the split of the queries, and attention over the rows with
    sinks: one planted row per query carries nearly all the weight (far back, at page borders, at the newest position,
    across decode partitions), partly through the rotated part alone; beside it rows where the sink takes the weight."""
    g = torch.Generator().manual_seed(R + H)
    md = getattr(torch, dt)
    bs, n, W, scale, eps = 16, 150, R + rot, 0.5, 0.05
    rj = {"dims": rot, "base": 300.0, "scaling": dict(factor=8.0, original=24, fast=3.0, slow=0.25)} if rot else None
    f, mag = ZO.RotCfg.from_json(rj).tables(dev)
    q, kv = torch.randn(n, H * (d + rot), generator=g), torch.randn(n, W, generator=g)
    w, sink = 1.0 + 0.2 * torch.randn(R, generator=g), torch.randn(H, generator=g)
    sink[0] = 4.0
    table = (torch.randperm(-(-n // bs) + 2, generator=g)[:-(-n // bs)]).tolist()
    cache = torch.full((len(table) + 2, bs, W), 9.0, device=dev, dtype=md)
    c = O.rms_norm(kv[:, :R].double(), w, eps)
    kr = O.rotate(kv[:, R:].double()[:, None], rj, True)[:, 0]
    rows = torch.cat([c, kr], 1)
    qr = O.rotate(q.double().reshape(n, H, d + rot)[:, :, d:], rj, True)
    part = (torch.empty(2 * H * 8, 2, device=dev), torch.empty(2 * H * 8, R, device=dev))
    wide = torch.cat([torch.randn(n, 2, generator=g), q, kv], 1).to(dev)
    qa_all = torch.randn(H, n, W, generator=g).double() * 0.05
    plant = {149: 0, 148: 15, 147: 16, 146: 146, 145: 64, 144: 63, 100: 3, 101: 101, 60: 31, 61: 32, 20: 20, 1: 0}
    rd = rows.float().to(md).double()
    for i, j in plant.items():
        qa_all[:, i, :R] += rd[j, :R] * (60.0 / max(1.0, float((rd[j, :R] ** 2).sum())))
    qa_all[:, :, R:] = qr.float().to(md).double().transpose(0, 1)
    qa_all = qa_all.float().to(md).double()
    got = torch.empty(H, n, R, device=dev, dtype=md)
    qn_got = torch.empty(n, H * d, device=dev, dtype=md)
    for n_dec, chunks, at in steps_of(n, [70, 2, 33, 20] + [1] * 25):
        m = 1 if n_dec else chunks[0]
        rws = list(range(at, at + m))
        slots = [table[p // bs] * bs + p % bs for p in rws]
        fb = _FB(n_dec, chunks, rws, [0], dev, slots, dec_bt=[table] if n_dec else None,
                 dec_lens=[at + 1] if n_dec else None, pf_bt=None if n_dec else [table], pf_ctx=None if n_dec else [at + m])
        qa = torch.zeros(H, m, W, device=dev, dtype=md)
        ws = wide[at:at + m]
        LA.latent_rope_append(ws[:, 2:2 + H * (d + rot)], ws[:, 2 + H * (d + rot):], H, d, rot, R, w.to(dev), eps, f, mag,
                              fb.positions, qn_got[at:at + m], qa, cache, fb.slots)
        if rot:
            close(qa[:, :, R:].float(), qr[at:at + m].transpose(0, 1), 1e-4 if dt == "float32" else 1e-2)
        qa[:, :, :R] = qa_all[:, at:at + m, :R].to(dev).to(md)
        LA.latent_attention(qa, cache, LA.Ragged(fb), scale, got[:, at:at + m], workspace=part, part_len=32,
                            sink=sink.to(dev))
    close(qn_got.float().reshape(n, H, d), q.reshape(n, H, d + rot)[:, :, :d], 1e-6 if dt == "float32" else 1e-2)
    stored = torch.stack([cache[table[p // bs], p % bs] for p in range(n)]).float()
    close(stored, rows, 1e-4 if dt == "float32" else 1e-2)
    want = torch.stack([O.softmax_rows(qa_all[h], rd, rd[:, :R], scale, sink=sink[h].double()) for h in range(H)])
    close(got.float(), want, 2e-4 if dt == "float32" else 2e-2)
    no_sink = torch.stack([O.softmax_rows(qa_all[h], rd, rd[:, :R], scale) for h in range(min(H, 2))])
    assert (no_sink[0, :20] - want[0, :20]).abs().max() > 0.3 * want.abs().max()  # (a sink left out shows)
    if dt == "bfloat16" and W % 8 == 0:  # the fp32 VALU kernel on the same operands
        again = torch.empty_like(got)
        fb = _FB(0, [n], list(range(n)), [0], dev, pf_bt=[table], pf_ctx=[n])
        LA.latent_attention(qa_all.float().to(md).to(dev), cache, LA.Ragged(fb), scale, again, impl=1, sink=sink.to(dev))
        close(again.float(), want, 2e-2)


@pytest.mark.parametrize("dev", DEVS)
def test_gate_per_number_and_per_head(dev):
    g = torch.Generator().manual_seed(6)
    H, T, dv = 3, 7, 10
    ov, gp = torch.randn(H, T, dv, generator=g), torch.randn(T, H * dv + 2, generator=g)
    flat = ov.double().permute(1, 0, 2).reshape(T, H * dv)
    for md, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        out = torch.empty(T, H * dv, device=dev, dtype=md)
        LA.head_gate_pack(ov.to(dev), gp.to(dev)[:, 2:], out)
        close(out.float(), flat * torch.sigmoid(gp.double()[:, 2:]), tol)
        LA.head_gate_pack(ov.to(dev), gp.to(dev)[:, 2:2 + H], out)
        close(out.float(), flat * torch.sigmoid(gp.double()[:, 2:2 + H]).repeat_interleave(dv, 1), tol)


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
@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_models_of_one_kind_of_layer(dev, dt, tol, kind):
    kw = dict(SHAPES["plain"], pattern=(kind,) * 3, kv_from={1: 0, 2: 0} if kind == "attention" else None, window=13,
              keep_first=2)
    cfg, tensors, model = build(dev, dt, seed=13, **kw)
    assert len(model.cache_ranks()) == (1 if kind == "attention" else 3)
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
    some beside single tokens of others; finished requests hand their pages on. Every request's logits equal those it
    gets alone."""
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
        # and the same request alone, in the same number format: no router tie falls differently here
        alone = run_cuts(eng, "alone-" + k, reqs[k], [len(reqs[k])])
        close(torch.cat(got[k]), alone, 2e-4 if dt == "float32" else 1e-2)
    assert eng.bm.num_free == eng.bm.num_blocks - 1 and len(eng.state_slots.free) == 3


@pytest.mark.parametrize("dev,dt,tol", RUNS)
def test_peaked_attention_far_keys_and_long_decode(dev, dt, tol):
    """Large score scales make single keys dominate, so a lost or shifted key anywhere in a long prompt (page borders,
    window edges, kept tokens, position 0) moves the logits; then 110 tokens decoded one by one, so that the window passes
    over decoded tokens only."""
    kw = dict(SHAPES["plain"], scale=1.5, l_scale=1.0, window={0: 50, 2: 90}, keep_first={0: 3, 2: 17})
    cfg, tensors, model = build(dev, dt, seed=21, **kw)
    t = toks(300, cfg.vocab, 8)
    want = oracle(cfg, tensors, t)
    eng = engine(model, max_tokens=304, seqs=2)
    got = run_cuts(eng, "x", t, [187, 3] + [1] * 110)
    close(got, want, tol * 2, rms=dt == "bfloat16")


@pytest.mark.parametrize("dev,dt,tol", RUNS)
@pytest.mark.parametrize("dim,vdim,heads,kv,rank,lrot", [(64, 128, 8, 2, 80, 48), (128, 64, 3, 1, 512, 64)])
def test_matrix_core_sizes_through_the_engine(dev, dt, tol, dim, vdim, heads, kv, rank, lrot):
    """Head sizes of 64 / 128 and latent rows of the matrix-core kernels: a prompt in portions that end inside 16-row
    tiles, decoded rows behind enough keys to be split into partitions."""
    kw = dict(hidden=128, vocab=211, pattern=("attention", "latent_attention", "attention"), kv_from={2: 0}, heads=heads,
              kv_heads=kv, dim=dim, vdim=vdim, scale=1.5 * dim ** -0.5, window=100, keep_first=6, rot_dims=dim // 2,
              rot_scaling=(2.0, 128.0, 16.0, 1.0), l_heads=6, l_dim=32, l_rot=lrot, l_vdim=24, kv_rank=rank,
              experts=4, top=2, groups=(2, 1), expert_ff=64, shared_ff=64, emb_scale=2.0)
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
        kind = rng.choice(["attention", "latent_attention"])
        pattern.append(kind)
        if kind == "attention":
            if owners and rng.random() < 0.4:
                kv_from[i] = rng.choice(owners)
            else:
                owners.append(i)
    kv, lrot = rng.choice([1, 2, 3]), rng.choice([2, 8, 16, 32])
    count = rng.choice([1, 2, 4])
    experts = count * rng.choice([1, 2, 3])
    keep = rng.randint(1, count)
    dim = rng.choice([16, 24, 32, 64])
    scaling = lambda: rng.choice([None, (2.0, 64.0, 8.0, 1.0), (16.0, 32.0, 4.0, 0.5), (1.5, 4096.0, 32.0, 1.0)])  # noqa: E731
    return dict(hidden=rng.choice([64, 96, 160]), vocab=rng.choice([97, 256, 1000]), pattern=tuple(pattern),
                kv_from=kv_from, heads=kv * rng.choice([1, 2, 3]), kv_heads=kv, dim=dim,
                vdim=rng.choice([16, 32, 64, 128]), scale=rng.choice([0.05, 0.1, 0.2]),
                window={i: rng.choice([0, 1, 5, 16, 40, 64, 130]) for i in range(nl)},
                keep_first={i: rng.choice([0, 1, 4, 16, 50]) for i in range(nl)}, rot_dims=rng.choice([0, 8, dim]),
                rot_base=rng.choice([100.0, 1e4, 1e6]), rot_scaling=scaling(), l_heads=rng.choice([1, 2, 5]),
                l_dim=rng.choice([8, 16, 40]), l_rot=lrot, l_vdim=rng.choice([8, 32, 48]),
                kv_rank=rng.choice([16, 33, 64, 160]), l_rot_base=rng.choice([100.0, 1e4]), l_rot_scaling=scaling(),
                mlps=tuple(rng.choice(["moe", "moe", None]) for _ in range(rng.randint(1, 3))), experts=experts,
                top=rng.randint(1, keep * (experts // count)), groups=(count, keep), expert_ff=rng.choice([16, 40]),
                limit=rng.choice([0.3, 1.0, 7.0]), shared_ff=rng.choice([0, 32, 96]), shared_limit=rng.choice([0.5, 4.0]),
                emb_scale=rng.choice([1.0, 6.0]), eps=rng.choice([1e-6, 1e-5]))


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("seed", [1, 2, 3])
def test_random_configurations_and_schedules(dev, seed):
    """Drawn sizes, layer orders, borrowed keys, windows and groups; five requests fed through four live slots in drawn
    portions (single tokens beside portions of up to 150, requests left out of steps, blocks handed on) in a pool that
    holds the four largest but not all five. fp32 only: every position agrees with the oracle."""
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
        close(torch.cat(got[k]), want[k], 2e-4)
    assert eng.bm.num_free == eng.bm.num_blocks - 1 and len(eng.state_slots.free) == 4


# ------------------------------------------------------------------------------------------------ serving path
@pytest.mark.parametrize("dev,dt", [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("native", [False, True])
def test_greedy_generation_through_the_scheduler(dev, dt, native):
    """engine.submit: chunked prefill, continuous batching of three requests, greedy sampling; each request's tokens
    equal the oracle's greedy continuation."""
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


@pytest.mark.parametrize("dev,dt", [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("native", [False, True])
def test_shared_prefix_reuses_pages(dev, dt, native):
    """Everything a sequence carries lies in its pages, so a prompt that begins like an earlier one takes that one's full
    pages over, window, kept tokens and latents alike; the tokens are those of a run from position 0."""
    cfg, tensors, model = build(dev, dt, seed=4, **SHAPES["plain"])
    ec = EngineConfig(max_num_seqs=2, max_batched_tokens=64, max_model_len=128, block_size=16, num_blocks=24,
                      use_graphs=False, native_scheduler=native, gemm_autotune=False, enable_prefix_cache=True)
    eng = LLMEngine(model, ByteTokenizer(cfg.vocab), ec)
    if native and not eng.native_sched:
        pytest.skip("native runtime not built")
    head = toks(40, cfg.vocab, 5)
    prompts = [head + toks(n, cfg.vocab, n) for n in (7, 3, 11)]
    got = []
    for p in prompts:
        h = eng.submit(Request(p, SamplingParams(temperature=0.0, ignore_eos=True), 8))
        eng.run_until_done()
        got.append([i for o in h for i in o.token_ids])
    assert eng.stats["cached_tokens_total"] == 2 * 32  # two full pages each for the second and third prompt
    for p, ids in zip(prompts, got):
        assert ids == greedy(cfg, tensors, p, 8)


@pytest.mark.gpu
def test_decode_graphs_replay_like_the_oracle():
    """Decode-only steps replay captured graphs (several buckets as requests come and go, eager prompt chunks
    between the replays); every request still yields the oracle's greedy tokens, also after pages were reused."""
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
    """The matrix-core decode kernels inside replayed graphs: many replays with the program's own work between them give
    the tokens of the eager engine (the same kernels, launched one by one)."""
    kw = dict(hidden=128, vocab=211, pattern=("attention", "latent_attention", "attention"), kv_from={2: 0}, heads=8,
              kv_heads=2, dim=64, vdim=64, window=40, keep_first=4, l_heads=5, l_dim=24, l_rot=16, l_vdim=40, kv_rank=80,
              experts=4, top=2, groups=(2, 1), expert_ff=64, shared_ff=64)
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
@pytest.mark.parametrize("prefix", [False, True])
def test_preempted_request_recomputes_its_pages(native, prefix):
    """A pool too small for both requests' growth: one is preempted, loses its blocks and is recomputed later, from
    position 0 or (prefix cache) from the full pages that are still cached; while it waits it must not hold on to those, or
    the other one could not grow. Both still produce the oracle's greedy tokens."""
    cfg, tensors, model = build("cpu", "float32", seed=8, **SHAPES["plain"])
    ec = EngineConfig(max_num_seqs=2, max_batched_tokens=64, max_model_len=128, block_size=16, num_blocks=8,
                      use_graphs=False, native_scheduler=native, gemm_autotune=False, enable_prefix_cache=prefix)
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
    cfg = ZO.make_config(**SHAPES["odd"])
    get = ZO.synthetic_source(cfg, 1)
    ZO.save_checkpoint(cfg, get, str(tmp_path))
    assert ZO.is_zomolix_dir(str(tmp_path))
    cfg2, get2 = ZO.dir_source(str(tmp_path))
    assert cfg2 == ZO.ZomolixConfig.from_json(cfg.to_json(), cfg2.name) and cfg2.to_json() == cfg.to_json()
    assert cfg2.layers[1].mlp is None and cfg2.layers[0].mlp.shared_ff is None and cfg2.layers[0].mlp.groups == (1, 1)
    assert cfg2.layers[1].mixer.window == 7 and cfg2.layers[2].mixer.window == 0 and cfg2.layers[0].mixer.rot.scaling is None
    assert torch.equal(get2("l1.mix.q"), get("l1.mix.q")) and get2("l1.norm2") is None and get2("l1.ls2") is None
    from localai_tfp_amd.models.loader import load_llm
    m, _tok, c, _ = load_llm(str(tmp_path), "cpu")
    assert isinstance(m, ZO.ZomolixModel) and c.layers[1].mixer.scale == 0.4
    assert m.cache_ranks() == [27, 3 * 64, 3 * 64]
    cfg3 = ZO.make_config(**SHAPES["plain"])
    j3 = cfg3.to_json()
    assert j3["layers"][2]["mixer"]["kv_from"] == 0 and j3["layers"][2]["mixer"]["mask"] == {"size": 11, "keep_first": 5}
    assert "l2.mix.k" not in ZO.tensor_shapes(cfg3) and ZO.tensor_shapes(cfg3)["l1.mix.dkv"] == (48, 64)
    assert [sorted(e) for e in ZO.ZomolixModel(cfg3).cache_spec()] == [["kv"], ["lat"], [], ["lat"]]
    for path, val in ((("layers", 0, "type"), "something_else"), (("layers", 1, "mlp", "kind"), "dense"),
                      (("layers", 2, "mixer", "kv_from"), 2), (("layers", 2, "mixer", "kv_from"), 1),
                      (("layers", 2, "mixer", "dim"), 8), (("layers", 0, "mixer", "kv_heads"), 3),
                      (("layers", 1, "mixer", "rot_dim"), 6), (("layers", 1, "mixer", "kv_rank"), 700),
                      (("layers", 0, "mixer", "rot", "dims"), 18), (("layers", 0, "mlp", "router", "top"), 5),
                      (("layers", 0, "mlp", "router", "groups", "count"), 3),
                      (("layers", 0, "mlp", "router", "groups", "keep"), 5)):
        bad = json.loads(json.dumps(j3))
        ZO.ZomolixConfig.from_json(bad)  # (valid until it is broken)
        node = bad
        for p in path[:-1]:
            node = node[p]
        node[path[-1]] = val
        with pytest.raises(ValueError):
            ZO.ZomolixConfig.from_json(bad)
    tensors = {k: get(k) for k in get.names}
    tensors["l1.mix.q"] = tensors["l1.mix.q"][:-1]
    with pytest.raises(ValueError):
        ZO.ZomolixModel.load(cfg, tensors.get, "cpu")
    m, _, c, _ = load_llm("synthetic:zomolix-tiny", "cpu")
    assert isinstance(m, ZO.ZomolixModel) and c.layers[2].mixer.kv_from == 0


def test_trace_runner_command_line(tmp_path):
    """bin/trace_run on a checkpoint directory: steps on stdin, one logits file per step that wants any."""
    cfg = ZO.make_config(**SHAPES["plain"])
    get = ZO.synthetic_source(cfg, 6)
    mdir, odir = str(tmp_path / "m"), str(tmp_path / "o")
    ZO.save_checkpoint(cfg, get, mdir)
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
    """The gRPC LLM worker loads a Zomolix checkpoint directory like any other model and streams a completion whose
    tokens are the oracle's greedy continuation (byte-level tokenizer: one token per prompt byte after BOS)."""
    from localai_tfp_amd.grpc import pb
    from localai_tfp_amd.grpc.client import BackendClient
    from localai_tfp_amd.grpc.server import AioServer
    from localai_tfp_amd.workers.llm import LLMServicer
    cfg = ZO.make_config(**dict(SHAPES["plain"], vocab=300))
    get = ZO.synthetic_source(cfg, 12)
    ZO.save_checkpoint(cfg, get, str(tmp_path))
    svc = LLMServicer(device="cpu")
    server = AioServer(svc, "127.0.0.1:0", max_workers=4)
    c = BackendClient(f"127.0.0.1:{server.port}")
    try:
        r = c.load_model(pb.ModelOptions(Model=str(tmp_path), ContextSize=256))
        assert r.success, r.message
        assert isinstance(svc.engine.model, ZO.ZomolixModel)
        o = pb.PredictOptions(Prompt="windows", Tokens=6, Temperature=0.0, IgnoreEOS=True)
        a = c.predict(o)
        chunks = list(c.predict_stream(o))
        assert a.tokens == 6 and b"".join(x.message for x in chunks) == a.message
        tok = svc.engine.tok
        seq = list(tok.encode("windows"))
        assert a.prompt_tokens == len(seq)
        want = greedy(cfg, {k: get(k) for k in get.names}, seq, 6)
        assert tok.decode(want).encode(errors="replace") == a.message or a.message == tok.decode(want).encode()
    finally:
        c.close()
        if svc.engine is not None:
            svc.engine.shutdown()
        server.stop()
