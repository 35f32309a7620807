"""Zomolix: a pre-norm decoder with layer scales whose layers draw their mixer from two kinds, every layer with a mixture
of clamped gated experts behind it:

    x  = scale * embed[token]
    x += ls1 * mixer(rms_norm(x; norm1))
    x += ls2 * ff(rms_norm(x; norm2))                 (absent when the layer has no feed-forward)
    logits = head rms_norm(x; final)

Mixers (`type`):
  attention         softmax attention with grouped key / value heads, biases on all four projections, rotary positions on
                    the pairs (i, i + rot.dims / 2) of a head's first rot.dims numbers, and a sliding window that keeps
                    the sequence's first tokens: the token at position i sees j <= i with i - j < mask.size or
                    j < mask.keep_first. A layer with `kv_from: j` has no key / value tensors: it attends over layer j's
                    paged keys and values with its own queries and mask.
  latent_attention  per token one latent c = rms_norm(W_dkv h) of kv_rank numbers and one rotated key part of rot_dim
                    numbers shared by all heads. Head h's key is (W_uk c, rotated part), its value W_uv c; its query has an
                    unrotated part of `dim` numbers and a rotated one (pairs (2i, 2i + 1)). Causal, with a learned sink
                    per head in the softmax denominator; the heads' outputs are multiplied by sigmoid(W_g h), one gate per
                    number.
Rotations may be scaled (`rot.scaling`, YaRN): the frequencies of slow pairs are divided by `factor`, with a linear ramp
between the pairs that make `fast` and `slow` turns over `original` positions, and sine and cosine are multiplied by
0.1 ln(factor) + 1.
Feed-forward (`mlp.kind` = moe): scores = softmax over all experts in fp32; experts form groups.count equal groups of
neighbours and only those of the groups.keep groups with the largest best scores can be chosen; the `top` largest keep
their scores as weights. Experts and the always-on shared expert are W_down (g sigmoid(1.702 g) (u + 1)) with
g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit).

How a layer maps onto launches (T rows of a ragged engine step; hin is the normed h, written by the add before it):

    y = hin W_in^T            every projection that reads h stacked into ONE GEMM (fp32 out)
    attention:  bias + rotary + paged append (one launch); masked attention (window, kept first tokens) -> cat
    latent:     latent norm + rotary + paged append of (c, rotated key part) beside the split of the queries (one launch);
                qa = q U_k per head (batched GEMM into the first kv_rank columns of the absorbed queries); attention whose
                keys are the cached rows and whose values are their first kv_rank numbers; U_v per head (batched GEMM);
                gate + pack -> cat
    o = cat W_o^T;  x += ls1 * (o + b), hin <- norm2(x)                                                 (one launch)
    y = hin W_ff^T            router | shared gate, up | every expert's gate, up as ONE GEMM
    routing weights [T, E]; clamped unit (shared); clamped unit (experts, each times its routing weight) -> cat
    o = cat W_down^T          shared and experts stacked along K: the sum over experts is the GEMM's accumulator
    x += ls2 * o, hin <- the next layer's norm1(x)                                                      (one launch)

The engine sees `cache_kind = "hybrid"`: paged key / value pools for the attention layers that own keys and one paged pool
of latent rows per latent layer (engine/kv_cache.py HybridCache). Nothing else is carried (`pages_only`), so the prefix
cache may share blocks between requests.
`dtype` bf16: GEMM operands, absorbed queries and the pools are bf16, everything between GEMMs fp32. `dtype` fp32: all fp32.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field

import torch

from ..ops import hybrid as HY
from ..ops import latent as LA
from ..ops.core import rope_inv_freq
from ..ops.dense import Dense
from ..ops.dense import bmm_f32

ARCH = "Zomolix"
UNIT_ALPHA = 1.702  # slope of the experts' sigmoid


@dataclass
class RotCfg:
    dims: int = 0
    base: float = 10000.0
    scaling: tuple | None = None  # (factor, original, fast, slow)

    @classmethod
    def from_json(cls, r) -> "RotCfg":
        if not r:
            return cls()
        s = r.get("scaling")
        return cls(int(r["dims"]), float(r["base"]),
                   (float(s["factor"]), float(s["original"]), float(s["fast"]), float(s["slow"])) if s else None)

    def to_json(self) -> dict | None:
        if not self.dims:
            return None
        d = {"dims": self.dims, "base": self.base}
        if self.scaling:
            d["scaling"] = dict(zip(("factor", "original", "fast", "slow"), self.scaling))
        return d

    def tables(self, device):
        """(frequency of every pair fp32 [dims / 2], factor on sine and cosine)."""
        if not self.scaling:
            f, mag = rope_inv_freq(self.dims, self.base)
        else:
            factor, original, fast, slow = self.scaling
            f, mag = rope_inv_freq(self.dims, self.base, 1.0 / factor, "yarn", original, beta_fast=fast, beta_slow=slow)
        return f.to(device), mag


@dataclass
class WindowAttnCfg:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: RotCfg
    window: int = 0  # 0: plain causal
    keep_first: int = 0
    kv_from: int | None = None


@dataclass
class RotLatentCfg:
    heads: int
    dim: int  # unrotated query / key size per head
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot: RotCfg


@dataclass
class ClampedMoeCfg:
    ff: int
    limit: float
    experts: int
    top: int
    groups: tuple = (1, 1)  # (count, keep)
    shared_ff: int | None = None
    shared_limit: float = 0.0


@dataclass
class ZomolixLayerCfg:
    type: str  # attention | latent_attention
    mixer: WindowAttnCfg | RotLatentCfg
    mlp: ClampedMoeCfg | None


def _need(cond: bool, what: str):
    if not cond:
        raise ValueError(f"Zomolix configuration: {what}")


@dataclass
class ZomolixConfig:
    name: str = "zomolix"
    arch: str = "zomolix"
    hidden: int = 256
    vocab: int = 512
    layers: list = field(default_factory=list)
    rms_eps: float = 1e-6
    emb_scale: float = 1.0
    ctx_train: int = 1 << 20  # rotary angles are computed from the position: the engine's max_model_len is the limit
    extra: dict = field(default_factory=dict)
    # fields the engine / workers read off every model config
    head_dim: int = 1
    n_heads: int = 1
    n_kv_heads: int = 1
    embed_scale: float = 1.0
    tie_embeddings: bool = False

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_json(cls, d: dict, name: str = "zomolix") -> "ZomolixConfig":
        if d.get("architecture") != ARCH:
            raise ValueError(f"not a {ARCH} configuration")
        layers = []
        for i, e in enumerate(d["layers"]):
            m = e["mixer"]
            rot = RotCfg.from_json(m.get("rot"))
            _need(rot.dims % 2 == 0, f"layer {i}: rot.dims is even")
            if e["type"] == "attention":
                mask, src = m.get("mask") or {}, m.get("kv_from")
                mixer = WindowAttnCfg(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]),
                                      float(m["scale"]), rot, int(mask.get("size") or 0), int(mask.get("keep_first") or 0),
                                      None if src is None else int(src))
                if not mixer.window:
                    mixer.keep_first = 0  # everything is visible
                _need(mixer.heads % mixer.kv_heads == 0, f"layer {i}: heads are a multiple of kv_heads")
                _need(rot.dims <= mixer.dim, f"layer {i}: rot.dims at most dim")
                _need(mixer.window >= 0 and mixer.keep_first >= 0, f"layer {i}: window sizes are not negative")
                if mixer.kv_from is not None:
                    j = mixer.kv_from
                    _need(0 <= j < i and layers[j].type == "attention" and layers[j].mixer.kv_from is None,
                          f"layer {i}: kv_from names an earlier attention layer with keys of its own")
                    o = layers[j].mixer
                    _need((o.kv_heads, o.dim, o.vdim) == (mixer.kv_heads, mixer.dim, mixer.vdim),
                          f"layer {i}: key / value sizes equal those of layer {j}")
            elif e["type"] == "latent_attention":
                mixer = RotLatentCfg(int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]),
                                     float(m["scale"]), rot)
                _need(rot.dims == mixer.rot_dim, f"layer {i}: rot.dims equals rot_dim")
                _need(mixer.kv_rank + mixer.rot_dim <= 640, f"layer {i}: cached rows of up to 640 numbers")
            else:
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            f = e.get("mlp")
            if f is None:
                mlp = None
            elif f.get("kind") == "moe":
                r, sh, gr = f["router"], f.get("shared"), f["router"].get("groups")
                mlp = ClampedMoeCfg(int(f["expert"]["ff"]), float(f["expert"]["limit"]), int(r["experts"]), int(r["top"]),
                                    (int(gr["count"]), int(gr["keep"])) if gr else (1, 1),
                                    int(sh["ff"]) if sh else None, float(sh["limit"]) if sh else 0.0)
                n, k = mlp.groups
                _need(0 < mlp.top <= mlp.experts, f"layer {i}: 1 <= top <= experts")
                _need(n >= 1 and mlp.experts % n == 0 and 1 <= k <= n and mlp.top <= k * (mlp.experts // n),
                      f"layer {i}: equal groups, and enough experts in the kept ones")
            else:
                raise ValueError(f"layer {i}: unknown feed-forward {f.get('kind')!r}")
            layers.append(ZomolixLayerCfg(e["type"], mixer, mlp))
        return cls(name=name, hidden=int(d["width"]), vocab=int(d["vocab"]), layers=layers,
                   rms_eps=float(d["norm"]["eps"]), emb_scale=float((d.get("embedding") or {}).get("scale", 1.0)))

    def to_json(self) -> dict:
        ls = []
        for L in self.layers:
            m = L.mixer
            if L.type == "attention":
                mj = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale}
                if m.window:
                    mj["mask"] = {"size": m.window, "keep_first": m.keep_first}
                if m.kv_from is not None:
                    mj["kv_from"] = m.kv_from
            else:
                mj = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank,
                      "scale": m.scale}
            if m.rot.dims:
                mj["rot"] = m.rot.to_json()
            f, fj = L.mlp, None
            if f is not None:
                fj = {"kind": "moe", "expert": {"ff": f.ff, "limit": f.limit},
                      "router": {"experts": f.experts, "top": f.top}}
                if f.groups != (1, 1):
                    fj["router"]["groups"] = {"count": f.groups[0], "keep": f.groups[1]}
                if f.shared_ff:
                    fj["shared"] = {"ff": f.shared_ff, "limit": f.shared_limit}
            ls.append({"type": L.type, "mixer": mj, "mlp": fj})
        return {"architecture": ARCH, "width": self.hidden, "vocab": self.vocab, "norm": {"eps": self.rms_eps},
                "embedding": {"scale": self.emb_scale}, "layers": ls}


def make_config(hidden=128, vocab=320, pattern=("latent_attention", "attention"), heads=4, kv_heads=2, dim=32, vdim=32,
                scale=None, window=96, keep_first=3, rot_dims=None, rot_base=10000.0, rot_scaling=None, kv_from=None,
                l_heads=4, l_dim=16, l_rot=16, l_vdim=32, kv_rank=64, l_scale=None, l_rot_base=10000.0,
                l_rot_scaling=None, mlps=("moe",), experts=4, top=2, groups=(1, 1), expert_ff=128, limit=7.0, shared_ff=128,
                shared_limit=None, emb_scale=1.0, eps=1e-6, name="zomolix") -> ZomolixConfig:
    """A configuration whose i-th layer has mixer pattern[i] and feed-forward mlps[i % len(mlps)] ("moe" | None);
    `kv_from` maps a layer index to the attention layer whose keys and values it reads; `window` and `keep_first` may be
    maps from the layer index. Rotation scalings are (factor, original, fast, slow)."""
    per = lambda v, i: v[i] if isinstance(v, dict) else v  # noqa: E731
    layers = []
    for i, t in enumerate(pattern):
        if t == "attention":
            rot = RotCfg(dim if rot_dims is None else rot_dims, float(rot_base), rot_scaling)
            mixer = WindowAttnCfg(heads, kv_heads, dim, vdim, float(scale if scale is not None else dim ** -0.5), rot,
                                  per(window, i), per(keep_first, i) if per(window, i) else 0, (kv_from or {}).get(i))
        else:
            mixer = RotLatentCfg(l_heads, l_dim, l_rot, l_vdim, kv_rank,
                                 float(l_scale if l_scale is not None else (l_dim + l_rot) ** -0.5),
                                 RotCfg(l_rot, float(l_rot_base), l_rot_scaling))
        mlp = None if mlps[i % len(mlps)] is None else ClampedMoeCfg(
            expert_ff, float(limit), experts, top, tuple(groups), shared_ff or None,
            float(limit if shared_limit is None else shared_limit) if shared_ff else 0.0)
        layers.append(ZomolixLayerCfg(t, mixer, mlp))
    return ZomolixConfig(name=name, hidden=hidden, vocab=vocab, layers=layers, rms_eps=eps, emb_scale=float(emb_scale))


# sizes of the order of a 1B / 7B decoder (bench / synthetic checkpoints): windowed attention, a layer that borrows its
# keys, and two latent layers in turn
_PAT = ("latent_attention", "attention", "attention", "latent_attention")
SYNTHETIC = {
    "zomolix-tiny": dict(hidden=160, vocab=352, pattern=("attention", "latent_attention", "attention"), kv_from={2: 0},
                         groups=(2, 1)),
    "zomolix-1b": dict(hidden=2048, vocab=32000, pattern=_PAT * 4, kv_from={i: i - 1 for i in range(2, 16, 4)}, heads=16,
                       kv_heads=4, dim=128, vdim=128, window=1024, keep_first=16, rot_dims=64,
                       rot_scaling=(4.0, 8192.0, 32.0, 1.0), l_heads=16, l_dim=128, l_rot=64, l_vdim=128, kv_rank=512,
                       l_rot_scaling=(16.0, 4096.0, 32.0, 1.0), experts=8, top=2, groups=(4, 2), expert_ff=2048,
                       shared_ff=4096),
    "zomolix-7b": dict(hidden=4096, vocab=32000, pattern=_PAT * 8, kv_from={i: i - 1 for i in range(2, 32, 4)}, heads=32,
                       kv_heads=8, dim=128, vdim=128, window=1024, keep_first=16, rot_dims=64,
                       rot_scaling=(4.0, 8192.0, 32.0, 1.0), l_heads=32, l_dim=128, l_rot=64, l_vdim=128, kv_rank=512,
                       l_rot_scaling=(16.0, 4096.0, 32.0, 1.0), experts=8, top=2, groups=(4, 2), expert_ff=3584,
                       shared_ff=7168),
}


@dataclass
class ZomolixWeights:
    """Device tensors of one layer, with the column layout of its stacked GEMMs."""
    norm1: torch.Tensor
    ls1: torch.Tensor
    w_in: Dense
    w_o: Dense
    cols: dict  # name -> first column of the projection in the input GEMM's output
    n_in: int
    k_o: int
    freqs: torch.Tensor  # rotary frequencies, one per pair
    mag: float
    bias: dict = field(default_factory=dict)  # attention: q, k, v, o (fp32)
    dkv_norm: torch.Tensor | None = None
    uk: torch.Tensor | None = None  # [H, dim, rank]
    uvt: torch.Tensor | None = None  # [H, rank, vdim]
    sink: torch.Tensor | None = None
    norm2: torch.Tensor | None = None
    ls2: torch.Tensor | None = None
    w_ff: Dense | None = None
    w_down: Dense | None = None
    ff_cols: dict | None = None
    n_ff: int = 0
    k_down: int = 0


class ZomolixWorkspace:
    """Step scratch sized for the largest step; forward() only takes views (static addresses for graph capture)."""

    def __init__(self, model: "ZomolixModel", max_tokens: int, max_seqs: int, logits_rows: int, max_parts: int = 64):
        cfg, dev, md = model.cfg, model.device, model.dtype
        T, C = max_tokens, cfg.hidden
        f32 = dict(dtype=torch.float32, device=dev)
        m16 = dict(dtype=md, device=dev)
        self.max_tokens, self.max_seqs = T, max_seqs
        self.logits_rows = S = max(max_seqs, logits_rows)
        Ws = list(model.weights.values())
        n_y = max(max(W.n_in, W.n_ff) for W in Ws)
        k_cat = max(max(W.k_o, W.k_down) for W in Ws)
        att = [L.mixer for L in cfg.layers if L.type == "attention"]
        lat = [L.mixer for L in cfg.layers if L.type == "latent_attention"]
        n_q = max([m.heads * m.dim for m in att + lat])
        n_e = max([L.mlp.experts for L in cfg.layers if L.mlp is not None] or [1])
        self.x = torch.empty((T, C), **f32)
        self.hin = torch.empty((T, C), **m16)
        self.y = torch.empty((T * n_y,), **f32)
        self.o = torch.empty((T, C), **f32)
        self.q = torch.empty((T * n_q,), **m16)
        self.qa = torch.empty((T * max([m.heads * (m.kv_rank + m.rot_dim) for m in lat] or [1]),), **m16)
        self.ol = torch.empty((T * max([m.heads * m.kv_rank for m in lat] or [1]),), **m16)
        self.ov = torch.empty((T * max([m.heads * m.vdim for m in lat] or [1]),), **f32)
        self.cat = torch.zeros((T * k_cat,), **m16)  # zero: padded columns are read, never written
        self.route = torch.empty((T * n_e,), **f32)
        self.hs = torch.empty((S, C), **m16)
        self.logits = torch.empty((S, cfg.vocab), **f32)
        # partial results of decode rows whose visible keys are split into partitions (one layer at a time)
        rows = 1
        if att:
            rows = HY.DECODE_WAVES + max_seqs * max(a.heads for a in att)
        if lat:
            rows = max(rows, max(m.heads for m in lat) * max(max_seqs * max_parts, 256))
        self.part_ml = torch.empty((rows, 2), **f32)
        self.part_o = torch.empty((rows * max([a.vdim for a in att] + [m.kv_rank for m in lat]),), **f32)

    def parts(self, n: int):
        """(maxima and sums, unnormalised outputs of n numbers) of the decode partitions."""
        return self.part_ml, self.part_o[:self.part_ml.shape[0] * n].view(-1, n)


class ZomolixModel:
    cache_kind = "hybrid"
    pages_only = True  # everything a sequence carries lies in its pages
    tp_size = 1
    n_kv = 1
    n_heads = 1

    def __init__(self, cfg: ZomolixConfig, device="cpu", dtype=None):
        self.cfg = cfg
        self.device = torch.device(device)
        if dtype is None:
            dtype = torch.bfloat16 if self.device.type == "cuda" else torch.float32
        if self.device.type != "cuda":
            dtype = torch.float32  # the CPU plumbing path runs everything in fp32
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Zomolix runs in bfloat16 or float32")
        self.dtype = dtype
        self.weights: dict[int, ZomolixWeights] = {}
        self.embed: torch.Tensor | None = None
        self.final_norm = None
        self.head: Dense | None = None
        self.last_hidden = None

    # ------------------------------------------------------------------ engine hooks
    def cache_spec(self) -> list:
        spec = []
        for L in self.cfg.layers:
            m = L.mixer
            if L.type == "latent_attention":
                spec.append({"lat": m.kv_rank + m.rot_dim})
            else:
                spec.append({} if m.kv_from is not None else {"kv": (m.kv_heads * m.dim, m.kv_heads * m.vdim)})
        return spec

    def make_cache(self, num_blocks: int, block_size: int, state_slots: int):
        from ..engine.kv_cache import HybridCache
        return HybridCache(self.cache_spec(), num_blocks, block_size, self.device, self.dtype, state_slots)

    def cache_ranks(self):
        """Pool numbers per token of every layer that keeps something per token."""
        from ..engine.kv_cache import HybridCache
        return HybridCache.pool_numbers(self.cache_spec())

    def make_workspace(self, max_tokens: int, max_seqs: int, logits_rows: int = 0, max_parts: int = 64):
        return ZomolixWorkspace(self, max_tokens, max_seqs, logits_rows, max_parts)

    def weight_bytes(self) -> int:
        n = self.embed.numel() * self.embed.element_size() + self.head.w.numel() * self.head.w.element_size()
        for W in self.weights.values():
            for t in [d.w for d in (W.w_in, W.w_o, W.w_ff, W.w_down) if d is not None] + [W.uk, W.uvt]:
                if t is not None:
                    n += t.numel() * t.element_size()
        return n

    # ------------------------------------------------------------------ loading
    @classmethod
    def load(cls, cfg: ZomolixConfig, get, device="cpu", dtype=None) -> "ZomolixModel":
        """`get(name)` -> torch tensor (any float dtype) of the checkpoint tensor `name`."""
        m = cls(cfg, device, dtype)
        dev, md = m.device, m.dtype
        C = cfg.hidden

        def t(name, shape):
            a = get(name)
            if a is None:
                raise KeyError(f"checkpoint has no tensor {name!r}")
            if tuple(a.shape) != tuple(shape):
                raise ValueError(f"{name}: shape {tuple(a.shape)}, configuration says {tuple(shape)}")
            return a.float()

        def f32(name, shape):
            return t(name, shape).contiguous().to(dev)

        def stack(parts):
            """[(key, weight)] -> (weight rows padded to whole 16-byte rows, first column of each key, row count)."""
            cols, n = {}, 0
            for key, w in parts:
                cols[key] = n
                n += w.shape[0]
            w = torch.cat([w for _, w in parts], 0)
            if n % 8:
                w = torch.cat([w, torch.zeros(8 - n % 8, C)], 0)
            return w, cols, w.shape[0]

        def along_k(outs):
            w = torch.cat(outs, 1)
            if w.shape[1] % 8:  # the padded columns of the operand are never written and stay zero
                w = torch.cat([w, torch.zeros(C, 8 - w.shape[1] % 8)], 1)
            return w

        for i, L in enumerate(cfg.layers):
            p, mx = f"l{i}.mix.", L.mixer
            H, dk, dv = mx.heads, mx.dim, mx.vdim
            kw = {}
            if L.type == "attention":
                G = mx.kv_heads
                sizes = [("q", H * dk)] + ([("k", G * dk), ("v", G * dv)] if mx.kv_from is None else [])
                parts = [(n, t(p + n, (r, C))) for n, r in sizes]
                kw["bias"] = {n: f32(p + n + ".b", (r,)) for n, r in sizes + [("o", C)]}
            else:
                R, rot = mx.kv_rank, mx.rot_dim
                parts = [("q", t(p + "q", (H * (dk + rot), C))), ("dkv", t(p + "dkv", (R + rot, C))),
                         ("g", t(p + "g", (H * dv, C)))]
                uk = t(p + "uk", (H * dk, R)).reshape(H, dk, R)
                uv = t(p + "uv", (H * dv, R)).reshape(H, dv, R)
                kw.update(dkv_norm=f32(p + "dkv.norm", (R,)), sink=f32(p + "sink", (H,)),
                          uk=uk.to(dev).to(md).contiguous(), uvt=uv.transpose(1, 2).to(dev).to(md).contiguous())
            w_in, cols, n_in = stack(parts)
            w_o = along_k([t(p + "o", (C, H * dv))])
            freqs, mag = mx.rot.tables(dev)
            f, q = L.mlp, f"l{i}.mlp."
            if f is not None:
                fparts, outs = [("router", t(q + "router", (f.experts, C)))], []
                if f.shared_ff:
                    fparts += [("sgate", t(q + "shared.gate", (f.shared_ff, C))),
                               ("sup", t(q + "shared.up", (f.shared_ff, C)))]
                    outs.append(t(q + "shared.down", (C, f.shared_ff)))
                fparts += [("egate", torch.cat([t(f"{q}e{e}.gate", (f.ff, C)) for e in range(f.experts)], 0)),
                           ("eup", torch.cat([t(f"{q}e{e}.up", (f.ff, C)) for e in range(f.experts)], 0))]
                outs += [t(f"{q}e{e}.down", (C, f.ff)) for e in range(f.experts)]
                w_ff, ff_cols, n_ff = stack(fparts)
                w_down = along_k(outs)
                kw.update(norm2=f32(f"l{i}.norm2", (C,)), ls2=f32(f"l{i}.ls2", (C,)), w_ff=Dense(w_ff, None, dev, md),
                          w_down=Dense(w_down, None, dev, md), ff_cols=ff_cols, n_ff=n_ff, k_down=w_down.shape[1])
            m.weights[i] = ZomolixWeights(norm1=f32(f"l{i}.norm1", (C,)), ls1=f32(f"l{i}.ls1", (C,)),
                                          w_in=Dense(w_in, None, dev, md), w_o=Dense(w_o, None, dev, md), cols=cols,
                                          n_in=n_in, k_o=w_o.shape[1], freqs=freqs, mag=mag, **kw)
        m.embed = t("embed", (cfg.vocab, C)).to(md).contiguous().to(dev)
        m.final_norm = f32("final.norm", (C,))
        m.head = Dense(t("head", (cfg.vocab, C)), None, dev, md)
        return m

    # ------------------------------------------------------------------ forward
    def forward(self, fb, cache, ws: ZomolixWorkspace) -> torch.Tensor:
        cfg = self.cfg
        T, C, eps = fb.T, cfg.hidden, cfg.rms_eps
        if T > ws.max_tokens:
            raise ValueError(f"step of {T} tokens, workspace holds {ws.max_tokens}")
        b16 = self.dtype != torch.float32
        rag = HY.Ragged(fb)
        x, hin, o = ws.x[:T], ws.hin[:T], ws.o[:T]
        h32, h16 = (None, hin) if b16 else (hin, None)
        HY.embed_rows(self.embed, fb.tokens, x, scale=cfg.emb_scale)
        if fb.embed_rows:
            for r0, e in fb.embed_rows:
                x[r0:r0 + e.shape[0]].copy_(e)
        n_run = len(cfg.layers) if fb.stop_layer is None else min(fb.stop_layer, len(cfg.layers))
        if n_run:
            HY.offset_rmsnorm(x, self.weights[0].norm1, eps, h32, h16, offset=0.0)
        for li in range(n_run):
            L, W = cfg.layers[li], self.weights[li]
            nxt = self.weights[li + 1].norm1 if li + 1 < n_run else None  # the norm the next layer reads
            y = ws.y[:T * W.n_in].view(T, W.n_in)
            W.w_in.into(hin, y)
            cat = ws.cat[:T * W.k_o].view(T, W.k_o)
            if L.type == "attention":
                own = li if L.mixer.kv_from is None else L.mixer.kv_from
                self._attention(L.mixer, W, y, fb, rag, cache.kv[own], ws, cat, eps)
            else:
                self._latent(L.mixer, W, y, fb, rag, cache.lat[li], ws, cat, eps)
            W.w_o.into(cat, o)
            f = L.mlp
            HY.scale_add_norm(o, W.bias.get("o"), W.ls1, x, nxt if f is None else W.norm2, eps, h32, h16)
            if f is None:
                continue
            c, E = W.ff_cols, f.experts
            y = ws.y[:T * W.n_ff].view(T, W.n_ff)
            W.w_ff.into(hin, y)
            cat = ws.cat[:T * W.k_down].view(T, W.k_down)
            Fs, k1 = f.shared_ff or 0, E * f.ff
            if Fs:
                HY.glu(y[:, c["sgate"]:c["sgate"] + Fs], y[:, c["sup"]:c["sup"] + Fs], None, None, cat[:, :Fs],
                       act="clamped", limit=f.shared_limit, alpha=UNIT_ALPHA)
            rw = ws.route[:T * E].view(T, E)
            HY.moe_route(y[:, c["router"]:c["router"] + E], f.top, 1.0, rw, 0.0, mode="scores", groups=f.groups)
            HY.glu(y[:, c["egate"]:c["egate"] + k1], y[:, c["eup"]:c["eup"] + k1], None, None, cat[:, Fs:Fs + k1],
                   scale=rw, group=f.ff, act="clamped", limit=f.limit, alpha=UNIT_ALPHA)
            W.w_down.into(cat, o)
            HY.scale_add_norm(o, None, W.ls2, x, nxt, eps, h32, h16)
        if fb.stop_layer is not None:
            return x
        S = fb.logits_idx.numel()
        if S > ws.logits_rows:
            raise ValueError(f"{S} logit rows asked, workspace holds {ws.logits_rows}")
        hs = ws.hs[:S]
        HY.offset_rmsnorm(x, self.final_norm, eps, out32=None if b16 else hs, out16=hs if b16 else None,
                          rows=fb.logits_idx, offset=0.0)
        if fb.want_hidden or fb.keep_hidden:
            if fb.want_hidden:
                return hs.float()
            self.last_hidden = hs.float()
        return self.head.into(hs, ws.logits[:S])

    def _attention(self, a: WindowAttnCfg, W, y, fb, rag, kv, ws, cat, eps):
        T = y.shape[0]
        H, G, dk, dv = a.heads, a.kv_heads, a.dim, a.vdim
        c, b = W.cols, W.bias
        q = ws.q[:T * H * dk].view(T, H * dk)
        own = a.kv_from is None
        HY.rope_norm_append(y[:, c["q"]:c["q"] + H * dk], y[:, c["k"]:c["k"] + G * dk] if own else None,
                            y[:, c["v"]:c["v"] + G * dv] if own else None, fb.positions, H, G, dk, dv, a.rot.dims,
                            a.rot.base, False, eps, q, kv[0] if own else None, kv[1] if own else None, fb.slots, half=True,
                            freqs=W.freqs, mag=W.mag, q_bias=b["q"], k_bias=b.get("k"), v_bias=b.get("v"))
        HY.masked_attention(q, kv[0], kv[1], rag, H, G, dk, dv, a.scale, cat[:, :H * dv], window=a.window,
                            keep=a.keep_first, workspace=ws.parts(dv))

    def _latent(self, m: RotLatentCfg, W, y, fb, rag, lat, ws, cat, eps):
        T = y.shape[0]
        H, d, dv, R, rot = m.heads, m.dim, m.vdim, m.kv_rank, m.rot_dim
        c = W.cols
        q = ws.q[:T * H * d].view(T, H * d)
        qa = ws.qa[:H * T * (R + rot)].view(H, T, R + rot)
        LA.latent_rope_append(y[:, c["q"]:c["q"] + H * (d + rot)], y[:, c["dkv"]:c["dkv"] + R + rot], H, d, rot, R,
                              W.dkv_norm, eps, W.freqs, W.mag, fb.positions, q, qa, lat, fb.slots)
        torch.bmm(q.view(T, H, d).transpose(0, 1), W.uk, out=qa[:, :, :R])
        ol = ws.ol[:H * T * R].view(H, T, R)
        LA.latent_attention(qa, lat, rag, m.scale, ol, workspace=ws.parts(R), sink=W.sink,
                            part_len=LA.decode_part_len(rag.n_dec, H, rag.dec_max_len) if rag.n_dec else 0)
        ov = ws.ov[:H * T * dv].view(H, T, dv)
        bmm_f32(ol, W.uvt, ov)
        LA.head_gate_pack(ov, y[:, c["g"]:c["g"] + H * dv], cat[:, :H * dv])


# ------------------------------------------------------------------------------------------------ sources
def is_zomolix_dir(path: str) -> bool:
    f = os.path.join(path, "config.json")
    if not (os.path.isdir(path) and os.path.isfile(f)):
        return False
    try:
        with open(f) as fh:
            return json.load(fh).get("architecture") == ARCH
    except (OSError, ValueError):
        return False


def dir_source(model_dir: str):
    """(ZomolixConfig, get) of a directory holding config.json and model.safetensors."""
    from .vosotar import tensor_getter
    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = ZomolixConfig.from_json(json.load(f), os.path.basename(os.path.normpath(model_dir)))
    return cfg, tensor_getter(model_dir)


def tensor_shapes(cfg: ZomolixConfig) -> dict:
    """name -> shape of every checkpoint tensor of a configuration."""
    C = cfg.hidden
    s = {"embed": (cfg.vocab, C), "final.norm": (C,), "head": (cfg.vocab, C)}
    for i, L in enumerate(cfg.layers):
        p, m = f"l{i}.mix.", L.mixer
        H = m.heads
        s.update({f"l{i}.norm1": (C,), f"l{i}.ls1": (C,), p + "o": (C, H * m.vdim)})
        if L.type == "attention":
            rows = {"q": H * m.dim}
            if m.kv_from is None:
                rows.update(k=m.kv_heads * m.dim, v=m.kv_heads * m.vdim)
            for n, r in rows.items():
                s.update({p + n: (r, C), p + n + ".b": (r,)})
            s[p + "o.b"] = (C,)
        else:
            s.update({p + "q": (H * (m.dim + m.rot_dim), C), p + "dkv": (m.kv_rank + m.rot_dim, C),
                      p + "dkv.norm": (m.kv_rank,), p + "uk": (H * m.dim, m.kv_rank), p + "uv": (H * m.vdim, m.kv_rank),
                      p + "sink": (H,), p + "g": (H * m.vdim, C)})
        f, q = L.mlp, f"l{i}.mlp."
        if f is not None:
            s.update({f"l{i}.norm2": (C,), f"l{i}.ls2": (C,), q + "router": (f.experts, C)})
            for e in range(f.experts):
                s.update({f"{q}e{e}.gate": (f.ff, C), f"{q}e{e}.up": (f.ff, C), f"{q}e{e}.down": (C, f.ff)})
            if f.shared_ff:
                s.update({q + "shared.gate": (f.shared_ff, C), q + "shared.up": (f.shared_ff, C),
                          q + "shared.down": (C, f.shared_ff)})
    return s


def synthetic_source(cfg: ZomolixConfig, seed: int = 0):
    """Random weights (bf16-representable) under the checkpoint's tensor names, made on first use."""
    made: dict = {}
    sh = tensor_shapes(cfg)
    order = sorted(sh)

    def get(name):
        if name not in sh:
            return None
        if name not in made:
            g = torch.Generator().manual_seed(seed * 1000003 + order.index(name))
            s = sh[name]
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm1", "norm2", "norm"):
                a = 1.0 + 0.1 * torch.randn(s, generator=g)
            elif leaf in ("ls1", "ls2"):
                a = 0.5 + 0.1 * torch.randn(s, generator=g)
            elif leaf == "sink":
                a = torch.randn(s, generator=g)
            elif leaf == "b":
                a = 0.5 * torch.randn(s, generator=g)
            elif leaf == "router":
                a = 2.0 * torch.randn(s, generator=g) * (s[-1] ** -0.5)
            elif name == "embed":
                a = torch.randn(s, generator=g)
            else:
                a = torch.randn(s, generator=g) * (s[-1] ** -0.5)
            made[name] = a.to(torch.bfloat16)
        return made[name]
    get.names = order
    return get


def save_checkpoint(cfg: ZomolixConfig, get, model_dir: str) -> None:
    """Write config.json + model.safetensors (bf16) of `get`'s tensors: the layout `dir_source` reads."""
    from safetensors.torch import save_file
    os.makedirs(model_dir, exist_ok=True)
    with open(os.path.join(model_dir, "config.json"), "w") as f:
        json.dump(cfg.to_json(), f, indent=1)
    save_file({k: get(k).contiguous() for k in get.names}, os.path.join(model_dir, "model.safetensors"))


def load_dir(model_dir: str, device="cpu", dtype=None) -> ZomolixModel:
    cfg, get = dir_source(model_dir)
    return ZomolixModel.load(cfg, get, device, dtype)
