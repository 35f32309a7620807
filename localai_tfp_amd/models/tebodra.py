"""Tebodra: a pre-norm decoder with one factor on everything that enters the residual, whose layers draw their mixer from
three kinds:

    x  = embed[token]
    x += m * mixer(norm(x; norm1))
    x += m * ff(norm(x; norm2))                 (absent when the layer has no feed-forward)
    logits = head norm(x; final)                 norm(x; w) = x / sqrt(mean(x^2) + eps) * (1 + w)

Mixers (`type`):
  attention    softmax attention with grouped heads whose values ARE its keys: queries and keys pass a short causal
               convolution over time (no activation), the convolved keys serve as values, and then both are rotated
               (pairs (i, i + rot.dims / 2)). Scores are capped, softcap * tanh(s / softcap). Causal.
  attention_2  softmax attention inside fixed chunks of positions (i sees j <= i with i // size == j // size): queries and
               keys are RMS-normed over the whole projection, then rotated; a learned sink per head in the softmax
               denominator. A layer with `kv_from: j` has no key / value tensors and reads layer j's cached keys and values
               under its own mask.
  mlstm        matrix memory with exponential gates: per head S <- a S + c k v^T, n <- a n + c k, o = S^T q /
               (max(|n . q|, exp(-m)) + 1e-6), where a = exp(f + m_before - m), c = exp(i - m) and m = max(f + m_before, i)
               is carried beside S and n; o is unit-RMS-normed per head and multiplied by a weight.
All three multiply their heads' concatenation by sigmoid(W_g h), one gate per number, before the output projection.
Rotations may be scaled (`rot.scaling`): every frequency divided by `factor`, or, with `low`, `high` and `original`, only
those of long wavelengths, with a blend in between.
Feed-forward (`mlp.kind` = dense): W_down gelu(W_up h), the exact gelu.

How a layer maps onto launches (T rows of a ragged engine step; hin is the normed h, written by the add before it):

    y = hin W_in^T            every projection of the mixer stacked into ONE GEMM (fp32 out)
    attention:    convolution (+ carried inputs) + rotary + paged append of rotated and plain keys (one launch, and one for
                  the carried inputs of prompt chunks); masked attention (score cap, gates in its epilogue) -> cat
    attention_2:  whole-row norms + rotary + paged append (one launch); masked attention (chunk, sink, gates) -> cat
    mlstm:        gates and running maximum; state scan with the normaliser as one more column of the state; division +
                  head norm * weight * sigmoid(gate) -> cat
    o = cat W_o^T;  x += m * o, hin <- norm2(x)                                                         (one launch)
    y = hin W_up^T;  gelu -> cat;  o = cat W_down^T;  x += m * o, hin <- the next layer's norm1(x)      (two launches)

The engine sees `cache_kind = "hybrid"`: paged key / value pools for the attention layers that own keys, one state slot per
live sequence for the memories, their running maxima and the convolutions' last inputs (engine/kv_cache.py HybridCache).
`dtype` bf16: GEMM operands and the pools are bf16, everything between GEMMs fp32. `dtype` fp32: all fp32.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field

import torch

from ..ops import hybrid as HY
from ..ops.core import rope_inv_freq
from ..ops.dense import Dense

ARCH = "Tebodra"
NORMALISER_EPS = 1e-6  # added to the matrix memory's divisor


@dataclass
class RotCfg:
    dims: int = 0
    base: float = 10000.0
    scaling: tuple | None = None  # (factor,) or (factor, low, high, original)

    KEYS = ("factor", "low", "high", "original")

    @classmethod
    def from_json(cls, r) -> "RotCfg":
        if not r:
            return cls()
        s = r.get("scaling")
        keys = cls.KEYS if s and "original" in s else cls.KEYS[:1]
        return cls(int(r["dims"]), float(r["base"]), tuple(float(s[k]) for k in keys) if s else None)

    def to_json(self) -> dict | None:
        if not self.dims:
            return None
        d = {"dims": self.dims, "base": self.base}
        if self.scaling:
            d["scaling"] = dict(zip(self.KEYS, self.scaling))
        return d

    def table(self, device) -> torch.Tensor:
        """Frequency of every pair, fp32 [dims / 2]."""
        s = self.scaling
        if not self.dims:
            return torch.empty(0, dtype=torch.float32, device=device)
        if s is None:
            f, _ = rope_inv_freq(self.dims, self.base)
        elif len(s) == 1:
            f, _ = rope_inv_freq(self.dims, self.base, 1.0 / s[0], "linear")
        else:
            f, _ = rope_inv_freq(self.dims, self.base, llama3={
                "factor": s[0], "low_freq_factor": s[1], "high_freq_factor": s[2], "original_max_position_embeddings": s[3]})
        return f.to(device)


@dataclass
class SoftmaxCfg:
    """Both attention mixers: `tied` (values are the convolved keys, capped scores) or chunked with normed rows and sinks."""
    tied: bool
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: RotCfg
    conv: int = 0  # tied: taps
    softcap: float = 0.0  # tied; 0: none
    chunk: int = 0  # chunked; 0: plain causal
    kv_from: int | None = None


@dataclass
class MlstmCfg:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass
class TebodraLayerCfg:
    type: str  # attention | attention_2 | mlstm
    mixer: SoftmaxCfg | MlstmCfg
    ff: int | None  # None: no feed-forward


def _need(cond: bool, what: str):
    if not cond:
        raise ValueError(f"Tebodra configuration: {what}")


@dataclass
class TebodraConfig:
    name: str = "tebodra"
    arch: str = "tebodra"
    hidden: int = 256
    vocab: int = 512
    layers: list = field(default_factory=list)
    rms_eps: float = 1e-6
    residual_mult: float = 1.0
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
    def from_json(cls, d: dict, name: str = "tebodra") -> "TebodraConfig":
        if d.get("architecture") != ARCH:
            raise ValueError(f"not a {ARCH} configuration")
        layers = []
        for i, e in enumerate(d["layers"]):
            m = e["mixer"]
            if e["type"] in ("attention", "attention_2"):
                tied, src, rot = e["type"] == "attention", m.get("kv_from"), RotCfg.from_json(m.get("rot"))
                mixer = SoftmaxCfg(tied, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]),
                                   float(m["scale"]), rot, kv_from=None if src is None else int(src))
                if tied:
                    mixer.conv, mixer.softcap = int(m["conv"]), float(m.get("softcap") or 0.0)
                    _need(1 <= mixer.conv <= 16, f"layer {i}: 1 to 16 taps")
                    _need(mixer.vdim == mixer.dim, f"layer {i}: values that are keys have the keys' size")
                    _need(mixer.softcap >= 0, f"layer {i}: the score cap is positive")
                else:
                    mixer.chunk = int((m.get("mask") or {}).get("size") or 0)
                    _need(mixer.chunk >= 0, f"layer {i}: the chunk size is not negative")
                _need(mixer.heads % mixer.kv_heads == 0, f"layer {i}: heads are a multiple of kv_heads")
                _need(rot.dims % 2 == 0 and rot.dims <= mixer.dim, f"layer {i}: rot.dims even, at most dim")
                if src is not None:
                    j = mixer.kv_from
                    _need(0 <= j < i and layers[j].type != "mlstm" and layers[j].mixer.kv_from is None,
                          f"layer {i}: kv_from names an earlier attention layer with keys of its own")
                    o = layers[j].mixer
                    _need((o.kv_heads, o.dim, o.vdim) == (mixer.kv_heads, mixer.dim, mixer.vdim),
                          f"layer {i}: key / value sizes equal those of layer {j}")
            elif e["type"] == "mlstm":
                mixer = MlstmCfg(int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"]))
                _need(mixer.dim <= 256, f"layer {i}: memory rows of up to 256 numbers")
                _need(mixer.gate_cap > 0, f"layer {i}: gate_cap > 0")
            else:
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            f = e.get("mlp")
            if f is not None and f.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {f.get('kind')!r}")
            layers.append(TebodraLayerCfg(e["type"], mixer, None if f is None else int(f["ff"])))
        return cls(name=name, hidden=int(d["width"]), vocab=int(d["vocab"]), layers=layers,
                   rms_eps=float(d["norm"]["eps"]), residual_mult=float(d["residual_mult"]))

    def to_json(self) -> dict:
        ls = []
        for L in self.layers:
            m = L.mixer
            if L.type == "mlstm":
                mj = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "gate_cap": m.gate_cap}
            else:
                mj = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale}
                if m.rot.dims:
                    mj["rot"] = m.rot.to_json()
                if m.tied:
                    mj["conv"] = m.conv
                    if m.softcap:
                        mj["softcap"] = m.softcap
                elif m.chunk:
                    mj["mask"] = {"size": m.chunk}
                if m.kv_from is not None:
                    mj["kv_from"] = m.kv_from
            ls.append({"type": L.type, "mixer": mj, "mlp": None if L.ff is None else {"kind": "dense", "ff": L.ff}})
        return {"architecture": ARCH, "width": self.hidden, "vocab": self.vocab, "norm": {"eps": self.rms_eps},
                "residual_mult": self.residual_mult, "layers": ls}


def make_config(hidden=128, vocab=320, pattern=("attention_2", "mlstm", "attention"), heads=4, kv_heads=2, dim=32, vdim=32,
                scale=None, chunk=48, rot_dims=None, rot_base=10000.0, rot_factor=None, kv_from=None, t_heads=None,
                t_kv_heads=None, t_dim=None, t_scale=None, t_rot_dims=None, t_rot_base=10000.0, t_scaling=None, conv=4,
                softcap=50.0, m_heads=4, m_dim=32, m_vdim=32, gate_cap=15.0, mlps=("dense",), ff=256, residual_mult=0.5,
                eps=1e-6, name="tebodra") -> TebodraConfig:
    """A configuration whose i-th layer has mixer pattern[i] and feed-forward mlps[i % len(mlps)] ("dense" | None).
    heads .. rot_factor describe the chunked layers (`chunk` may be a map from the layer index, `rot_factor` is a linear
    scaling), t_* .. softcap the layers with values tied to keys (sizes as the chunked ones' when not given; `t_scaling` =
    (factor, low, high, original)), m_* and gate_cap the memories; `kv_from` maps a layer index to the layer whose keys and
    values it reads."""
    layers = []
    for i, t in enumerate(pattern):
        if t == "attention_2":
            rot = RotCfg(dim if rot_dims is None else rot_dims, float(rot_base),
                         (float(rot_factor),) if rot_factor else None)
            mixer = SoftmaxCfg(False, heads, kv_heads, dim, vdim, float(scale if scale is not None else dim ** -0.5), rot,
                               chunk=chunk[i] if isinstance(chunk, dict) else chunk, kv_from=(kv_from or {}).get(i))
        elif t == "attention":
            d = t_dim or dim
            rot = RotCfg(d if t_rot_dims is None else t_rot_dims, float(t_rot_base),
                         tuple(float(x) for x in t_scaling) if t_scaling else None)
            mixer = SoftmaxCfg(True, t_heads or heads, t_kv_heads or kv_heads, d, d,
                               float(t_scale if t_scale is not None else d ** -0.5), rot, conv=conv,
                               softcap=float(softcap or 0.0), kv_from=(kv_from or {}).get(i))
        else:
            mixer = MlstmCfg(m_heads, m_dim, m_vdim, float(gate_cap))
        layers.append(TebodraLayerCfg(t, mixer, None if mlps[i % len(mlps)] is None else ff))
    return TebodraConfig(name=name, hidden=hidden, vocab=vocab, layers=layers, rms_eps=eps,
                         residual_mult=float(residual_mult))


# sizes of the order of a 1B / 7B decoder (bench / synthetic checkpoints): a chunked layer, one that borrows its keys, a
# memory and a layer with values tied to keys in turn
_PAT = ("attention_2", "attention_2", "mlstm", "attention")
SYNTHETIC = {
    "tebodra-tiny": dict(hidden=144, vocab=352, pattern=("attention_2", "mlstm", "attention", "attention_2"), kv_from={3: 0},
                         mlps=("dense", None)),
    "tebodra-1b": dict(hidden=2048, vocab=32000, pattern=_PAT * 4, kv_from={i: i - 1 for i in range(1, 16, 4)}, heads=16,
                       kv_heads=4, dim=128, vdim=128, chunk=2048, rot_factor=2.0, rot_base=1e5, t_rot_dims=64,
                       t_rot_base=1e5, t_scaling=(8.0, 1.0, 4.0, 8192.0), softcap=50.0, m_heads=8, m_dim=128, m_vdim=256,
                       ff=8192, residual_mult=0.25),
    "tebodra-7b": dict(hidden=4096, vocab=32000, pattern=_PAT * 8, kv_from={i: i - 1 for i in range(1, 32, 4)}, heads=32,
                       kv_heads=8, dim=128, vdim=128, chunk=2048, rot_factor=2.0, rot_base=1e5, t_rot_dims=64,
                       t_rot_base=1e5, t_scaling=(8.0, 1.0, 4.0, 8192.0), softcap=50.0, m_heads=16, m_dim=128, m_vdim=256,
                       ff=14336, residual_mult=0.18),
}


@dataclass
class TebodraWeights:
    """Device tensors of one layer, with the column layout of its stacked GEMM."""
    norm1: torch.Tensor
    w_in: Dense
    w_o: Dense
    cols: dict  # name -> first column of the projection in the input GEMM's output
    n_in: int
    k_o: int
    freqs: torch.Tensor | None = None  # rotary frequencies, one per pair
    conv_w: torch.Tensor | None = None  # [taps, channels], queries first
    q_norm: torch.Tensor | None = None  # over the whole projection
    k_norm: torch.Tensor | None = None
    sink: torch.Tensor | None = None
    i_b: torch.Tensor | None = None
    f_b: torch.Tensor | None = None
    mix_norm: torch.Tensor | None = None
    norm2: torch.Tensor | None = None
    w_up: Dense | None = None
    w_down: Dense | None = None
    n_ff: int = 0  # rows of w_up, padded to whole 16-byte rows


class TebodraWorkspace:
    """Step scratch sized for the largest step; forward() only takes views (static addresses for graph capture)."""

    def __init__(self, model: "TebodraModel", max_tokens: int, max_seqs: int, logits_rows: int):
        cfg, dev, md = model.cfg, model.device, model.dtype
        T, C = max_tokens, cfg.hidden
        f32 = dict(dtype=torch.float32, device=dev)
        m16 = dict(dtype=md, device=dev)
        self.max_tokens, self.max_seqs = T, max_seqs
        self.logits_rows = R = max(max_seqs, logits_rows)
        Ws = list(model.weights.values())
        n_y = max([max(W.n_in, W.n_ff) for W in Ws] or [1])
        k_cat = max([max(W.k_o, W.n_ff) for W in Ws] or [1])
        att = [L.mixer for L in cfg.layers if L.type != "mlstm"]
        mem = [L.mixer for L in cfg.layers if L.type == "mlstm"]
        self.x = torch.empty((T, C), **f32)
        self.hin = torch.empty((T, C), **m16)
        self.y = torch.empty((T * n_y,), **f32)
        self.o = torch.empty((T, C), **f32)
        self.q = torch.empty((T * max([a.heads * a.dim for a in att] or [1]),), **m16)
        self.scan = torch.empty((T * max([r.heads * r.vdim for r in mem] or [1]),), **f32)
        n_h = max([r.heads for r in mem] or [1])
        self.decay, self.coef, self.floor, self.nq = (torch.empty((T * n_h,), **f32) for _ in range(4))
        self.cat = torch.zeros((T * k_cat,), **m16)  # zero: padded columns are read, never written
        self.hs = torch.empty((R, C), **m16)
        self.logits = torch.empty((R, cfg.vocab), **f32)
        rows = HY.DECODE_WAVES + max_seqs * max([a.heads for a in att] or [1])
        self.part_ml = torch.empty((rows, 2), **f32)
        self.part_o = torch.empty((rows, max([a.vdim for a in att] or [1])), **f32)


class TebodraModel:
    cache_kind = "hybrid"
    tp_size = 1
    n_kv = 1
    n_heads = 1

    def __init__(self, cfg: TebodraConfig, device="cpu", dtype=None):
        self.cfg = cfg
        self.device = torch.device(device)
        if dtype is None:
            dtype = torch.bfloat16 if self.device.type == "cuda" else torch.float32
        if self.device.type != "cuda":
            dtype = torch.float32  # the CPU plumbing path runs everything in fp32
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Tebodra runs in bfloat16 or float32")
        self.dtype = dtype
        # everything a sequence carries lies in its pages when no layer has a memory or a convolution longer than one tap
        self.pages_only = all(L.type == "attention_2" or (L.type == "attention" and L.mixer.conv == 1) for L in cfg.layers)
        self.weights: dict[int, TebodraWeights] = {}
        self.embed: torch.Tensor | None = None
        self.final_norm = None
        self.head: Dense | None = None
        self.last_hidden = None

    # ------------------------------------------------------------------ engine hooks
    def cache_spec(self) -> list:
        spec = []
        for L in self.cfg.layers:
            m, e = L.mixer, {}
            if L.type == "mlstm":  # one more column than values: the normaliser
                e = {"state": (m.heads, m.vdim + 1, m.dim), "peak": m.heads}
            else:
                if m.kv_from is None:
                    e["kv"] = (m.kv_heads * m.dim, m.kv_heads * m.vdim)
                if m.tied:
                    e["tails"] = (m.conv - 1, (m.heads + (m.kv_heads if m.kv_from is None else 0)) * m.dim)
            spec.append(e)
        return spec

    def make_cache(self, num_blocks: int, block_size: int, state_slots: int):
        from ..engine.kv_cache import HybridCache
        return HybridCache(self.cache_spec(), num_blocks, block_size, self.device, self.dtype, state_slots)

    def cache_ranks(self):
        """Pool numbers per token of every layer that owns keys and values."""
        from ..engine.kv_cache import HybridCache
        return HybridCache.pool_numbers(self.cache_spec())

    def make_workspace(self, max_tokens: int, max_seqs: int, logits_rows: int = 0, max_parts: int = 64):
        return TebodraWorkspace(self, max_tokens, max_seqs, logits_rows)

    def weight_bytes(self) -> int:
        n = self.embed.numel() * self.embed.element_size() + self.head.w.numel() * self.head.w.element_size()
        for W in self.weights.values():
            for t in [d.w for d in (W.w_in, W.w_o, W.w_up, W.w_down) if d is not None] + [W.conv_w]:
                if t is not None:
                    n += t.numel() * t.element_size()
        return n

    # ------------------------------------------------------------------ loading
    @classmethod
    def load(cls, cfg: TebodraConfig, get, device="cpu", dtype=None) -> "TebodraModel":
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

        def along_k(w):
            if w.shape[1] % 8:  # the padded columns of the operand are never written and stay zero
                w = torch.cat([w, torch.zeros(C, 8 - w.shape[1] % 8)], 1)
            return w

        for i, L in enumerate(cfg.layers):
            p, mx = f"l{i}.mix.", L.mixer
            H, dk, dv = mx.heads, mx.dim, mx.vdim
            kw = {}
            if L.type == "mlstm":
                sizes = [("q", H * dk), ("k", H * dk), ("v", H * dv), ("g", H * dv), ("i", H), ("f", H)]
                kw.update(i_b=f32(p + "i.b", (H,)), f_b=f32(p + "f.b", (H,)), mix_norm=f32(p + "norm", (H * dv,)))
            else:
                G, own = mx.kv_heads, mx.kv_from is None
                sizes = [("q", H * dk)] + ([("k", G * dk)] if own else [])
                kw["freqs"] = mx.rot.table(dev)
                if mx.tied:
                    conv = [t(p + n + ".conv", (r, mx.conv)) for n, r in sizes]
                    kw["conv_w"] = torch.cat(conv, 0).t().contiguous().to(dev)
                else:
                    kw.update(q_norm=f32(p + "q.norm", (H * dk,)), sink=f32(p + "sink", (H,)))
                    if own:
                        sizes.append(("v", G * dv))
                        kw["k_norm"] = f32(p + "k.norm", (G * dk,))
                sizes.append(("g", H * dv))
            w_in, cols, n_in = stack([(n, t(p + n, (r, C))) for n, r in sizes])
            w_o = along_k(t(p + "o", (C, H * dv)))
            if L.ff is not None:
                w_up, _, n_ff = stack([("up", t(f"l{i}.mlp.up", (L.ff, C)))])
                kw.update(norm2=f32(f"l{i}.norm2", (C,)), w_up=Dense(w_up, None, dev, md), n_ff=n_ff,
                          w_down=Dense(along_k(t(f"l{i}.mlp.down", (C, L.ff))), None, dev, md))
            m.weights[i] = TebodraWeights(norm1=f32(f"l{i}.norm1", (C,)), w_in=Dense(w_in, None, dev, md),
                                          w_o=Dense(w_o, None, dev, md), cols=cols, n_in=n_in, k_o=w_o.shape[1], **kw)
        m.embed = t("embed", (cfg.vocab, C)).to(md).contiguous().to(dev)
        m.final_norm = f32("final.norm", (C,))
        m.head = Dense(t("head", (cfg.vocab, C)), None, dev, md)
        return m

    # ------------------------------------------------------------------ forward
    def forward(self, fb, cache, ws: TebodraWorkspace) -> torch.Tensor:
        cfg = self.cfg
        T, eps, mult = fb.T, cfg.rms_eps, cfg.residual_mult
        if T > ws.max_tokens:
            raise ValueError(f"step of {T} tokens, workspace holds {ws.max_tokens}")
        b16 = self.dtype != torch.float32
        rag = HY.Ragged(fb)
        x, hin, o = ws.x[:T], ws.hin[:T], ws.o[:T]
        h32, h16 = (None, hin) if b16 else (hin, None)
        HY.embed_rows(self.embed, fb.tokens, x)
        if fb.embed_rows:
            for r0, e in fb.embed_rows:
                x[r0:r0 + e.shape[0]].copy_(e)
        n_run = len(cfg.layers) if fb.stop_layer is None else min(fb.stop_layer, len(cfg.layers))
        if n_run:
            HY.offset_rmsnorm(x, self.weights[0].norm1, eps, h32, h16)
        for li in range(n_run):
            L, W = cfg.layers[li], self.weights[li]
            nxt = self.weights[li + 1].norm1 if li + 1 < n_run else None  # the norm the next layer reads
            y = ws.y[:T * W.n_in].view(T, W.n_in)
            W.w_in.into(hin, y)
            cat = ws.cat[:T * W.k_o].view(T, W.k_o)
            if L.type == "mlstm":
                self._mlstm(L.mixer, W, y, rag, cache.state[li], cache.peak[li], ws, cat, eps)
            else:
                own = li if L.mixer.kv_from is None else L.mixer.kv_from
                self._attention(L.mixer, W, y, rag, cache.kv[own], cache.tails[li], ws, cat, eps)
            W.w_o.into(cat, o)
            HY.scale_add_norm(o, None, None, x, nxt if L.ff is None else W.norm2, eps, h32, h16, offset=1.0, mult=mult)
            if L.ff is None:
                continue
            y = ws.y[:T * W.n_ff].view(T, W.n_ff)
            W.w_up.into(hin, y)
            cat = ws.cat[:T * W.n_ff].view(T, W.n_ff)
            HY.glu(y, None, None, None, cat, act="gelu")  # (padded columns: gelu(0) = 0)
            W.w_down.into(cat, o)
            HY.scale_add_norm(o, None, None, x, nxt, eps, h32, h16, offset=1.0, mult=mult)
        if fb.stop_layer is not None:
            return x
        R = fb.logits_idx.numel()
        if R > ws.logits_rows:
            raise ValueError(f"{R} logit rows asked, workspace holds {ws.logits_rows}")
        hs = ws.hs[:R]
        HY.offset_rmsnorm(x, self.final_norm, eps, out32=None if b16 else hs, out16=hs if b16 else None,
                          rows=fb.logits_idx)
        if fb.want_hidden or fb.keep_hidden:
            if fb.want_hidden:
                return hs.float()
            self.last_hidden = hs.float()
        return self.head.into(hs, ws.logits[:R])

    def _attention(self, a: SoftmaxCfg, W, y, rag, kv, tails, ws, cat, eps):
        T = y.shape[0]
        H, G, dk, dv = a.heads, a.kv_heads, a.dim, a.vdim
        c, own = W.cols, a.kv_from is None
        q = ws.q[:T * H * dk].view(T, H * dk)
        col = lambda n, w: y[:, c[n]:c[n] + w] if n in c else None  # noqa: E731
        HY.row_rope_append(col("q", H * dk), col("k", G * dk), col("v", G * dv), rag, H, G, dk, dv, W.freqs, 1.0, q,
                           kv[0] if own else None, kv[1] if own else None, W.q_norm, W.k_norm, eps, W.conv_w, tails)
        HY.masked_attention(q, kv[0], kv[1], rag, H, G, dk, dv, a.scale, cat[:, :H * dv], chunk=a.chunk,
                            sink=False if a.tied else W.sink, softcap=a.softcap, gate=col("g", H * dv),
                            workspace=(ws.part_ml, ws.part_o), p32=True)

    def _mlstm(self, r: MlstmCfg, W, y, rag, state, peak, ws, cat, eps):
        T = y.shape[0]
        H, dk, dv = r.heads, r.dim, r.vdim
        c = W.cols
        nk, nv = H * dk, H * dv
        decay, coef, floor, nq = (b[:T * H].view(T, H) for b in (ws.decay, ws.coef, ws.floor, ws.nq))
        HY.mlstm_gates(y[:, c["i"]:c["i"] + H], y[:, c["f"]:c["f"] + H], W.i_b, W.f_b, r.gate_cap, peak, rag, decay, coef,
                       floor)
        o = ws.scan[:T * nv].view(T, nv)
        HY.state_scan(y[:, c["k"]:c["k"] + nk], y[:, c["q"]:c["q"] + nk], y[:, c["v"]:c["v"] + nv], decay, coef, None, state,
                      rag, o, H, H, dk, dv, delta=False, q_scale=dk ** -0.5, norm_out=nq)
        HY.gated_group_norm(o, y[:, c["g"]:c["g"] + nv], W.mix_norm, eps, dv, cat[:, :nv], gate_first=False, act="sigmoid",
                            den=nq, den_min=floor, den_eps=NORMALISER_EPS)


# ------------------------------------------------------------------------------------------------ sources
def is_tebodra_dir(path: str) -> bool:
    f = os.path.join(path, "config.json")
    if not (os.path.isdir(path) and os.path.isfile(f)):
        return False
    try:
        with open(f) as fh:
            return json.load(fh).get("architecture") == ARCH
    except (OSError, ValueError):
        return False


def dir_source(model_dir: str):
    """(TebodraConfig, get) of a directory holding config.json and model.safetensors."""
    from .vosotar import tensor_getter
    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = TebodraConfig.from_json(json.load(f), os.path.basename(os.path.normpath(model_dir)))
    return cfg, tensor_getter(model_dir)


def tensor_shapes(cfg: TebodraConfig) -> dict:
    """name -> shape of every checkpoint tensor of a configuration."""
    C = cfg.hidden
    s = {"embed": (cfg.vocab, C), "final.norm": (C,), "head": (cfg.vocab, C)}
    for i, L in enumerate(cfg.layers):
        p, m = f"l{i}.mix.", L.mixer
        nq, nv = m.heads * m.dim, m.heads * m.vdim
        s.update({f"l{i}.norm1": (C,), p + "q": (nq, C), p + "g": (nv, C), p + "o": (C, nv)})
        if L.type == "mlstm":
            s.update({p + "k": (nq, C), p + "v": (nv, C), p + "norm": (nv,), p + "i": (m.heads, C), p + "i.b": (m.heads,),
                      p + "f": (m.heads, C), p + "f.b": (m.heads,)})
        else:
            nk, own = m.kv_heads * m.dim, m.kv_from is None
            if own:
                s[p + "k"] = (nk, C)
            if m.tied:
                s[p + "q.conv"] = (nq, m.conv)
                if own:
                    s[p + "k.conv"] = (nk, m.conv)
            else:
                s.update({p + "q.norm": (nq,), p + "sink": (m.heads,)})
                if own:
                    s.update({p + "k.norm": (nk,), p + "v": (m.kv_heads * m.vdim, C)})
        if L.ff is not None:
            s.update({f"l{i}.norm2": (C,), f"l{i}.mlp.up": (L.ff, C), f"l{i}.mlp.down": (C, L.ff)})
    return s


def synthetic_source(cfg: TebodraConfig, seed: int = 0):
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
            if leaf in ("norm1", "norm2") or name == "final.norm":
                a = 0.1 * torch.randn(s, generator=g)
            elif leaf == "norm":
                a = 1.0 + 0.1 * torch.randn(s, generator=g)
            elif leaf == "sink":
                a = torch.randn(s, generator=g)
            elif leaf == "conv":
                a = torch.randn(s, generator=g) * (s[-1] ** -0.5)
            elif name.endswith(".f.b"):
                a = 3.0 + torch.randn(s, generator=g)  # forget gates near one, as a trained layer keeps them
            elif leaf == "b":
                a = torch.randn(s, generator=g)
            elif name == "embed":
                a = torch.randn(s, generator=g)
            else:
                a = torch.randn(s, generator=g) * (s[-1] ** -0.5)
            made[name] = a.to(torch.bfloat16)
        return made[name]
    get.names = order
    return get


def save_checkpoint(cfg: TebodraConfig, get, model_dir: str) -> None:
    """Write config.json + model.safetensors (bf16) of `get`'s tensors: the layout `dir_source` reads."""
    from safetensors.torch import save_file
    os.makedirs(model_dir, exist_ok=True)
    with open(os.path.join(model_dir, "config.json"), "w") as f:
        json.dump(cfg.to_json(), f, indent=1)
    save_file({k: get(k).contiguous() for k in get.names}, os.path.join(model_dir, "model.safetensors"))


def load_dir(model_dir: str, device="cpu", dtype=None) -> TebodraModel:
    cfg, get = dir_source(model_dir)
    return TebodraModel.load(cfg, get, device, dtype)
