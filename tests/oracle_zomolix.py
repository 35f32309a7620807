"""Plain float64 whole-sequence oracle of the Zomolix decoder, one function per mechanism, written from the model's
equations and sharing no code with the package. `forward(config dict, get, tokens)` -> logits [T, vocab]; `get(name)`
returns a checkpoint tensor. Everything is recomputed from position 0 for every call: no cache, no pages, and the latent
layers build every head's keys and values instead of absorbing the projections into the query."""
import math

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.to(F64)


def frequencies(rot):
    """([dims / 2] angles per position, factor on cos and sin) of a `rot` entry, with or without frequency scaling."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return torch.tensor(f, dtype=F64), 1.0

    def turns(t):  # the (fractional) dimension whose pair makes t turns over the original length
        return dims * math.log(s["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(turns(s["fast"])), 0), min(math.ceil(turns(s["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = (i - lo) / max(hi - lo, 0.001)
        r = 0.0 if r < 0.0 else 1.0 if r > 1.0 else r
        out.append(fi / s["factor"] * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, rot, interleaved, positions=None):
    """x [T, heads, d]: turns the pairs of the first rot.dims numbers of every head, (2i, 2i + 1) when interleaved, else
    (i, i + dims / 2), by the row's position (0, 1, .. when not given)."""
    if not rot or not rot["dims"]:
        return x
    n = rot["dims"] // 2
    f, mag = frequencies(rot)
    p = torch.arange(x.shape[0], dtype=F64) if positions is None else torch.as_tensor(positions, dtype=F64)
    out = x.clone()
    for i in range(n):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + n)
        c, s = (torch.cos(p * f[i]) * mag)[:, None], (torch.sin(p * f[i]) * mag)[:, None]
        out[:, :, a] = x[:, :, a] * c - x[:, :, b] * s
        out[:, :, b] = x[:, :, b] * c + x[:, :, a] * s
    return out


def visible(i, mask):
    """Key positions the query at position i attends to."""
    if not mask or not mask.get("size"):
        return list(range(i + 1))
    return [j for j in range(i + 1) if i - j < mask["size"] or j < mask.get("keep_first", 0)]


def softmax_rows(q, k, v, scale, mask=None, sink=None):
    """One head: q, k [T, d], v [T, e]; `sink` is one more score in the denominator, without a value."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F64)
    for i in range(q.shape[0]):
        js = visible(i, mask)
        s = (k[js] @ q[i]) * scale
        m = s.max() if sink is None else torch.maximum(s.max(), sink)
        e = torch.exp(s - m)
        den = e.sum() + (0.0 if sink is None else torch.exp(sink - m))
        out[i] = (e / den) @ v[js]
    return out


def grouped_attention(q, k, v, scale, mask):
    """q [T, H, d], k [T, G, d], v [T, G, e]: head h reads key / value head h // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    return torch.stack([softmax_rows(q[:, h], k[:, h // (H // G)], v[:, h // (H // G)], scale, mask)
                        for h in range(H)], 1)


def attention_mixer(m, get, p, h, kv_of):
    """`kv_of`: layer index -> (rotated keys, values) of the attention layers run so far."""
    T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def proj(n):
        return h @ get(p + "mix." + n).to(F64).T + get(p + "mix." + n + ".b").to(F64)
    q = rotate(proj("q").reshape(T, H, d), m.get("rot"), False)
    src = m.get("kv_from")
    if src is None:
        k, v = rotate(proj("k").reshape(T, G, d), m.get("rot"), False), proj("v").reshape(T, G, e)
    else:
        k, v = kv_of[src]
    o = grouped_attention(q, k, v, m["scale"], m.get("mask")).reshape(T, H * e)
    return o @ get(p + "mix.o").to(F64).T + get(p + "mix.o.b").to(F64), (k, v)


def latent_mixer(m, get, p, h, eps):
    T, H, d, r, e, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    w = lambda n: get(p + "mix." + n).to(F64)  # noqa: E731
    q = (h @ w("q").T).reshape(T, H, d + r)
    qr = rotate(q[:, :, d:], m["rot"], True)
    down = h @ w("dkv").T
    c = rms_norm(down[:, :R], w("dkv.norm"), eps)
    kr = rotate(down[:, R:].reshape(T, 1, r), m["rot"], True)[:, 0]
    kn, v = (c @ w("uk").T).reshape(T, H, d), (c @ w("uv").T).reshape(T, H, e)
    heads = [softmax_rows(torch.cat([q[:, i, :d], qr[:, i]], 1), torch.cat([kn[:, i], kr], 1), v[:, i], m["scale"],
                          sink=w("sink")[i]) for i in range(H)]
    o = torch.cat(heads, 1) * torch.sigmoid(h @ w("g").T)
    return o @ w("o").T


def clamped_unit(g, u, limit):
    """Gated unit of an expert before its output projection."""
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def expert(get, p, h, limit):
    return clamped_unit(h @ get(p + "gate").to(F64).T, h @ get(p + "up").to(F64).T, limit) @ get(p + "down").to(F64).T


def route(z, top, groups=None):
    """[(expert, weight)] for one token's logits z [E]: softmax scores over all experts; only the experts of the best
    groups (by their largest score) can be chosen; the chosen keep their scores."""
    s = torch.softmax(z, -1)
    E = s.numel()
    allowed = list(range(E))
    if groups:
        n = E // groups["count"]
        best = sorted(range(groups["count"]), key=lambda gr: (-float(s[gr * n:(gr + 1) * n].max()), gr))[:groups["keep"]]
        allowed = [e for e in allowed if e // n in best]
    return [(e, s[e]) for e in sorted(allowed, key=lambda e: (-float(s[e]), e))[:top]]


def mixture(f, get, p, h):
    p += "mlp."
    r = f["router"]
    z = h @ get(p + "router").to(F64).T
    y = torch.zeros_like(h)
    outs = [expert(get, p + f"e{e}.", h, f["expert"]["limit"]) for e in range(r["experts"])]
    for t in range(h.shape[0]):
        for e, wgt in route(z[t], r["top"], r.get("groups")):
            y[t] += wgt * outs[e][t]
    if f.get("shared"):
        y = y + expert(get, p + "shared.", h, f["shared"]["limit"])
    return y


def forward(d, get, tokens, layers=None):
    """Logits of every position; `layers` (a list) receives the residual after every layer."""
    eps = d["norm"]["eps"]
    x = get("embed").to(F64)[torch.as_tensor(tokens)] * d["embedding"]["scale"]
    kv = {}
    for i, L in enumerate(d["layers"]):
        p = f"l{i}."
        h = rms_norm(x, get(p + "norm1"), eps)
        if L["type"] == "attention":
            y, kv[i] = attention_mixer(L["mixer"], get, p, h, kv)
        else:
            y = latent_mixer(L["mixer"], get, p, h, eps)
        x = x + get(p + "ls1").to(F64) * y
        if L["mlp"] is not None:
            x = x + get(p + "ls2").to(F64) * mixture(L["mlp"], get, p, rms_norm(x, get(p + "norm2"), eps))
        if layers is not None:
            layers.append(x)
    return rms_norm(x, get("final.norm"), eps) @ get("head").to(F64).T
