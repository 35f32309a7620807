"""Plain float64 whole-sequence oracle of the Tebodra decoder, one function per mechanism, written from the model's
equations and sharing no code with the package. `forward(config dict, get, tokens)` -> logits [T, vocab]; `get(name)`
returns a checkpoint tensor. Everything is recomputed from position 0 for every call: no cache, no pages, no carried state.
The matrix-memory layers run without their running maximum (float64 holds the plain exponentials); `mlstm_stabilised`
is the form with it."""
import math

import torch

F64 = torch.float64


def offset_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * (1.0 + w.to(F64))


def plain_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.to(F64)


def gelu(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def short_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start; no activation."""
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for t in range(u.shape[0]):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j].to(F64) * u[s]
    return y


def frequencies(rot):
    """Angle per position of every pair. Scaling: none, linear (`factor` alone), or by wavelength (`low`, `high`,
    `original`): short waves kept, long ones divided by the factor, a blend between."""
    f = [rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)]
    s = rot.get("scaling")
    if s and "original" not in s:
        f = [x / s["factor"] for x in f]
    elif s:
        out = []
        for x in f:
            wave = 2.0 * math.pi / x
            if wave < s["original"] / s["high"]:
                out.append(x)
            elif wave > s["original"] / s["low"]:
                out.append(x / s["factor"])
            else:
                r = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
                out.append((1.0 - r) * x / s["factor"] + r * x)
        f = out
    return torch.tensor(f, dtype=F64)


def rotate(x, rot, positions=None):
    """x [T, heads, d]: turns the pairs (i, i + dims / 2) of the first rot.dims numbers of every head."""
    if not rot or not rot["dims"]:
        return x
    n, f = rot["dims"] // 2, frequencies(rot)
    p = torch.arange(x.shape[0], dtype=F64) if positions is None else torch.as_tensor(positions, dtype=F64)
    out = x.clone()
    for i in range(n):
        c, s = torch.cos(p * f[i])[:, None], torch.sin(p * f[i])[:, None]
        out[:, :, i] = x[:, :, i] * c - x[:, :, i + n] * s
        out[:, :, i + n] = x[:, :, i + n] * c + x[:, :, i] * s
    return out


def visible(i, chunk):
    """Key positions the query at position i attends to."""
    return [j for j in range(i + 1) if not chunk or j // chunk == i // chunk]


def softmax_rows(q, k, v, scale, softcap=None, chunk=None, sink=None):
    """One head: q, k [T, d], v [T, e]; `sink` is one more score in the denominator, neither scaled nor capped, without a
    value."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F64)
    for i in range(q.shape[0]):
        js = visible(i, chunk)
        s = (k[js] @ q[i]) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        m = s.max() if sink is None else torch.maximum(s.max(), sink)
        e = torch.exp(s - m)
        den = e.sum() + (0.0 if sink is None else torch.exp(sink - m))
        out[i] = (e / den) @ v[js]
    return out


def grouped_attention(q, k, v, scale, softcap=None, chunk=None, sink=None):
    """q [T, H, d], k [T, G, d], v [T, G, e]: head h reads key / value head h // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    return torch.stack([softmax_rows(q[:, h], k[:, h // (H // G)], v[:, h // (H // G)], scale, softcap, chunk,
                                     None if sink is None else sink[h]) for h in range(H)], 1)


def gated_output(o, h, get, p):
    return (o * torch.sigmoid(h @ get(p + "g").to(F64).T)) @ get(p + "o").to(F64).T


def tied_mixer(m, get, p, h, kv_of):
    """Attention whose values are its keys as the convolution leaves them. `kv_of`: layer index -> (keys as they are scored,
    values) of the attention layers run so far."""
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = short_conv(h @ get(p + "q").to(F64).T, get(p + "q.conv")).reshape(T, H, d)
    if m.get("kv_from") is None:
        v = short_conv(h @ get(p + "k").to(F64).T, get(p + "k.conv")).reshape(T, G, d)
        k = rotate(v, m.get("rot"))
    else:
        k, v = kv_of[m["kv_from"]]
    o = grouped_attention(rotate(q, m.get("rot")), k, v, m["scale"], m.get("softcap"))
    return gated_output(o.reshape(T, H * d), h, get, p), (k, v)


def chunked_mixer(m, get, p, h, eps, kv_of):
    T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate(plain_norm(h @ get(p + "q").to(F64).T, get(p + "q.norm"), eps).reshape(T, H, d), m.get("rot"))
    if m.get("kv_from") is None:
        k = rotate(plain_norm(h @ get(p + "k").to(F64).T, get(p + "k.norm"), eps).reshape(T, G, d), m.get("rot"))
        v = (h @ get(p + "v").to(F64).T).reshape(T, G, e)
    else:
        k, v = kv_of[m["kv_from"]]
    o = grouped_attention(q, k, v, m["scale"], None, (m.get("mask") or {}).get("size"), get(p + "sink").to(F64))
    return gated_output(o.reshape(T, H * e), h, get, p), (k, v)


def mlstm_gates(zi, zf, cap):
    """(log input gate, log forget gate) of pre-activations with biases."""
    return cap * torch.tanh(zi / cap), torch.nn.functional.logsigmoid(cap * torch.tanh(zf / cap))


def mlstm_plain(q, k, v, i, f):
    """One head, q, k [T, d] (q scaled), v [T, e], log gates i, f [T]: the recurrence without the running maximum. With
    m_t = ln(scale of the stored state) the stabilised form divides S, n by exp(m_t) and bounds |n . q| by exp(-m_t), so
    its result is this one's with the bound 1 and the 1e-6 scaled by exp(m_t)."""
    T = q.shape[0]
    S, n, m = torch.zeros(q.shape[1], v.shape[1], dtype=F64), torch.zeros(q.shape[1], dtype=F64), 0.0
    out = torch.zeros(T, v.shape[1], dtype=F64)
    for t in range(T):
        m = max(float(f[t]) + m, float(i[t]))
        S = torch.exp(f[t]) * S + torch.exp(i[t]) * torch.outer(k[t], v[t])
        n = torch.exp(f[t]) * n + torch.exp(i[t]) * k[t]
        out[t] = (S.T @ q[t]) / (torch.clamp((n @ q[t]).abs(), min=1.0) + 1e-6 * math.exp(m))
    return out


def mlstm_stabilised(q, k, v, i, f):
    T = q.shape[0]
    S, n, m = torch.zeros(q.shape[1], v.shape[1], dtype=F64), torch.zeros(q.shape[1], dtype=F64), torch.zeros((), dtype=F64)
    out = torch.zeros(T, v.shape[1], dtype=F64)
    for t in range(T):
        new = torch.maximum(f[t] + m, i[t])
        a, c = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        S, n, m = a * S + c * torch.outer(k[t], v[t]), a * n + c * k[t], new
        out[t] = (S.T @ q[t]) / (torch.maximum((n @ q[t]).abs(), torch.exp(-m)) + 1e-6)
    return out


def mlstm_mixer(m, get, p, h, eps):
    T, H, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    w = lambda n: get(p + n).to(F64)  # noqa: E731
    q = (h @ w("q").T).reshape(T, H, d) * d ** -0.5
    k, v = (h @ w("k").T).reshape(T, H, d), (h @ w("v").T).reshape(T, H, e)
    i, f = mlstm_gates(h @ w("i").T + w("i.b"), h @ w("f").T + w("f.b"), m["gate_cap"])
    o = torch.stack([mlstm_plain(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]) for a in range(H)], 1)
    o = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps)
    return gated_output(o.reshape(T, H * e) * w("norm"), h, get, p)


def dense_unit(get, p, h):
    return gelu(h @ get(p + "up").to(F64).T) @ get(p + "down").to(F64).T


def forward(d, get, tokens, layers=None):
    """Logits of every position; `layers` (a list) receives the residual after every layer."""
    eps, mult = d["norm"]["eps"], d["residual_mult"]
    x = get("embed").to(F64)[torch.as_tensor(tokens)]
    kv = {}
    for i, L in enumerate(d["layers"]):
        p = f"l{i}.mix."
        h = offset_norm(x, get(f"l{i}.norm1"), eps)
        if L["type"] == "attention":
            y, kv[i] = tied_mixer(L["mixer"], get, p, h, kv)
        elif L["type"] == "attention_2":
            y, kv[i] = chunked_mixer(L["mixer"], get, p, h, eps, kv)
        else:
            y = mlstm_mixer(L["mixer"], get, p, h, eps)
        x = x + mult * y
        if L["mlp"] is not None:
            x = x + mult * dense_unit(get, f"l{i}.mlp.", offset_norm(x, get(f"l{i}.norm2"), eps))
        if layers is not None:
            layers.append(x)
    return offset_norm(x, get("final.norm"), eps) @ get("head").to(F64).T
