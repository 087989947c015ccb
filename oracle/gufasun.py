"""The Gufasun decoder family, restated plainly on the CPU in float64: one function per mechanism,
whole sequences at once, no cache.  The GPU library's kernels and the engine are tested against
this file; it shares no code with them.

A model is a list of layers, each  x += mixer(u + conv(u)) + ff(LN2(x)),  u = LN1(x): both sublayers
read the same x.  LN is a layer norm with a weight and no bias, conv a causal per-channel
convolution of the mixer's input.  Two mixers:

* attention: grouped-query softmax attention over a sliding window, without rotation.  q, k and v
  have biases and pass a causal per-channel convolution each; q and k are RMS-normed per head; q
  grows with the logarithm of its position; scores are capped smoothly, and each head takes off a
  logarithm of the distance.  A layer may read another layer's keys and values.
* mlstm: a matrix memory per head with an exponential input gate and a sigmoid forget gate, kept
  in range by a running maximum of the gates' logarithms, read through a normalizer.

The feed-forward's activation mixes the normed first three powers of its hidden vector.
"""
import math

import torch

F64 = torch.float64


def layer_norm(x, w, eps):
    x = x.to(F64)
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt(d.pow(2).mean(-1, keepdim=True) + eps) * w.to(F64)


def rms_norm(x, w, eps):
    x = x.to(F64)
    y = x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w.to(F64)


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    u, w = u.to(F64), w.to(F64)
    taps, T = w.shape[1], u.shape[0]
    y = torch.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y


def query_temperature(pos, coef, every):
    steps = (torch.as_tensor(pos).long() + 1) // every
    return 1 + coef * torch.log(steps.to(F64) + 1)


def window_scores(q, k, pos_q, scale, softcap, r1, r2, window):
    """q [n, H, d] at positions pos_q against k [T, H, d] -> scores [H, n, T], -inf where not seen."""
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    if softcap:
        s = softcap * torch.tanh(s / softcap)
    dist = torch.as_tensor(pos_q).long()[:, None] - torch.arange(k.shape[0])[None, :]
    away = dist.clamp_min(0).to(F64)
    s = s - r1.to(F64)[:, None, None] * torch.log(1 + r2.to(F64)[:, None, None] * away)
    seen = (dist >= 0) & (dist < window if window else dist >= 0)
    return s.masked_fill(~seen[None], -math.inf)


def projected(h, t, name):
    """A projection with its bias and, after it, its convolution."""
    u = h.to(F64) @ t[name].to(F64).T + t[name + ".b"].to(F64)
    return causal_conv(u, t[name + ".conv"])


def keys_values(h, m, t):
    """The keys and values an attention layer caches: [T, G, dk], [T, G, dv]."""
    T, G = h.shape[0], m["kv_heads"]
    k = rms_norm(projected(h, t, "k").view(T, G, m["dim"]), t["k.norm"], m["eps"])
    return k, projected(h, t, "v").view(T, G, m["vdim"])


def attention(h, m, t, pos, kv=None):
    """h [T, W] -> [T, W].  kv: another layer's (keys, values) to read instead of this one's."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = rms_norm(projected(h, t, "q").view(T, H, m["dim"]), t["q.norm"], m["eps"])
    qt = m.get("q_temp")
    if qt:
        q = q * query_temperature(pos, qt["coef"], qt["every"])[:, None, None]
    k, v = kv if kv is not None else keys_values(h, m, t)
    k, v = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)   # head h reads kv head h // (H/G)
    s = window_scores(q, k, pos, m["scale"], m.get("softcap"), t["r1"], t["r2"], (m.get("mask") or {}).get("size"))
    o = torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v)
    return o.reshape(T, H * m["vdim"]) @ t["o"].to(F64).T


def mlstm_gates(h, t, cap):
    """Logarithms of the input and the forget gate, [T, H] each."""
    zi = h.to(F64) @ t["i"].to(F64).T + t["i.b"].to(F64)
    zf = h.to(F64) @ t["f"].to(F64).T + t["f.b"].to(F64)
    return cap * torch.tanh(zi / cap), torch.nn.functional.logsigmoid(cap * torch.tanh(zf / cap))


def mlstm_read(q, k, v, li, lf):
    """q, k [T, H, dk] (q scaled), v [T, H, dv], gate logarithms [T, H] -> read vectors [T, H, dv]."""
    T, H, dk = q.shape
    S, n, m = torch.zeros(H, dk, v.shape[2], dtype=F64), torch.zeros(H, dk, dtype=F64), torch.zeros(H, dtype=F64)
    out = []
    for i in range(T):
        m_new = torch.maximum(lf[i] + m, li[i])
        keep, add = torch.exp(lf[i] + m - m_new), torch.exp(li[i] - m_new)
        S = keep[:, None, None] * S + add[:, None, None] * k[i][:, :, None] * v[i][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[i]
        m = m_new
        den = torch.maximum((n * q[i]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out.append((S * q[i][:, :, None]).sum(1) / den[:, None])
    return torch.stack(out)


def mlstm(h, m, t):
    T, H, dk, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    h = h.to(F64)
    q = (h @ t["q"].to(F64).T).view(T, H, dk) * dk ** -0.5
    k, v = (h @ t["k"].to(F64).T).view(T, H, dk), (h @ t["v"].to(F64).T).view(T, H, dv)
    li, lf = mlstm_gates(h, t, m["gate_cap"])
    o = rms_norm(mlstm_read(q, k, v, li, lf), None, m["eps"]).reshape(T, H * dv) * t["norm"].to(F64)
    return (o * torch.sigmoid(h @ t["g"].to(F64).T)) @ t["o"].to(F64).T


def poly_norm(z, act, eps):
    a, b, c, e = (act.to(F64)[i] for i in range(4))
    z = z.to(F64)
    return a * rms_norm(z, None, eps) + b * rms_norm(z * z, None, eps) + c * rms_norm(z * z * z, None, eps) + e


def feed_forward(h, t, eps):
    z = h.to(F64) @ t["up"].to(F64).T + t["up.b"].to(F64)
    return poly_norm(z, t["act"], eps) @ t["down"].to(F64).T + t["down.b"].to(F64)


def sub(state, prefix):
    return {k[len(prefix):]: v for k, v in state.items() if k.startswith(prefix)}


def forward(cfg, state, tokens, layer_out=None):
    """tokens [T] of one sequence -> logits [T, vocab] (float64)."""
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    pos = torch.arange(tokens.numel())
    eps = cfg["norm"]["eps"]
    x = state["embed"].to(F64)[tokens] * cfg["embedding"]["scale"]
    kept = {}                                            # keys and values of the layers others read
    for i, l in enumerate(cfg["layers"]):
        pre = f"l{i}."
        m, t = dict(l["mixer"], eps=eps), sub(state, pre + "mix.")
        h = layer_norm(x, state[pre + "norm1"], eps)
        h = h + causal_conv(h, state[pre + "canon1"])
        if l["type"] == "attention":
            src = m.get("kv_from")
            if src is None:
                kept[i] = keys_values(h, m, t)
            y = attention(h, m, t, pos, kv=kept[i if src is None else src])
        elif l["type"] == "mlstm":
            y = mlstm(h, m, t)
        else:
            raise ValueError(l["type"])
        if l.get("mlp"):
            y = y + feed_forward(layer_norm(x, state[pre + "norm2"], eps), sub(state, pre + "mlp."), eps)
        x = x + y
        if layer_out is not None:
            layer_out.append(x.clone())
    return layer_norm(x, state["final.norm"], eps) @ state["head"].to(F64).T


def random_tensors(cfg, seed=0):
    """Seeded random tensors (bfloat16 values, as float32) under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)

    def rn(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * s).to(torch.bfloat16).float()

    W, st = cfg["width"], {}
    st["embed"], st["head"], st["final.norm"] = rn(cfg["vocab"], W), rn(cfg["vocab"], W, s=W ** -0.5), 1 + rn(W, s=0.1)
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        st[p + "norm1"], st[p + "canon1"] = 1 + rn(W, s=0.1), rn(W, cfg["canon"]["taps"], s=0.4)
        if l["type"] == "attention":
            G, taps = m["kv_heads"], m["conv"]
            names = [("q", H * dk)] + ([("k", G * dk), ("v", G * dv)] if m.get("kv_from") is None else [])
            for n, rows in names:
                st[p + "mix." + n], st[p + f"mix.{n}.b"] = rn(rows, W, s=W ** -0.5), rn(rows, s=0.3)
                st[p + f"mix.{n}.conv"] = rn(rows, taps, s=0.6)
                if n != "v":
                    st[p + f"mix.{n}.norm"] = 1 + rn(dk, s=0.1)
            st[p + "mix.r1"], st[p + "mix.r2"] = rn(H, s=0.5).abs(), rn(H, s=0.5).abs()
        else:
            for n, rows in (("q", H * dk), ("k", H * dk), ("v", H * dv), ("g", H * dv), ("i", H), ("f", H)):
                st[p + "mix." + n] = rn(rows, W, s=W ** -0.5)
            st[p + "mix.i.b"], st[p + "mix.f.b"], st[p + "mix.norm"] = rn(H), rn(H) + 3.0, 1 + rn(H * dv, s=0.1)
        st[p + "mix.o"] = rn(W, H * dv, s=(H * dv) ** -0.5)
        if l.get("mlp"):
            F = l["mlp"]["ff"]
            st[p + "norm2"], st[p + "mlp.act"] = 1 + rn(W, s=0.1), torch.cat([rn(3, s=0.6), rn(1, s=0.2)])
            st[p + "mlp.up"], st[p + "mlp.up.b"] = rn(F, W, s=W ** -0.5), rn(F, s=0.2)
            st[p + "mlp.down"], st[p + "mlp.down.b"] = rn(W, F, s=F ** -0.5), rn(W, s=0.2)
    return st
