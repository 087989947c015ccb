"""The Tovapel decoder family, restated plainly on the CPU in float64: one function per mechanism,
whole sequences at once, no cache.  The GPU library's kernels and the engine are tested against
this file; it shares no code with them.

A model keeps `streams` copies of the residual.  Every sublayer reads one weighted sum of them,
    u = sum_s a_s x_s,   y = sublayer(N(u)),   x_t <- sum_s M[s, t] x_s + b_t y,
with an RMS norm N whose weight is stored around zero.  A mixer is two mixers on one input: softmax
attention over a window that keeps the first tokens (biased projections, q and k normed per head,
capped scores, a learned sink, one gate per head) and linear attention with a decay per key channel;
its result is half the sum of the two, each normed over the width.  Feed-forwards: a gated one, or
routed experts with clamped activations among which some are the identity.
"""
import math

import torch

F64 = torch.float64


def rms(x, eps):
    x = x.to(F64)
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    """A plain weight."""
    return rms(x, eps) * w.to(F64)


def offset_rms_norm(x, w, eps):
    """A weight stored around zero."""
    return rms(x, eps) * (1 + w.to(F64))


def soft_cap(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def visible(i, j, size, keep):
    """Whether the query at position i sees the key at position j: a window of `size` tokens, the
    query's own included (0: no window), and the sequence's first `keep` tokens."""
    return j <= i and (size <= 0 or i - j < size or j < keep)


def attend(q, k, v, pos_q, scale, size=0, keep=0, cap=0.0, sink=None):
    """q [n, H, dk] at positions pos_q against keys k [T, G, dk] / values v [T, G, dv] at positions
    0..T-1 -> [n, H, dv].  Head h reads key head h // (H/G).  sink [H]: one more term exp(sink) in
    the denominator."""
    H, (T, G, _) = q.shape[1], k.shape
    k, v = k.to(F64).repeat_interleave(H // G, 1), v.to(F64).repeat_interleave(H // G, 1)
    s = soft_cap(torch.einsum("ihd,jhd->hij", q.to(F64), k) * scale, cap)
    i, j = torch.as_tensor(pos_q).long()[:, None], torch.arange(T)[None, :]
    seen = (j <= i) & ((i - j < size) | (j < keep)) if size > 0 else j <= i   # visible(), all pairs at once
    s = s.masked_fill(~seen[None], -math.inf)
    top = s.max(-1).values
    if sink is not None:
        top = torch.maximum(top, sink.to(F64)[:, None])
    e = torch.exp(s - top[..., None])
    den = e.sum(-1)
    if sink is not None:
        den = den + torch.exp(sink.to(F64)[:, None] - top)
    return torch.einsum("hij,jhd->ihd", e / den[..., None], v)


def window_attention(h, m, t, pos):
    """h [T, W] -> [T, W].  m: the mixer's sizes and constants; t: its tensors by short name."""
    n, h = h.shape[0], h.to(F64)
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def proj(name, heads, d):
        return (h @ t[name].to(F64).T + t[name + ".b"].to(F64)).view(n, heads, d)
    q = rms_norm(proj("q", H, dk), t["q.norm"], m["eps"])
    k = rms_norm(proj("k", G, dk), t["k.norm"], m["eps"])
    mask = m.get("mask") or {}
    o = attend(q, k, proj("v", G, dv), pos, m["scale"], mask.get("size", 0), mask.get("keep_first", 0),
               m.get("softcap", 0.0), t["sink"])
    gate = torch.sigmoid(h @ t["g"].to(F64).T)                                       # [T, H]
    return (o * gate[..., None]).reshape(n, H * dv) @ t["o"].to(F64).T


def channel_decays(h, m, t):
    """[T, H, dk]: sigmoid(z)^(1/tau)."""
    z = (h.to(F64) @ t["a1"].to(F64).T) @ t["a2"].to(F64).T + t["a2.b"].to(F64)
    return torch.exp(torch.nn.functional.logsigmoid(z) / m["tau"]).view(h.shape[0], m["heads"], m["dim"])


def decayed_reads(q, k, v, decay, state=None):
    """S <- diag(decay_t) S + k_t v_t^T;  o_t = S^T q_t, a token at a time.  q, k, decay [T, H, dk],
    v [T, H, dv]; state [H, dk, dv] (or None: zero).  Returns (o [T, H, dv], the last S)."""
    n, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[2], dtype=F64) if state is None else state.to(F64).clone()
    out = torch.empty(n, H, v.shape[2], dtype=F64)
    q, k, v, decay = q.to(F64), k.to(F64), v.to(F64), decay.to(F64)
    for i in range(n):
        S = decay[i][:, :, None] * S + k[i][:, :, None] * v[i][:, None, :]
        out[i] = (S * q[i][:, :, None]).sum(1)
    return out, S


def linear_attention(h, m, t):
    n, h = h.shape[0], h.to(F64)
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ t["q"].to(F64).T).view(n, H, dk) * dk ** -0.5
    k, v = (h @ t["k"].to(F64).T).view(n, H, dk), (h @ t["v"].to(F64).T).view(n, H, dv)
    o, _ = decayed_reads(q, k, v, channel_decays(h, m, t))
    g = h @ t["g"].to(F64).T
    return (rms_norm(o, t["norm"], m["eps"]).reshape(n, H * dv) * g * torch.sigmoid(g)) @ t["o"].to(F64).T


def parallel_mixer(h, m, t, pos):
    a = window_attention(h, dict(m["left"], eps=m["eps"]), sub(t, "left."), pos)
    b = linear_attention(h, dict(m["right"], eps=m["eps"]), sub(t, "right."))
    return 0.5 * (rms_norm(a, t["left.out"], m["eps"]) + rms_norm(b, t["right.out"], m["eps"]))


def dense_ff(h, t):
    h = h.to(F64)
    g = h @ t["gate"].to(F64).T
    return (g * torch.sigmoid(g) * (h @ t["up"].to(F64).T)) @ t["down"].to(F64).T


def clamped_expert(h, gate, up, down, limit):
    h = h.to(F64)
    g = torch.clamp(h @ gate.to(F64).T, max=limit)
    u = torch.clamp(h @ up.to(F64).T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ down.to(F64).T


def route(h, w_router, correction, top):
    """(chosen outputs [T, top], their weights [T, top]): the choice sees the correction, the weights
    do not, and they are not renormalized."""
    s = torch.softmax(h.to(F64) @ w_router.to(F64).T, -1)
    idx = (s + correction.to(F64)).topk(top, -1).indices
    return idx, s.gather(-1, idx)


def experts_ff(h, mlp, t):
    r, n = mlp["router"], mlp["router"]["experts"]
    h = h.to(F64)
    idx, wt = route(h, t["router"], t["correction"], r["top"])
    out = torch.zeros_like(h)
    for e in range(n + r.get("identity", 0)):
        rows, slot = (idx == e).nonzero(as_tuple=True)
        if rows.numel():
            y = h[rows] if e >= n else clamped_expert(h[rows], t[f"e{e}.gate"], t[f"e{e}.up"], t[f"e{e}.down"],
                                                      mlp["expert"]["limit"])
            out[rows] += wt[rows, slot][:, None] * y
    return out


def read_streams(x, w_in):
    """x [T, S, W] -> [T, W]."""
    return (x * w_in.to(F64)[None, :, None]).sum(1)


def update_streams(x, y, mix, out):
    """x_t <- sum_s mix[s, t] x_s + out_t y for every t, x on the right as it was."""
    return torch.einsum("nsw,st->ntw", x, mix.to(F64)) + out.to(F64)[None, :, None] * y[:, None, :]


def sub(state, prefix):
    return {k[len(prefix):]: v for k, v in state.items() if k.startswith(prefix)}


def forward(cfg, state, tokens, layer_out=None):
    """tokens [T] of one sequence -> logits [T, vocab] (float64).  layer_out receives the sum of the
    streams after every layer."""
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    pos, eps = torch.arange(tokens.numel()), cfg["norm"]["eps"]
    x = state["embed"].to(F64)[tokens][:, None, :].repeat(1, cfg["streams"], 1)
    for i, l in enumerate(cfg["layers"]):
        pre = f"l{i}."

        def sublayer(x, n, f):
            hc = sub(state, f"{pre}hc{n}.")
            y = f(offset_rms_norm(read_streams(x, hc["in"]), state[f"{pre}norm{n}"], eps))
            return update_streams(x, y, hc["mix"], hc["out"])
        if l["type"] != "parallel":
            raise ValueError(l["type"])
        x = sublayer(x, 1, lambda h: parallel_mixer(h, dict(l["mixer"], eps=eps), sub(state, pre + "mix."), pos))
        mlp, t = l.get("mlp"), sub(state, pre + "mlp.")
        if mlp:
            x = sublayer(x, 2, (lambda h: dense_ff(h, t)) if mlp["kind"] == "dense" else (lambda h: experts_ff(h, mlp, t)))
        if layer_out is not None:
            layer_out.append(x.sum(1))
    z = offset_rms_norm(x.sum(1), state["final.norm"], eps) @ state["head"].to(F64).T
    return soft_cap(z, cfg.get("logit_softcap", 0.0))


def random_tensors(cfg, ranks, seed=0):
    """Seeded random tensors (bfloat16 values, as float32) under the checkpoint's names.  ranks: the
    inner size of every layer's low-rank pair."""
    g = torch.Generator().manual_seed(seed)

    def rn(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * s).to(torch.bfloat16).float()

    W, S, st = cfg["width"], cfg["streams"], {}
    st["embed"], st["head"], st["final.norm"] = rn(cfg["vocab"], W), rn(cfg["vocab"], W, s=W ** -0.5), rn(W, s=0.1)
    for i, l in enumerate(cfg["layers"]):
        p, a, b, mlp = f"l{i}.", l["mixer"]["left"], l["mixer"]["right"], l.get("mlp")
        for n in (1, 2) if mlp else (1,):
            st[p + f"norm{n}"] = rn(W, s=0.1)
            st[p + f"hc{n}.in"], st[p + f"hc{n}.out"] = rn(S, s=0.3) + 0.5, rn(S, s=0.3) + 0.75
            st[p + f"hc{n}.mix"] = torch.eye(S) + rn(S, S, s=0.2)
        q = p + "mix.left."
        for n, heads, d in (("q", a["heads"], a["dim"]), ("k", a["kv_heads"], a["dim"]), ("v", a["kv_heads"], a["vdim"])):
            st[q + n], st[q + n + ".b"] = rn(heads * d, W, s=W ** -0.5), rn(heads * d, s=0.3)
        st[q + "q.norm"], st[q + "k.norm"] = 1 + rn(a["dim"], s=0.2), 1 + rn(a["dim"], s=0.2)
        st[q + "sink"], st[q + "g"] = rn(a["heads"]), rn(a["heads"], W, s=W ** -0.5)
        st[q + "o"], st[q + "out"] = rn(W, a["heads"] * a["vdim"], s=(a["heads"] * a["vdim"]) ** -0.5), 1 + rn(W, s=0.2)
        q, H, dk, dv = p + "mix.right.", b["heads"], b["dim"], b["vdim"]
        for n, rows in (("q", H * dk), ("k", H * dk), ("v", H * dv), ("g", H * dv)):
            st[q + n] = rn(rows, W, s=W ** -0.5)
        st[q + "o"], st[q + "out"], st[q + "norm"] = rn(W, H * dv, s=(H * dv) ** -0.5), 1 + rn(W, s=0.2), 1 + rn(dv, s=0.2)
        st[q + "a1"], st[q + "a2"] = rn(ranks[i], W, s=W ** -0.5), rn(H * dk, ranks[i], s=ranks[i] ** -0.5)
        st[q + "a2.b"] = rn(H * dk) + 1.0
        if not mlp:
            continue
        q = p + "mlp."
        if mlp["kind"] == "dense":
            F = mlp["ff"]
            st[q + "gate"], st[q + "up"], st[q + "down"] = rn(F, W, s=W ** -0.5), rn(F, W, s=W ** -0.5), rn(W, F, s=F ** -0.5)
            continue
        E, F, n_id = mlp["router"]["experts"], mlp["expert"]["ff"], mlp["router"].get("identity", 0)
        st[q + "router"], st[q + "correction"] = rn(E + n_id, W, s=2 * W ** -0.5), rn(E + n_id, s=0.1)
        for e in range(E):
            st[q + f"e{e}.gate"], st[q + f"e{e}.up"] = rn(F, W, s=1.5 * W ** -0.5), rn(F, W, s=1.5 * W ** -0.5)
            st[q + f"e{e}.down"] = rn(W, F, s=F ** -0.5)
    return {k: v.to(torch.bfloat16).float() for k, v in st.items()}
