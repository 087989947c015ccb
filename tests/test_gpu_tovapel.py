"""The Tovapel decoder family on the GPU against the plain CPU restatement in oracle/tovapel.py:
every mechanism alone through its entry point, then whole models through the engine (prompts
whole, token by token, in portions, in mixed batches, over reused slots and pages) and through
the worker and scheduler.  Small random models of several shapes; where random weights would hide
a fault (one far key among many, a window's edge, the first tokens, a sink, decays that are strong or
almost one, identity experts, streams that are all alike) the inputs are made so that it shows."""

import pytest
import torch

from oracle import tovapel as O

pytestmark = pytest.mark.gpu

DEV = "cuda"
PAGE = 16
F64 = torch.float64


def dev(t, dtype=None):
    return t.to(dtype or t.dtype).contiguous().to(DEV)


def i32(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


def rel(a, b):
    a, b = a.double().cpu(), b.double().cpu()
    return ((a - b).pow(2).mean().sqrt() / b.pow(2).mean().sqrt().clamp_min(1e-30)).item()


# ------------------------------------------------------------------ model shapes
def dense(ff=24):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=2, ff=20, limit=1.0, identity=2):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "identity": identity}, "expert": {"ff": ff, "limit": limit}}


def layer(heads=4, kv_heads=2, dim=8, vdim=12, window=13, keep=3, scale=0.4, cap=20.0, rh=3, rdim=8, rvdim=10, tau=8.0,
          mlp=None, rank=6):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, softcap=cap,
                mask={"size": window, "keep_first": keep})
    return {"type": "parallel", "mixer": {"left": left, "right": dict(heads=rh, dim=rdim, vdim=rvdim, tau=tau)}, "mlp": mlp,
            "rank": rank}


def model_cfg(layers, width=32, vocab=80, streams=3, eps=1e-5, cap=25.0):
    return {"architecture": "Tovapel", "width": width, "vocab": vocab, "norm": {"eps": eps}, "streams": streams,
            "logit_softcap": cap, "layers": layers}


SHAPES = {
    "two_kinds": model_cfg([layer(mlp=dense()), layer(window=21, keep=5, mlp=moe()), layer(mlp=None), layer(mlp=moe(top=3))]),
    # sizes that divide nothing; every pair of sizes that may coincide made different; three heads on a kv
    # head; no feed-forward, no identity expert, more identity experts than others
    "odd": model_cfg([layer(heads=6, kv_heads=2, dim=11, vdim=19, window=18, keep=1, rh=2, rdim=21, rvdim=37, tau=3.0, rank=5,
                            mlp=moe(experts=7, top=3, ff=13, identity=0)),
                      layer(heads=5, kv_heads=5, dim=10, vdim=7, window=1, keep=0, scale=0.2, cap=5.0, rh=5, rdim=6, rvdim=3,
                            tau=1.0, rank=1, mlp=dense(33)),
                      layer(heads=3, kv_heads=1, dim=17, vdim=23, window=40, keep=29, rh=4, rdim=33, rvdim=17, tau=16.0, rank=20,
                            mlp=moe(experts=2, top=4, ff=9, limit=0.5, identity=5)), layer(mlp=None)],
                     width=41, vocab=131, streams=5, eps=1e-6, cap=12.0),
    # one head, one channel, one stream, one expert, a window of one token
    "ones": model_cfg([layer(heads=1, kv_heads=1, dim=1, vdim=1, window=1, keep=1, scale=1.0, rh=1, rdim=1, rvdim=1, tau=1.0,
                             rank=1, mlp=moe(experts=1, top=1, ff=1, limit=3.0, identity=0)),
                       layer(heads=1, kv_heads=1, dim=1, vdim=1, window=2, keep=0, rh=1, rdim=1, rvdim=1, mlp=dense(1))],
                      width=24, vocab=50, streams=1),
    # widths that are multiples of 32: bfloat16 serving takes the tiled linear kernels; output matrices of equal
    # input widths (stacked) and of unequal ones
    "aligned": model_cfg([layer(heads=4, kv_heads=2, dim=16, vdim=16, rh=2, rdim=16, rvdim=32, rank=8, mlp=moe(ff=32)),
                          layer(heads=4, kv_heads=2, dim=24, vdim=16, rh=4, rdim=40, rvdim=8, rank=16, mlp=dense(96)),
                          layer(heads=4, kv_heads=4, dim=16, vdim=16, rh=4, rdim=16, rvdim=16, mlp=None)],
                         width=64, vocab=178, streams=4),
    # heads wider than a wave, values wider than two tiles of columns, nine heads on a kv head, large keep
    "wide": model_cfg([layer(heads=9, kv_heads=1, dim=72, vdim=136, window=30, keep=40, rh=2, rdim=130, rvdim=72, mlp=dense()),
                       layer(heads=16, kv_heads=2, dim=130, vdim=300, window=70, keep=2, rh=1, rdim=256, rvdim=260, rank=70,
                             mlp=moe(experts=12, top=5))], width=48, vocab=64, streams=9),
    # no window at all, no caps, keys kept beyond the window's size
    "open": model_cfg([layer(window=0, keep=0, cap=0.0, mlp=dense()), layer(window=4, keep=50, mlp=moe())], cap=0.0, streams=2),
    # the head sizes of larger models: bfloat16 prompts take the matrix-core attention
    "heads128": model_cfg([layer(heads=4, kv_heads=2, dim=128, vdim=128, window=37, keep=5, scale=0.088, cap=30.0, rh=2, rdim=128,
                                 rvdim=128, mlp=moe(ff=64)),
                           layer(heads=4, kv_heads=1, dim=64, vdim=128, window=100, keep=3, scale=0.125, rh=3, rdim=64, rvdim=192,
                                 mlp=dense(64))], width=96, vocab=160, streams=2),
}


def ranks_of(cfg):
    return [l["rank"] for l in cfg["layers"]]


def tensors(cfg, seed=0):
    return O.random_tensors(cfg, ranks_of(cfg), seed)


def build(cfg, dtype=torch.float32, seed=0, tiled=True, st=None, **eng_kw):
    from vllm_omni_draft_amd import config, weights
    from vllm_omni_draft_amd.seq_engine import SeqEngine, SeqEngineConfig
    st = st or tensors(cfg, seed)
    mc = config.tovapel_config(cfg, {k: tuple(v.shape) for k, v in st.items()})
    w = weights.seq_from_state_dict(mc, st, DEV, dtype, tiled=tiled)
    kw = dict(max_seqs=4, max_tokens=1024)
    kw.update(eng_kw)
    return st, SeqEngine(w, SeqEngineConfig(**kw))


def prompt(cfg, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def fill_pages(rows, units, pages_of):
    """rows [n, units*d] of one sequence in slot 0 -> cache [pages, units, PAGE, d], written here
    (not through the library): token j lies in page pages_of[j // PAGE], row j % PAGE."""
    n, d = rows.shape[0], rows.shape[1] // units
    cache = torch.zeros(max(pages_of) + 1, units, PAGE, d, dtype=rows.dtype)
    for j in range(n):
        cache[pages_of[j // PAGE], :, j % PAGE] = rows[j].view(units, d)
    return cache.to(DEV)


def table(pages_of):
    bt = torch.zeros(2, len(pages_of), dtype=torch.int32, device=DEV)
    bt[0] = i32(pages_of)
    return bt


def plain_attention(q, k, v, pos, H, G, scale, window, keep, cap, sink, gates=None):
    n = q.shape[0]
    o = O.attend(q.view(n, H, -1), k.view(k.shape[0], G, -1), v.view(v.shape[0], G, -1), pos, scale, window, keep, cap, sink)
    if gates is not None:
        o = o * torch.sigmoid(gates.to(F64))[..., None]
    return o.reshape(n, -1)


# ------------------------------------------------------------------ attention alone
@pytest.mark.parametrize("H,G,dk,dv,window,keep,cap", [
    (4, 2, 16, 16, 13, 4, 5.0), (3, 1, 12, 20, 0, 0, 0.0), (2, 2, 72, 136, 70, 20, 2.0), (9, 1, 8, 8, 1, 1, 0.0),
    (16, 2, 8, 300, 64, 3, 3.0), (4, 2, 128, 128, 33, 17, 10.0), (8, 1, 128, 64, 100, 50, 0.0), (5, 5, 64, 128, 17, 200, 4.0),
    (6, 2, 96, 80, 20, 16, 8.0), (4, 1, 64, 64, 1, 0, 1.0)])
@pytest.mark.parametrize("cdt", [torch.float32, torch.bfloat16])
def test_attention_with_kept_tokens_sink_and_gates(H, G, dk, dv, window, keep, cap, cdt):
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(H * 100 + dk)
    n = 140
    q = torch.randn(n, H * dk, generator=g)
    k, v = torch.randn(n, G * dk, generator=g).to(cdt), torch.randn(n, G * dv, generator=g).to(cdt)
    sink, gates = torch.randn(H, generator=g) * 2, torch.randn(n, H, generator=g) * 2
    pages = [5, 1, 3, 8, 0, 2, 9, 4, 7]                 # pages out of order
    kc, vc, bt = fill_pages(k, G, pages), fill_pages(v, G, pages), table(pages)
    for sunk, gated in ((True, True), (False, False), (True, False)):
        want = plain_attention(q, k, v, torch.arange(n), H, G, 0.3, window, keep, cap, sink if sunk else None,
                               gates if gated else None)
        for rows in (list(range(n)), list(range(17, 90)), [n - 1], [0, 15, 16, 17, 31, 32, 44]):   # prompts, decoded rows
            for split in (True, False):
                kw = dict(sinks=dev(sink)) if sunk else {}
                if gated:
                    kw["gates"] = dev(gates[rows])
                if split and len(rows) > 64:                 # (with the rows' portion, where they are one)
                    kw["entries"] = i32([[0, 0, len(rows), rows[0]]])
                args = (dev(q[rows]), kc, vc, i32(rows), i32([0] * len(rows)), bt, H, G, dk, dv, 0.3, window, keep, cap)
                got = ops.gated_softmax_attention(*args, split=split, ldo=H * dv + 7, **kw)
                assert rel(got, want[rows]) < 5e-6, (len(rows), split, sunk, gated)
                assert rel(ops.gated_softmax_attention(*args, split=split, bf16_only=True, **kw), want[rows]) < 4e-3


def test_visibility_with_one_hot_values():
    """Value of key j is the unit vector j: a row's output shows which keys it saw.  Every edge of the
    window and of the kept tokens, in prompts of one portion (whole and from the middle on) and as single
    decoded rows, over page borders."""
    from vllm_omni_draft_amd import ops
    n, dk = 300, 128
    pages = torch.randperm(19, generator=torch.Generator().manual_seed(1)).tolist()
    for window, keep in ((1, 0), (1, 1), (2, 15), (15, 16), (16, 17), (17, 3), (31, 33), (33, 31), (64, 128), (65, 129), (79, 1),
                         (80, 140), (128, 2), (200, 300), (400, 5), (0, 0)):
        for cdt in (torch.float32, torch.bfloat16):
            kc = torch.zeros(19, 1, PAGE, dk, dtype=cdt, device=DEV)
            bt = table(pages)
            for half in (0, 1, 2):                         # (value columns 128 * half ..)
                v = torch.zeros(n, 128, dtype=cdt)
                lo = 128 * half
                for j in range(lo, min(lo + 128, n)):
                    v[j, j - lo] = 1
                vc = fill_pages(v, 1, pages)
                for rows in (list(range(n)), list(range(130, n)), [n - 1], [30, 31, 32, 250]):
                    got = ops.gated_softmax_attention(
                        torch.zeros(len(rows), 2 * dk, device=DEV), kc, vc, i32(rows), i32([0] * len(rows)), bt, 2, 1, dk, 128,
                        1.0, window, keep, 7.0, sinks=torch.zeros(2, device=DEV),
                        entries=i32([[0, 0, len(rows), rows[0]]]) if len(rows) > 64 else None)
                    i = torch.tensor(rows)[:, None]
                    j = torch.arange(lo, lo + 128)[None, :]
                    seen = (j <= i) & (j < n) & ((i - j < window) | (j < keep) | torch.tensor(window == 0))
                    full = torch.arange(n)[None, :]
                    count = ((full <= i) & ((i - full < window) | (full < keep) | torch.tensor(window == 0))).sum(1, keepdim=True)
                    want = seen.double() / (count + 1)      # (the sink is one more term of the same size)
                    got = got.double().cpu().view(len(rows), 2, 128)
                    for h in range(2):
                        assert ((got[:, h] > 0) == seen).all(), (window, keep, len(rows), half)
                        assert (got[:, h] - want).abs().max() < 3e-6, (window, keep, len(rows), half)


@pytest.mark.parametrize("cdt", [torch.float32, torch.bfloat16])
def test_a_kept_key_far_away_and_a_large_sink(cdt):
    """700 keys, a window of 50 and five kept tokens: head 0 points at the kept key 3, head 1 at key 5, which
    is not kept (only its neighbours' noise remains), head 2's sink takes nearly everything."""
    from vllm_omni_draft_amd import ops
    n, H, dk, dv, window, keep = 700, 3, 64, 64, 50, 5
    g = torch.Generator().manual_seed(11)
    k = torch.randn(n, dk, generator=g)
    k = (k / k.norm(dim=-1, keepdim=True)).to(cdt)
    v = torch.randn(n, dv, generator=g).to(cdt)
    pages = list(range(44))[::-1]
    kc, vc, bt = fill_pages(k, 1, pages), fill_pages(v, 1, pages), table(pages)
    rows = list(range(600, 700))
    sink = torch.tensor([0.0, -1.0, 9.0])
    q = torch.cat([40.0 * k[3].float(), 40.0 * k[5].float(), torch.zeros(dk)]).repeat(len(rows), 1)
    q += 0.1 * torch.randn(len(rows), H * dk, generator=g)
    want = plain_attention(q, k, v, torch.tensor(rows), H, 1, 1.0, window, keep, 50.0, sink)
    for sel in (slice(None), slice(99, 100), slice(0, 3), slice(7, 93)):
        got = ops.gated_softmax_attention(dev(q[sel]), kc, vc, i32(rows[sel]), i32([0] * len(rows[sel])), bt, H, 1, dk, dv, 1.0,
                                          window, keep, 50.0, sinks=dev(sink), entries=i32([[0, 0, len(rows[sel]), rows[sel][0]]]))
        assert rel(got, want[sel]) < (2e-5 if cdt == torch.bfloat16 else 5e-6)
        assert rel(got[:, :dv], v[3].float().expand(len(rows[sel]), dv)) < 1e-3
        assert rel(got[:, dv:2 * dv], v[5].float().expand(len(rows[sel]), dv)) > 0.5
        assert got[:, 2 * dv:].abs().max() < 0.05


@pytest.mark.parametrize("H,G,dk,dv", [(4, 1, 128, 128), (3, 3, 40, 64), (6, 2, 64, 104), (4, 2, 128, 56), (3, 1, 10, 12)])
def test_portions_of_several_sequences_in_one_launch(H, G, dk, dv):
    """Portions of four sequences: a long one, a single token, one that starts at its first token, two
    tokens; each row against the plain attention over its own sequence."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(dk + dv)
    n, window, keep = 300, 61, 20
    k, v = torch.randn(4, n, G * dk, generator=g).to(torch.bfloat16), torch.randn(4, n, G * dv, generator=g).to(torch.bfloat16)
    order = torch.randperm(76, generator=g).view(4, 19).tolist()
    kc = torch.zeros(76, G, PAGE, dk, dtype=torch.bfloat16)
    vc = torch.zeros(76, G, PAGE, dv, dtype=torch.bfloat16)
    for s in range(4):
        for j in range(n):
            kc[order[s][j // PAGE], :, j % PAGE] = k[s, j].view(G, dk)
            vc[order[s][j // PAGE], :, j % PAGE] = v[s, j].view(G, dv)
    portions = [(2, 190, 70), (0, 299, 1), (3, 0, 33), (1, 17, 2)]        # slot, first position, rows
    total = sum(p[2] for p in portions)
    q, gates, sink = torch.randn(total, H * dk, generator=g), torch.randn(total, H, generator=g), torch.randn(H, generator=g)
    ents, pos, slots, want, at = [], [], [], [], 0
    for s, p0, m in portions:
        ents.append([s, at, m, p0])
        pos += range(p0, p0 + m)
        slots += [s] * m
        want.append(plain_attention(q[at:at + m], k[s, :p0 + m], v[s, :p0 + m], torch.arange(p0, p0 + m), H, G, 0.2, window,
                                    keep, 4.0, sink, gates[at:at + m]))
        at += m
    got = ops.gated_softmax_attention(dev(q), kc.to(DEV), vc.to(DEV), i32(pos), i32(slots), i32(order), H, G, dk, dv, 0.2, window,
                                      keep, 4.0, sinks=dev(sink), gates=dev(gates), entries=i32(ents))
    for (s, p0, m), (_, a, _, _), w in zip(portions, ents, want):
        assert rel(got[a:a + m], w) < 5e-6, (s, p0, m)


# ------------------------------------------------------------------ linear attention alone
@pytest.mark.parametrize("H,dk,dv,rank", [(2, 16, 24, 6), (3, 21, 37, 1), (1, 1, 1, 3), (2, 130, 72, 17), (4, 256, 260, 64),
                                          (1, 5, 400, 70), (2, 128, 128, 16), (2, 64, 192, 8), (3, 32, 64, 20), (1, 96, 40, 2)])
@pytest.mark.parametrize("form", ["chunks", "whole", "step"])
@pytest.mark.parametrize("strength", ["usual", "strong", "almost_one"])
def test_linear_attention(H, dk, dv, rank, form, strength):
    """Decays from the low-rank pair, then the recurrence in portions of two interleaved sequences (down
    to single tokens), in chunks, in one go, and with single tokens in their fused launch; from slots an
    earlier request left full; decays that forget everything within a token among ordinary ones."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(H * 1000 + dk)
    T, eps = 233, 1e-5
    rn = lambda *s: torch.randn(*s, generator=g)
    q, k, v, gate = rn(2, T, H * dk), rn(2, T, H * dk), rn(2, T, H * dv), rn(2, T, H * dv)
    a1, a2, b = rn(2, T, rank), rn(H * dk, rank) * rank ** -0.5, rn(H * dk) + 1
    tau = 8.0
    if strength == "strong":
        b, tau = b * 20 - 20, 1.0                         # down to e^-60 per token beside factors of nearly one
    elif strength == "almost_one":
        b, a2 = b + 9, a2 * 0.1
    w = 1 + 0.2 * rn(dv)
    S = torch.full((3, H, dk, dv), 5.0, device=DEV)
    got = [[], []]
    for lo, hi in ((0, 1), (1, 2), (2, 70), (70, 71), (71, 73), (73, 74), (74, 139), (139, 203), (203, T)):
        n = hi - lo
        cat = lambda t: dev(torch.cat([t[0, lo:hi], t[1, lo:hi]]))
        if form == "step" and n == 1:
            y = ops.decay_step_rows(cat(q), cat(k), cat(v), cat(gate), cat(a1), dev(a2), dev(b), tau, S, dev(w), eps,
                                    i32([lo, lo]), i32([2, 0]), q_scale=dk ** -0.5)
        else:
            d = ops.low_rank_decay(cat(a1), dev(a2), dev(b), tau)
            o = ops.decay_chunks(cat(q), cat(k), cat(v), d, S, i32([[2, 0, n, lo], [0, n, n, lo]]), q_scale=dk ** -0.5,
                                 cut=form != "whole")
            y = ops.head_post(o, cat(gate), H, dv, norm_w=dev(w), unit_norm=True, eps=eps, gate="silu")
        for s in range(2):
            got[s].append(y[s * n:(s + 1) * n])
    for s in range(2):
        z = a1[s].double() @ a2.double().T + b.double()
        decay = torch.exp(torch.nn.functional.logsigmoid(z) / tau).view(T, H, dk)
        d = ops.low_rank_decay(dev(a1[s]), dev(a2), dev(b), tau)
        assert rel(d, decay.reshape(T, -1)) < 1e-6
        o, last = O.decayed_reads(q[s].view(T, H, dk) * dk ** -0.5, k[s].view(T, H, dk), v[s].view(T, H, dv), decay)
        gd = gate[s].double()
        want = O.rms_norm(o, w, eps).reshape(T, H * dv) * gd * torch.sigmoid(gd)
        gs = torch.cat(got[s])
        rows = sorted(rel(gs[t], want[t]) for t in range(T))
        assert rel(gs, want) < 2e-5 and rows[T // 2] < 4e-6, (rel(gs, want), rows[T // 2])
        assert rel(S[2 if s == 0 else 0], last) < 4e-6
    assert (S[1] == 5.0).all()


def test_chunked_form_of_long_portions():
    """Portions long enough for the long chunks, unequal, beside single tokens."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(3)
    H, dk, dv = 40, 32, 16
    lens, pos0 = [700, 1, 129, 64, 2], [0, 9, 3, 0, 100]
    n = sum(lens)
    q, k, v = torch.randn(n, H * dk, generator=g), torch.randn(n, H * dk, generator=g), torch.randn(n, H * dv, generator=g)
    decay = torch.sigmoid(torch.randn(n, H * dk, generator=g) * 2 + 2)
    S0 = torch.randn(6, H, dk, dv, generator=g)
    slots = [4, 0, 5, 1, 2]
    ents, at = [], 0
    for s, m, p in zip(slots, lens, pos0):
        ents.append([s, at, m, p])
        at += m
    outs = []
    for cut in (True, False):
        S = dev(S0.clone())
        outs.append(ops.decay_chunks(dev(q), dev(k), dev(v), dev(decay), S, i32(ents), cut=cut))
        for (s, a, m, p) in ents:
            want, last = O.decayed_reads(q[a:a + m].view(m, H, dk), k[a:a + m].view(m, H, dk), v[a:a + m].view(m, H, dv),
                                         decay[a:a + m].view(m, H, dk), S0[s] if p else None)
            assert rel(outs[-1][a:a + m], want.reshape(m, -1)) < 2e-6 and rel(S[s], last) < 2e-6, (cut, m)
        assert torch.equal(S[3].cpu(), S0[3])
    assert rel(outs[0], outs[1]) < 2e-6


def test_the_state_keeps_a_first_token_for_hundreds():
    """Decays of exactly one for half the channels: 600 tokens later a query along the first key still
    reads the first value."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(7)
    T, dk, dv = 600, 32, 32
    k, v = torch.zeros(T, dk), torch.randn(T, dv, generator=g)
    k[0, :16] = torch.randn(16, generator=g)
    k[1:, 16:] = torch.randn(T - 1, 16, generator=g)
    q = torch.zeros(T, dk)
    q[:, :16] = k[0, :16] / k[0].norm() ** 2
    d = torch.full((T, dk), 0.5)
    d[:, :16] = 1.0
    S = torch.zeros(1, 1, dk, dv, device=DEV)
    outs = [ops.decay_chunks(dev(q[lo:hi]), dev(k[lo:hi]), dev(v[lo:hi]), dev(d[lo:hi]), S, i32([[0, 0, hi - lo, lo]]))
            for lo, hi in ((0, 1), (1, 300), (300, 301), (301, T))]
    o = torch.cat(outs).cpu()
    assert rel(o[-1], v[0]) < 1e-5 and rel(o[299], v[0]) < 1e-5


@pytest.mark.parametrize("H,G,dk,dv", [(4, 2, 16, 24), (3, 3, 10, 7), (9, 1, 72, 136), (1, 1, 1, 1), (5, 5, 300, 500), (16, 2, 64, 64)])
@pytest.mark.parametrize("wdt", [torch.float32, torch.bfloat16])
def test_biased_preparation(H, G, dk, dv, wdt):
    """Biases, norms per head, append; alone and with the linear attention's step in the same launch."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(H * 10 + dk)
    n, eps, rh, rk, rv, rank = 7, 1e-5, 3, 20, 33, 5
    rn = lambda *s: torch.randn(*s, generator=g)
    q, k, v = rn(n, H * dk), rn(n, G * dk), rn(n, G * dv)
    bias = [rn(t.shape[1]).to(wdt) for t in (q, k, v)]
    qw, kw = (1 + 0.3 * rn(dk)).to(wdt), (1 + 0.3 * rn(dk)).to(wdt)
    pos, slots = [0, 17, 31, 32, 5, 16, 40], [1, 0, 0, 2, 2, 1, 2]
    bt = i32([[3, 8, 1], [0, 2, 7], [6, 5, 4]])
    sq, sk, sv, sg, a1 = rn(n, rh * rk), rn(n, rh * rk), rn(n, rh * rv), rn(n, rh * rv), rn(n, rank)
    a2, ab, w = rn(rh * rk, rank).to(wdt), rn(rh * rk), (1 + 0.2 * rn(rv)).to(wdt)
    for with_step in (False, True):
        kc = torch.zeros(9, G, PAGE, dk, dtype=wdt, device=DEV)
        vc = torch.zeros(9, G, PAGE, dv, dtype=wdt, device=DEV)
        rows = [0, 1, 3] if with_step else list(range(n))       # (rows alone in their entries: distinct slots)
        S = torch.full((3, rh, rk, rv), 2.0, device=DEV)
        step = (dev(sq[rows]), dev(sk[rows]), dev(sv[rows]), dev(sg[rows]), dev(a1[rows]), dev(a2), dev(ab), 4.0, S, dev(w),
                rk ** -0.5) if with_step else None
        p, s = [pos[r] for r in rows], [slots[r] for r in rows]
        for with_bias in (True, False):
            b = [dev(t) for t in bias] if with_bias else [None] * 3
            if with_step:
                S.fill_(2.0)
            got = ops.biased_qkv_prep(dev(q[rows]), dev(k[rows]), dev(v[rows]), b, G, dk, dv, dev(qw), dev(kw), eps, kc, vc,
                                      i32(p), i32(s), bt, step=step)
            if with_step:
                got, y = got
                S2 = torch.full((3, rh, rk, rv), 2.0, device=DEV)
                y2 = ops.decay_step_rows(*step[:8], S2, step[9], eps, i32(p), i32(s), q_scale=rk ** -0.5)
                assert torch.equal(y, y2) and torch.equal(S, S2)
            add = [t.double() if with_bias else 0.0 for t in bias]
            wq = O.rms_norm((q[rows].double() + add[0]).view(-1, H, dk), qw, eps)
            wk = O.rms_norm((k[rows].double() + add[1]).view(-1, G, dk), kw, eps)
            wv = (v[rows].double() + add[2]).view(-1, G, dv)
            tol = 3e-6 if wdt == torch.float32 else 6e-3
            assert rel(got, wq.reshape(len(rows), -1)) < 2e-6
            for i in range(len(rows)):
                pg = int(bt[s[i], p[i] // PAGE])
                assert rel(kc[pg, :, p[i] % PAGE], wk[i]) < tol and rel(vc[pg, :, p[i] % PAGE], wv[i]) < tol


# ------------------------------------------------------------------ streams, experts
@pytest.mark.parametrize("W,S", [(5, 1), (72, 3), (1000, 2), (2048, 4), (4100, 6), (6002, 3), (260, 16), (8192, 5)])
@pytest.mark.parametrize("wdt", [torch.float32, torch.bfloat16])
def test_streams_update(W, S, wdt):
    """Entry from the embedding; a pair of normed results; a plain sum; experts with identity ones; rows
    of a list with the streams left as they are.  The mix matrix is far from symmetric."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(W + S)
    rn = lambda *s: torch.randn(*s, generator=g)
    n, eps, E = 6, 1e-5, 4
    x, a, b, h = rn(n, S, W), rn(n, W), rn(n, W) * 3, rn(n, W)
    wa, wb, wn = (1 + 0.3 * rn(W)).to(wdt), (1 + 0.3 * rn(W)).to(wdt), (0.3 * rn(W)).to(wdt)
    mix, out, cin = rn(S, S), rn(S), rn(S).abs() + 0.1     # (factors that do not cancel on equal streams)
    norm = lambda t: O.offset_rms_norm(O.read_streams(t, cin), wn, eps)
    emb, toks = rn(11, W).to(wdt), [3, 0, 10, 3, 7, 1]
    dx = torch.empty(n, S, W, device=DEV)
    gh, cp = ops.streams_residual(dx, tokens=i32(toks), embed=dev(emb), in_=dev(cin), w_next=dev(wn), eps=eps, want_copy=True)
    ex = emb.double()[toks][:, None, :].repeat(1, S, 1)
    assert torch.equal(dx.cpu(), ex.float()) and rel(gh, norm(ex)) < 2e-6 and rel(cp, ex.sum(1)) < 1e-6
    y = 0.5 * (O.rms_norm(a, wa, eps) + O.rms_norm(b, wb, eps))
    want = O.update_streams(x.double(), y, mix, out)
    kw = dict(mix=dev(mix), out=dev(out), in_=dev(cin), w_next=dev(wn), eps=eps)
    dx = dev(x)
    gh, cp = ops.streams_residual(dx, a=dev(a), b=dev(b), w_a=dev(wa), w_b=dev(wb), want_copy=True, **kw)
    assert rel(dx, want) < 1e-6 and rel(gh, norm(want)) < 3e-6 and rel(cp, want.sum(1)) < 2e-6
    dx = dev(x)
    gb, _ = ops.streams_residual(dx, a=dev(a), b=dev(b), w_a=dev(wa), w_b=dev(wb), bf16=True, **kw)
    assert rel(gb, norm(want)) < 4e-3
    # the sum of three rows each, then the same with chosen experts: indices from E on are the identity
    a3 = rn(n * 3, W)
    dx = dev(x)
    ops.streams_residual(dx, a=dev(a3), n_a=3, **kw)
    assert rel(dx, O.update_streams(x.double(), a3.double().view(n, 3, W).sum(1), mix, out)) < 1e-6
    sel = torch.tensor([[0, 1, 2], [4, 3, 5], [5, 4, 6], [3, 6, 0], [1, 4, 2], [6, 0, 5]], dtype=torch.int32)
    sw = torch.rand(n, 3, generator=g)
    y = torch.where((sel < E)[..., None], a3.double().view(n, 3, W), sw.double()[..., None] * h.double()[:, None, :]).sum(1)
    nan = a3.clone().view(n, 3, W)
    nan[sel >= E] = float("nan")                           # (rows of identity experts are never read)
    want = O.update_streams(x.double(), y, mix, out)
    dx, dh = dev(x), dev(h)
    gh, _ = ops.streams_residual(dx, a=dev(nan.view(n * 3, W)), n_a=3, sel=(dev(sel), dev(sw), E), input=dh, h=dh, **kw)
    assert rel(dx, want) < 1e-6 and rel(dh, norm(want)) < 3e-6 and gh is dh
    # some rows only, every stream with factor one, x left as it is
    dx = dev(x)
    gh, _ = ops.streams_residual(dx, a=dev(a3), n_a=3, mix=dev(mix), out=dev(out), w_next=dev(wn), eps=eps, rows=i32([4, 1]))
    w = O.update_streams(x.double(), a3.double().view(n, 3, W).sum(1), mix, out)[[4, 1]].sum(1)
    assert rel(gh, O.offset_rms_norm(w, wn, eps)) < 3e-6 and torch.equal(dx, dev(x))
    gh, _ = ops.streams_residual(dx, w_next=dev(wn), eps=eps, rows=i32([5]))
    assert rel(gh, O.offset_rms_norm(x.double()[[5]].sum(1), wn, eps)) < 3e-6


@pytest.mark.parametrize("E,n_id,top,W", [(5, 2, 2, 32), (1, 0, 1, 24), (8, 3, 4, 41), (3, 9, 5, 64), (70, 6, 6, 96)])
@pytest.mark.parametrize("wdt", [torch.float32, torch.bfloat16])
def test_router_with_correction(E, n_id, top, W, wdt):
    """The choice follows score + correction, the weights do not; a correction that overrules the scores."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(E + W)
    n, N = 33, E + n_id
    h = torch.randn(n, W, generator=g).to(torch.bfloat16).float()
    wr = (torch.randn(N, W, generator=g) * 2 * W ** -0.5).to(wdt)
    for scale in (0.0, 0.05, 3.0):
        corr = torch.randn(N, generator=g) * scale if scale < 1 else torch.randperm(N, generator=g) * scale
        idx, wt = O.route(h, wr, corr, top)
        e, w, z = ops.moe_route_rows_corrected(dev(h), dev(wr), dev(corr), top)
        s = torch.softmax(h.double() @ wr.double().T, -1)
        c = (s + corr.double()).sort(-1, descending=True).values
        clear = torch.ones(n, dtype=torch.bool) if top == N else (c[:, top - 1] - c[:, top]) > 1e-6
        assert clear.sum() > n // 2
        assert torch.equal(e.cpu().long().sort(-1).values[clear], idx.sort(-1).values[clear])
        assert rel(w, s.gather(-1, e.cpu().long())) < 1e-5
        assert rel(z, h.double() @ wr.double().T) < 1e-5
        if scale == 3.0 and top < N:
            assert (e.cpu()[0].sort().values == e.cpu().sort(-1).values).all()      # the same experts for every row


@pytest.mark.parametrize("W,F,E,n", [(32, 20, 5, 40), (41, 13, 3, 5), (64, 96, 4, 70), (256, 64, 6, 7), (96, 32, 2, 200), (24, 1, 1, 3)])
@pytest.mark.parametrize("wdt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("limit", [0.4, 3.0])
def test_clamped_experts(W, F, E, n, wdt, limit):
    """Every form of the products (few assignments, grouped tiles, matrix cores); chosen indices from E on
    are left out, wherever they stand in a row."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(W + n)
    top = 3
    x = torch.randn(n, W, generator=g).to(torch.bfloat16).float()
    gu = (torch.randn(E, 2 * F, W, generator=g) * 1.5 * W ** -0.5).to(wdt)
    dn = (torch.randn(E, W, F, generator=g) * F ** -0.5).to(wdt)
    sel = torch.randint(0, E + 2, (n, top), generator=g, dtype=torch.int32)
    sel[0], sel[n - 1] = E, E + 1                          # rows of identity experts alone
    sel[1] = torch.tensor([E, 0, E + 1])
    sw = torch.rand(n, top, generator=g)
    for bf16_copy in (False, True):
        got = ops.moe_experts_clamped(dev(x), dev(sel), dev(sw), dev(gu), dev(dn), limit, bf16_copy=bf16_copy).cpu()
        assert torch.isnan(got[sel >= E]).all()
        for e in range(E):
            r, j = (sel == e).nonzero(as_tuple=True)
            if r.numel():
                want = sw[r, j].double()[:, None] * O.clamped_expert(x[r], gu[e, :F], gu[e, F:], dn[e], limit)
                assert rel(got[r, j], want) < (3e-6 if wdt == torch.float32 else 1e-2), e


def test_capped_rows():
    from vllm_omni_draft_amd import ops
    z = torch.randn(3, 1001, generator=torch.Generator().manual_seed(1)) * 60
    d = dev(z.clone())
    ops.cap_rows(d, 30.0)
    assert rel(d, O.soft_cap(z.double(), 30.0)) < 1e-6


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("shape", list(SHAPES))
def test_prompt_logits_match_the_plain_model(shape):
    cfg = SHAPES[shape]
    st, eng = build(cfg)
    toks = prompt(cfg, 150)
    lo = []
    want = O.forward(cfg, st, toks, lo)
    got, trace = eng.step([("a", toks, list(range(len(toks))))], layer_out=True)
    assert trace.shape[0] == len(lo) == len(cfg["layers"])
    tol = 4e-5 if shape == "ones" else 1e-5           # (norms over one channel amplify what rounds near zero)
    for i, x in enumerate(lo):
        assert rel(trace[i], x) < tol, f"residual after layer {i}"
    assert rel(got, want) < tol
    eng.finish("a")
    assert rel(eng.step([("a", toks, [0, 77, 149])]), want[[0, 77, 149]]) < tol    # without the per-layer copies


@pytest.mark.parametrize("shape,tiled", [("two_kinds", False), ("odd", False), ("ones", False), ("aligned", True),
                                         ("aligned", False), ("wide", False), ("heads128", True), ("open", True)])
def test_bfloat16_serving_stays_close(shape, tiled):
    cfg = SHAPES[shape]
    st, eng = build(cfg, torch.bfloat16, tiled=tiled)
    toks = prompt(cfg, 150, 1)
    want = O.forward(cfg, st, toks)
    got = eng.step([("a", toks, list(range(len(toks))))])
    rows = sorted(rel(got[r], want[r]) for r in range(len(toks)))
    assert rows[len(rows) // 2] < 2e-2 and rows[int(len(rows) * 0.9)] < 5e-2, rows[-5:]


@pytest.mark.parametrize("shape,dtype,tiled", [("two_kinds", torch.float32, True), ("odd", torch.float32, True),
                                               ("ones", torch.float32, True), ("wide", torch.float32, True),
                                               ("heads128", torch.float32, True), ("heads128", torch.bfloat16, True),
                                               ("open", torch.float32, True), ("odd", torch.bfloat16, False),
                                               ("aligned", torch.bfloat16, True)])
def test_cut_anywhere_batched_anyhow(shape, dtype, tiled):
    """The logits of a position are the same however its prompt was cut into steps (down to two
    tokens and to single decoded tokens), whatever else shares the batch and whichever slot and
    pages the request got."""
    cfg = SHAPES[shape]
    st, eng = build(cfg, dtype, tiled=tiled)
    pa, pb, pc = prompt(cfg, 157, 1), prompt(cfg, 134, 2), prompt(cfg, 9, 3)
    whole = {}
    for name, p in (("a", pa), ("b", pb), ("c", pc)):
        whole[name] = eng.step([(name, p, list(range(len(p))))])
        eng.finish(name)
    if dtype == torch.float32:
        for name, p in (("a", pa), ("b", pb), ("c", pc)):
            assert rel(whole[name], O.forward(cfg, st, p)) < (4e-5 if shape == "ones" else 1e-5)

    def same(x, y, what):
        # (few rows cut their keys over workgroups and merge them, many rows sweep them; a portion's
        # tokens are summed in blocks that start where it starts: the last bits differ, and in
        # bfloat16 a router's close call may fall the other way for a row)
        if dtype == torch.float32:
            assert rel(x, y) < (4e-5 if shape == "ones" else 1e-5), what
        else:
            rows = sorted(rel(x[r], y[r]) for r in range(x.shape[0]))
            assert rows[int(len(rows) * 0.9)] < 1.5e-2, what
    eng.step([("pad", prompt(cfg, 20, 9), [])])       # another slot and other pages than before
    got = torch.cat([eng.step([("a", [t], [0])]) for t in pa])
    same(got, whole["a"], "token by token")
    eng.finish("a")
    cuts_a = [0, 2, 4, 17, 19, 32, 33, 48, 57, 122, 157]
    cuts_b = [0, 16, 17, 18, 20, 34, 99, 101, 134]
    got_a, got_b, got_c = [], [], []
    ia = ib = ic = 0
    while ia < len(cuts_a) - 1 or ib < len(cuts_b) - 1 or ic < len(pc):
        entries, kinds = [], []
        if ia < len(cuts_a) - 1:
            lo, hi = cuts_a[ia], cuts_a[ia + 1]
            entries.append(("a", pa[lo:hi], list(range(hi - lo))))
            kinds.append(got_a)
            ia += 1
        if ic < len(pc):
            entries.append(("c", pc[ic:ic + 1], [0]))
            kinds.append(got_c)
            ic += 1
        if ib < len(cuts_b) - 1:
            lo, hi = cuts_b[ib], cuts_b[ib + 1]
            entries.append(("b", pb[lo:hi], list(range(hi - lo))))
            kinds.append(got_b)
            ib += 1
        out = eng.step(entries)
        at = 0
        for (_, t, _), dst in zip(entries, kinds):
            dst.append(out[at:at + len(t)])
            at += len(t)
    same(torch.cat(got_a), whole["a"], "portions of a")
    same(torch.cat(got_b), whole["b"], "portions of b")
    same(torch.cat(got_c), whole["c"], "single tokens of c")


@pytest.mark.parametrize("shape", ["two_kinds", "open"])
def test_slots_and_pages_are_used_again(shape):
    cfg = SHAPES[shape]
    st, eng = build(cfg, max_seqs=3, max_tokens=12 * PAGE, max_seq_len=6 * PAGE)
    ref = {}
    for r in range(10):
        p = prompt(cfg, 1 if r == 7 else 20 + 7 * (r % 5), r)
        ref[r] = (p, O.forward(cfg, st, p)[-1])
    live, nxt, done = {}, 0, 0
    while done < 10:
        while len(live) < 3 and nxt < 10:
            live[nxt] = 0
            nxt += 1
        entries = []
        for r in list(live):
            p = ref[r][0]
            n = min(len(p) - live[r], 13 if r % 2 else 1000)
            entries.append((str(r), p[live[r]:live[r] + n], [n - 1] if live[r] + n == len(p) else []))
            live[r] += n
        out = eng.step(entries)
        at = 0
        for rid, _, want in entries:
            if want:
                assert rel(out[at], ref[int(rid)][1]) < 1e-5, rid
                at += 1
                eng.finish(rid)
                del live[int(rid)]
                done += 1
    assert eng.free_slots == 3 and eng.cache.allocator.num_free == 12


def test_a_step_larger_than_a_pass():
    cfg = SHAPES["two_kinds"]
    st, eng = build(cfg, max_rows=16)
    pa, pb = prompt(cfg, 45, 4), prompt(cfg, 21, 5)
    out = eng.step([("a", pa, [0, 15, 16, 44]), ("b", pb, [20])])
    assert eng.passes == 5
    wa, wb = O.forward(cfg, st, pa), O.forward(cfg, st, pb)
    assert rel(out[:4], wa[[0, 15, 16, 44]]) < 1e-5 and rel(out[4], wb[20]) < 1e-5


def test_a_request_left_out_of_steps_goes_on():
    cfg = SHAPES["two_kinds"]
    st, eng = build(cfg)
    pa, pb = prompt(cfg, 40, 4), prompt(cfg, 60, 5)
    eng.step([("a", pa[:17], []), ("b", pb[:3], [])])
    for t in pb[3:50]:
        eng.step([("b", [t], [])])
    got = eng.step([("a", pa[17:], list(range(23))), ("b", pb[50:], [9])])
    assert rel(got[:23], O.forward(cfg, st, pa)[17:]) < 1e-5 and rel(got[23], O.forward(cfg, st, pb)[-1]) < 1e-5


def quiet_right(st, i=0):
    """Layer i's linear attention adds nothing."""
    st[f"l{i}.mix.right.out"] = st[f"l{i}.mix.right.out"] * 0


@pytest.mark.parametrize("window,keep", [(16, 2), (17, 1), (33, 4), (64, 0)])
def test_edges_of_window_and_kept_tokens_in_prompts_and_decoding(window, keep):
    """One layer whose linear attention is silenced, scores nearly flat: the last position's logits
    move with the oldest token of the window and with the last kept token, and not with the token before
    the window nor with the first that is not kept; in a whole prompt, cut before, at and behind each
    edge, and in single decoded tokens."""
    cfg = model_cfg([layer(heads=2, kv_heads=1, dim=8, vdim=8, window=window, keep=keep, cap=0.0, scale=0.1, tau=1.0)])
    st = tensors(cfg, 5)
    quiet_right(st)
    n = 2 * window + 9
    base = prompt(cfg, n, 6)
    edge = n - window                                     # the oldest token the last position's window holds
    w0 = O.forward(cfg, st, base)[-1]
    spots = [(edge - 1, False), (edge, True), (edge + 1, True), (keep, False)] + ([(keep - 1, True), (0, True)] if keep else [])
    for at, moves in spots:
        changed = list(base)
        changed[at] = (base[at] + 1) % cfg["vocab"]
        w1 = O.forward(cfg, st, changed)[-1]
        assert (rel(w1, w0) > 1e-5) == moves
        _, eng = build(cfg, st=st, max_seqs=2, max_tokens=1024)
        for cut in (0, max(keep, 1), edge - 1, edge, edge + 1, n - 1):
            if cut:
                eng.step([("x", changed[:cut], [])])
            got = eng.step([("x", changed[cut:], [n - 1 - cut])])[0]
            assert rel(got, w1) < 3e-6, (at, cut)
            eng.finish("x")
        eng.step([("y", changed[:5], [])])
        got = torch.cat([eng.step([("y", [t], [0])]) for t in changed[5:]])[-1]
        assert rel(got, w1) < 3e-6, at


def test_a_far_first_token_through_the_state():
    """300 positions, decays near one, a window of one token: two prompts that differ in their first
    token only differ at the end, in the plain model and, decoded token by token, in the engine."""
    cfg = model_cfg([layer(window=1, keep=0)])
    st = tensors(cfg, 5)
    st["l0.mix.right.a2.b"] = torch.full_like(st["l0.mix.right.a2.b"], 9.0)
    st["l0.mix.right.a2"] = st["l0.mix.right.a2"] * 0.1
    base, other = prompt(cfg, 300, 6), prompt(cfg, 300, 6)
    other[0] = (base[0] + 1) % cfg["vocab"]
    wa, wb = O.forward(cfg, st, base), O.forward(cfg, st, other)
    assert rel(wa[-1], wb[-1]) > 1e-4
    _, eng = build(cfg, st=st, max_seqs=2, max_tokens=1024)
    eng.step([("a", base[:100], [])])
    ga = torch.cat([eng.step([("a", [t], [0])]) for t in base[100:]])
    gb = eng.step([("b", other, [299])])
    assert rel(ga, wa[100:]) < 1e-5 and rel(gb[0], wb[-1]) < 1e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_long_decoding(dtype):
    cfg = SHAPES["heads128"] if dtype == torch.bfloat16 else SHAPES["odd"]
    st, eng = build(cfg, dtype)
    toks = prompt(cfg, 330, 7)
    want = O.forward(cfg, st, toks)
    eng.step([("a", toks[:10], [])])
    got = torch.cat([eng.step([("a", [t], [0])]) for t in toks[10:]])
    if dtype == torch.float32:
        assert rel(got, want[10:]) < 1e-5 and rel(got[-1], want[-1]) < 1e-5
    else:
        rows = sorted(rel(got[r], want[10 + r]) for r in range(320))
        assert rows[160] < 2e-2 and rows[288] < 5e-2


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_decode_steps_replayed_as_graphs(dtype):
    cfg = SHAPES["aligned"]
    st, plain = build(cfg, dtype, use_graph=False)
    _, graphed = build(cfg, dtype, use_graph=True)
    ps = [prompt(cfg, n, i) for i, n in enumerate((7, 19, 3))]
    for eng in (plain, graphed):
        eng.step([(str(i), p[:-1], []) for i, p in enumerate(ps)])
    nxt = [p[-1] for p in ps]
    for step in range(12):
        a = plain.step([(str(i), [t], [0]) for i, t in enumerate(nxt)])
        b = graphed.step([(str(i), [t], [0]) for i, t in enumerate(nxt)])
        assert torch.equal(a, b), step
        nxt = a.argmax(1).tolist()
    assert graphed.graph_replays >= 10


def test_greedy_generation_through_worker_and_scheduler():
    from vllm_omni_draft_amd import config, weights
    from vllm_omni_draft_amd.scheduler import SpecDecodeScheduler
    from vllm_omni_draft_amd.seq_engine import SeqWorker, SeqWorkerConfig
    cfg = SHAPES["two_kinds"]
    st = tensors(cfg, 3)
    mc = config.tovapel_config(cfg, {k: tuple(v.shape) for k, v in st.items()})
    worker = SeqWorker(SeqWorkerConfig(weights.seq_from_state_dict(mc, st, DEV, torch.float32), max_num_seqs=3,
                                       max_model_len=128))
    worker.init_device()
    worker.load_model()
    sched = SpecDecodeScheduler.for_worker(worker)
    prompts = [prompt(cfg, n, i) for i, n in enumerate((5, 33, 1, 18, 64, 9, 2))]   # more requests than slots
    reqs = sched.generate(prompts, max_tokens=10)
    assert worker.engine.free_slots == 3
    for p, r in zip(prompts, reqs):
        assert len(r.output_token_ids) == 10 and r.finish_reason == "length"
        toks = list(p)
        for tok in r.output_token_ids:
            logits = O.forward(cfg, st, toks)[-1]
            best = int(logits.argmax())
            if tok != best:                      # legitimate only at a near-tie of the plain model
                top = torch.topk(logits, 2).values
                assert (top[0] - top[1]) / logits.std() < 1e-4
                break
            toks.append(tok)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_command_line(tmp_path, dtype):
    """bin/trace_run on a checkpoint folder: the class chosen by config.json, steps read from
    standard input (portions beside single tokens, requests ended and their pages used again by a
    pool that holds two requests at most), logits written per step."""
    import json
    import os
    import subprocess
    import sys
    import numpy as np
    from safetensors.torch import save_file
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = SHAPES["two_kinds"]
    st = tensors(cfg, 6)
    model, out = tmp_path / "model", tmp_path / "out"
    model.mkdir()
    (model / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in st.items()}, str(model / "model.safetensors"))
    pa, pb, pc = prompt(cfg, 70, 1), prompt(cfg, 50, 2), prompt(cfg, 64, 3)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": pa[:33], "want": [0, 32]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": pa[33:35], "want": [1]}, {"id": "b", "tokens": pb[:49], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": pb[49:], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": pa[35:], "want": [34]}, {"id": "c", "tokens": pc, "want": [63]}], "end": ["a", "c"]}]
    run = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(model), "--dtype", dtype,
                          "--out", str(out), "--max-tokens", "192"], input="".join(json.dumps(s) + "\n" for s in steps),
                         capture_output=True, text=True, timeout=300)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    wa, wb, wc = (O.forward(cfg, st, p) for p in (pa, pb, pc))
    want = {0: wa[[0, 32]], 1: wa[[34]], 2: wb[[49]], 3: torch.stack([wa[69], wc[63]])}
    for n, w in want.items():
        got = torch.from_numpy(np.fromfile(str(out / f"{n}.f32"), dtype="<f4").reshape(w.shape[0], cfg["vocab"]).copy())
        assert rel(got, w) < (1e-5 if dtype == "float32" else 5e-2), n
