"""The Gufasun decoder family on the GPU against the plain CPU restatement in oracle/gufasun.py:
every mechanism alone through its entry point, then whole models through the engine (prompts
whole, token by token, in portions, in mixed batches, over reused slots and pages) and through
the worker and scheduler.  Small random models of several shapes; where random weights would hide
a fault (one far key among many, a window's edge, the first tokens, the oldest input of a
convolution, a memory that must be kept for hundreds of tokens) the inputs are made so that it shows."""

import pytest
import torch

from oracle import gufasun as G

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
def att(heads=4, kv_heads=2, dim=8, vdim=12, conv=3, scale=0.4, softcap=20.0, window=13, temp=(0.6, 7), kv_from=None, ff=24):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv, scale=scale, softcap=softcap,
             mask={"size": window} if window else None, q_temp={"coef": temp[0], "every": temp[1]} if temp else None)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def mem(heads=3, dim=8, vdim=10, cap=8.0, ff=20):
    return {"type": "mlstm", "mixer": dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap),
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model_cfg(layers, width=32, vocab=80, eps=1e-5, taps=4, scale=2.0):
    return {"architecture": "Gufasun", "width": width, "vocab": vocab, "norm": {"eps": eps}, "canon": {"taps": taps},
            "embedding": {"scale": scale}, "layers": layers}


SHAPES = {
    "two_kinds": model_cfg([att(), mem(), att(kv_from=0, window=21), mem(ff=0)]),
    # sizes that divide nothing; every pair of sizes that may coincide made different; three heads on a
    # kv head; layers that read the keys of one with other windows, scales and convolutions; no feed-forward
    "odd": model_cfg([mem(heads=2, dim=21, vdim=37, cap=3.0, ff=10),
                      att(heads=6, kv_heads=2, dim=12, vdim=20, conv=5, window=18, ff=0),
                      att(heads=6, kv_heads=2, dim=12, vdim=20, conv=2, scale=0.2, softcap=5.0, window=40, temp=(0.3, 3),
                          kv_from=1, ff=9),
                      mem(heads=5, dim=6, vdim=3, cap=20.0, ff=0),
                      att(heads=5, kv_heads=5, dim=10, vdim=7, conv=3, window=1, temp=None, ff=33),
                      att(heads=6, kv_heads=2, dim=12, vdim=20, conv=1, window=0, softcap=0.0, kv_from=1, ff=12)],
                     width=41, vocab=131, eps=1e-6, taps=3, scale=0.7),
    # one head, one channel, one tap, a window of one token, one token per step of the position factor
    "ones": model_cfg([att(heads=1, kv_heads=1, dim=1, vdim=1, conv=1, scale=1.0, window=1, temp=(1.0, 1), ff=1),
                       mem(heads=1, dim=1, vdim=1, cap=1.0, ff=4)], width=24, vocab=50, taps=1, scale=1.0),
    # widths that are multiples of 32: bfloat16 serving takes the tiled linear kernels
    "aligned": model_cfg([att(heads=4, kv_heads=2, dim=16, vdim=16, ff=64), mem(heads=2, dim=16, vdim=32, ff=96),
                          att(heads=4, kv_heads=2, dim=16, vdim=16, kv_from=0, ff=32), mem(heads=4, dim=24, vdim=16, ff=0)],
                         width=64, vocab=178),
    # heads wider than a wave, values wider than two tiles of columns, nine heads on a kv head, many taps
    "wide": model_cfg([att(heads=9, kv_heads=1, dim=72, vdim=136, conv=7, window=30), mem(heads=2, dim=130, vdim=72),
                       att(heads=16, kv_heads=2, dim=130, vdim=300, window=70, ff=40), mem(heads=1, dim=256, vdim=260, ff=40)],
                      width=48, vocab=64, taps=9),
    # one kind only: no pages at all, no recurrent state at all
    "memories": model_cfg([mem(heads=2, dim=32, vdim=64), mem(heads=2, dim=32, vdim=64, ff=0)], taps=2),
    "attentions": model_cfg([att(window=33), att(window=64, kv_from=0, ff=0)], taps=3),
    # the head sizes of larger models: bfloat16 prompts take the matrix-core kernels
    "heads128": model_cfg([att(heads=4, kv_heads=2, dim=128, vdim=128, scale=0.088, window=100, temp=(0.2, 50), ff=64),
                           mem(heads=2, dim=128, vdim=128, ff=64),
                           att(heads=4, kv_heads=2, dim=128, vdim=128, scale=0.088, window=37, kv_from=0, ff=64),
                           mem(heads=2, dim=64, vdim=128, ff=64)], width=96, vocab=160),
}


def build(cfg, dtype=torch.float32, seed=0, tiled=True, st=None, **eng_kw):
    from vllm_omni_draft_amd import config, weights
    from vllm_omni_draft_amd.seq_engine import SeqEngine, SeqEngineConfig
    st = st or G.random_tensors(cfg, seed)
    mc = config.gufasun_config(cfg, {k: tuple(v.shape) for k, v in st.items()})
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


def plain_attention(q, k, v, pos, H, Gk, scale, softcap, r1, r2, window):
    dk, dv, n = q.shape[1] // H, v.shape[1] // Gk, q.shape[0]
    q = q.to(F64).view(n, H, dk)
    k, v = (t.to(F64).view(t.shape[0], Gk, -1).repeat_interleave(H // Gk, 1) for t in (k, v))
    s = G.window_scores(q, k, pos, scale, softcap, r1, r2, window)
    return torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v).reshape(n, H * dv)


# ------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("H,Gk,dk,dv,window,cap", [(4, 2, 16, 16, 13, 5.0), (3, 1, 12, 20, 0, 0.0), (2, 2, 72, 136, 70, 2.0),
                                                   (9, 1, 8, 8, 1, 0.0), (16, 2, 8, 300, 64, 3.0), (4, 2, 128, 128, 33, 10.0),
                                                   (8, 1, 128, 64, 100, 0.0), (5, 5, 64, 128, 17, 4.0), (6, 2, 96, 80, 0, 8.0)])
@pytest.mark.parametrize("cdt", [torch.float32, torch.bfloat16])
def test_distance_attention_random(H, Gk, dk, dv, window, cap, cdt):
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(H * 100 + dk)
    n = 140
    q = torch.randn(n, H * dk, generator=g)
    k, v = torch.randn(n, Gk * dk, generator=g).to(cdt), torch.randn(n, Gk * dv, generator=g).to(cdt)
    r1, r2 = torch.rand(H, generator=g) * 2, torch.rand(H, generator=g) * 3
    pages = [5, 1, 3, 8, 0, 2, 9, 4, 7]                 # pages out of order
    kc, vc, bt = fill_pages(k, Gk, pages), fill_pages(v, Gk, pages), table(pages)
    for dist in (True, False):
        a, b = (r1, r2) if dist else (torch.zeros(H), torch.zeros(H))
        want = plain_attention(q, k, v, torch.arange(n), H, Gk, 0.3, cap, a, b, window)
        for rows in (list(range(n)), list(range(17, 90)), [n - 1], [0, 15, 16, 17, 31, 32, 44]):   # prompts, decoded rows
            for split in (True, False):                       # (split: with the rows' portion, where they are one)
                kw = dict(dist1=dev(a), dist2=dev(b)) if dist else {}
                if split and len(rows) > 64:
                    kw["entries"] = i32([[0, 0, len(rows), rows[0]]])
                got = ops.distance_softmax_attention(dev(q[rows]), kc, vc, i32(rows), i32([0] * len(rows)), bt, H, Gk, dk, dv,
                                                     0.3, window, cap, split=split, ldo=H * dv + 7, **kw)
                assert rel(got, want[rows]) < 5e-6, (len(rows), split, dist)
                gb = ops.distance_softmax_attention(dev(q[rows]), kc, vc, i32(rows), i32([0] * len(rows)), bt, H, Gk, dk, dv,
                                                    0.3, window, cap, split=split, bf16_only=True, **kw)
                assert rel(gb, want[rows]) < 4e-3


def test_window_visibility_with_one_hot_values():
    """Value of key j is the unit vector j: a row's output shows which keys it saw.  Every window edge
    in prompts of one portion and as single decoded rows, over page borders."""
    from vllm_omni_draft_amd import ops
    n, dk = 80, 128
    pages = [2, 0, 1, 4, 3]
    for window in (1, 2, 15, 16, 17, 31, 33, 64, 79, 80, 200):
        for cdt in (torch.float32, torch.bfloat16):
            k, v = torch.zeros(n, dk, dtype=cdt), torch.zeros(n, 128, dtype=cdt)
            v[torch.arange(n), torch.arange(n)] = 1
            kc, vc, bt = fill_pages(k, 1, pages), fill_pages(v, 1, pages), table(pages)
            r1, r2 = torch.tensor([0.5, 0.0]), torch.tensor([1.5, 2.0])
            for rows in (list(range(n)), [n - 1], [30, 31, 32]):
                got = ops.distance_softmax_attention(torch.zeros(len(rows), 2 * dk, device=DEV), kc, vc, i32(rows),
                                                     i32([0] * len(rows)), bt, 2, 1, dk, 128, 1.0, window, 7.0, dev(r1), dev(r2),
                                                     entries=i32([[0, 0, n, 0]]) if len(rows) == n else None)
                got = got.double().cpu().view(len(rows), 2, 128)
                for a, i in enumerate(rows):
                    for h in range(2):
                        w = torch.zeros(128, dtype=F64)
                        for j in range(max(0, i - window + 1), i + 1):
                            w[j] = (1 + float(r2[h]) * (i - j)) ** -float(r1[h])
                        w = w / w.sum()
                        assert (got[a, h] - w).abs().max() < 3e-6, (window, i, h)
                        assert ((got[a, h] > 0) == (w > 0)).all(), (window, i, h)


@pytest.mark.parametrize("cdt", [torch.float32, torch.bfloat16])
def test_a_far_key_among_hundreds(cdt):
    """700 keys, no window: head 0 points at key 3 with a score that outweighs the distance's loss and
    all others together; head 1 points at key 650."""
    from vllm_omni_draft_amd import ops
    n, H, dk, dv = 700, 2, 64, 64
    g = torch.Generator().manual_seed(11)
    k = torch.randn(n, dk, generator=g)
    k = (k / k.norm(dim=-1, keepdim=True)).to(cdt)
    v = torch.randn(n, dv, generator=g).to(cdt)
    pages = list(range(44))[::-1]
    kc, vc, bt = fill_pages(k, 1, pages), fill_pages(v, 1, pages), table(pages)
    rows = list(range(600, 700))
    r1, r2 = torch.tensor([1.5, 0.3]), torch.tensor([0.7, 5.0])
    q = torch.cat([60.0 * k[3].float(), 60.0 * k[650].float()]).repeat(len(rows), 1) + 0.1 * torch.randn(len(rows), 2 * dk, generator=g)
    want = plain_attention(q, k, v, torch.tensor(rows), H, 1, 1.0, 50.0, r1, r2, 0)
    for sel in (slice(None), slice(99, 100), slice(0, 3), slice(7, 93)):
        got = ops.distance_softmax_attention(dev(q[sel]), kc, vc, i32(rows[sel]), i32([0] * len(rows[sel])), bt, H, 1, dk, dv,
                                             1.0, 0, 50.0, dev(r1), dev(r2), entries=i32([[0, 0, len(rows[sel]), rows[sel][0]]]))
        assert rel(got, want[sel]) < 2e-5 if cdt == torch.bfloat16 else 5e-6
        assert rel(got[:, :dv], v[3].float().expand(len(rows[sel]), dv)) < 1e-3


@pytest.mark.parametrize("H,Gk,dk,dv", [(4, 1, 128, 128), (3, 3, 40, 64), (6, 2, 64, 104), (4, 2, 128, 56)])
def test_portions_of_several_sequences_on_the_matrix_cores(H, Gk, dk, dv):
    """One launch over portions of four sequences: a long one, single tokens, two tokens, one that
    starts at its first token; each row against the plain attention over its own sequence."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(dk + dv)
    n, window = 300, 61
    k, v = torch.randn(4, n, Gk * dk, generator=g).to(torch.bfloat16), torch.randn(4, n, Gk * dv, generator=g).to(torch.bfloat16)
    order = torch.randperm(76, generator=g).view(4, 19).tolist()
    kc = torch.zeros(76, Gk, PAGE, dk, dtype=torch.bfloat16, device=DEV)
    vc = torch.zeros(76, Gk, PAGE, dv, dtype=torch.bfloat16, device=DEV)
    for s in range(4):
        for j in range(n):
            kc[order[s][j // PAGE], :, j % PAGE] = k[s, j].view(Gk, dk).to(DEV)
            vc[order[s][j // PAGE], :, j % PAGE] = v[s, j].view(Gk, dv).to(DEV)
    bt = i32(order)
    portions = [(2, 190, 70), (0, 299, 1), (3, 0, 33), (1, 17, 2)]        # slot, first position, rows
    q = torch.randn(sum(p[2] for p in portions), H * dk, generator=g)
    r1, r2 = torch.rand(H, generator=g), torch.rand(H, generator=g) * 3
    ents, pos, slots, want, at = [], [], [], [], 0
    for s, p0, m in portions:
        ents.append([s, at, m, p0])
        pos += range(p0, p0 + m)
        slots += [s] * m
        want.append(plain_attention(q[at:at + m], k[s, :p0 + m], v[s, :p0 + m], torch.arange(p0, p0 + m), H, Gk, 0.2, 4.0, r1,
                                    r2, window))
        at += m
    got = ops.distance_softmax_attention(dev(q), kc, vc, i32(pos), i32(slots), bt, H, Gk, dk, dv, 0.2, window, 4.0, dev(r1),
                                         dev(r2), entries=i32(ents))
    assert rel(got, torch.cat(want)) < 5e-6
    for (s, p0, m), (_, a, _, _), w in zip(portions, ents, want):
        assert rel(got[a:a + m], w) < 5e-6, (s, p0, m)


@pytest.mark.parametrize("W,taps", [(5, 1), (72, 3), (1000, 2), (2048, 4), (4100, 6), (6002, 3)])
@pytest.mark.parametrize("wdt", [torch.float32, torch.bfloat16])
def test_residual_update_with_two_norms(W, taps, wdt):
    """The update, both layer norms, and the input convolution of single rows: two sequences decoded
    for a few tokens from the first one on, each against its whole sequence."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(W)
    T, eps = 9, 1e-5
    xs, a = torch.randn(2, T, W, generator=g) + 3.0, torch.randn(2, T, W, generator=g)   # (a mean that matters)
    w1, w2, ab = ((1 + 0.2 * torch.randn(W, generator=g)).to(wdt) for _ in range(3))
    cw = torch.randn(W, taps, generator=g).to(wdt)
    want_x = xs.double() + a.double() + ab.double()
    u = torch.stack([G.layer_norm(want_x[s], w1.float(), eps) for s in range(2)])
    hc = torch.stack([u[s] + G.causal_conv(u[s], cw.float()) for s in range(2)])
    h2 = torch.stack([G.layer_norm(want_x[s], w2.float(), eps) for s in range(2)])
    st = torch.full((3, max(taps - 1, 1), W), 7.0, device=DEV)          # (what an earlier request left)
    for t in range(T):
        x = dev(xs[:, t].clone())
        g1, g2, cp = ops.joint_residual(x, dev(a[:, t]), dev(ab), dev(w1), dev(w2), eps, x_copy=True, conv_w=dev(cw.t()),
                                        conv_state=st, row_pos=i32([t, t]), row_slot=i32([2, 0]))
        assert rel(x, want_x[:, t]) < 2e-7 and torch.equal(cp, x)
        assert rel(g1, hc[:, t]) < 2e-6 and rel(g2, h2[:, t]) < 2e-6, t
    # prompts: norms, then the convolution in its own launch, cut after four rows
    st.fill_(7.0)
    got = []
    for lo, hi in ((0, 4), (4, 5), (5, T)):
        n = hi - lo
        x = dev(torch.cat([xs[0, lo:hi], xs[1, lo:hi]]))
        av = dev(torch.cat([a[0, lo:hi], a[1, lo:hi]]))
        g1, _, _ = ops.joint_residual(x, av, dev(ab), dev(w1), dev(w2), eps)
        pos, slot = list(range(lo, hi)) * 2, [1] * n + [2] * n
        got.append(ops.conv_add_rows(g1, dev(cw.t()), st, i32(pos), i32(slot), i32([[1, 0, n, lo], [2, n, n, lo]])).view(2, n, W))
    assert rel(torch.cat(got, 1), hc) < 2e-6
    # some rows only, x left as it is
    x = dev(xs[0].clone())
    g1, _, _ = ops.joint_residual(x, dev(a[0]), dev(ab), dev(w1), None, eps, rows=i32([7, 2]))
    assert rel(g1, u[0, [7, 2]]) < 2e-6 and torch.equal(x, dev(xs[0]))
    g1, g2, _ = ops.joint_residual(x, None, None, dev(w1), dev(w2), eps, bf16=True)
    assert rel(g1, G.layer_norm(xs[0], w1.float(), eps)) < 4e-3 and g2.dtype == torch.bfloat16


@pytest.mark.parametrize("F,wdt", [(1, torch.float32), (37, torch.bfloat16), (256, torch.float32), (5001, torch.bfloat16),
                                   (8192, torch.bfloat16), (14336, torch.float32), (20004, torch.bfloat16)])
def test_activation_of_normed_powers(F, wdt):
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(F)
    z, b = torch.randn(5, F, generator=g) * 2, (torch.randn(F, generator=g) * 0.5).to(wdt)
    coef = torch.tensor([0.7, -0.4, 0.9, 0.3])
    want = G.poly_norm(z.double() + b.double(), coef, 1e-4)
    assert rel(ops.poly_norm_rows(dev(z), dev(coef), 1e-4, bias=dev(b)), want) < 2e-6
    assert rel(ops.poly_norm_rows(dev(z), dev(coef), 1e-4, bias=dev(b), bf16=True), want) < 4e-3
    assert rel(ops.poly_norm_rows(dev(z), dev(coef), 1e-4), G.poly_norm(z, coef, 1e-4)) < 2e-6
    # each power alone, so that none hides behind another
    for i in range(3):
        c = torch.zeros(4)
        c[i] = 1.0
        assert rel(ops.poly_norm_rows(dev(z), dev(c), 1e-4), G.poly_norm(z, c, 1e-4)) < 2e-6, i


@pytest.mark.parametrize("H,Gk,dk,dv,taps,temp,shared", [(4, 2, 16, 24, 3, (0.5, 4), False), (3, 3, 10, 7, 1, (0.0, 0), False),
                                                         (9, 1, 72, 136, 5, (1.0, 1), False), (6, 2, 130, 4, 4, (0.3, 9), True),
                                                         (1, 1, 1, 1, 2, (0.5, 3), False), (5, 5, 300, 500, 2, (0.2, 100), False)])
@pytest.mark.parametrize("wdt", [torch.float32, torch.bfloat16])
def test_convolved_preparation(H, Gk, dk, dv, taps, temp, shared, wdt):
    """Bias, convolution, norms, position factor and append, in portions (also single tokens) of two
    interleaved sequences, against whole sequences; the activation that rides along; the state an
    earlier request left behind does not show."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(H * 10 + dk)
    T, eps, nk = 37, 1e-5, 0 if shared else Gk
    Cq = H * dk + nk * (dk + dv)
    proj = torch.randn(2, T, Cq, generator=g)
    b, cw = torch.randn(Cq, generator=g).to(wdt), torch.randn(Cq, taps, generator=g).to(wdt)
    qw, kw = (1 + 0.3 * torch.randn(dk, generator=g)).to(wdt), (1 + 0.3 * torch.randn(dk, generator=g)).to(wdt)
    z, zb, coef = torch.randn(2, T, 19, generator=g), torch.randn(19, generator=g).to(wdt), torch.tensor([0.5, 0.4, -0.3, 0.1])
    kc = torch.zeros(8, Gk, PAGE, dk, dtype=wdt, device=DEV)
    vc = torch.zeros(8, Gk, PAGE, dv, dtype=wdt, device=DEV)
    bt = torch.zeros(3, 3, dtype=torch.int32, device=DEV)
    bt[2], bt[0] = i32([4, 0, 2]), i32([1, 7, 5])
    st = torch.full((3, max(taps - 1, 1), Cq), 9.0, device=DEV)
    got = [[], []]
    for lo, hi in ((0, 1), (1, 3), (3, 20), (20, 21), (21, 22), (22, T)):
        n = hi - lo
        act = torch.empty(2 * n, 19, device=DEV)
        q = ops.conv_attn_prep(dev(torch.cat([proj[0, lo:hi], proj[1, lo:hi]])), dev(cw.t()), st, H, Gk, dk, dv, dev(qw), dev(kw), eps,
                               None if shared else kc, None if shared else vc, i32(list(range(lo, hi)) * 2), i32([2] * n + [0] * n),
                               i32([[2, 0, n, lo], [0, n, n, lo]]), None if shared else bt, bias=dev(b), temp=temp,
                               act=(dev(torch.cat([z[0, lo:hi], z[1, lo:hi]])), dev(coef), dev(zb), act))
        for s in range(2):
            got[s].append(q[s * n:(s + 1) * n])
            assert rel(act[s * n:(s + 1) * n], G.poly_norm(z[s, lo:hi].double() + zb.double(), coef, eps)) < 2e-6
    for s, pages in ((0, [4, 0, 2]), (1, [1, 7, 5])):
        y = G.causal_conv(proj[s].double() + b.double(), cw.float())
        wq = G.rms_norm(y[:, :H * dk].reshape(T, H, dk), qw.float(), eps)
        if temp[1]:
            wq = wq * G.query_temperature(torch.arange(T), *temp)[:, None, None]
        assert rel(torch.cat(got[s]), wq.reshape(T, -1)) < 2e-6
        if shared:
            continue
        wk = G.rms_norm(y[:, H * dk:(H + Gk) * dk].reshape(T, Gk, dk), kw.float(), eps)
        wv = y[:, (H + Gk) * dk:].reshape(T, Gk, dv)
        tol = 3e-6 if wdt == torch.float32 else 6e-3
        ck = torch.stack([kc[pages[p // PAGE], :, p % PAGE] for p in range(T)])
        cv = torch.stack([vc[pages[p // PAGE], :, p % PAGE] for p in range(T)])
        assert rel(ck, wk) < tol and rel(cv, wv) < tol


@pytest.mark.parametrize("H,dk,dv", [(2, 16, 24), (3, 21, 37), (1, 1, 1), (2, 130, 72), (4, 256, 260), (1, 5, 400), (2, 128, 128),
                                     (2, 64, 192), (3, 32, 64), (1, 96, 40)])
@pytest.mark.parametrize("form", ["chunks", "tokens", "step"])
def test_matrix_memory(H, dk, dv, form):
    """Scan (in chunks, token by token, single tokens in one launch) and read-out in portions of two interleaved sequences (down to single tokens), from slots
    an earlier request left full, against the plain recurrence; the activation that rides along."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(H * 1000 + dk)
    T, cap, eps = 233, 9.0, 1e-5
    rn = lambda *s: torch.randn(*s, generator=g)
    q, k, v, gate = rn(2, T, H * dk), rn(2, T, H * dk), rn(2, T, H * dv), rn(2, T, H * dv)
    zi, zf = rn(2, T, H) * 4, rn(2, T, H) * 4
    bi, bf = rn(H), rn(H) + 2
    w, coef = 1 + 0.2 * rn(H * dv), torch.tensor([0.5, 0.4, -0.3, 0.1])
    z = rn(2, T, 23)
    S, N, M = (torch.full((3, H) + s, 5.0, device=DEV) for s in ((dk, dv), (dk,), ()))
    got = [[], []]
    for lo, hi in ((0, 1), (1, 2), (2, 70), (70, 71), (71, 73), (73, 74), (74, 139), (139, 203), (203, T)):
        n = hi - lo
        cat = lambda t: dev(torch.cat([t[0, lo:hi], t[1, lo:hi]]))
        if form == "step" and n == 1:
            y, a = ops.mlstm_step(cat(q), cat(k), cat(v), cat(zi), cat(zf), dev(bi), dev(bf), cap, S, N, M, i32([lo, lo]),
                                  i32([2, 0]), cat(gate), dev(w), eps, q_scale=dk ** -0.5, act=(cat(z), dev(coef), None))
            for s in range(2):
                got[s].append(y[s:s + 1])
                assert rel(a[s:s + 1], G.poly_norm(z[s, lo:hi], coef, eps)) < 2e-6
            continue
        num, mr = ops.mlstm_scan(cat(q), cat(k), cat(v), cat(zi), cat(zf), dev(bi), dev(bf), cap, S, N, M,
                                 i32([[2, 0, n, lo], [0, n, n, lo]]), q_scale=dk ** -0.5, chunks=form == "chunks")
        y, a = ops.mlstm_read(num, mr, M, i32([2] * n + [0] * n), cat(gate), dev(w), eps, act=(cat(z), dev(coef), None))
        for s in range(2):
            got[s].append(y[s * n:(s + 1) * n])
            assert rel(a[s * n:(s + 1) * n], G.poly_norm(z[s, lo:hi], coef, eps)) < 2e-6
    for s in range(2):
        li = cap * torch.tanh((zi[s].double() + bi.double()) / cap)
        lf = torch.nn.functional.logsigmoid(cap * torch.tanh((zf[s].double() + bf.double()) / cap))
        o = G.mlstm_read(q[s].double().view(T, H, dk) * dk ** -0.5, k[s].double().view(T, H, dk), v[s].double().view(T, H, dv), li, lf)
        want = G.rms_norm(o, None, eps).reshape(T, H * dv) * w.double() * torch.sigmoid(gate[s].double())
        gs = torch.cat(got[s])
        assert rel(gs, want) < 5e-5
        # (a head whose numerator nearly cancels is only as exact as its terms: most rows are far closer)
        rows = sorted(rel(gs[t], want[t]) for t in range(T))
        assert rows[T // 2] < 4e-6, rows[T // 2]


def test_the_memory_keeps_a_first_token_for_hundreds():
    """Forget gates near one and input gates near zero after the first token: 600 tokens later the
    memory still returns the first token's value."""
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(7)
    T, H, dk, dv, cap = 600, 1, 32, 32, 15.0
    k = torch.randn(T, dk, generator=g)
    q, v = k[0].repeat(T, 1) / k[0].norm() ** 2, torch.randn(T, dv, generator=g)
    zi, zf = torch.full((T, 1), -200.0), torch.full((T, 1), 200.0)
    zi[0] = 200.0
    S, N, M = (torch.zeros((1, H) + s, device=DEV) for s in ((dk, dv), (dk,), ()))
    outs = []
    for lo, hi in ((0, 1), (1, 300), (300, 301), (301, T)):
        num, mr = ops.mlstm_scan(dev(q[lo:hi]), dev(k[lo:hi]), dev(v[lo:hi]), dev(zi[lo:hi]), dev(zf[lo:hi]), torch.zeros(1, device=DEV),
                                 torch.zeros(1, device=DEV), cap, S, N, M, i32([[0, 0, hi - lo, lo]]))
        ops.mlstm_read(num, mr, M, i32([0] * (hi - lo)), torch.zeros(hi - lo, dv, device=DEV), torch.ones(dv, device=DEV), 1e-5)
        outs.append((num[:, 0, :dv] / num[:, 0, dv:]).cpu())
    o = torch.cat(outs)
    assert rel(o[-1], v[0]) < 1e-4 and rel(o[299], v[0]) < 1e-4


def test_two_inputs_of_one_stacked_product():
    from vllm_omni_draft_amd import ops
    g = torch.Generator().manual_seed(2)
    for M, n1, n2, K in ((1, 16, 5, 32), (4, 208, 96, 64), (16, 5008, 4096, 1024), (7, 32, 17, 2080)):
        w = (torch.randn(n1 + n2, K, generator=g) * K ** -0.5).to(torch.bfloat16)
        x, x2 = torch.randn(M, K, generator=g).to(torch.bfloat16), torch.randn(M, K, generator=g).to(torch.bfloat16)
        got = ops.linear_two_inputs(ops.tile_weights(dev(w), ops.TILE_PLAIN), dev(x), dev(x2), n1)
        want = torch.cat([x.double() @ w[:n1].double().T, x2.double() @ w[n1:].double().T], 1)
        assert rel(got, want) < 1e-5 and rel(got[:, n1:], want[:, n1:]) < 1e-5, (M, n1, n2, K)


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("shape", list(SHAPES))
def test_prompt_logits_match_the_plain_model(shape):
    cfg = SHAPES[shape]
    st, eng = build(cfg)
    toks = prompt(cfg, 150)
    lo = []
    want = G.forward(cfg, st, toks, lo)
    got, trace = eng.step([("a", toks, list(range(len(toks))))], layer_out=True)
    assert trace.shape[0] == len(lo) == len(cfg["layers"])
    for i, x in enumerate(lo):
        assert rel(trace[i], x) < 1e-5, f"residual after layer {i}"
    assert rel(got, want) < 1e-5
    eng.finish("a")
    assert rel(eng.step([("a", toks, [0, 77, 149])]), want[[0, 77, 149]]) < 1e-5   # without the per-layer copies


@pytest.mark.parametrize("shape,tiled", [("two_kinds", False), ("odd", False), ("ones", False), ("aligned", True),
                                         ("aligned", False), ("wide", False), ("heads128", True), ("memories", True)])
def test_bfloat16_serving_stays_close(shape, tiled):
    cfg = SHAPES[shape]
    st, eng = build(cfg, torch.bfloat16, tiled=tiled)
    toks = prompt(cfg, 150, 1)
    want = G.forward(cfg, st, toks)
    got = eng.step([("a", toks, list(range(len(toks))))])
    rows = sorted(rel(got[r], want[r]) for r in range(len(toks)))
    assert rows[len(rows) // 2] < 2e-2 and rows[int(len(rows) * 0.9)] < 5e-2, rows[-5:]


@pytest.mark.parametrize("shape,dtype,tiled", [("two_kinds", torch.float32, True), ("odd", torch.float32, True),
                                               ("ones", torch.float32, True), ("wide", torch.float32, True),
                                               ("heads128", torch.float32, True), ("heads128", torch.bfloat16, True),
                                               ("odd", torch.bfloat16, False), ("aligned", torch.bfloat16, True)])
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
            assert rel(whole[name], G.forward(cfg, st, p)) < 1e-5

    def same(x, y, what):
        # (few rows cut their keys over workgroups and merge them, many rows sweep them; a portion's
        # tokens are summed in chunks that start where it starts: the last bits differ)
        assert rel(x, y) < (1e-5 if dtype == torch.float32 else 1.5e-2), what
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


@pytest.mark.parametrize("shape", ["two_kinds", "memories"])
def test_slots_and_pages_are_used_again(shape):
    cfg = SHAPES[shape]
    st, eng = build(cfg, max_seqs=3, max_tokens=12 * PAGE, max_seq_len=6 * PAGE)
    ref = {}
    for r in range(10):
        p = prompt(cfg, 1 if r == 7 else 20 + 7 * (r % 5), r)
        ref[r] = (p, G.forward(cfg, st, p)[-1])
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
    wa, wb = G.forward(cfg, st, pa), G.forward(cfg, st, pb)
    assert rel(out[:4], wa[[0, 15, 16, 44]]) < 1e-5 and rel(out[4], wb[20]) < 1e-5


def test_a_request_left_out_of_steps_goes_on():
    cfg = SHAPES["two_kinds"]
    st, eng = build(cfg)
    pa, pb = prompt(cfg, 40, 4), prompt(cfg, 60, 5)
    eng.step([("a", pa[:17], []), ("b", pb[:3], [])])
    for t in pb[3:50]:
        eng.step([("b", [t], [])])
    got = eng.step([("a", pa[17:], list(range(23))), ("b", pb[50:], [9])])
    assert rel(got[:23], G.forward(cfg, st, pa)[17:]) < 1e-5 and rel(got[23], G.forward(cfg, st, pb)[-1]) < 1e-5


@pytest.mark.parametrize("window", [16, 17, 33, 64])
def test_a_windows_edge_in_prompts_and_decoding(window):
    """One attention layer without convolutions (one tap), scores nearly flat: the last position's logits move with the
    token window - 1 before it and do not move with the token window before it; in a whole prompt, cut
    before, at and behind the edge, and in single decoded tokens."""
    cfg = model_cfg([att(heads=2, kv_heads=1, dim=8, vdim=8, conv=1, window=window, softcap=0.0, scale=0.1, ff=0)], taps=1)
    st = G.random_tensors(cfg, 5)
    st["l0.mix.r1"] = st["l0.mix.r1"] * 0.1
    n = 2 * window + 5
    base = prompt(cfg, n, 6)
    edge = n - window                                     # the oldest token the last position sees
    w0 = G.forward(cfg, st, base)[-1]
    for at, moves in ((edge - 1, False), (edge, True), (edge + 1, True)):
        changed = list(base)
        changed[at] = (base[at] + 1) % cfg["vocab"]
        w1 = G.forward(cfg, st, changed)[-1]
        assert (rel(w1, w0) > 1e-5) == moves
        _, eng = build(cfg, st=st, max_seqs=2, max_tokens=1024)
        for cut in (0, edge - 1, edge, edge + 1, n - 1):
            if cut:
                eng.step([("x", changed[:cut], [])])
            got = eng.step([("x", changed[cut:], [n - 1 - cut])])[0]
            assert rel(got, w1) < 3e-6, (at, cut)
            eng.finish("x")
        eng.step([("y", changed[:5], [])])
        got = torch.cat([eng.step([("y", [t], [0])]) for t in changed[5:]])[-1]
        assert rel(got, w1) < 3e-6, at


def test_the_oldest_input_of_a_convolution():
    """Nothing but convolutions reaches back here (a window of one token, one layer): the logits at a
    position move with the token taps - 1 + taps' - 1 before it and with none earlier, in a prompt
    cut between them and in single tokens."""
    cfg = model_cfg([att(heads=2, kv_heads=2, dim=8, vdim=8, conv=4, window=1, ff=0)], taps=3)
    st = G.random_tensors(cfg, 8)
    base = prompt(cfg, 30, 6)
    reach = (4 - 1) + (3 - 1)
    w0 = G.forward(cfg, st, base)
    for back, moves in ((reach + 1, False), (reach, True), (1, True)):
        changed = list(base)
        changed[29 - back] = (base[29 - back] + 1) % cfg["vocab"]
        w1 = G.forward(cfg, st, changed)
        assert (rel(w1[29], w0[29]) > 1e-5) == moves
        _, eng = build(cfg, st=st, max_seqs=2, max_tokens=256)
        for cut in range(22, 30):
            eng.step([("x", changed[:cut], [])])
            assert rel(eng.step([("x", changed[cut:], [29 - cut])])[0], w1[29]) < 3e-6, (back, cut)
            eng.finish("x")
        got = torch.cat([eng.step([("y", [t], [0])]) for t in changed])
        assert rel(got, w1) < 3e-6                         # (the first tokens of the sequence among them)
        assert rel(eng.step([("z", changed[:1], [0])]), w1[:1]) < 3e-6


def test_a_far_first_token_through_the_memory():
    """300 positions, forget gates near one: two prompts that differ in their first token only differ
    at the end, in the plain model and, decoded token by token, in the engine."""
    cfg = model_cfg([mem(heads=2, dim=8, vdim=8, cap=15.0, ff=0)], taps=2)
    st = G.random_tensors(cfg, 5)
    st["l0.mix.f.b"], st["l0.mix.f"] = torch.full((2,), 8.0), st["l0.mix.f"] * 0.1
    base, other = prompt(cfg, 300, 6), prompt(cfg, 300, 6)
    other[0] = (base[0] + 1) % cfg["vocab"]
    wa, wb = G.forward(cfg, st, base), G.forward(cfg, st, other)
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
    want = G.forward(cfg, st, toks)
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
    st = G.random_tensors(cfg, 3)
    mc = config.gufasun_config(cfg, {k: tuple(v.shape) for k, v in st.items()})
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
            logits = G.forward(cfg, st, toks)[-1]
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
    st = {k: v.to(torch.bfloat16).float() for k, v in G.random_tensors(cfg, 6).items()}
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
    wa, wb, wc = (G.forward(cfg, st, p) for p in (pa, pb, pc))
    want = {0: wa[[0, 32]], 1: wa[[34]], 2: wb[[49]], 3: torch.stack([wa[69], wc[63]])}
    for n, w in want.items():
        got = torch.from_numpy(np.fromfile(str(out / f"{n}.f32"), dtype="<f4").reshape(w.shape[0], cfg["vocab"]).copy())
        assert rel(got, w) < (1e-5 if dtype == "float32" else 5e-2), n
