"""Host-side parts of the Gufasun family that need no GPU: the configuration reader and model
registry, the caches' shapes, the stacked weights, and the plain CPU model's own consistency
(causality, the convolutions, the window, the query's position factor, the distance's logarithm,
shared keys, the matrix memory against its unscaled form, the activation)."""
import json
import math
import os
import subprocess

import pytest
import torch

from oracle import gufasun as G

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64

ATT = {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 10, "conv": 4, "scale": 0.4, "softcap": 20.0, "mask": {"size": 9},
       "q_temp": {"coef": 0.7, "every": 5}}
CFG = {"architecture": "Gufasun", "width": 40, "vocab": 70, "norm": {"eps": 1e-6}, "canon": {"taps": 5},
       "embedding": {"scale": 3.0},
       "layers": [
           {"type": "attention", "mixer": ATT, "mlp": {"kind": "dense", "ff": 24}},
           {"type": "mlstm", "mixer": {"heads": 3, "dim": 8, "vdim": 12, "gate_cap": 6.0}, "mlp": None},
           {"type": "attention", "mixer": dict(ATT, kv_from=0, mask={"size": 20}, conv=2, scale=0.3),
            "mlp": {"kind": "dense", "ff": 17}},
       ]}


def toks(n, seed=0):
    return torch.randint(0, CFG["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def rn(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


def test_plain_model_is_causal():
    st = G.random_tensors(CFG, 1)
    t = toks(40)
    whole = G.forward(CFG, st, t)
    for n in (1, 2, 5, 9, 10, 23):
        assert torch.allclose(G.forward(CFG, st, t[:n]), whole[:n], atol=1e-9, rtol=0)
    assert not torch.allclose(G.forward(CFG, st, t[1:])[-1], whole[-1], atol=1e-6)     # what came before is remembered


def test_causal_convolution_written_out():
    u, w = rn(7, 3), rn(3, 4, seed=1)
    y = G.causal_conv(u, w)
    for t in range(7):
        for c in range(3):
            want = sum(w[c, j] * u[t - 3 + j, c] for j in range(4) if t - 3 + j >= 0)
            assert abs(y[t, c] - want) < 1e-12
    assert torch.allclose(G.causal_conv(u, w[:, 3:]), w[:, 3] * u)                     # one tap: a factor per channel
    assert torch.allclose(G.causal_conv(u[:2], w), y[:2])                              # fewer tokens than taps


def test_window_and_distance_of_the_scores():
    q, k = rn(3, 2, 4), rn(30, 2, 4, seed=1)
    r1, r2 = torch.tensor([0.5, 0.0], dtype=F64), torch.tensor([2.0, 3.0], dtype=F64)
    pos = [4, 12, 29]
    s = G.window_scores(q, k, pos, 0.5, 3.0, r1, r2, 6)
    for h in range(2):
        for a, i in enumerate(pos):
            for j in range(30):
                if not 0 <= i - j < 6:
                    assert s[h, a, j] == -math.inf
                    continue
                raw = 3.0 * math.tanh(float(q[a, h] @ k[j, h]) * 0.5 / 3.0)
                assert abs(float(s[h, a, j]) - (raw - float(r1[h]) * math.log(1 + float(r2[h]) * (i - j)))) < 1e-12
    assert (G.window_scores(q, k, pos, 0.5, 0.0, r1, r2, None)[:, 2] > -math.inf).all()   # no window: all before


def test_query_temperature_steps():
    f = G.query_temperature(torch.arange(12), 0.5, 5)
    for p in range(12):
        assert abs(float(f[p]) - (1 + 0.5 * math.log((p + 1) // 5 + 1))) < 1e-14
    assert f[3] == 1 and f[4] > 1 and f[8] == f[4] and f[9] > f[8]


def test_matrix_memory_equals_its_unscaled_form():
    """The running maximum only keeps numbers in range: with S and n multiplied back by e^m the read
    vector is S^T q / (max(|n . q|, 1) + 1e-6 e^m)."""
    T, H, dk, dv = 25, 2, 4, 5
    q, k, v = rn(T, H, dk), rn(T, H, dk, seed=1), rn(T, H, dv, seed=2)
    li, lf = rn(T, H, seed=3) * 2, -rn(T, H, seed=4).abs()
    got = G.mlstm_read(q, k, v, li, lf)
    for h in range(H):
        S, n, m = torch.zeros(dk, dv, dtype=F64), torch.zeros(dk, dtype=F64), 0.0
        for t in range(T):
            keep, add = math.exp(float(lf[t, h])), math.exp(float(li[t, h]))
            S, n = keep * S + add * torch.outer(k[t, h], v[t, h]), keep * n + add * k[t, h]
            m = max(float(lf[t, h]) + m, float(li[t, h]))
            den = max(abs(float(n @ q[t, h])), 1.0) + 1e-6 * math.exp(m)
            assert torch.allclose(got[t, h], S.T @ q[t, h] / den, atol=1e-12)


def test_gates_are_capped():
    t = {"i": rn(2, 3) * 100, "i.b": rn(2), "f": rn(2, 3, seed=1) * 100, "f.b": rn(2)}
    li, lf = G.mlstm_gates(rn(6, 3, seed=2) * 10, t, 4.0)
    assert li.abs().max() <= 4.0 and lf.max() <= 0 and lf.min() >= -math.log(1 + math.exp(4.0)) - 1e-12


def test_activation_of_normed_powers():
    z, act, eps = rn(3, 7), torch.tensor([0.5, -0.4, 0.3, 0.2]), 1e-3
    got = G.poly_norm(z, act, eps)
    for r in range(3):
        want = torch.full((7,), float(act[3]), dtype=F64)
        for p in range(3):
            y = z[r] ** (p + 1)
            want = want + float(act[p]) * y / math.sqrt(float((y * y).mean()) + eps)
        assert torch.allclose(got[r], want, atol=1e-12)


def test_both_sublayers_read_the_same_residual():
    cfg = dict(CFG, layers=CFG["layers"][:1])
    st = G.random_tensors(cfg, 6)
    t = toks(12)
    lo = []
    G.forward(cfg, st, t, lo)
    x = st["embed"].double()[t] * 3.0
    u = G.layer_norm(x, st["l0.norm1"], 1e-6)
    y = G.attention(u + G.causal_conv(u, st["l0.canon1"]), dict(ATT, eps=1e-6), G.sub(st, "l0.mix."), torch.arange(12))
    f = G.feed_forward(G.layer_norm(x, st["l0.norm2"], 1e-6), G.sub(st, "l0.mlp."), 1e-6)
    assert torch.allclose(lo[0], x + y + f, atol=1e-12)
    # a layer norm, not an RMS norm: a constant added to every channel changes nothing
    assert torch.allclose(G.layer_norm(x + 5.0, st["l0.norm1"], 0.0), G.layer_norm(x, st["l0.norm1"], 0.0), atol=1e-9)


def test_shared_keys_are_the_source_layers():
    st = G.random_tensors(CFG, 3)
    m0, m2 = dict(CFG["layers"][0]["mixer"], eps=1e-6), dict(CFG["layers"][2]["mixer"], eps=1e-6)
    h0, h2 = rn(15, 40), rn(15, 40, seed=1)
    t0, t2 = G.sub(st, "l0.mix."), G.sub(st, "l2.mix.")
    assert "k" not in t2 and "v" not in t2 and "k.conv" not in t2
    kv = G.keys_values(h0, m0, t0)
    got = G.attention(h2, m2, t2, torch.arange(15), kv=kv)
    own = dict(t2, **{n: t0[n] for n in ("k", "v", "k.b", "v.b", "k.conv", "v.conv", "k.norm")})
    assert not torch.allclose(got, G.attention(h2, m2, own, torch.arange(15)), atol=1e-3)
    assert torch.allclose(got, G.attention(h2, m2, own, torch.arange(15), kv=G.keys_values(h0, m2, own)), atol=1e-12)


def test_config_reader_and_registry(tmp_path):
    from safetensors.torch import save_file
    from vllm_omni_draft_amd import config
    st = G.random_tensors(CFG, 2)
    (tmp_path / "config.json").write_text(json.dumps(CFG))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in st.items()}, str(tmp_path / "model.safetensors"))
    mc = config.load_model_config(str(tmp_path))
    assert isinstance(mc, config.SeqModelConfig) and (mc.arch, mc.block, mc.n_layers) == ("gufasun", "joint", 3)
    assert (mc.embed_scale, mc.tied_head, mc.norm_eps, mc.n_runs) == (3.0, False, 1e-6, 3)
    a, b, c = (l.mixer for l in mc.layers)
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.softcap, a.window, a.conv_taps, a.q_temp_coef,
            a.q_temp_every, a.kv_from) == ("softmax_attention", 4, 2, 6, 10, 0.4, 20.0, 9, 4, 0.7, 5, -1)
    assert a.qk_head_norm and a.qkv_bias and a.distance_bias and not (a.qk_full_norm or a.proj_bias or a.sink)
    assert (b.kind, b.heads, b.dim, b.vdim, b.gate_cap) == ("mlstm", 3, 8, 12, 6.0)
    assert (c.kv_from, c.window, c.conv_taps, c.scale) == (0, 20, 2, 0.3)
    assert [l.ff for l in mc.layers] == [24, 0, 17] and all(l.in_taps == 5 and l.ff_act == "polynorm" for l in mc.layers)
    assert a.conv_channels == 4 * 6 + 2 * (6 + 10) and c.conv_channels == 24
    assert mc.state_bytes_per_seq() == 4 * (3 * 4 * 40 + 3 * 56 + 1 * 24 + 3 * (8 * 13 + 1))
    assert mc.param_count() == sum(v.numel() for v in st.values())


def test_parts_that_may_be_absent():
    from vllm_omni_draft_amd import config
    cfg = json.loads(json.dumps(CFG))
    m = cfg["layers"][0]["mixer"]
    m["softcap"] = m["q_temp"] = m["mask"] = None
    cfg["canon"] = None
    mc = config.gufasun_config(cfg)
    a = mc.layers[0].mixer
    assert (a.softcap, a.q_temp_every, a.window, mc.layers[0].in_taps) == (0.0, 0, 0, 0)


@pytest.mark.parametrize("path,value", [
    (("layers", 0, "type"), "conv"),
    (("layers", 0, "mixer", "kv_heads"), 3),
    (("layers", 0, "mixer", "conv"), 0),
    (("layers", 0, "mixer", "dim"), 513),
    (("layers", 1, "mixer", "gate_cap"), 0.0),
    (("layers", 1, "mixer", "dim"), 300),
    (("layers", 2, "mixer", "kv_from"), 2),                     # itself
    (("layers", 2, "mixer", "kv_from"), 1),                     # a layer of the other kind
    (("layers", 2, "mixer", "kv_heads"), 4),                    # another head layout than its source
    (("layers", 0, "mlp", "kind"), "moe"),
])
def test_config_reader_refuses(path, value):
    from vllm_omni_draft_amd import config
    cfg = json.loads(json.dumps(CFG))
    node = cfg
    for k in path[:-1]:
        node = node[k]
    node[path[-1]] = value
    with pytest.raises(ValueError):
        config.gufasun_config(cfg)


def test_what_a_sequence_keeps():
    from vllm_omni_draft_amd import _lib, config
    from vllm_omni_draft_amd.kv_cache import PAGE, SeqCache
    if not os.path.exists(_lib.lib_path()):
        subprocess.run(["make", "-C", ROOT, "-j8"], check=True)
    mc = config.gufasun_config(CFG)
    c = SeqCache(mc, torch.bfloat16, max_seqs=3, num_pages=7, max_seq_len=4 * PAGE, device="cpu")
    assert c.has_pages and sorted(c.k) == sorted(c.v) == [0] and c.kv_source == {2: 0} and c.keys_of(2) is c.k[0]
    assert c.k[0].shape == (7, 2, PAGE, 6) and c.v[0].shape == (7, 2, PAGE, 10) and c.k[0].dtype == torch.bfloat16
    assert c.conv[0].shape == (3, 3, 56) and c.conv[2].shape == (3, 1, 24) and sorted(c.conv) == [0, 2]
    assert [c.in_conv[i].shape for i in range(3)] == [(3, 4, 40)] * 3
    assert c.state[1].shape == (3, 3, 8, 12) and c.nstate[1].shape == (3, 3, 8) and c.mstate[1].shape == (3, 3)
    assert all(t.dtype == torch.float32 for d in (c.conv, c.in_conv, c.state, c.nstate, c.mstate) for t in d.values())
    per_slot = mc.state_bytes_per_seq()
    assert c.nbytes() == 3 * per_slot + 2 * (c.k[0].numel() + c.v[0].numel())


def test_weights_are_stacked_per_layer():
    from vllm_omni_draft_amd import config, weights
    st = G.random_tensors(CFG, 3)
    mc = config.gufasun_config(CFG)
    w = weights.seq_from_state_dict(mc, st, "cpu", torch.float32)
    a, b, c = w.layers
    assert a.mix_rows == 64 and a.w_in.shape == (64 + 24, 40) and a.w_in[56:64].abs().sum() == 0    # padded to 16 rows
    assert torch.equal(a.w_in[46 - 10:46], st["l0.mix.v"][:10]) and torch.equal(a.w_in[64:], st["l0.mlp.up"])
    assert torch.equal(a.w_o, torch.cat([st["l0.mix.o"], st["l0.mlp.down"]], 1)) and torch.equal(a.w_o_bias, st["l0.mlp.down.b"])
    assert a.conv_w.shape == (4, 56) and torch.equal(a.conv_w[:, 24:36].t(), st["l0.mix.k.conv"])
    assert torch.equal(a.w_in_bias, torch.cat([st["l0.mix.q.b"], st["l0.mix.k.b"], st["l0.mix.v.b"]]))
    assert torch.equal(a.dist1, st["l0.mix.r1"]) and torch.equal(a.ff_coef, st["l0.mlp.act"]) and a.ff_coef.dtype == torch.float32
    assert b.mix_rows == 128 and b.w_in.shape == (128, 40) and b.w_in[126:].abs().sum() == 0
    assert torch.equal(b.w_in[120:123], st["l1.mix.i"]) and torch.equal(b.w_in[123:126], st["l1.mix.f"])
    assert torch.equal(b.gate_bias, torch.cat([st["l1.mix.i.b"], st["l1.mix.f.b"]])) and b.w_o.shape == (40, 36)
    assert b.norm2_w is None and b.w_o_bias is None and b.ff_coef is None
    assert c.mix_rows == 32 and c.conv_w.shape == (2, 24) and c.k_norm_w is None and c.w_in_bias.shape == (24,)
    st2 = weights.seq_random_state(mc, 0)
    assert {k: tuple(v.shape) for k, v in st2.items()} == {k: tuple(v.shape) for k, v in st.items()}
    del st["l1.mix.f.b"]
    with pytest.raises(KeyError):
        weights.seq_from_state_dict(mc, st, "cpu", torch.float32)
