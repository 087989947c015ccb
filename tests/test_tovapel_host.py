"""Host-side parts of the Tovapel family that need no GPU: the configuration reader and model
registry, the caches' shapes, the stacked weights, and the plain CPU model's own consistency
(causality, visibility, the sink, the recurrence in portions, the streams' update, identity experts,
the corrected choice, the clamped activation)."""
import json
import math
import os
import subprocess

import pytest
import torch

from oracle import tovapel as O

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64

LEFT = {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 10, "scale": 0.4, "softcap": 20.0, "mask": {"size": 9, "keep_first": 2}}
RIGHT = {"heads": 3, "dim": 5, "vdim": 7, "tau": 4.0}
CFG = {"architecture": "Tovapel", "width": 40, "vocab": 70, "norm": {"eps": 1e-6}, "streams": 2, "logit_softcap": 15.0,
       "layers": [
           {"type": "parallel", "mixer": {"left": LEFT, "right": RIGHT}, "mlp": {"kind": "dense", "ff": 24}},
           {"type": "parallel", "mixer": {"left": dict(LEFT, kv_heads=4, mask={"size": 20, "keep_first": 0}),
                                          "right": dict(RIGHT, heads=5, vdim=8)},
            "mlp": {"kind": "moe", "router": {"experts": 3, "top": 2, "identity": 2}, "expert": {"ff": 11, "limit": 0.7}}},
           {"type": "parallel", "mixer": {"left": dict(LEFT, heads=2), "right": dict(RIGHT, heads=2, vdim=10)}, "mlp": None},
       ]}
RANKS = [3, 4, 1]


def state(seed=0, cfg=CFG):
    return O.random_tensors(cfg, RANKS, seed)


def toks(n, seed=0):
    return torch.randint(0, CFG["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def rn(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


def test_plain_model_is_causal():
    st = state(1)
    t = toks(40)
    whole = O.forward(CFG, st, t)
    for n in (1, 2, 5, 9, 10, 23):
        assert torch.allclose(O.forward(CFG, st, t[:n]), whole[:n], atol=1e-9, rtol=0)
    assert not torch.allclose(O.forward(CFG, st, t[1:])[-1], whole[-1], atol=1e-6)     # what came before is remembered
    assert whole.abs().max() < 15.0


def test_window_kept_tokens_cap_and_sink_written_out():
    q, k, v = rn(3, 2, 4), rn(30, 1, 4, seed=1), rn(30, 1, 5, seed=2)
    sink, pos = torch.tensor([0.5, -2.0], dtype=F64), [4, 12, 29]
    got = O.attend(q, k, v, pos, 0.5, 6, 3, 2.0, sink)
    for a, i in enumerate(pos):
        for h in range(2):
            num, den = torch.zeros(5, dtype=F64), math.exp(float(sink[h]))
            for j in range(i + 1):
                assert O.visible(i, j, 6, 3) == (i - j < 6 or j < 3)
                if O.visible(i, j, 6, 3):
                    w = math.exp(2.0 * math.tanh(float(q[a, h] @ k[j, 0]) * 0.5 / 2.0))
                    num, den = num + w * v[j, 0], den + w
            assert torch.allclose(got[a, h], num / den, atol=1e-12)
    assert not O.visible(5, 6, 6, 9) and O.visible(29, 2, 6, 3) and not O.visible(29, 3, 6, 3) and O.visible(29, 0, 0, 0)


def test_recurrence_in_portions_and_written_out():
    q, k, v = rn(9, 2, 3), rn(9, 2, 3, seed=1), rn(9, 2, 4, seed=2)
    d = torch.sigmoid(rn(9, 2, 3, seed=3))
    o, S = O.decayed_reads(q, k, v, d)
    o1, S1 = O.decayed_reads(q[:4], k[:4], v[:4], d[:4])
    o2, S2 = O.decayed_reads(q[4:], k[4:], v[4:], d[4:], S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)
    want = sum((q[8, 1] * k[s, 1] * d[s + 1:, 1].prod(0)).sum() * v[s, 1] for s in range(9))
    assert torch.allclose(o[8, 1], want, atol=1e-12)


def test_channel_decays():
    t = {"a1": rn(2, 4), "a2": rn(6, 2, seed=1), "a2.b": rn(6, seed=2)}
    h = rn(3, 4, seed=3)
    z = torch.einsum("cr,tr->tc", t["a2"], torch.einsum("rw,tw->tr", t["a1"], h)) + t["a2.b"]
    got = O.channel_decays(h, dict(heads=2, dim=3, tau=4.0), t)
    assert torch.allclose(got.reshape(3, 6), torch.sigmoid(z) ** 0.25, atol=1e-12)


def test_streams_are_mixed_from_the_old_ones():
    x, y = rn(2, 3, 4), rn(2, 4, seed=1)
    mix, out = rn(3, 3, seed=2), rn(3, seed=3)
    got = O.update_streams(x, y, mix, out)
    for t in range(3):
        want = sum(mix[s, t] * x[:, s] for s in range(3)) + out[t] * y
        assert torch.allclose(got[:, t], want, atol=1e-12)
    # one stream with unit factors: the plain residual sum
    one = torch.ones(1, dtype=F64)
    assert torch.allclose(O.update_streams(x[:, :1], y, one[:, None], one)[:, 0], x[:, 0] + y)
    assert torch.allclose(O.read_streams(x, out), sum(out[s] * x[:, s] for s in range(3)))


def test_corrected_choice_and_identity_experts():
    mlp = {"router": {"experts": 2, "top": 2, "identity": 2}, "expert": {"limit": 0.7}}
    t = {"router": rn(4, 6), "correction": torch.tensor([0.0, -9.0, 9.0, 0.0]), "e0.gate": rn(5, 6, seed=1),
         "e0.up": rn(5, 6, seed=2), "e0.down": rn(6, 5, seed=3), "e1.gate": rn(5, 6, seed=4), "e1.up": rn(5, 6, seed=5),
         "e1.down": rn(6, 5, seed=6)}
    h = rn(7, 6, seed=7)
    idx, wt = O.route(h, t["router"], t["correction"], 2)
    s = torch.softmax(h @ t["router"].T, -1)
    assert (idx[:, 0] == 2).all() and (idx != 1).all()
    assert torch.allclose(wt[:, 0], s[:, 2]) and (wt.sum(-1) < 1).all()                # scores as they are
    out = O.experts_ff(h, mlp, t)
    for r in range(7):
        other = int(idx[r, 1])
        y = h[r] if other == 3 else O.clamped_expert(h[r:r + 1], t["e0.gate"], t["e0.up"], t["e0.down"], 0.7)[0]
        assert torch.allclose(out[r], s[r, 2] * h[r] + s[r, other] * y, atol=1e-12)


def test_clamped_activation():
    eye, big = torch.eye(3, dtype=F64), torch.tensor([[5.0, -5.0, 0.3]], dtype=F64)
    got = O.clamped_expert(big, eye, eye, eye, 1.0)[0]
    for c, z in enumerate((5.0, -5.0, 0.3)):
        g, u = min(z, 1.0), max(min(z, 1.0), -1.0)         # the gate is bounded above only
        assert abs(float(got[c]) - g / (1 + math.exp(-1.702 * g)) * (u + 1)) < 1e-12


def test_config_reader_and_registry(tmp_path):
    from safetensors.torch import save_file
    from vllm_omni_draft_amd import config
    st = state(2)
    (tmp_path / "config.json").write_text(json.dumps(CFG))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in st.items()}, str(tmp_path / "model.safetensors"))
    mc = config.load_model_config(str(tmp_path))
    assert isinstance(mc, config.SeqModelConfig) and (mc.arch, mc.block, mc.n_layers) == ("tovapel", "streams", 3)
    assert (mc.streams, mc.logit_softcap, mc.tied_head, mc.norm_eps, mc.n_runs) == (2, 15.0, False, 1e-6, 3)
    a, b, c = (l.mixer for l in mc.layers)
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.softcap, a.window, a.keep_first) == \
        ("parallel", 4, 2, 6, 10, 0.4, 20.0, 9, 2)
    assert a.qk_head_norm and a.qkv_bias and a.sink and a.head_gate and a.ssd is None
    assert (a.linear.heads, a.linear.dim, a.linear.vdim, a.linear.rank, a.linear.tau) == (3, 5, 7, 3, 4.0)
    assert (b.kv_heads, b.window, b.keep_first, b.linear.rank) == (4, 20, 0, 4) and c.linear.rank == 1
    ex = mc.layers[1].experts
    assert (ex.experts, ex.identity, ex.outputs, ex.top, ex.ff, ex.limit, ex.act, ex.score) == \
        (3, 2, 5, 2, 11, 0.7, "clamped_gate", "softmax")
    assert ex.correction and not ex.renorm and not ex.scale_input and [l.ff for l in mc.layers] == [24, 0, 0]
    assert mc.state_bytes_per_seq() == 4 * (3 * 5 * 7 + 5 * 5 * 8 + 2 * 5 * 10)
    assert mc.param_count() == sum(v.numel() for v in st.values())


def test_parts_that_may_be_absent():
    from vllm_omni_draft_amd import config
    cfg = json.loads(json.dumps(CFG))
    m = cfg["layers"][0]["mixer"]
    m["left"]["softcap"] = m["left"]["mask"] = cfg["logit_softcap"] = None
    m["right"]["rank"] = 3
    for l in cfg["layers"][1:]:
        l["mixer"]["right"]["rank"] = 2
    del cfg["layers"][1]["mlp"]["router"]["identity"]
    mc = config.tovapel_config(cfg)
    a = mc.layers[0].mixer
    assert (a.softcap, a.window, a.keep_first, mc.logit_softcap, mc.layers[1].experts.outputs) == (0.0, 0, 0, 0.0, 3)


@pytest.mark.parametrize("path,value", [
    (("layers", 0, "type"), "attention"),
    (("layers", 0, "mixer", "left", "kv_heads"), 3),
    (("layers", 0, "mixer", "left", "dim"), 513),
    (("layers", 0, "mixer", "left", "mask", "keep_first"), -1),
    (("layers", 0, "mixer", "right", "dim"), 257),
    (("layers", 0, "mixer", "right", "tau"), 0.0),
    (("layers", 1, "mlp", "router", "top"), 6),                 # more than experts and identity experts
    (("layers", 1, "mlp", "expert", "limit"), 0.0),
    (("layers", 0, "mlp", "kind"), "sparse"),
    (("streams",), 17),
])
def test_config_reader_refuses(path, value):
    from vllm_omni_draft_amd import config
    cfg = json.loads(json.dumps(CFG))
    node = cfg
    for k in path[:-1]:
        node = node[k]
    node[path[-1]] = value
    with pytest.raises(ValueError):
        config.tovapel_config(cfg, {f"l{i}.mix.right.a1": (r, 40) for i, r in enumerate(RANKS)})


def test_streams_parts_belong_to_streams_models():
    from vllm_omni_draft_amd import config
    ex = config.ExpertsSpec(experts=4, top=2, ff=8, identity=1)
    m = config.MixerSpec(kind="softmax_attention", heads=2, dim=8, vdim=8)
    with pytest.raises(ValueError):
        config.SeqModelConfig("x", 16, 10, [config.SeqLayerSpec(m, 0, ex)], block="sandwich").validate()
    with pytest.raises(ValueError):
        config.SeqModelConfig("x", 16, 10, [config.SeqLayerSpec(m, 0)], block="sandwich", streams=2).validate()


def reader(cfg=CFG):
    from vllm_omni_draft_amd import config
    return config.tovapel_config(cfg, {f"l{i}.mix.right.a1": (r, 40) for i, r in enumerate(RANKS)})


def test_what_a_sequence_keeps():
    from vllm_omni_draft_amd import _lib
    from vllm_omni_draft_amd.kv_cache import PAGE, SeqCache
    if not os.path.exists(_lib.lib_path()):
        subprocess.run(["make", "-C", ROOT, "-j8"], check=True)
    mc = reader()
    c = SeqCache(mc, torch.bfloat16, max_seqs=3, num_pages=7, max_seq_len=4 * PAGE, device="cpu")
    assert c.has_pages and sorted(c.k) == sorted(c.v) == sorted(c.state) == [0, 1, 2] and not c.conv and not c.kv_source
    assert c.k[0].shape == (7, 2, PAGE, 6) and c.v[1].shape == (7, 4, PAGE, 10) and c.k[0].dtype == torch.bfloat16
    assert [c.state[i].shape for i in range(3)] == [(3, 3, 5, 7), (3, 5, 5, 8), (3, 2, 5, 10)]
    assert all(t.dtype == torch.float32 for t in c.state.values())
    assert c.nbytes() == 3 * mc.state_bytes_per_seq() + 2 * sum(c.k[i].numel() + c.v[i].numel() for i in range(3))


def test_weights_are_stacked_per_layer():
    from vllm_omni_draft_amd import weights
    st, mc = state(3), reader()
    w = weights.seq_from_state_dict(mc, st, "cpu", torch.float32)
    a, b, c = w.layers
    names = ["left.q", "left.k", "left.v", "right.q", "right.k", "right.v", "right.g", "right.a1", "left.g"]
    assert torch.equal(a.w_in, torch.cat([st["l0.mix." + n] for n in names]))
    assert torch.equal(a.w_in_bias, torch.cat([st[f"l0.mix.left.{n}.b"] for n in "qkv"]))
    assert not a.out_stacked and torch.equal(a.w_o, st["l0.mix.left.o"]) and torch.equal(a.w_o2, st["l0.mix.right.o"])
    assert torch.equal(a.hc_mix, st["l0.hc1.mix"]) and torch.equal(a.hc2_out, st["l0.hc2.out"]) and a.sinks.dtype == torch.float32
    assert torch.equal(a.w_ff_in, torch.cat([st["l0.mlp.gate"], st["l0.mlp.up"]])) and torch.equal(a.out_norm2_w, st["l0.mix.right.out"])
    assert b.w_gate_up.shape == (3, 22, 40) and torch.equal(b.w_gate_up[2, 11:], st["l1.mlp.e2.up"])
    assert b.w_router.shape == (5, 40) and torch.equal(b.route_correction, st["l1.mlp.correction"])
    # equal input widths, but a width that is no multiple of 16: not stacked
    assert not c.out_stacked and c.norm2_w is None and c.hc2_in is None
    wide = json.loads(json.dumps(CFG))
    wide["width"] = 48
    st48 = state(3, wide)
    c48 = weights.seq_from_state_dict(reader(wide), st48, "cpu", torch.float32).layers[2]
    assert c48.out_stacked and c48.w_o2 is None and torch.equal(c48.w_o[48:], st48["l2.mix.right.o"])
    st2 = weights.seq_random_state(mc, 0)
    assert {k: tuple(v.shape) for k, v in st2.items()} == {k: tuple(v.shape) for k, v in st.items()}
    del st["l1.mlp.correction"]
    with pytest.raises(KeyError):
        weights.seq_from_state_dict(mc, st, "cpu", torch.float32)
