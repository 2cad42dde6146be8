"""Host side of the layer-list models, no GPU: the safetensors reader, the configuration reader's mapping onto layer descriptors, the ctypes
mirror of the descriptors against the C header, and the plain statement's own invariances."""
import ctypes as C
import json
import os
import subprocess

import numpy as np
import pytest

import seq_oracle
from powerserve_amd import hip, safetensors_io, seqmodel, synth

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
L = synth.seq_layer
CFG = synth.seq_config(24, 30, [L("delta", 20, heads=4, kv_heads=2, dim=6, vdim=10, conv=4), L("wkv", None, heads=3, dim=8),
                                L("latent_attention", 16, heads=2, dim=6, vdim=10, q_rank=7, kv_rank=9, rot_dim=4, rot={"base": 77.0, "dims": 4},
                                  mask={"size": 5}, scale=0.25)], taps=2, eps=1e-5, logit_scale=0.75)


def test_safetensors_round_trip_and_rounding(tmp_path):
    a = np.array([1.0, 1.00390625, 1.01171875, -3.0e-5, 65504.0, 0.0], dtype=np.float32)  # 1 + 2^-8 ties to even (down), 1 + 3 * 2^-8 ties up
    bits = safetensors_io.f32_to_bf16_bits(a)
    back = (bits.astype(np.uint32) << 16).view(np.float32)
    assert back[1] == 1.0 and back[2] == np.float32(1.015625) and back[0] == 1.0 and back[5] == 0.0
    t = {"w": np.arange(12, dtype=np.float32).reshape(3, 4), "idx": np.arange(5, dtype=np.int32)}
    p = str(tmp_path / "x.safetensors")
    safetensors_io.write(p, t)
    st = safetensors_io.SafeTensors(p)
    assert st.dtype("w") == "BF16" and st.dtype("idx") == "I32" and st.shape("w") == (3, 4)
    assert np.array_equal(st.f32("w"), t["w"]) and np.array_equal(st.raw("idx"), t["idx"])
    with pytest.raises(ValueError):
        st.bf16_bits("idx")


class FakeUp:
    def __init__(self):
        self.vecs, self.mats = [], []

    def vec(self, a):
        self.vecs.append(np.array(a))
        return len(self.vecs)

    def mat(self, bits):
        self.mats.append(np.array(bits))
        return 1000 + len(self.mats)


def test_configuration_maps_onto_layer_descriptors(tmp_path):
    t = synth.write_seq_model_dir(str(tmp_path), CFG, 1)
    cfg = seqmodel.read_config(str(tmp_path))
    up = FakeUp()
    layers, top = seqmodel.ARCHITECTURES[cfg["architecture"]](cfg, safetensors_io.SafeTensors(str(tmp_path / "model.safetensors")), up)
    assert (top["width"], top["vocab"], top["canon_taps"], top["norm_offset"]) == (24, 30, 2, 1.0)
    assert abs(top["norm_eps"] - 1e-5) < 1e-12 and top["logit_scale"] == 0.75
    d, w, a = layers
    assert (d.kind, d.heads, d.kv_heads, d.dim, d.vdim, d.conv_taps, d.ff_kind, d.ff) == (seqmodel.MIX_DELTA, 4, 2, 6, 10, 4, seqmodel.FF_DENSE_XIELU, 20)
    assert (w.kind, w.heads, w.dim, w.vdim, w.decay_rank, w.ff_kind) == (seqmodel.MIX_WKV, 3, 8, 8, 8, seqmodel.FF_NONE)
    assert (a.kind, a.q_rank, a.kv_rank, a.rot_dim, a.rot_dims, a.window) == (seqmodel.MIX_LATENT, 7, 9, 4, 4, 5)
    assert abs(a.rot_base - 77.0) < 1e-6 and abs(a.scale - 0.25) < 1e-9
    # the fused input projection of the delta mixer: rows q | k | v | g | b | a
    cat = up.mats[d.in_cat - 1001]
    assert cat.shape == (2 * 2 * 6 + 2 * 4 * 10 + 2 * 4, 24)
    want = np.concatenate([safetensors_io.f32_to_bf16_bits(t["l0.mix." + n]) for n in ("q", "k", "v", "g", "b", "a")])
    assert np.array_equal(cat, want)
    assert up.mats[a.ukv - 1001].shape == (2 * 6 + 2 * 10, 9) and up.mats[a.in_cat - 1001].shape == (7 + 9 + 4, 24)
    assert up.vecs[w.mu - 1].shape == (5, 24)


def test_unknown_names_are_refused(tmp_path):
    bad = dict(CFG, architecture="Somethingelse")
    synth.write_seq_model_dir(str(tmp_path), bad, 1, tensors=synth.seq_tensors(CFG, 1))
    with pytest.raises(seqmodel.ConfigError):
        seqmodel.read_config(str(tmp_path))
    bad = json.loads(json.dumps(CFG))
    bad["layers"][1]["type"] = "conveyor"
    with open(tmp_path / "config.json", "w") as f:
        json.dump(bad, f)
    with pytest.raises(seqmodel.ConfigError):
        seqmodel.ARCHITECTURES["Ranutar"](bad, safetensors_io.SafeTensors(str(tmp_path / "model.safetensors")), FakeUp())
    bad = json.loads(json.dumps(CFG))
    bad["canon"]["taps"] = 3  # the file's tensors have two taps
    with pytest.raises(seqmodel.ConfigError):
        seqmodel.ARCHITECTURES["Ranutar"](bad, safetensors_io.SafeTensors(str(tmp_path / "model.safetensors")), FakeUp())


def test_ctypes_descriptors_match_the_header(tmp_path):
    src = tmp_path / "sz.c"
    src.write_text('#include <stdio.h>\n#include <stddef.h>\n#include "ps_hip.h"\nint main(void){printf("%zu %zu %zu %zu %zu %zu %zu %zu %zu %zu %zu\\n", sizeof(ps_seq_layer), '
                   'offsetof(ps_seq_layer, norm1), offsetof(ps_seq_layer, kvnorm), sizeof(ps_seq_desc), offsetof(ps_seq_desc, embed), offsetof(ps_seq_desc, layers), '
                   'offsetof(ps_seq_layer, beside), offsetof(ps_seq_layer, in_bias), offsetof(ps_seq_layer, tau), offsetof(ps_seq_desc, embed_scale), '
                   'offsetof(ps_seq_desc, max_context));'
                   'printf("%zu %zu %zu %zu %zu %zu %zu\\n", offsetof(ps_seq_layer, res_scale), offsetof(ps_seq_layer, depth_mix), offsetof(ps_seq_layer, softcap), '
                   'offsetof(ps_seq_layer, qtemp_every), offsetof(ps_seq_layer, experts), offsetof(ps_seq_layer, shared_down), offsetof(ps_seq_desc, norm_groups));'
                   'printf("%zu %zu %zu %zu %zu %zu %zu\\n", offsetof(ps_seq_layer, head_norm), offsetof(ps_seq_layer, yarn_factor), offsetof(ps_seq_layer, yarn_original), '
                   'offsetof(ps_seq_layer, ff_up_bias), offsetof(ps_seq_layer, moe_identity), offsetof(ps_seq_layer, moe_correction), offsetof(ps_seq_desc, norm_center));'
                   'printf("%zu %zu %zu %zu %zu %zu %zu %zu %zu\\n", offsetof(ps_seq_layer, moe_scale), offsetof(ps_seq_layer, out_bias), offsetof(ps_seq_layer, dist_slope), '
                   'offsetof(ps_seq_layer, keep_first), offsetof(ps_seq_layer, kv_from), offsetof(ps_seq_layer, norm_parts), offsetof(ps_seq_layer, skip), '
                   'offsetof(ps_seq_desc, bigram), offsetof(ps_seq_desc, logit_softcap));return 0;}\n')
    exe = str(tmp_path / "sz")
    subprocess.run(["gcc", "-I" + os.path.join(ROOT, "include"), str(src), "-o", exe], check=True)
    got = [int(x) for x in subprocess.run([exe], check=True, capture_output=True, text=True).stdout.split()]
    assert got == [C.sizeof(hip.SeqLayer), hip.SeqLayer.norm1.offset, hip.SeqLayer.kvnorm.offset, C.sizeof(hip.SeqDesc), hip.SeqDesc.embed.offset,
                   hip.SeqDesc.layers.offset, hip.SeqLayer.beside.offset, hip.SeqLayer.in_bias.offset, hip.SeqLayer.tau.offset, hip.SeqDesc.embed_scale.offset,
                   hip.SeqDesc.max_context.offset,
                   hip.SeqLayer.res_scale.offset, hip.SeqLayer.depth_mix.offset, hip.SeqLayer.softcap.offset, hip.SeqLayer.qtemp_every.offset, hip.SeqLayer.experts.offset,
                   hip.SeqLayer.shared_down.offset, hip.SeqDesc.norm_groups.offset,
                   hip.SeqLayer.head_norm.offset, hip.SeqLayer.yarn_factor.offset, hip.SeqLayer.yarn_original.offset, hip.SeqLayer.ff_up_bias.offset,
                   hip.SeqLayer.moe_identity.offset, hip.SeqLayer.moe_correction.offset, hip.SeqDesc.norm_center.offset,
                   hip.SeqLayer.moe_scale.offset, hip.SeqLayer.out_bias.offset, hip.SeqLayer.dist_slope.offset, hip.SeqLayer.keep_first.offset, hip.SeqLayer.kv_from.offset,
                   hip.SeqLayer.norm_parts.offset, hip.SeqLayer.skip.offset, hip.SeqDesc.bigram.offset, hip.SeqDesc.logit_softcap.offset]


def test_plain_statement_is_causal_and_windowed():
    """what a later token is does not change earlier logits; a token outside every window and with the recurrent layers cut out does not matter"""
    t = synth.seq_tensors(CFG, 2)
    rng = np.random.default_rng(0)
    a = rng.integers(0, 30, 20)
    b = a.copy()
    b[12] = (b[12] + 1) % 30
    la, lb = seq_oracle.run(CFG, t, a), seq_oracle.run(CFG, t, b)
    assert np.array_equal(la[:12], lb[:12]) and np.abs(la[12:] - lb[12:]).max() > 1e-3
    only = synth.seq_config(24, 30, [CFG["layers"][2]], taps=2)
    t2 = synth.seq_tensors(only, 2)
    la, lb = seq_oracle.run(only, t2, a), seq_oracle.run(only, t2, b)
    # window 5 and a 2-tap input filter in front of the mixer and of the feed-forward: token 12 reaches positions 12 .. 12 + 4 + 1 + 1
    assert np.abs(la[19:] - lb[19:]).max() < 1e-12 and np.abs(la[12:19] - lb[12:19]).max() > 1e-6


PCFG = synth.parallel_config(24, 30, [
    synth.parallel_layer(20, dict(heads=4, kv_heads=2, dim=6, vdim=10, mask={"size": 5, "pool": 3}, rot={"base": 77.0, "dims": 4, "scaling": {"factor": 2.0}}, scale=0.25),
                         dict(heads=3, dim=8, vdim=4, tau=5.0), 1.25, 0.5),
    synth.parallel_layer(None, dict(heads=2, kv_heads=2, dim=6, vdim=6, mask={"size": 4, "pool": 2}, rot={"base": 9.0, "dims": 6}, scale=0.5),
                         dict(heads=1, dim=5, vdim=7, tau=1.0))], taps=2, eps=1e-5, embed_scale=3.0, loop=(0, 1, 2))


def test_parallel_configuration_maps_onto_layer_descriptors(tmp_path):
    t = synth.write_seq_model_dir(str(tmp_path), PCFG, 1)
    cfg = seqmodel.read_config(str(tmp_path))
    up = FakeUp()
    layers, top = seqmodel.ARCHITECTURES[cfg["architecture"]](cfg, safetensors_io.SafeTensors(str(tmp_path / "model.safetensors")), up)
    assert (top["width"], top["vocab"], top["canon_taps"], top["norm_offset"], top["embed_scale"]) == (24, 30, 2, 0.0, 3.0)
    assert (top["loop_start"], top["loop_stop"], top["loop_times"]) == (0, 1, 2)
    a, b = layers
    assert (a.form, a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.pool, a.rot_dims, a.rot_pairing, a.gated) == \
        (seqmodel.LAYER_PARALLEL, seqmodel.MIX_WINATTN, 4, 2, 6, 10, 5, 3, 4, seqmodel.ROT_NEIGHBOURS, 1)
    assert abs(a.rot_base - 77.0) < 1e-6 and a.rot_factor == 2.0 and a.scale == 0.25 and a.mix_scale == 1.25 and b.rot_factor == 1.0
    r = a.beside.contents
    assert (r.kind, r.heads, r.dim, r.vdim, r.decay_rank, r.tau, r.mix_scale) == (seqmodel.MIX_GLA, 3, 8, 4, 8, 5.0, 0.5)
    assert (a.ff_kind, a.ff, b.ff_kind) == (seqmodel.FF_DENSE_SWIGLU, 20, seqmodel.FF_NONE)
    # stacked input projections: q | k | v | gate with their biases (the gate has none), and q | k | v | g | a1
    cat = up.mats[a.in_cat - 1001]
    assert cat.shape == (4 * 6 + 2 * 6 + 2 * 10 + 4, 24)
    assert np.array_equal(cat, np.concatenate([safetensors_io.f32_to_bf16_bits(t["l0.mix.left." + n]) for n in ("q", "k", "v", "g")]))
    bias = up.vecs[a.in_bias - 1]
    assert bias.shape == (60,) and np.array_equal(bias[:24], t["l0.mix.left.q.b"]) and not bias[56:].any()
    assert up.mats[r.in_cat - 1001].shape == (2 * 3 * 8 + 2 * 3 * 4 + 8, 24)
    # the feed-forward's gate and up rows alternate
    both = up.mats[a.ff_up - 1001]
    assert both.shape == (40, 24)
    assert np.array_equal(both[0::2], safetensors_io.f32_to_bf16_bits(t["l0.mlp.gate"])) and np.array_equal(both[1::2], safetensors_io.f32_to_bf16_bits(t["l0.mlp.up"]))
    # what the file does not have does not exist
    st = safetensors_io.SafeTensors(str(tmp_path / "model.safetensors"))
    less = {n: st.f32(n) for n in st.names() if not n.endswith((".b", "temp", "sink", "q.norm", "left.g"))}
    cfg2 = json.loads(json.dumps(PCFG))
    del cfg2["loop"], cfg2["layers"][0]["mixer"]["left"]["rot"]
    synth.write_seq_model_dir(str(tmp_path / "less"), cfg2, 1, tensors=less)
    layers, top = seqmodel.ARCHITECTURES["Vobisun"](cfg2, safetensors_io.SafeTensors(str(tmp_path / "less" / "model.safetensors")), FakeUp())
    a = layers[0]
    assert (a.gated, a.in_bias, a.temp, a.sink, a.qnorm, a.rot_dims, top["loop_times"]) == (0, None, None, None, None, 0, 1) and a.knorm is not None
    bad = json.loads(json.dumps(PCFG))
    bad["layers"][0]["mixer"]["left"]["heads"] = 5
    with pytest.raises(seqmodel.ConfigError):
        seqmodel.ARCHITECTURES["Vobisun"](bad, st, FakeUp())


def test_plain_parallel_statement_reach():
    """causal; with the recurrent mixer switched off, a token reaches exactly as far as its window, then only through its block's mean; the layers of a loop run in order"""
    assert seq_oracle.layer_runs(PCFG) == [0, 0, 1] and seq_oracle.layer_runs({"layers": [0, 0, 0, 0], "loop": {"start": 1, "stop": 3, "times": 3}}) == [0, 1, 2, 1, 2, 1, 2, 3]
    assert list(seq_oracle.visible_tokens(9, 4)) == [6, 7, 8, 9] and list(seq_oracle.visible_blocks(9, 4, 3)) == [0, 1] and list(seq_oracle.visible_blocks(8, 4, 3)) == [0]
    assert list(seq_oracle.visible_blocks(3, 4, 3)) == [] and list(seq_oracle.visible_tokens(2, 4)) == [0, 1, 2]
    one = synth.parallel_config(24, 30, [synth.parallel_layer(None, PCFG["layers"][0]["mixer"]["left"], PCFG["layers"][0]["mixer"]["right"], 1.0, 0.0)], taps=1)
    t = synth.seq_tensors(one, 2)
    rng = np.random.default_rng(0)
    a = rng.integers(0, 30, 24)
    b = a.copy()
    b[7] = (b[7] + 1) % 30
    la, lb = seq_oracle.run_parallel(one, t, a), seq_oracle.run_parallel(one, t, b)
    changed = [i for i in range(24) if np.abs(la[i] - lb[i]).max() > 1e-9]
    # window 5: positions 7 .. 11 see token 7 itself; its block 6 .. 8 is seen from 8 + 5 = 13 on; 12 sees neither
    assert changed == [7, 8, 9, 10, 11] + list(range(13, 24))
    la, lb = seq_oracle.run_parallel(one, t, a, pool=0), seq_oracle.run_parallel(one, t, b, pool=0)
    assert [i for i in range(24) if np.abs(la[i] - lb[i]).max() > 1e-9] == [7, 8, 9, 10, 11]


ZCFG = synth.zusolix_config(24, 30, [
    synth.zusolix_layer("attention", synth.zusolix_attention(4, 2, 6, 10, 0.25, 7.0, (0.3, 9)), moe=(3, 2, 8), shared=5),
    synth.zusolix_layer("mingru", {"width": 14}, ff=20),
    synth.zusolix_layer("attention", synth.zusolix_attention(2, 2, 6, 6, 0.5))], groups=3, eps=1e-5, embed_scale=3.0, residual_mult=0.4)


def test_zusolix_configuration_maps_onto_layer_descriptors(tmp_path):
    t = synth.write_seq_model_dir(str(tmp_path), ZCFG, 1)
    cfg = seqmodel.read_config(str(tmp_path))
    up = FakeUp()
    st = safetensors_io.SafeTensors(str(tmp_path / "model.safetensors"))
    layers, top = seqmodel.ARCHITECTURES[cfg["architecture"]](cfg, st, up)
    bits = safetensors_io.f32_to_bf16_bits
    assert (top["width"], top["vocab"], top["canon_taps"], top["norm_offset"], top["embed_scale"], top["norm_groups"]) == (24, 30, 1, 0.0, 3.0, 3)
    a, g, c = layers
    assert all(abs(x.res_scale - 0.4) < 1e-7 and x.form == seqmodel.LAYER_PARALLEL and x.canon1 is None for x in layers)
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.pool, a.rot_dims, a.gated, a.qtemp_every) == (seqmodel.MIX_WINATTN, 4, 2, 6, 10, 0, 0, 0, 0, 9)
    assert abs(a.softcap - 7.0) < 1e-6 and abs(a.qtemp_coef - 0.3) < 1e-6 and a.scale == 0.25 and (c.softcap, c.qtemp_every, c.qtemp_coef) == (0.0, 0, 0.0)
    assert (a.qnorm, a.knorm, a.temp, a.sink) == (None, None, None, None)
    bias = up.vecs[a.in_bias - 1]
    assert bias.shape == (24 + 12 + 20,) and np.array_equal(bias[24:36], t["l0.mix.k.b"])
    # the depth average's weights: one more per layer
    assert [up.vecs[x.depth_mix - 1].shape for x in layers] == [(2,), (3,), (4,)] and a.norm2 is not None and c.norm2 is None and c.ff_kind == seqmodel.FF_NONE
    # the recurrence: z | x | g stacked, one bias vector (g has none)
    assert (g.kind, g.heads, g.dim, g.ff_kind, g.ff) == (seqmodel.MIX_MINGRU, 1, 14, seqmodel.FF_DENSE_SWIGLU, 20)
    assert np.array_equal(up.mats[g.in_cat - 1001], np.concatenate([bits(t["l1.mix." + n]) for n in ("z", "x", "g")]))
    gb = up.vecs[g.in_bias - 1]
    assert gb.shape == (42,) and np.array_equal(gb[14:28], t["l1.mix.x.b"]) and not gb[28:].any()
    # the experts: one matrix each way, expert after expert, gate / up rows alternating inside an expert; the router and the shared gate stay fp32 vectors
    assert (a.ff_kind, a.ff, a.experts, a.top, a.shared_ff, a.moe_norm_top) == (seqmodel.FF_MOE_SWIGLU, 8, 3, 2, 5, 0)
    ups, downs = up.mats[a.ff_up - 1001], up.mats[a.ff_down - 1001]
    assert ups.shape == (3 * 16, 24) and downs.shape == (3 * 24, 8)
    assert np.array_equal(ups[16:32:2], bits(t["l0.mlp.e1.gate"])) and np.array_equal(ups[33:48:2], bits(t["l0.mlp.e2.up"])) and np.array_equal(downs[24:48], bits(t["l0.mlp.e1.down"]))
    assert up.vecs[a.router - 1].shape == (3, 24) and up.vecs[a.shared_gate - 1].shape == (24,) and up.mats[a.shared_up - 1001].shape == (10, 24)
    # what the file and the configuration do not have does not exist
    less = {n: st.f32(n) for n in st.names() if not n.endswith((".b", "dwa", "shared.sg"))}
    cfg2 = json.loads(json.dumps(ZCFG))
    del cfg2["layers"][0]["mixer"]["softcap"], cfg2["layers"][0]["mixer"]["q_temp"], cfg2["norm"]["groups"]
    synth.write_seq_model_dir(str(tmp_path / "less"), cfg2, 1, tensors=less)
    layers, top = seqmodel.ARCHITECTURES["Zusolix"](cfg2, safetensors_io.SafeTensors(str(tmp_path / "less" / "model.safetensors")), FakeUp())
    a, g, _ = layers
    assert (a.in_bias, g.in_bias, a.depth_mix, a.shared_gate, a.softcap, a.qtemp_every, top["norm_groups"]) == (None, None, None, None, 0.0, 0, 1) and a.shared_up is not None
    for key, val in (("type", "conveyor"), ("mlp", {"kind": "sparse", "ff": 8})):
        bad = json.loads(json.dumps(ZCFG))
        bad["layers"][1][key] = val
        with pytest.raises(seqmodel.ConfigError):
            seqmodel.ARCHITECTURES["Zusolix"](bad, st, FakeUp())
    bad = json.loads(json.dumps(ZCFG))
    bad["layers"][0]["mlp"]["router"]["top"] = 4
    with pytest.raises(seqmodel.ConfigError):
        seqmodel.ARCHITECTURES["Zusolix"](bad, st, FakeUp())


def test_plain_zusolix_statement_reach_and_pieces():
    """causal, and every later token sees a changed one (nothing limits the reach); the norm's groups are on their own; the temperature steps where it should;
    the largest scores are the ones chosen"""
    t = synth.seq_tensors(ZCFG, 2)
    rng = np.random.default_rng(0)
    a = rng.integers(0, 30, 20)
    b = a.copy()
    b[6] = (b[6] + 1) % 30
    la, lb = seq_oracle.run_zusolix(ZCFG, t, a), seq_oracle.run_zusolix(ZCFG, t, b)
    assert np.array_equal(la[:6], lb[:6]) and min(np.abs(la[i] - lb[i]).max() for i in range(6, 20)) > 1e-6
    x = rng.standard_normal((4, 12))
    y = x.copy()
    y[:, 4:8] *= 7.0  # scaling one part changes nothing (up to eps), inside or outside it
    assert np.abs(seq_oracle.grouped_norm(x, np.ones(12), 3, 0.0) - seq_oracle.grouped_norm(y, np.ones(12), 3, 0.0)).max() < 1e-12
    assert np.abs(seq_oracle.grouped_norm(x, np.ones(12), 1, 0.0) - seq_oracle.grouped_norm(y, np.ones(12), 1, 0.0)).max() > 0.1
    assert [round(float(seq_oracle.query_temperature(p, 1.0, 4)), 6) for p in (0, 2, 3, 6, 7)] == [1.0, 1.0, round(1 + np.log(2), 6), round(1 + np.log(2), 6), round(1 + np.log(3), 6)]
    W = {k: np.asarray(v, np.float64) for k, v in t.items()}
    h = rng.standard_normal((5, 24))
    mlp = ZCFG["layers"][0]["mlp"]
    full = seq_oracle.expert_mixture(W, "l0.mlp.", h, mlp, use_shared=False)
    for i in range(5):
        s = seq_oracle.sigmoid(W["l0.mlp.router"] @ h[i])
        keep = np.argsort(-s)[:2]
        assert np.allclose(full[i], sum(seq_oracle.one_expert(W, "l0.mlp.e%d." % e, s[e] * h[i]) for e in keep))


KCFG = synth.pokatar_config(24, 30, [
    synth.pokatar_layer("attention", synth.pokatar_attention(4, 2, 6, 10, 0.25), moe=(3, 2, 8, 2, 5, 2), shared=5),
    synth.pokatar_layer("latent_attention", synth.pokatar_latent(3, 6, 4, 5, 7, 0.3, 77.0, (3.0, 40, 8.0, 0.5)), ff=20),
    synth.pokatar_layer("latent_attention", synth.pokatar_latent(2, 4, 6, 4, 9, 0.5, 9.0))], eps=1e-5)


def test_pokatar_configuration_maps_onto_layer_descriptors(tmp_path):
    t = synth.write_seq_model_dir(str(tmp_path), KCFG, 1)
    cfg = seqmodel.read_config(str(tmp_path))
    up = FakeUp()
    st = safetensors_io.SafeTensors(str(tmp_path / "model.safetensors"))
    layers, top = seqmodel.ARCHITECTURES[cfg["architecture"]](cfg, st, up)
    bits = safetensors_io.f32_to_bf16_bits
    assert (top["width"], top["vocab"], top["canon_taps"], top["norm_offset"], top["norm_center"], top["logit_scale"]) == (24, 30, 1, 0.0, 1, 1.0)
    assert top["head"] == top["embed"]  # the logits are taken against the embedding table
    a, b, c = layers
    assert all(x.form == seqmodel.LAYER_PRENORM and x.canon1 is None and x.norm1b is None and x.depth_mix is None for x in layers)
    # attention: q | k | v | g stacked, a gate row per output element, norms per head with [dim] weights, unit values, a sink of zeros
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.pool, a.rot_dims, a.gated, a.head_norm, a.v_unit) == (seqmodel.MIX_WINATTN, 4, 2, 6, 10, 0, 0, 0, 2, 1, 1)
    assert up.mats[a.in_cat - 1001].shape == (24 + 12 + 20 + 40, 24) and np.array_equal(up.mats[a.in_cat - 1001][56:], bits(t["l0.mix.g"]))
    assert up.vecs[a.qnorm - 1].shape == (6,) and up.vecs[a.knorm - 1].shape == (6,) and not up.vecs[a.sink - 1].any() and up.vecs[a.sink - 1].shape == (4,) and a.in_bias is None
    # latent attention: q | dkv | g stacked, no query latent, everything before the token, the scaling constants
    assert (b.kind, b.heads, b.dim, b.vdim, b.q_rank, b.kv_rank, b.rot_dim, b.rot_dims, b.window, b.gated) == (seqmodel.MIX_LATENT, 3, 6, 5, 0, 7, 4, 4, 0, 1)
    assert (b.yarn_factor, b.yarn_original, b.yarn_fast, b.yarn_slow, b.rot_base) == (3.0, 40, 8.0, 0.5, 77.0) and (c.yarn_factor, c.yarn_original) == (0.0, 0)
    assert np.array_equal(up.mats[b.in_cat - 1001], np.concatenate([bits(t["l1.mix." + n]) for n in ("q", "dkv", "g")])) and up.mats[b.in_cat - 1001].shape == (30 + 11 + 3, 24)
    assert np.array_equal(up.mats[b.ukv - 1001], np.concatenate([bits(t["l1.mix.uk"]), bits(t["l1.mix.uv"])])) and b.uq is None and b.qnorm is None
    # the dense feed-forward: gate / up rows alternating, their biases alike, a bias on the way down
    assert (b.ff_kind, b.ff, c.ff_kind) == (seqmodel.FF_DENSE_RELU_GLU, 20, seqmodel.FF_NONE)
    ub = up.vecs[b.ff_up_bias - 1]
    assert ub.shape == (40,) and np.array_equal(ub[0::2], t["l1.mlp.gate.b"]) and np.array_equal(ub[1::2], t["l1.mlp.up.b"]) and np.array_equal(up.vecs[b.ff_down_bias - 1], t["l1.mlp.down.b"])
    assert np.array_equal(up.mats[b.ff_up - 1001][1::2], bits(t["l1.mlp.up"]))
    # the experts: one matrix each way; the router has rows for the identity experts too; groups over all of them
    assert (a.ff_kind, a.ff, a.experts, a.top, a.shared_ff, a.moe_identity, a.moe_softmax, a.moe_groups, a.moe_keep, a.moe_weight_output) == (seqmodel.FF_MOE_RELU2, 8, 3, 2, 5, 2, 1, 5, 2, 1)
    assert up.mats[a.ff_up - 1001].shape == (3 * 8, 24) and up.mats[a.ff_down - 1001].shape == (3 * 24, 8) and np.array_equal(up.mats[a.ff_up - 1001][8:16], bits(t["l0.mlp.e1.up"]))
    assert up.vecs[a.router - 1].shape == (5, 24) and up.vecs[a.moe_correction - 1].shape == (5,) and up.mats[a.shared_up - 1001].shape == (5, 24) and a.shared_gate is None
    # what the file and the configuration do not have does not exist
    less = {n: st.f32(n) for n in st.names() if not n.endswith((".b", "correction", ".g", "q.norm"))}
    cfg2 = json.loads(json.dumps(KCFG))
    del cfg2["layers"][0]["mlp"]["router"]["groups"], cfg2["layers"][0]["mlp"]["router"]["identity"], cfg2["layers"][0]["mlp"]["shared"], cfg2["layers"][1]["mixer"]["rot"]["scaling"]
    less["l0.mlp.router"] = less["l0.mlp.router"][:3]
    synth.write_seq_model_dir(str(tmp_path / "less"), cfg2, 1, tensors=less)
    layers, _ = seqmodel.ARCHITECTURES["Pokatar"](cfg2, safetensors_io.SafeTensors(str(tmp_path / "less" / "model.safetensors")), FakeUp())
    a, b, _ = layers
    assert (a.gated, b.gated, a.qnorm, a.moe_correction, a.moe_groups, a.moe_identity, a.shared_up, b.ff_up_bias, b.ff_down_bias, b.yarn_factor) == (0, 0, None, None, 0, 0, None, None, None, 0.0)
    assert a.knorm is not None
    for key, val in (("type", "conveyor"), ("mlp", {"kind": "sparse", "ff": 8})):
        bad = json.loads(json.dumps(KCFG))
        bad["layers"][1][key] = val
        with pytest.raises(seqmodel.ConfigError):
            seqmodel.ARCHITECTURES["Pokatar"](bad, st, FakeUp())
    for key, val in (("top", 6), ("groups", {"count": 2, "keep": 1}), ("groups", {"count": 5, "keep": 1})):  # more than the router has; groups that do not divide; top beyond what stays
        bad = json.loads(json.dumps(KCFG))
        bad["layers"][0]["mlp"]["router"][key] = val
        with pytest.raises(seqmodel.ConfigError):
            seqmodel.ARCHITECTURES["Pokatar"](bad, st, FakeUp())


def test_plain_pokatar_statement_reach_and_pieces():
    """causal, and every later token sees a changed one; the layer norm ignores a shift; the sink takes its share; the frequency ramp ends where it should; the
    router's choice stays inside the best groups and an identity expert hands its input on"""
    t = synth.seq_tensors(KCFG, 2)
    rng = np.random.default_rng(0)
    a = rng.integers(0, 30, 20)
    b = a.copy()
    b[6] = (b[6] + 1) % 30
    la, lb = seq_oracle.run_pokatar(KCFG, t, a), seq_oracle.run_pokatar(KCFG, t, b)
    assert np.array_equal(la[:6], lb[:6]) and min(np.abs(la[i] - lb[i]).max() for i in range(6, 20)) > 1e-6
    x = rng.standard_normal((4, 12))
    assert np.abs(seq_oracle.centred_norm(x, np.ones(12), 0.0) - seq_oracle.centred_norm(x + 5.0, np.ones(12), 0.0)).max() < 1e-12
    assert abs(np.mean(seq_oracle.centred_norm(x, np.ones(12), 1e-5))) < 1e-12
    p = seq_oracle.sink_softmax(np.array([0.0, 0.0, 0.0]))
    assert np.allclose(p, 0.25) and np.allclose(seq_oracle.sink_softmax(np.array([50.0])), 1.0) and np.allclose(seq_oracle.sink_softmax(np.array([-50.0])), 0.0, atol=1e-20)
    # base 100, 8 dims: f = 1, 100^-1/4, 100^-1/2, 100^-3/4; original 40: pairs turning more than 8 times in 40 positions keep their frequency, fewer than 1/2 are divided
    f, mag = seq_oracle.yarn_frequencies({"dims": 8, "base": 100.0, "scaling": {"factor": 4.0, "original": 40, "fast": 8.0, "slow": 0.5}})
    plain = 100.0 ** (-np.arange(4) / 4.0)
    lo, hi = max(np.floor(8 * np.log(40 / (2 * np.pi * 8.0)) / (2 * np.log(100.0))), 0), min(np.ceil(8 * np.log(40 / (2 * np.pi * 0.5)) / (2 * np.log(100.0))), 7)
    assert (lo, hi) == (0, 3) and np.allclose(f, plain * (1 - np.arange(4) / 3) + plain / 4 * np.arange(4) / 3) and abs(mag - (0.1 * np.log(4.0) + 1)) < 1e-12
    assert np.allclose(seq_oracle.yarn_frequencies({"dims": 8, "base": 100.0})[0], plain)
    v = rng.standard_normal(8)
    r = seq_oracle.rotate_halves(v, 3, plain, 1.0)
    assert np.allclose(np.hypot(r[:4], r[4:]), np.hypot(v[:4], v[4:])) and np.allclose(seq_oracle.rotate_halves(v, 0, plain, 1.5), 1.5 * v)
    # five router rows in five groups of one of which two stay: exactly the two best corrected scores; with one group of five the same two
    s, corr = np.array([0.1, 0.3, 0.15, 0.25, 0.2]), np.array([0.0, -0.2, 0.0, 0.0, 0.2])
    assert seq_oracle.grouped_choice(s, corr, {"top": 2, "groups": {"count": 5, "keep": 2}}) == [4, 3]
    assert seq_oracle.grouped_choice(s, 0.0, {"top": 2}) == [1, 3]
    # six rows in three pairs, one pair stays: the best single row decides the pair, the second choice is its neighbour however small
    s6 = np.array([0.05, 0.3, 0.25, 0.2, 0.1, 0.1])
    assert seq_oracle.grouped_choice(s6, 0.0, {"top": 2, "groups": {"count": 3, "keep": 1}}) == [1, 0]
    W = {k: np.asarray(v, np.float64) for k, v in t.items()}
    h = rng.standard_normal((6, 24))
    mlp = KCFG["layers"][0]["mlp"]
    full = seq_oracle.routed_experts(W, "l0.mlp.", h, mlp, use_shared=False)
    for i in range(6):
        z = W["l0.mlp.router"] @ h[i]
        sc = np.exp(z) / np.exp(z).sum()
        keep = np.argsort(-(sc + W["l0.mlp.correction"]))[:2]  # (five groups of one, two stay: the group limit changes nothing here)
        assert np.allclose(full[i], sum(sc[e] * (seq_oracle.squared_relu_expert(W, "l0.mlp.e%d." % e, h[i]) if e < 3 else h[i]) for e in keep))


UCFG = synth.pupidra_config(24, 30, [
    synth.pupidra_layer("mamba2", synth.pupidra_mamba2(6, 5, 7, 3, 4, 2), (3, 2, 8, 1.5), 5),
    synth.pupidra_layer("attention", synth.pupidra_attention(4, 2, 6, 10, 0.25, 9, 3), (4, 1, 6, 2.0)),
    synth.pupidra_layer("latent_attention", synth.pupidra_latent(3, 6, 4, 5, 7, 0.3, 77.0)),
    synth.pupidra_layer("attention", synth.pupidra_attention(2, 2, 6, 10, 0.5, 5, 8, kv_from=1))], bigram=(11, 3, 2), softcap=20.0, eps=1e-5)


def test_pupidra_configuration_maps_onto_layer_descriptors(tmp_path):
    t = synth.write_seq_model_dir(str(tmp_path), UCFG, 1)
    cfg = seqmodel.read_config(str(tmp_path))
    up = FakeUp()
    st = safetensors_io.SafeTensors(str(tmp_path / "model.safetensors"))
    layers, top = seqmodel.ARCHITECTURES[cfg["architecture"]](cfg, st, up)
    bits = safetensors_io.f32_to_bf16_bits
    assert (top["width"], top["vocab"], top["norm_offset"], top["logit_softcap"], top["bigram_buckets"], top["bigram_mul_prev"], top["bigram_mul_cur"]) == (24, 30, 0.0, 20.0, 11, 3, 2)
    assert up.mats[top["bigram"] - 1001].shape == (12, 24) and top["head"] != top["embed"]
    m, a, b, c = layers
    assert all(x.form == seqmodel.LAYER_POSTNORM and x.norm1 is None and x.norm2 is None and x.canon1 is None for x in layers)
    # the layer scale is part of the output norm's weight
    assert np.array_equal(up.vecs[m.norm1b - 1], t["l0.norm1"] * t["l0.ls1"]) and np.array_equal(up.vecs[m.norm2b - 1], t["l0.norm2"] * t["l0.ls2"]) and b.norm2b is None
    # the recurrence: one stacked projection as the file has it
    assert (m.kind, m.heads, m.vdim, m.dim, m.kv_heads, m.conv_taps, m.norm_parts) == (seqmodel.MIX_SSD, 6, 5, 7, 3, 4, 2)
    assert up.mats[m.in_cat - 1001].shape == (30 + 30 + 21 + 21 + 6, 24) and up.vecs[m.conv - 1].shape == (72, 4) and up.vecs[m.conv_bias - 1].shape == (72,)
    assert all(up.vecs[getattr(m, n) - 1].shape == (6,) for n in ("a_log", "dt_bias", "skip")) and up.vecs[m.onorm - 1].shape == (30,)
    # attention: q | k | v stacked with their biases, a bias on the way out, unit weights for the norms, a slope per head
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, a.pool, a.rot_dims, a.gated, a.head_norm, a.v_unit, a.kv_from) == (
        seqmodel.MIX_WINATTN, 4, 2, 6, 10, 9, 3, 0, 0, 0, 1, 0, 0)
    assert np.array_equal(up.mats[a.in_cat - 1001], np.concatenate([bits(t["l1.mix." + n]) for n in "qkv"])) and up.mats[a.in_cat - 1001].shape == (24 + 12 + 20, 24)
    assert np.array_equal(up.vecs[a.in_bias - 1], np.concatenate([t["l1.mix." + n + ".b"] for n in "qkv"])) and np.array_equal(up.vecs[a.out_bias - 1], t["l1.mix.o.b"])
    assert np.array_equal(up.vecs[a.dist_slope - 1], np.float32([2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8])) and np.array_equal(up.vecs[a.qnorm - 1], np.ones(6)) and np.array_equal(up.vecs[a.knorm - 1], np.ones(6))
    # a layer on another one's keys and values has queries only
    assert (c.kv_from, c.heads, c.kv_heads, c.window, c.keep_first, c.knorm) == (2, 2, 2, 5, 8, None)
    assert np.array_equal(up.mats[c.in_cat - 1001], bits(t["l3.mix.q"])) and np.array_equal(up.vecs[c.in_bias - 1], t["l3.mix.q.b"])
    assert (b.kind, b.q_rank, b.kv_rank, b.rot_dim, b.rot_dims, b.rot_pairing, b.gated, b.window, b.yarn_factor) == (seqmodel.MIX_LATENT, 0, 7, 4, 4, seqmodel.ROT_NEIGHBOURS, 1, 0, 0.0)
    assert (m.ff_kind, m.ff, m.experts, m.top, m.shared_ff, m.moe_softmax, m.moe_weight_output, m.moe_identity, m.moe_groups, m.moe_norm_top, m.moe_scale) == (
        seqmodel.FF_MOE_RELU2, 8, 3, 2, 5, 1, 1, 0, 0, 0, 1.5)
    assert b.ff_kind == c.ff_kind == seqmodel.FF_NONE and a.shared_up is None and a.moe_scale == 2.0
    # what the file and the configuration do not have does not exist
    less = {n: st.f32(n) for n in st.names() if not n.endswith(".b") and ".ls" not in n and n != "bigram"}
    cfg2 = json.loads(json.dumps(UCFG))
    del cfg2["embedding"], cfg2["logit_softcap"], cfg2["layers"][1]["mixer"]["mask"], cfg2["layers"][0]["mlp"]["router"]["scale"]
    synth.write_seq_model_dir(str(tmp_path / "less"), cfg2, 1, tensors=less)
    layers, top = seqmodel.ARCHITECTURES["Pupidra"](cfg2, safetensors_io.SafeTensors(str(tmp_path / "less" / "model.safetensors")), FakeUp())
    m, a, b, c = layers
    assert "bigram" not in top and top["logit_softcap"] == 0.0 and (a.window, a.keep_first, a.in_bias, a.out_bias, c.in_bias, m.moe_scale) == (0, 0, None, None, None, 1.0)
    for i, key, val in ((1, "type", "conveyor"), (1, "mlp", {"kind": "dense", "ff": 8}), (3, "kv_from", 2), (3, "kv_from", 3), (3, "kv_from", 7), (3, "dim", 7), (3, "kv_heads", 1), (0, "groups", 4), (0, "norm_groups", 4)):
        bad = json.loads(json.dumps(UCFG))
        (bad["layers"][i] if key in ("type", "mlp") else bad["layers"][i]["mixer"])[key] = val
        with pytest.raises(seqmodel.ConfigError):
            seqmodel.ARCHITECTURES["Pupidra"](bad, st, FakeUp())


def test_plain_pupidra_statement_reach_and_pieces():
    """causal; the window with its kept first tokens by hand; the slopes of a head count that is no power of two; the bigram rows; the recurrence against its closed
    form; the gate in front of the norm"""
    t = synth.seq_tensors(UCFG, 2)
    rng = np.random.default_rng(0)
    a = rng.integers(0, 30, 20)
    b = a.copy()
    b[6] = (b[6] + 1) % 30
    la, lb = seq_oracle.run_pupidra(UCFG, t, a), seq_oracle.run_pupidra(UCFG, t, b)
    assert np.array_equal(la[:6], lb[:6]) and min(np.abs(la[i] - lb[i]).max() for i in range(6, 20)) > 1e-6 and np.abs(la).max() < 20.0
    mask = seq_oracle.kept_window_mask(8, 3, 2)
    assert [list(np.flatnonzero(r)) for r in mask] == [[0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 3, 4, 5], [0, 1, 4, 5, 6], [0, 1, 5, 6, 7]]
    assert np.allclose(seq_oracle.distance_slopes(3), [2 ** (-8 / 3), 2 ** (-16 / 3), 2 ** -8.0])
    assert seq_oracle.bigram_rows([4, 9, 0], {"buckets": 11, "mul_prev": 3, "mul_cur": 2}) == [11, (4 * 3 + 9 * 2) % 11, (9 * 3) % 11]
    # S_t = sum_s prod_(s < r <= t) g_r dt_s B_s x_s^T
    T, H, P, G, N = 9, 4, 3, 2, 5
    x, B, C, dt = rng.standard_normal((T, H, P)), rng.standard_normal((T, G, N)), rng.standard_normal((T, G, N)), rng.random((T, H)) + 0.1
    al, D = rng.standard_normal(H), rng.standard_normal(H)
    y = seq_oracle.state_space_scan(x, B, C, dt, al, D)
    for hd in range(H):
        cum = np.cumsum(-np.exp(al[hd]) * dt[:, hd])
        for i in range(T):
            want = sum(np.exp(cum[i] - cum[j]) * dt[j, hd] * (C[i, hd // 2] @ B[j, hd // 2]) * x[j, hd] for j in range(i + 1)) + D[hd] * x[i, hd]
            assert np.allclose(y[i, hd], want)
    u, z = rng.standard_normal((2, 6)), rng.standard_normal((2, 6))
    n = seq_oracle.gated_part_norm(u, z, np.ones(6), 3, 0.0)
    assert np.allclose(np.mean(n.reshape(2, 3, 2) ** 2, axis=-1), 1.0) and np.allclose(n, seq_oracle.gated_part_norm(2.0 * u, z, np.ones(6), 3, 0.0))


def test_the_small_library_exports_what_its_models_need():
    if not os.path.exists(hip.SEQ_LIB_PATH):
        pytest.skip("lib/libps_hip_seq.so not built")
    lib = C.CDLL(hip.SEQ_LIB_PATH)
    assert not [n for n in hip.SEQ_EXPORTS if not hasattr(lib, n)]


SCFG = synth.sogavik_config(24, 30, [
    synth.sogavik_layer(synth.sogavik_attention(4, 2, 6, 10, 0.25, 9, 4, 100.0, (4.0, 40, 8.0, 0.5)), moe=(3, 2, 8)),
    synth.sogavik_layer(synth.sogavik_attention(3, 3, 6, 5, 0.5, 7, 2, 77.0), synth.sogavik_memory(5, 4, 3, 6.0), (4, 1, 6)),
    synth.sogavik_layer(synth.sogavik_attention(2, 1, 6, 10, 0.25, 5, 6))], side=5, eps=1e-5)


def test_sogavik_configuration_maps_onto_layer_descriptors(tmp_path):
    t = synth.write_seq_model_dir(str(tmp_path), SCFG, 1)
    cfg = seqmodel.read_config(str(tmp_path))
    up = FakeUp()
    st = safetensors_io.SafeTensors(str(tmp_path / "model.safetensors"))
    layers, top = seqmodel.ARCHITECTURES[cfg["architecture"]](cfg, st, up)
    bits = safetensors_io.f32_to_bf16_bits
    assert (top["width"], top["vocab"], top["norm_offset"], top["norm_center"], top["side_dim"]) == (24, 30, 0.0, 1, 5) and top["head"] != top["embed"]
    assert up.mats[top["side_embed"] - 1001].shape == (30, 15) and np.array_equal(up.vecs[top["final_norm_bias"] - 1], t["final.norm.b"])
    a, b, c = layers
    for i, x in enumerate(layers):
        assert x.form == seqmodel.LAYER_POSTNORM and x.norm1 is None and x.norm2 is None and x.canon1 is None
        assert np.array_equal(up.vecs[x.norm1b - 1], t[f"l{i}.norm1"]) and np.array_equal(up.vecs[x.norm1b_bias - 1], t[f"l{i}.norm1.b"])
        assert up.mats[x.side_gate - 1001].shape == (5, 24) and up.mats[x.side_proj - 1001].shape == (24, 5) and np.array_equal(up.vecs[x.side_norm - 1], t[f"l{i}.side.norm"])
    assert np.array_equal(up.vecs[a.norm2b_bias - 1], t["l0.norm2.b"]) and c.norm2b is None and c.ff_kind == seqmodel.FF_NONE
    # attention: q | k | v | gate stacked, biases alike (none for the gate), norms over the whole projections, frequencies scaled by wavelength
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.rot_dims, a.rot_pairing, a.gated, a.head_norm, a.yarn_factor, a.yarn_original, a.yarn_fast, a.yarn_slow) == (
        seqmodel.MIX_WINATTN, 4, 2, 6, 10, 9, 4, seqmodel.ROT_HALVES, 1, 0, 4.0, 40, 8.0, 0.5)
    assert np.array_equal(up.mats[a.in_cat - 1001], np.concatenate([bits(t["l0.mix." + n]) for n in "qkvg"]))
    assert np.array_equal(up.vecs[a.in_bias - 1], np.concatenate([t["l0.mix." + n + ".b"] for n in "qkv"] + [np.zeros(4, np.float32)]))
    assert up.vecs[a.qnorm - 1].shape == (24,) and up.vecs[a.knorm - 1].shape == (12,) and not a.beside and a.mix_scale == 1.0 and a.mix_onorm is None
    # the pair: half of each side's output behind a norm of its own
    r = b.beside.contents
    assert (b.kind, b.gated, b.yarn_factor, b.mix_scale, r.mix_scale) == (seqmodel.MIX_WINATTN, 0, 0.0, 0.5, 0.5)
    assert np.array_equal(up.vecs[b.mix_onorm - 1], t["l1.mix.left.out"]) and np.array_equal(up.vecs[r.mix_onorm - 1], t["l1.mix.right.out"])
    assert (r.kind, r.heads, r.dim, r.vdim, r.gate_cap) == (seqmodel.MIX_MLSTM, 5, 4, 3, 6.0)
    assert np.array_equal(up.mats[r.in_cat - 1001], np.concatenate([bits(t["l1.mix.right." + n]) for n in "qkvgif"]))
    assert np.array_equal(up.vecs[r.in_bias - 1], np.concatenate([np.zeros(70, np.float32), t["l1.mix.right.i.b"], t["l1.mix.right.f.b"]])) and up.vecs[r.onorm - 1].shape == (15,)
    # the experts
    assert (a.ff_kind, a.ff, a.experts, a.top, a.moe_softmax, a.moe_weight_output, a.moe_norm_top, b.top) == (seqmodel.FF_MOE_SWIGLU, 8, 3, 2, 2, 1, 0, 1)
    assert np.array_equal(up.vecs[a.router_bias - 1], t["l0.mlp.router.b"]) and up.mats[a.ff_up - 1001].shape == (48, 24)
    # what the file and the configuration do not have does not exist
    less = {n: st.f32(n) for n in st.names() if not n.endswith(".b") and "side." not in n and n != "l0.mix.g"}
    cfg2 = json.loads(json.dumps(SCFG))
    del cfg2["token_side"], cfg2["layers"][0]["mixer"]["rot"]["scaling"]
    synth.write_seq_model_dir(str(tmp_path / "less"), cfg2, 1, tensors=less)
    layers, top = seqmodel.ARCHITECTURES["Sogavik"](cfg2, safetensors_io.SafeTensors(str(tmp_path / "less" / "model.safetensors")), FakeUp())
    a, b, c = layers
    assert "side_embed" not in top and top["final_norm_bias"] is None and (a.side_gate, a.norm1b_bias, a.in_bias, a.router_bias, a.gated, a.yarn_factor, b.beside.contents.in_bias) == (
        None, None, None, None, 0, 0.0, None)
    for i, path, val in ((0, ("type",), "conveyor"), (0, ("mlp",), {"kind": "sparse", "ff": 8}), (0, ("mixer", "kv_heads"), 3), (0, ("mixer", "dim"), 7), (1, ("mixer", "right", "heads"), 4),
                         (1, ("mixer", "right", "vdim"), 4), (0, ("mlp", "router", "top"), 4)):
        bad = json.loads(json.dumps(SCFG))
        at = bad["layers"][i]
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = val
        with pytest.raises(seqmodel.ConfigError):
            seqmodel.ARCHITECTURES["Sogavik"](bad, st, FakeUp())
    for val in (4, 6):
        with pytest.raises(seqmodel.ConfigError):
            seqmodel.ARCHITECTURES["Sogavik"](dict(SCFG, token_side={"dim": val}), st, FakeUp())


def test_plain_sogavik_statement_reach_and_pieces():
    """causal; the layer norm takes the mean off in front of its bias; the memory against its closed form, with a denominator that has a floor; the running maximum changes nothing but the
    range; the chosen soft-max; the side input reads the layer's own stretch"""
    t = synth.seq_tensors(SCFG, 2)
    rng = np.random.default_rng(0)
    a = rng.integers(0, 30, 20)
    b = a.copy()
    b[6] = (b[6] + 1) % 30
    la, lb = seq_oracle.run_sogavik(SCFG, t, a), seq_oracle.run_sogavik(SCFG, t, b)
    assert np.array_equal(la[:6], lb[:6]) and min(np.abs(la[i] - lb[i]).max() for i in range(6, 20)) > 1e-6
    x = rng.standard_normal((4, 12))
    n = seq_oracle.biased_layer_norm(x + 3.0, np.ones(12), 0.25, 1e-9)
    assert np.allclose(n.mean(-1), 0.25) and np.allclose(np.var(n, axis=-1), 1.0)
    z = np.linspace(-4, 4, 9)
    assert np.allclose(seq_oracle.gelu_tanh(z) - seq_oracle.gelu_tanh(-z), z) and seq_oracle.gelu_tanh(np.float64(1.0)) == pytest.approx(0.841192, abs=1e-6)
    assert np.allclose(seq_oracle.log_sigmoid(z), np.log(1 / (1 + np.exp(-z)))) and abs(seq_oracle.capped(1e9, 5.0) - 5.0) < 1e-12
    # o_t = sum_s D_ts (q_t . k_s) v_s / (max(|sum_s D_ts (q_t . k_s)|, 1) + tiny),  D_ts = exp(f_(s+1) + .. + f_t + i_s): the maximum cancels but for the 1e-6
    T, H, d, dv = 9, 2, 3, 4
    q, k, v = rng.standard_normal((T, H, d)), rng.standard_normal((T, H, d)), rng.standard_normal((T, H, dv))
    i, f = rng.standard_normal((T, H)), seq_oracle.log_sigmoid(rng.standard_normal((T, H)))
    o = seq_oracle.matrix_memory_scan(q, k, v, i, f)
    for h in range(H):
        c = np.cumsum(f[:, h])
        for s in range(T):
            w = np.exp(c[s] - c[:s + 1] + i[:s + 1, h]) * (k[:s + 1, h] @ q[s, h])
            assert np.allclose(o[s, h], w @ v[:s + 1, h] / max(abs(w.sum()), 1.0), rtol=1e-4, atol=1e-6)
    assert np.allclose(o, seq_oracle.matrix_memory_scan(q, k, v, i, f, m0=-50.0), rtol=1e-4, atol=1e-6)
    W = {n: np.asarray(u, np.float64) for n, u in t.items()}
    h = rng.standard_normal((5, 24))
    moe = SCFG["layers"][0]["mlp"]
    got = seq_oracle.chosen_softmax_experts(W, "l0.mlp.", h, moe)
    for r in range(5):
        zr = W["l0.mlp.router"] @ h[r] + W["l0.mlp.router.b"]
        e0, e1 = np.argsort(-zr)[:2]
        w0 = 1.0 / (1.0 + np.exp(zr[e1] - zr[e0]))
        y = [seq_oracle.gated_feed_forward(W, f"l0.mlp.e{e}.", h[r]) for e in (e0, e1)]
        assert np.allclose(got[r], w0 * y[0] + (1 - w0) * y[1])
    u = seq_oracle.token_side_input(W, "l1.side.", h, a[:5], 1, 5, 1e-5)
    other = dict(W, **{"side.embed": np.where(np.arange(15) // 5 == 1, W["side.embed"], 0.0)})
    assert np.allclose(u, seq_oracle.token_side_input(other, "l1.side.", h, a[:5], 1, 5, 1e-5)) and np.allclose(np.mean((u / W["l1.side.norm"]) ** 2, axis=-1), 1.0, atol=1e-3)
