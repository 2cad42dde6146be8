"""Pupidra (post-norm layers with a layer scale; a hashed bigram table beside the embedding; a state-space recurrence with a scalar decay per head; attention over a
sliding window and the first tokens of the sequence with a penalty per token of distance, unit-rms queries and keys, biases, possibly on another layer's keys and
values; latent attention with neighbour-pair rotary and a gate per head; squared-relu experts whose soft-max scores are taken times a constant; soft-capped
logits) on the GPU against the plain float64 statement in tests/seq_oracle.py: small configurations and weights made here, each mechanism alone, every schedule
(whole prompts, token by token, portions down to two tokens, interleaved requests, reused slots, long decoding, greedy generation), and hand-made models in which
one key or one state decides the logits, so that a lost one shows."""
import numpy as np
import pytest

import seq_oracle
from powerserve_amd import hip, host, seqmodel, synth
from powerserve_amd.safetensors_io import f32_to_bf16_bits

pytestmark = pytest.mark.gpu

UL, UM, UA, ULA, UC = synth.pupidra_layer, synth.pupidra_mamba2, synth.pupidra_attention, synth.pupidra_latent, synth.pupidra_config

CONFIGS = {
    # sizes that are multiples of nothing (scalar state pieces, per-key attention, 64 x 64 mat-mul, the expanded single-token latent step), one key / value head and
    # kv_heads == heads, dim != vdim, layers without feed-forward, a reader with a wider window and more first tokens than the layer it reads, one convolution tap
    "odd": UC(40, 50, [UL("mamba2", UM(3, 10, 7, 1, 3, 2), (5, 2, 12, 1.7), 20), UL("attention", UA(3, 1, 10, 6, 0.3, 9, 3)), UL("latent_attention", ULA(3, 10, 6, 7, 12, 0.25, 1000.0), (4, 1, 9, 0.6)),
                       UL("attention", UA(6, 1, 10, 6, 0.4, 17, 5, kv_from=1), (3, 3, 8, 1.0), 6), UL("mamba2", UM(4, 5, 12, 4, 1, 4)), UL("attention", UA(4, 4, 6, 10, 0.4, 12, 0)),
                       UL("attention", UA(4, 4, 6, 10, 0.2, 5, 1, kv_from=5), (5, 2, 12, 2.0))], bigram=(37, 5, 3), softcap=9.0, eps=1e-5),
    # sizes the matrix-core and chunked kernels take (inputs that are multiples of 64, state and value sizes that are multiples of 16)
    "aligned": UC(128, 96, [UL("latent_attention", ULA(4, 48, 32, 16, 48, 0.15, 10000.0), (8, 2, 64, 2.2), 64), UL("mamba2", UM(8, 16, 32, 2, 4, 2), (6, 3, 64, 1.5), 128),
                            UL("attention", UA(8, 2, 16, 32, 0.3, 24, 10), (4, 1, 128, 3.0), 64), UL("attention", UA(4, 2, 16, 32, 0.35, 40, 18, kv_from=2), (4, 2, 64, 1.0)),
                            UL("mamba2", UM(4, 48, 64, 4, 2, 1), (8, 4, 64, 2.0), 64)], bigram=(211, 29, 13), softcap=12.0),
    # a state of 160 over 6 heads in 3 groups, 20 heads on one key / value head, 18 latent heads; no bigram table, no soft cap
    "manyheads": UC(64, 40, [UL("mamba2", UM(6, 32, 160, 3, 4, 6)), UL("attention", UA(20, 1, 16, 8, 0.3, 30, 4), (2, 1, 16, 2.0), 16), UL("latent_attention", ULA(18, 16, 16, 8, 32, 0.2, 100.0), (3, 2, 32, 1.5))]),
    # 128 value columns per head, a latent wider than the model, the widest state the scan takes, heads == groups == 1
    "wide": UC(96, 40, [UL("attention", UA(2, 2, 48, 128, 0.15, 20, 33), (3, 2, 40, 1.0)), UL("latent_attention", ULA(3, 48, 16, 128, 160, 0.1), (4, 2, 32, 0.5), 24),
                        UL("mamba2", UM(1, 80, 256, 1, 5, 5), (4, 3, 32, 2.0))], bigram=(1, 7, 11), softcap=30.0),
}
TOL = {"float32": 2e-4, "bfloat16": 1e-1}  # fp32: a few ulps of fp32 sums; bfloat16: 8-bit mantissas in models this narrow


def err(got, want):
    """centred rms of the difference over the rms of the logits, worst row"""
    return max(rows(got, want, range(len(want))))


def rows(got, want, which):
    d = np.asarray(got, dtype=np.float64) - want
    d = d - d.mean(-1, keepdims=True)
    s = np.sqrt(np.mean((want - want.mean(-1, keepdims=True)) ** 2))
    r = np.sqrt(np.mean(d * d, -1)) / s
    return [float(r[i]) for i in which]


def close(got, want, dtype):
    """float32: every row within TOL.  bfloat16: nine rows in ten within TOL and none beyond the logits' own spread -- where two scores of a router are closer
    than 8-bit mantissas resolve, the choice may go the other way and the rows behind it move; the same schedules are held to 2e-4 in float32."""
    if dtype == "float32":
        return err(got, want) < TOL[dtype]
    r = rows(got, want, range(len(want)))
    return float(np.quantile(r, 0.9)) < TOL[dtype] and max(r) < 1.0


@pytest.fixture(scope="module")
def made(ctx, tmp_path_factory):
    cache = {}

    def get(name, dtype="float32", max_batch=16, cfg=None, tensors=None, max_context=600):
        key = (name, dtype, max_batch, max_context)
        if key not in cache:
            c = cfg or CONFIGS[name]
            d = str(tmp_path_factory.mktemp("u"))
            t = synth.write_seq_model_dir(d, c, 0, tensors)
            cache[key] = (seqmodel.load_model(ctx, d, dtype=dtype, max_batch=max_batch, n_slots=3, max_context=max_context), c, t)
        return cache[key]

    yield get
    for m, _, _ in cache.values():
        m.close()


def tokens_for(cfg, n, seed=1, lo=0):
    return np.random.default_rng(seed).integers(lo, cfg["vocab"], n).astype(np.int32)


def run_portions(m, toks, sizes):
    s, out, at, i = m.acquire(), [], 0, 0
    while at < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - at)
        out.append(m.forward(s, toks[at:at + n], np.arange(n)))
        at, i = at + n, i + 1
    m.release(s)
    return np.concatenate(out)


def bf16(t):
    return {k: (f32_to_bf16_bits(np.asarray(v, np.float32)).astype(np.uint32) << 16).view(np.float32).reshape(np.shape(v)) for k, v in t.items()}


def layer_adds(m, toks, sizes):
    """what the first (only) layer adds to the embedding, fed in portions"""
    m.capture_layers(True)
    s, got, at, i = m.acquire(), [], 0, 0
    while at < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - at)
        m.forward(s, toks[at:at + n])
        got.append(m.layers(n)[0].astype(np.float64))
        at, i = at + n, i + 1
    m.release(s)
    m.capture_layers(False)
    return np.concatenate(got)


# ---------------------------------------------------------------------------------------------------------------- mechanisms, one at a time
ALONE = {
    "state_space": UL("mamba2", UM(6, 10, 9, 3, 4, 4)),
    "state_space_chunked": UL("mamba2", UM(6, 32, 48, 3, 4, 2)),
    "state_space_wide": UL("mamba2", UM(2, 64, 256, 1, 2, 1)),
    "attention": UL("attention", UA(3, 1, 10, 6, 0.3, 11, 4)),
    "attention_mfma": UL("attention", UA(6, 2, 16, 8, 0.3, 21, 6)),
    "attention_unmasked": UL("attention", UA(4, 2, 16, 8, 0.3, 0, 0)),
    "latent": UL("latent_attention", ULA(3, 10, 6, 7, 12, 0.25, 100.0)),
    "latent_mfma": UL("latent_attention", ULA(4, 16, 16, 8, 32, 0.2, 10000.0)),
    "mixture": UL("attention", UA(3, 1, 10, 6, 0.3, 11, 4), (6, 2, 14, 1.9)),
    "mixture_aligned": UL("attention", UA(3, 1, 10, 6, 0.3, 11, 4), (6, 3, 64, 0.7), 64),
    "mixture_top1": UL("attention", UA(3, 1, 10, 6, 0.3, 11, 4), (5, 1, 12, 3.0)),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", list(ALONE))
def test_each_mechanism_alone(made, which, dtype):
    """one layer in which only one sublayer contributes (the mixer's layer scale is zero, or there is no feed-forward): what it adds to the embedding against that
    mechanism's own plain function, in one portion, in portions and token by token"""
    layer = ALONE[which]
    W_ = 64 if which.endswith(("mfma", "aligned", "chunked")) else 40
    cfg = UC(W_, 32, [layer], eps=1e-5)
    t = synth.seq_tensors(cfg, 3)
    if layer["mlp"]:
        t["l0.ls1"] = np.zeros_like(t["l0.ls1"])
    m, _, _ = made("alone_" + which, dtype, max_batch=200, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 150, seed=3)
    W = {k: np.asarray(v, np.float64) for k, v in t.items()}
    x0 = W["embed"][toks]
    mc, n = layer["mixer"], "2" if layer["mlp"] else "1"
    if layer["mlp"]:
        y = seq_oracle.scaled_experts(W, "l0.mlp.", x0, layer["mlp"])
    elif layer["type"] == "mamba2":
        y = seq_oracle.state_space_mixer(W, "l0.mix.", x0, mc, 1e-5)
    elif layer["type"] == "attention":
        y = seq_oracle.kept_window_attention(W, "l0.mix.", x0, mc, 1e-5, size=mc["mask"]["size"] or len(toks))[0]
    else:
        y = seq_oracle.neighbour_latent_attention(W, "l0.mix.", x0, mc, 1e-5)
    want = seq_oracle.plain_norm(y, W["l0.norm" + n], 1e-5) * W["l0.ls" + n]
    for sizes in ([150], [1], [70, 3, 2, 33, 1]):
        got = layer_adds(m, toks, sizes) - x0
        bad = np.abs(got - want).max(axis=1) / np.abs(want).max()
        if dtype == "float32":
            assert bad.max() < 2e-4, sizes
        else:  # (the norm behind the sublayer stretches rows whose output is small; a router's close call may flip)
            assert np.quantile(bad, 0.9) < 6e-2, sizes


def test_what_the_plain_statement_is_sensitive_to(made):
    """every mechanism of the design left out of the plain statement in turn moves its logits far from the right ones; the library agrees with the right ones"""
    m, cfg, t = made("odd", "float32", max_batch=32)
    toks = tokens_for(cfg, 30, seed=8)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    for kw in ({"use_bigram": False}, {"use_previous": False}, {"use_layer_scale": False}, {"use_cap": False}, {"attn_kw": {"use_slopes": False}},
               {"attn_kw": {"use_unit": False}}, {"attn_kw": {"use_bias": False}}, {"attn_kw": {"keep": 0}}, {"attn_kw": {"size": 30}}, {"latent_kw": {"use_rotation": False}},
               {"latent_kw": {"use_gate": False}}, {"latent_kw": {"use_latent_norm": False}}, {"ssm_kw": {"carry": False}}, {"ssm_kw": {"use_D": False}}, {"ssm_kw": {"use_filter": False}},
               {"ssm_kw": {"gate_first": False}}, {"ssm_kw": {"one_group": True}}, {"moe_kw": {"use_scale": False}}, {"moe_kw": {"use_shared": False}}, {"moe_kw": {"renormalise": True}}):
        assert err(seq_oracle.run_pupidra(cfg, t, toks, **kw), want) > 5e-3, kw
    assert err(run_portions(m, toks, [30]), want) < TOL["float32"]
    assert err(run_portions(m, toks, [1]), want) < TOL["float32"]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_against_the_plain_statement(made, name, dtype):
    m, cfg, t = made(name, dtype, max_batch=64)
    toks = tokens_for(cfg, 90)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    s = m.acquire()
    got = m.forward(s, toks, np.arange(len(toks)))
    m.release(s)
    assert close(got, want, dtype)


@pytest.mark.parametrize("name", ["odd", "aligned", "wide"])
def test_the_residual_stream_after_every_layer(made, name):
    m, cfg, t = made(name, "float32", max_batch=64)
    toks = tokens_for(cfg, 45, seed=5)
    per = []
    seq_oracle.run_pupidra(cfg, t, toks, per_layer=per)
    assert m.n_runs == len(per) == len(cfg["layers"])
    m.capture_layers(True)
    s = m.acquire()
    m.forward(s, toks)
    got = m.layers(len(toks))
    m.release(s)
    m.capture_layers(False)
    for i, want in enumerate(per):
        assert np.abs(got[i] - want).max() < 2e-4 * np.abs(want).max(), i


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_token_by_token_and_portions_give_the_whole_prompts_logits(made, name, dtype):
    m, cfg, t = made(name, dtype, max_batch=16)  # 16: a 50-token portion is also cut inside the library
    toks = tokens_for(cfg, 90, seed=2)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    for sizes in ([1], [2], [3, 1, 7, 2], [50, 2, 23], [16, 17, 15], [9, 8, 10]):  # (9 and 10 tokens: the smallest tiled mixtures, 8: the widest mat-vec)
        assert close(run_portions(m, toks, sizes), want, dtype), sizes


@pytest.mark.parametrize("name", ["aligned", "manyheads", "wide"])
def test_portions_around_the_chunks_of_the_recurrence(made, name):
    """portions just below, at and above whole chunks of the chunked recurrence (64 tokens), with scanned portions and single tokens between them"""
    m, cfg, t = made(name, "float32", max_batch=256)
    toks = tokens_for(cfg, 330, seed=12)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    for sizes in ([330], [63, 65], [64, 1, 128, 2], [31, 32, 33, 129], [200, 7]):
        assert err(run_portions(m, toks, sizes), want) < TOL["float32"], sizes


def test_first_tokens_of_a_sequence(made):
    """the first token takes the bigram table's last row and sees itself alone"""
    m, cfg, t = made("aligned", "float32")
    for n in (1, 2, 3, 5):
        toks = tokens_for(cfg, n, seed=10 + n)
        want = seq_oracle.run_pupidra(cfg, t, toks)
        assert err(seq_oracle.run_pupidra(cfg, dict(t, bigram=np.roll(t["bigram"], 1, axis=0)), toks), want) > 1e-2
        assert err(run_portions(m, toks, [n]), want) < TOL["float32"]
        assert err(run_portions(m, toks, [1]), want) < TOL["float32"]


def test_interleaved_requests_and_reused_slots(made):
    """requests of unequal length fed in turns through the scheduler against each alone; then every slot is used again and must start from nothing (no previous
    token, no convolution tail, no state, no kept first tokens of the request before)"""
    m, cfg, t = made("aligned", "float32", max_batch=16)
    seqs = [tokens_for(cfg, n, seed=20 + n) for n in (61, 9, 88)]
    want = [seq_oracle.run_pupidra(cfg, t, s) for s in seqs]
    sched = seqmodel.RequestScheduler(m)
    got, at = [[] for _ in seqs], [0, 0, 0]
    steps, i = [5, 2, 11, 1, 3], 0
    while any(a < len(s) for a, s in zip(at, seqs)):
        r = i % 3
        if at[r] < len(seqs[r]):
            n = min(steps[i % len(steps)], len(seqs[r]) - at[r])
            got[r].append(sched.feed("req%d" % r, seqs[r][at[r]:at[r] + n], np.arange(n)))
            at[r] += n
            if at[r] == len(seqs[r]):
                sched.finish("req%d" % r)
        i += 1
    for g, w in zip(got, want):
        assert err(np.concatenate(g), w) < TOL["float32"]
    for r in range(4):
        which = 2 if r % 2 == 0 else 1
        assert err(sched.feed("again", seqs[which], np.arange(len(seqs[which]))), want[which]) < TOL["float32"]
        sched.finish("again")
    with pytest.raises(hip.PSHipError):
        [m.acquire() for _ in range(4)]
    for s in range(3):
        m.release(s)


# ---------------------------------------------------------------------------------------------------------------- weights made so that a fault shows
def mark_embedding(t, cfg, rng):
    """Token 0 is a MARK: its embedding alone has feature 0; feature 1 is the same constant for every token; nothing a layer puts out touches the two."""
    V, W = cfg["vocab"], cfg["width"]
    e = rng.standard_normal((V, W)).astype(np.float32) * 0.5
    e[:, 0], e[:, 1], e[0, 0] = 0.0, 4.0, 8.0
    t["embed"] = e
    for i, lc in enumerate(cfg["layers"]):
        for n in ("1", "2"):
            if f"l{i}.ls{n}" in t:
                t[f"l{i}.ls{n}"] = np.where(np.arange(W) < 2, 0.0, t[f"l{i}.ls{n}"]).astype(np.float32)


def mark_attention(t, p, mc, W, rng):
    """Every key reads feature 0 into the last channel of its head and every query reads feature 1 into that channel: with unit-rms vectors a query's score for a
    mark is about dim x scale, for anything else about 0.  Every value channel reads feature 0."""
    H, G, d, dv, c = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"], mc["dim"] - 1
    q = rng.standard_normal((H * d, W)).astype(np.float32) * 0.02
    q[:, :2] = 0.0
    q[c::d, 1] = 2.0
    t[p + "q"], t[p + "q.b"] = q, np.zeros(H * d, np.float32)
    if mc.get("kv_from") is None:
        k = rng.standard_normal((G * d, W)).astype(np.float32) * 0.05
        k[:, :2] = 0.0
        k[c::d, 0] = 2.0
        v = rng.standard_normal((G * dv, W)).astype(np.float32) * 0.2
        v[:, 0] = 1.5
        t[p + "k"], t[p + "k.b"], t[p + "v"] = k, np.zeros(G * d, np.float32), v


MASK = {"own": (24, 7), "reader": (37, 13)}


def marked_attention_model(aligned, seed=0):
    """an attention layer and one that reads its keys with a wider window and more first tokens"""
    rng = np.random.default_rng(seed)
    W = 64 if aligned else 30
    H, G, d, dv = (4, 2, 16, 8) if aligned else (3, 1, 10, 6)
    cfg = UC(W, 24, [UL("attention", UA(H, G, d, dv, 1.2, *MASK["own"])), UL("attention", UA(2 * H, G, d, dv, 1.2, *MASK["reader"], kv_from=0))], eps=1e-5)
    t = synth.seq_tensors(cfg, seed)
    mark_embedding(t, cfg, rng)
    for i in (0, 1):
        mark_attention(t, f"l{i}.mix.", cfg["layers"][i]["mixer"], W, rng)
    return cfg, bf16(t)


def with_masks(cfg, own, reader):
    layers = [dict(lc, mixer=dict(lc["mixer"], mask={"size": s, "keep_first": k})) for lc, (s, k) in zip(cfg["layers"], (own, reader))]
    return dict(cfg, layers=layers)


@pytest.mark.parametrize("aligned", [False, True])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_window_and_first_token_edges_in_prompts_and_in_decoding(made, dtype, aligned):
    """One mark, at the last kept position, at the first that is not kept, or in the middle: the statement whose window or number of kept tokens is one off (either
    layer) is far off on the row that its edge moves and right up to there; the library agrees with the right one, in portions cut anywhere (edges across portion
    and tile borders, the kept tokens brought by several portions) and token by token."""
    cfg, t = marked_attention_model(aligned)
    m, _, _ = made("marked%d" % aligned, dtype, max_batch=64, cfg=cfg, tensors=t)
    tol = 1e-3 if dtype == "float32" else TOL[dtype]
    (so, ko), (sr, kr) = MASK["own"], MASK["reader"]
    for mark in (ko - 1, ko, kr - 1, kr, 50):
        toks = tokens_for(cfg, 130, seed=30 + mark, lo=1)
        toks[mark] = 0
        want = seq_oracle.run_pupidra(cfg, t, toks)
        wrong = [(with_masks(cfg, (so + 1, ko), (sr, kr)), mark + so), (with_masks(cfg, (so - 1, ko), (sr, kr)), mark + so - 1),
                 (with_masks(cfg, (so, ko), (sr + 1, kr)), mark + sr), (with_masks(cfg, (so, ko), (sr - 1, kr)), mark + sr - 1)]
        for bad, row in wrong:
            r = rows(seq_oracle.run_pupidra(bad, t, toks), want, range(len(toks)))
            own = bad["layers"][0]["mixer"]["mask"] != cfg["layers"][0]["mixer"]["mask"]
            assert max(r[mark:row]) < 0.01, (mark, row)  # (the mark is seen either way and outweighs the other key at the edge)
            if mark >= (ko if own else kr):
                assert r[row] > 0.3, (mark, row)
        for own, bad, off in ((True, with_masks(cfg, (so, ko - 1), (sr, kr)), -1), (True, with_masks(cfg, (so, ko + 1), (sr, kr)), 0),
                              (False, with_masks(cfg, (so, ko), (sr, kr - 1)), -1), (False, with_masks(cfg, (so, ko), (sr, kr + 1)), 0)):
            if mark == (ko if own else kr) + off:
                r = rows(seq_oracle.run_pupidra(bad, t, toks), want, range(len(toks)))
                assert np.median(r[mark + (so if own else sr):]) > 0.1 and max(r[:mark + (so if own else sr)]) < 1e-9, (mark, off)
        for sizes in ([130], [1], [3, 2, 5], [61, 2, 1, 30]):
            assert max(rows(run_portions(m, toks, sizes), want, range(len(toks)))) < tol, (mark, sizes)


@pytest.mark.parametrize("aligned", [False, True])
def test_a_reader_uses_the_layer_it_names(made, aligned):
    """two attention layers with keys of their own and one that reads the first's: the statement that reads the second's is far off"""
    W = 64 if aligned else 30
    H, G, d, dv = (4, 2, 16, 8) if aligned else (3, 1, 10, 6)
    cfg = UC(W, 24, [UL("attention", UA(H, G, d, dv, 0.5, 9, 2)), UL("attention", UA(H, G, d, dv, 0.5, 14, 3), (3, 2, 16, 1.5)), UL("mamba2", UM(2, 16, 16, 1, 3, 1)),
                     UL("attention", UA(H, G, d, dv, 0.5, 20, 4, kv_from=0))], eps=1e-5)
    t = synth.seq_tensors(cfg, 4)
    m, _, _ = made("reader%d" % aligned, "float32", max_batch=32, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 80, seed=5)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    assert np.median(rows(seq_oracle.run_pupidra(cfg, t, toks, share=False), want, range(len(toks)))) > 0.05
    for sizes in ([80], [1], [7, 2, 30]):
        assert err(run_portions(m, toks, sizes), want) < TOL["float32"], sizes


def marked_latent_model(aligned, seed=0):
    """one latent layer whose latent channel 0 reads feature 0; the key expansion sends it to the last plain channel of every head, where the query reads feature 1"""
    rng = np.random.default_rng(seed)
    W = 64 if aligned else 30
    H, d, dr, dv, R = (4, 16, 16, 8, 16) if aligned else (3, 10, 6, 6, 9)
    cfg = UC(W, 24, [UL("latent_attention", ULA(H, d, dr, dv, R, 0.9))], eps=1e-5)
    t = synth.seq_tensors(cfg, seed)
    mark_embedding(t, cfg, rng)
    p, c = "l0.mix.", d - 1
    dkv = rng.standard_normal((R + dr, W)).astype(np.float32) * 0.1
    dkv[:, :2] = 0.0
    dkv[0, 0] = 3.0
    q = rng.standard_normal((H * (d + dr), W)).astype(np.float32) * 0.1
    q[:, :2] = 0.0
    q[c::d + dr, 1] = 1.0
    uk = rng.standard_normal((H * d, R)).astype(np.float32) * 0.1
    uv = rng.standard_normal((H * dv, R)).astype(np.float32) * 0.2
    uk[:, 0], uv[:, 0] = 0.0, 1.5
    uk[c::d, 0] = 2.0
    t[p + "q"], t[p + "dkv"], t[p + "uk"], t[p + "uv"], t[p + "dkv.norm"] = q, dkv, uk, uv, np.ones(R, np.float32)
    return cfg, bf16(t)


@pytest.mark.parametrize("aligned", [False, True])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_latent_key_among_hundreds(made, dtype, aligned):
    cfg, t = marked_latent_model(aligned)
    m, _, _ = made("latentmark%d" % aligned, dtype, max_batch=64, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 470, seed=3, lo=1)
    toks[4] = 0
    want = seq_oracle.run_pupidra(cfg, t, toks)
    for reach in (64, 256, 300):
        wrong = seq_oracle.run_pupidra(cfg, t, toks, latent_kw={"reach": reach})
        assert np.median(rows(wrong, want, range(4 + reach, 470))) > 0.05 and max(rows(wrong, want, range(0, reach))) < 1e-9
    tol = 1e-3 if dtype == "float32" else TOL[dtype]
    s = m.acquire()
    got = [m.forward(s, toks[:300], np.arange(300))] + [m.forward(s, toks[i:i + 1], [0]) for i in range(300, 470)]
    m.release(s)
    assert max(rows(np.concatenate(got), want, range(len(toks)))) < tol
    for sizes in ([470], [64], [61, 2, 100]):
        assert max(rows(run_portions(m, toks, sizes), want, range(len(toks)))) < tol, sizes


@pytest.mark.parametrize("aligned", [False, True])
def test_rotation_far_from_the_start(made, aligned):
    """a latent layer whose rotated parts carry the scores, 400 tokens: the statement without rotation, or with halves in the place of neighbours, is off"""
    la = ULA(4, 16, 32, 8, 32, 0.15, 10000.0) if aligned else ULA(3, 6, 10, 7, 12, 0.3, 200.0)
    cfg = UC(64 if aligned else 40, 32, [UL("latent_attention", la)], eps=1e-5)
    t = synth.seq_tensors(cfg, 5)
    H, d, dr, R = la["heads"], la["dim"], la["rot_dim"], la["kv_rank"]
    q = t["l0.mix.q"].reshape(H, d + dr, -1).copy()
    q[:, d:] *= 3.0
    t["l0.mix.q"] = q.reshape(H * (d + dr), -1)
    t["l0.mix.dkv"] = t["l0.mix.dkv"].copy()
    t["l0.mix.dkv"][R:] *= 3.0
    t = bf16(t)
    m, _, _ = made("rot%d" % aligned, "float32", max_batch=64, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 400, seed=4)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    assert err(seq_oracle.run_pupidra(cfg, t, toks, latent_kw={"use_rotation": False}), want) > 0.05
    halves = np.concatenate([np.arange(0, dr, 2), np.arange(1, dr, 2)])  # the same weights read as if pair i were (i, i + dr / 2)
    other = dict(t, **{"l0.mix.q": t["l0.mix.q"].reshape(H, d + dr, -1)[:, np.r_[np.arange(d), d + np.argsort(halves)]].reshape(H * (d + dr), -1),
                       "l0.mix.dkv": t["l0.mix.dkv"][np.r_[np.arange(R), R + np.argsort(halves)]]})
    assert err(seq_oracle.run_pupidra(cfg, other, toks), want) > 0.05
    for sizes in ([64], [1], [61, 2, 100, 1, 1]):
        assert max(rows(run_portions(m, toks, sizes), want, range(len(toks)))) < 1e-3, sizes


@pytest.mark.parametrize("which", ["scan", "chunked"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_state_is_carried_for_hundreds_of_tokens(made, dtype, which):
    """slow decays (a few thousandths per token): the statement that loses its state once, at a portion's or a chunk's edge, is far off on hundreds of rows behind it"""
    mc = UM(3, 10, 14, 1, 3, 1) if which == "scan" else UM(4, 32, 48, 2, 4, 2)
    cfg = UC(64, 24, [UL("mamba2", mc)], eps=1e-5)
    t = synth.seq_tensors(cfg, 6)
    t["l0.mix.A_log"] = np.linspace(-5.5, -4.5, mc["heads"]).astype(np.float32)
    t["l0.mix.D"] = t["l0.mix.D"] * 0.1
    t = bf16(t)
    m, _, _ = made("slow_" + which, dtype, max_batch=128, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 420, seed=9)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    for at in (64, 128, 200):
        r = rows(seq_oracle.run_pupidra(cfg, t, toks, ssm_kw={"lose_at": at}), want, range(len(toks)))
        assert max(r[:at]) < 1e-9 and np.median(r[at:at + 200]) > 0.1, at
    for sizes in ([420], [64], [1], [200, 1, 1, 2, 70]):
        assert max(rows(run_portions(m, toks, sizes), want, range(len(toks)))) < (1e-3 if dtype == "float32" else TOL[dtype]), sizes


def test_fast_and_slow_decays_side_by_side(made):
    """decays from one part in a thousand to e^-40 per token, large steps: nothing overflows and the chunked recurrence agrees with the scan"""
    mc = UM(8, 32, 32, 2, 4, 1)
    cfg = UC(64, 24, [UL("mamba2", mc)], eps=1e-5)
    t = synth.seq_tensors(cfg, 7)
    t["l0.mix.A_log"] = np.linspace(-6.0, 3.0, 8).astype(np.float32)
    t["l0.mix.dt_bias"] = np.linspace(2.0, -3.0, 8).astype(np.float32)[[0, 7, 1, 6, 2, 5, 3, 4]]
    t = bf16(t)
    m, _, _ = made("decays", "float32", max_batch=256, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 256, seed=11)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    for sizes in ([256], [1], [100, 3]):
        assert err(run_portions(m, toks, sizes), want) < TOL["float32"], sizes


def test_the_previous_token_crosses_portions(made):
    """a model in which the bigram row decides: portions of every size, single tokens, and the captured greedy step all see the token before"""
    cfg = UC(40, 30, [UL("attention", UA(2, 1, 8, 8, 0.3, 6, 1))], bigram=(101, 13, 7), eps=1e-5)
    t = synth.seq_tensors(cfg, 8)
    t["embed"] = t["embed"] * 0.1
    t = bf16(t)
    m, _, _ = made("bigram", "float32", max_batch=8, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 40, seed=2)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    assert min(rows(seq_oracle.run_pupidra(cfg, t, toks, use_previous=False), want, range(1, 40))) > 0.2
    for sizes in ([40], [1], [2], [8, 1, 5]):
        assert err(run_portions(m, toks, sizes), want) < TOL["float32"], sizes
    ids = m.generate(toks[:7], 12)
    s = m.acquire()
    m.forward(s, toks[:6])
    first = m.decode_greedy(s, int(toks[6]), 5)
    rest = m.decode_greedy(s, int(first[-1]), 7)  # a second call goes on from the slot's own memory of the last token
    m.release(s)
    assert np.array_equal(np.concatenate([first, rest]), ids)
    full = np.concatenate([toks[:7], ids])
    want = seq_oracle.run_pupidra(cfg, t, full[:-1])
    assert all(want[6 + i].max() - want[6 + i][tok] < 1e-4 * (want.max() - want.min()) for i, tok in enumerate(ids))


def test_long_decoding_keeps_the_caches(made):
    m, cfg, t = made("aligned", "float32", max_batch=16)
    toks = tokens_for(cfg, 260, seed=6)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    assert err(run_portions(m, toks, [13, 1, 1, 1, 1, 1, 1, 1]), want) < TOL["float32"]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["aligned", "odd"])
def test_greedy_generation_through_the_entry_point(made, name, dtype):
    """SeqModel.generate (prefill, then the captured single-token step feeding its own arg-max) picks, at every step, a token whose logit in the
    plain statement is the largest up to rounding; eager launches and a host sampler set to top-1 give the same ids."""
    m, cfg, t = made(name, dtype, max_batch=16)
    prompt = tokens_for(cfg, 29, seed=7)
    ids = m.generate(prompt, 40)
    assert ids.shape == (40,)
    full = np.concatenate([prompt, ids])
    want = seq_oracle.run_pupidra(cfg, t, full[:-1])
    spread = want.max() - want.min()
    off = [(want[len(prompt) - 1 + i].max() - want[len(prompt) - 1 + i][tok]) / spread for i, tok in enumerate(ids)]
    assert max(off) < 1e-4 if dtype == "float32" else np.quantile(off, 0.9) < 3e-2
    m.set_mode(1)
    assert np.array_equal(m.generate(prompt, 40), ids)
    m.set_mode(0)
    assert np.array_equal(m.generate(prompt, 40), ids)  # the captured sequence replayed on a slot that was used before
    sm = host.Sampler(host.SamplerCfg.make(cfg["vocab"], seed=1, temperature=1.0, top_p=1.0, top_k=1))
    assert np.array_equal(m.generate(prompt, 40, sampler=sm.sample), ids)
    sm.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["aligned", "manyheads", "wide"])
def test_matrix_core_forms_agree_with_the_plain_kernels(made, name, dtype):
    """mode bit 1 keeps the per-key attention, the expanded single-token latent step, the token-by-token scan and the 64 x 64 mat-mul (also for the experts' grouped
    products): the faster forms of a portion and of a single token must give the same logits (fp32: up to the order of sums)"""
    m, cfg, t = made(name, dtype, max_batch=128)
    toks = tokens_for(cfg, 250, seed=9)
    cuts = ([128], [1], [70, 1, 1, 1, 9])
    fast = [run_portions(m, toks, sizes) for sizes in cuts]
    m.set_mode(2)
    plain = [run_portions(m, toks, sizes) for sizes in cuts]
    m.set_mode(0)
    want = seq_oracle.run_pupidra(cfg, t, toks)
    for a, b in zip(fast, plain):
        assert err(a, b) < 1e-4 if dtype == "float32" else close(a, b.astype(np.float64), dtype)
        assert close(a, want, dtype)


def test_host_facade_loads_and_generates_the_same(made, tmp_path):
    m, cfg, t = made("odd", "float32", max_batch=16)
    synth.write_seq_model_dir(str(tmp_path), cfg, 0, t)
    hm = host.HostSeqModel(str(tmp_path), dtype="float32", max_batch=16, n_slots=2, max_context=600)
    prompt = tokens_for(cfg, 19, seed=7)
    ids = m.generate(prompt, 12)
    assert np.array_equal(hm.generate(prompt, 12), ids)
    s, s2 = hm.acquire(), m.acquire()
    a, b = hm.forward(s, prompt, [0, 5, 18]), m.forward(s2, prompt, [0, 5, 18])
    hm.release(s)
    m.release(s2)
    assert np.array_equal(a, b)
    hm.close()


def test_a_sequence_fills_its_context_and_no_more(ctx, tmp_path):
    """(more first tokens asked for than the context holds, and windows beyond it)"""
    cfg = UC(40, 50, [UL("attention", UA(3, 1, 10, 6, 0.3, 9, 64)), UL("latent_attention", ULA(3, 10, 6, 7, 12, 0.25)), UL("attention", UA(3, 1, 10, 6, 0.3, 500, 5, kv_from=0))], eps=1e-5)
    t = synth.write_seq_model_dir(str(tmp_path), cfg, 0)
    m = seqmodel.load_model(ctx, str(tmp_path), dtype="float32", max_batch=8, n_slots=1, max_context=20)
    toks = tokens_for(cfg, 20)
    s = m.acquire()
    got = [m.forward(s, toks[:18], np.arange(18))]
    with pytest.raises(hip.PSHipError):
        m.forward(s, [1, 2, 3])
    got.append(m.forward(s, toks[18:], [0, 1]))
    m.release(s)
    assert err(np.concatenate(got), seq_oracle.run_pupidra(cfg, t, toks)) < TOL["float32"]
    m.close()
