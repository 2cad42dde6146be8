"""Sogavik (post-norm layers whose layer norms have a weight and a bias; an input of every layer's own for the token itself; attention over a sliding window with biases,
RMS norms over the whole q / k projections, rotate-half rotary scaled by wavelength and a gate per head; two mixers side by side -- such an attention and a matrix
memory with exponential gates -- normed one by one and averaged; SiLU-gated experts weighted by the soft-max over the chosen logits) on the GPU against the plain
float64 statement in tests/seq_oracle.py: small configurations and weights made here, each mechanism alone, every schedule (whole prompts, token by token, portions
down to two tokens, interleaved requests, reused slots, long decoding, greedy generation), and hand-made models in which one key or one written token decides the
logits, so that a lost one shows."""
import numpy as np
import pytest

import seq_oracle
from powerserve_amd import hip, host, seqmodel, synth
from test_gpu_pupidra import TOL, bf16, close, err, layer_adds, rows, run_portions, tokens_for

pytestmark = pytest.mark.gpu

SL, SA, SM, SC = synth.sogavik_layer, synth.sogavik_attention, synth.sogavik_memory, synth.sogavik_config
YARN = (4.0, 60, 8.0, 0.5)

CONFIGS = {
    # sizes that are multiples of nothing (scalar state pieces, per-key attention, 64 x 64 mat-mul, a joint input projection whose parts need padding), one key / value
    # head and kv_heads == heads, dim != vdim on both sides, a rotation of every number of a head and of two, layers without feed-forward, a scaling on the left side too
    "odd": SC(40, 50, [SL(SA(3, 1, 10, 6, 0.3, 9, 4, 100.0, YARN), moe=(5, 2, 12)), SL(SA(6, 3, 10, 7, 0.25, 17, 10, 1000.0), SM(3, 7, 5, 6.0), (3, 3, 9)), SL(SA(4, 4, 6, 10, 0.4, 12, 2)),
                       SL(SA(2, 1, 6, 5, 0.4, 5, 6, 50.0, YARN), SM(5, 12, 4, 15.0)), SL(SA(5, 5, 4, 3, 0.5, 1, 4), moe=(4, 1, 10))], side=7, eps=1e-5),
    # sizes the matrix-core and chunked kernels take (inputs that are multiples of 64, state and value sizes that are multiples of 16)
    "aligned": SC(128, 96, [SL(SA(4, 2, 32, 16, 0.2, 24, 16, 10000.0), SM(4, 48, 32, 9.0), (8, 2, 64)), SL(SA(8, 2, 16, 32, 0.3, 40, 8, 500.0, (2.5, 256, 24.0, 1.5)), moe=(6, 3, 64)),
                            SL(SA(2, 2, 64, 64, 0.15, 33, 64, 10000.0, YARN), SM(6, 16, 64, 4.0), (4, 1, 128))], side=64),
    # 20 heads on one key / value head beside 18 memories of 160, a token input of one number per layer; an odd number of gate rows in front of the second mixer
    "manyheads": SC(64, 40, [SL(SA(20, 1, 16, 8, 0.3, 30, 8), SM(18, 160, 8, 12.0)), SL(SA(3, 3, 16, 8, 0.3, 70, 16, 200.0), moe=(7, 2, 16))], side=1),
    # 128 value columns per head, a memory of the widest keys and of values beyond one block's 128 columns, heads == 1; no token input
    "wide": SC(96, 40, [SL(SA(2, 2, 48, 128, 0.15, 20, 32), SM(1, 256, 140, 30.0), (4, 3, 32)), SL(SA(1, 1, 48, 128, 0.15, 300, 48, 10000.0, YARN), moe=(3, 2, 40))], side=None),
}


@pytest.fixture(scope="module")
def made(ctx, tmp_path_factory):
    cache = {}

    def get(name, dtype="float32", max_batch=16, cfg=None, tensors=None, max_context=600):
        key = (name, dtype, max_batch, max_context)
        if key not in cache:
            c = cfg or CONFIGS[name]
            d = str(tmp_path_factory.mktemp("s"))
            t = synth.write_seq_model_dir(d, c, 0, tensors)
            cache[key] = (seqmodel.load_model(ctx, d, dtype=dtype, max_batch=max_batch, n_slots=3, max_context=max_context), c, t)
        return cache[key]

    yield get
    for m, _, _ in cache.values():
        m.close()


# ---------------------------------------------------------------------------------------------------------------- mechanisms, one at a time
ALONE = {
    "attention": SL(SA(3, 1, 10, 6, 0.3, 11, 4, 100.0, YARN)),
    "attention_mfma": SL(SA(6, 2, 16, 8, 0.3, 21, 16, 100.0, YARN)),
    "left": SL(SA(6, 3, 10, 6, 0.3, 13, 10), SM(2, 5, 3, 8.0)),
    "left_mfma": SL(SA(4, 4, 32, 16, 0.2, 40, 16), SM(3, 16, 12, 8.0)),
    "memory": SL(SA(3, 3, 10, 6, 0.3, 11, 4), SM(3, 9, 5, 6.0)),
    "memory_chunked": SL(SA(2, 1, 16, 16, 0.3, 11, 4), SM(5, 48, 32, 9.0)),
    "memory_wide": SL(SA(2, 1, 16, 16, 0.3, 11, 4), SM(2, 256, 200, 12.0)),
    "mixture": SL(SA(3, 1, 10, 6, 0.3, 11, 4), moe=(6, 2, 14)),
    "mixture_aligned": SL(SA(3, 1, 10, 6, 0.3, 11, 4), moe=(6, 3, 64)),
    "mixture_top1": SL(SA(3, 1, 10, 6, 0.3, 11, 4), moe=(5, 1, 12)),
    "side": SL(SA(3, 1, 10, 6, 0.3, 11, 4)),
    "side_aligned": SL(SA(3, 1, 10, 6, 0.3, 11, 4)),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", list(ALONE))
def test_each_mechanism_alone(made, which, dtype):
    """one layer in which only one sublayer (or one side of a pair) contributes -- the weights and biases behind the others are zero: what it adds to the embedding against
    that mechanism's own plain function, in one portion, in portions and token by token"""
    layer, eps, aligned = ALONE[which], 1e-5, which.endswith(("mfma", "aligned", "chunked", "wide"))
    side = (64 if aligned else 9) if which.startswith("side") else None
    cfg = SC(64 if aligned else 40, 32, [layer], side=side, eps=eps)
    t = synth.seq_tensors(cfg, 3)
    zero = {"mixture": ["l0.norm1", "l0.norm1.b"], "side": ["l0.norm1", "l0.norm1.b"], "left": ["l0.mix.right.out"], "memory": ["l0.mix.left.out"]}.get(which.split("_")[0], [])
    for n in zero:
        t[n] = np.zeros_like(t[n])
    m, _, _ = made("alone_" + which, dtype, max_batch=200, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 150, seed=3)
    W = {k: np.asarray(v, np.float64) for k, v in t.items()}
    x0 = W["embed"][toks]
    mc = layer["mixer"]
    if layer["mlp"]:
        want = seq_oracle.biased_layer_norm(seq_oracle.chosen_softmax_experts(W, "l0.mlp.", x0, layer["mlp"]), W["l0.norm2"], W["l0.norm2.b"], eps)
    elif side:
        want = seq_oracle.token_side_input(W, "l0.side.", x0, toks, 0, side, eps)
    else:
        if layer["type"] == "attention":
            y = seq_oracle.normed_window_attention(W, "l0.mix.", x0, mc, eps)
        elif which.startswith("left"):
            y = 0.5 * seq_oracle.plain_norm(seq_oracle.normed_window_attention(W, "l0.mix.left.", x0, mc["left"], eps), W["l0.mix.left.out"], eps)
        else:
            y = 0.5 * seq_oracle.plain_norm(seq_oracle.matrix_memory_mixer(W, "l0.mix.right.", x0, mc["right"], eps), W["l0.mix.right.out"], eps)
        want = seq_oracle.biased_layer_norm(y, W["l0.norm1"], W["l0.norm1.b"], eps)
    for sizes in ([150], [1], [70, 3, 2, 33, 1]):
        got = layer_adds(m, toks, sizes) - x0
        bad = np.abs(got - want).max(axis=1) / np.abs(want).max()
        if dtype == "float32":
            assert bad.max() < 2e-4, sizes
        else:  # (the norm behind the sublayer stretches rows whose output is small; a router's close call may flip)
            assert np.quantile(bad, 0.9) < 6e-2, sizes


WRONG = [{"use_mean": False}, {"use_norm_bias": False}, {"use_side": False}, {"side_kw": {"use_gate": False}},
         {"attn_kw": {"use_bias": False}}, {"attn_kw": {"use_norm": False}}, {"attn_kw": {"per_head": True}}, {"attn_kw": {"use_rotation": False}}, {"attn_kw": {"use_scaling": False}},
         {"attn_kw": {"use_gate": False}}, {"attn_kw": {"size": 30}}, {"pair_kw": {"use_out_norms": False}}, {"pair_kw": {"use_left": False}}, {"pair_kw": {"use_right": False}},
         {"pair_kw": {"left_kw": {"use_bias": False}}}, {"pair_kw": {"left_kw": {"size": 30}}}, {"pair_kw": {"left_kw": {"per_head": True}}}, {"pair_kw": {"left_kw": {"use_rotation": False}}},
         {"pair_kw": {"right_kw": {"use_cap": False}}}, {"pair_kw": {"right_kw": {"use_norm": False}}}, {"pair_kw": {"right_kw": {"use_gate": False}}}, {"pair_kw": {"right_kw": {"carry": False}}},
         {"moe_kw": {"use_bias": False}}, {"moe_kw": {"equal": True}}, {"moe_kw": {"on_input": True}}]


def test_what_the_plain_statement_is_sensitive_to(made):
    """every mechanism of the design left out of the plain statement in turn moves its logits far from the right ones; the library agrees with the right ones"""
    m, cfg, t = made("odd", "float32", max_batch=32)
    toks = tokens_for(cfg, 30, seed=8)
    want = seq_oracle.run_sogavik(cfg, t, toks)
    for kw in WRONG:
        assert err(seq_oracle.run_sogavik(cfg, t, toks, **kw), want) > 5e-3, kw
    shifted = dict(t, **{"side.embed": np.roll(t["side.embed"], cfg["token_side"]["dim"], axis=1)})  # every layer reads its neighbour's stretch
    assert err(seq_oracle.run_sogavik(cfg, shifted, toks), want) > 5e-2
    assert err(run_portions(m, toks, [30]), want) < TOL["float32"]
    assert err(run_portions(m, toks, [1]), want) < TOL["float32"]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_against_the_plain_statement(made, name, dtype):
    m, cfg, t = made(name, dtype, max_batch=64)
    toks = tokens_for(cfg, 90)
    want = seq_oracle.run_sogavik(cfg, t, toks)
    s = m.acquire()
    got = m.forward(s, toks, np.arange(len(toks)))
    m.release(s)
    assert close(got, want, dtype)


@pytest.mark.parametrize("name", ["odd", "aligned", "wide"])
def test_the_residual_stream_after_every_layer(made, name):
    m, cfg, t = made(name, "float32", max_batch=64)
    toks = tokens_for(cfg, 45, seed=5)
    per = []
    seq_oracle.run_sogavik(cfg, t, toks, per_layer=per)
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
    want = seq_oracle.run_sogavik(cfg, t, toks)
    for sizes in ([1], [2], [3, 1, 7, 2], [50, 2, 23], [16, 17, 15], [9, 8, 10]):  # (9 and 10 tokens: the smallest tiled mixtures, 8: the widest mat-vec)
        assert close(run_portions(m, toks, sizes), want, dtype), sizes


@pytest.mark.parametrize("name", ["aligned", "manyheads", "wide"])
def test_portions_around_the_chunks_of_the_memory(made, name):
    """portions just below, at and above whole chunks of the chunked recurrence (64 tokens), with scanned portions and single tokens between them"""
    m, cfg, t = made(name, "float32", max_batch=256)
    toks = tokens_for(cfg, 330, seed=12)
    want = seq_oracle.run_sogavik(cfg, t, toks)
    for sizes in ([330], [63, 65], [64, 1, 128, 2], [31, 32, 33, 129], [200, 7]):
        assert err(run_portions(m, toks, sizes), want) < TOL["float32"], sizes


def test_more_chunks_than_waves(made):
    """a portion of more chunks than the gates' block has waves"""
    cfg = SC(32, 40, [SL(SA(2, 1, 16, 8, 0.3, 9, 4), SM(3, 16, 12, 7.0))], side=None)
    m, _, t = made("long_portion", "float32", max_batch=1200, cfg=cfg, max_context=1300)
    toks = tokens_for(cfg, 1190, seed=3)
    want = seq_oracle.run_sogavik(cfg, t, toks)
    for sizes in ([1190], [1100, 90]):
        assert err(run_portions(m, toks, sizes), want) < TOL["float32"], sizes


def test_first_tokens_of_a_sequence(made):
    """the first token sees itself alone and a memory of nothing"""
    m, cfg, t = made("aligned", "float32")
    for n in (1, 2, 3, 5):
        toks = tokens_for(cfg, n, seed=10 + n)
        want = seq_oracle.run_sogavik(cfg, t, toks)
        assert err(run_portions(m, toks, [n]), want) < TOL["float32"]
        assert err(run_portions(m, toks, [1]), want) < TOL["float32"]


def test_interleaved_requests_and_reused_slots(made):
    """requests of unequal length fed in turns through the scheduler against each alone; then every slot is used again and must start from nothing (no memory, no running
    maximum, no keys of the request before)"""
    m, cfg, t = made("aligned", "float32", max_batch=16)
    seqs = [tokens_for(cfg, n, seed=20 + n) for n in (61, 9, 88)]
    want = [seq_oracle.run_sogavik(cfg, t, s) for s in seqs]
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
    for n in t:
        if n.split(".", 1)[-1] in ("norm1", "norm1.b", "norm2", "norm2.b", "side.norm") and n[0] == "l":
            t[n] = np.where(np.arange(W) < 2, 0.0, t[n]).astype(np.float32)


def mark_attention(t, p, mc, W, rng):
    """Every key reads feature 0 into the last (never rotated) channel of its head and every query reads feature 1 into that channel: normed over the whole projection, a query's
    score for a mark is about dim x scale, for anything else 0 up to the queries' small other numbers.  Every value channel reads feature 0."""
    H, G, d, dv, c = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"], mc["dim"] - 1
    assert mc["rot"]["dims"] < d
    q = rng.standard_normal((H * d, W)).astype(np.float32) * 0.02
    q[:, :2] = 0.0
    q[c::d, 1] = 2.0
    k = rng.standard_normal((G * d, W)).astype(np.float32) * 0.05
    k[:, :2], k[c::d] = 0.0, 0.0
    k[c::d, 0] = 2.0
    v = rng.standard_normal((G * dv, W)).astype(np.float32) * 0.2
    v[:, 0] = 1.5
    t[p + "q"], t[p + "k"], t[p + "v"] = q, k, v
    t[p + "q.b"], t[p + "k.b"] = np.zeros(H * d, np.float32), np.zeros(G * d, np.float32)
    t[p + "q.norm"], t[p + "k.norm"] = np.ones(H * d, np.float32), np.ones(G * d, np.float32)


WINDOWS = (24, 37)


def marked_model(aligned, seed=0):
    """an attention layer and a pair whose left side has a wider window"""
    rng = np.random.default_rng(seed)
    W = 64 if aligned else 30
    H, G, d, dv, memory = (4, 2, 16, 8, SM(2, 16, 16, 8.0)) if aligned else (3, 1, 10, 6, SM(2, 7, 5, 8.0))
    cfg = SC(W, 24, [SL(SA(H, G, d, dv, 1.2, WINDOWS[0], d - 4)), SL(SA(2 * H, G, d, dv, 1.2, WINDOWS[1], 4), memory)], side=None, eps=1e-5)
    t = synth.seq_tensors(cfg, seed)
    mark_embedding(t, cfg, rng)
    mark_attention(t, "l0.mix.", cfg["layers"][0]["mixer"], W, rng)
    mark_attention(t, "l1.mix.left.", cfg["layers"][1]["mixer"]["left"], W, rng)
    return cfg, bf16(t)


@pytest.mark.parametrize("aligned", [False, True])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_window_edges_in_prompts_and_in_decoding(made, dtype, aligned):
    """One mark in the sequence: the statement whose window is one off (either layer) is far off on the row that its edge moves and agrees right up to there; the library agrees
    with the right one, in portions cut anywhere (the edge across portion and tile borders) and token by token."""
    cfg, t = marked_model(aligned)
    m, _, _ = made("marked%d" % aligned, dtype, max_batch=64, cfg=cfg, tensors=t)
    tol = 1e-3 if dtype == "float32" else TOL[dtype]
    s0, s1 = WINDOWS
    for mark in (0, 1, 15, 16, 50):
        toks = tokens_for(cfg, 130, seed=30 + mark, lo=1)
        toks[mark] = 0
        want = seq_oracle.run_sogavik(cfg, t, toks)
        for kw, row in (({"attn_kw": {"size": s0 + 1}}, mark + s0), ({"attn_kw": {"size": s0 - 1}}, mark + s0 - 1),
                        ({"pair_kw": {"left_kw": {"size": s1 + 1}}}, mark + s1), ({"pair_kw": {"left_kw": {"size": s1 - 1}}}, mark + s1 - 1)):
            r = rows(seq_oracle.run_sogavik(cfg, t, toks, **kw), want, range(len(toks)))
            assert r[row] > 0.15 and max(r[mark:row], default=0.0) < 0.05, (mark, kw, r[row])
        for sizes in ([130], [1], [3, 2, 5], [61, 2, 1, 30]):
            assert max(rows(run_portions(m, toks, sizes), want, range(len(toks)))) < tol, (mark, sizes)


@pytest.mark.parametrize("aligned", [False, True])
def test_rotation_far_from_the_start(made, aligned):
    """a layer whose rotated numbers carry the scores, 400 tokens: the statement without rotation, without the scaling of the frequencies, or with neighbours in the place of
    halves, is off"""
    sa = SA(4, 2, 32, 8, 0.4, 200, 32, 10000.0, (2.5, 256, 24.0, 1.5)) if aligned else SA(3, 1, 10, 7, 0.6, 150, 10, 200.0, YARN)
    cfg = SC(64 if aligned else 40, 32, [SL(sa)], side=None, eps=1e-5)
    t = bf16(synth.seq_tensors(cfg, 5))
    m, _, _ = made("rot%d" % aligned, "float32", max_batch=64, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 400, seed=4)
    want = seq_oracle.run_sogavik(cfg, t, toks)
    H, G, d, dims = sa["heads"], sa["kv_heads"], sa["dim"], sa["rot"]["dims"]
    assert err(seq_oracle.run_sogavik(cfg, t, toks, attn_kw={"use_rotation": False}), want) > 0.05
    assert err(seq_oracle.run_sogavik(cfg, t, toks, attn_kw={"use_scaling": False}), want) > 0.05
    order = np.r_[np.arange(0, dims, 2), np.arange(1, dims, 2), np.arange(dims, d)]  # the same weights read as if pair i were (2 i, 2 i + 1)
    other = dict(t)
    for n, heads in (("q", H), ("k", G)):
        at = (np.arange(heads)[:, None] * d + order).reshape(-1)
        for suffix in ("", ".b", ".norm"):
            other["l0.mix." + n + suffix] = t["l0.mix." + n + suffix][at]
    assert err(seq_oracle.run_sogavik(cfg, other, toks), want) > 0.05
    for sizes in ([64], [1], [61, 2, 100, 1, 1]):
        assert max(rows(run_portions(m, toks, sizes), want, range(len(toks)))) < 1e-3, sizes


def memory_alone(mc, W, seed, **made_up):
    """a pair of which only the memory contributes, tensors of the right side replaced by `made_up`"""
    cfg = SC(W, 24, [SL(SA(2, 1, 16, 8, 0.3, 9, 4), mc)], side=None, eps=1e-5)
    t = synth.seq_tensors(cfg, seed)
    t["l0.mix.left.out"] = np.zeros_like(t["l0.mix.left.out"])
    t.update({"l0.mix.right." + k.replace("_b", ".b"): np.asarray(v, np.float32) for k, v in made_up.items()})
    return cfg, bf16(t)


@pytest.mark.parametrize("which", ["scan", "chunked", "wide"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_memory_is_carried_for_hundreds_of_tokens(made, dtype, which):
    """forget gates of a few parts in a thousand: the statement that loses its memory once, at a portion's or a chunk's edge, is far off on hundreds of rows behind it"""
    mc = {"scan": SM(3, 10, 14, 9.0), "chunked": SM(4, 32, 48, 12.0), "wide": SM(2, 64, 132, 12.0)}[which]
    cfg, t = memory_alone(mc, 64, 6, f=np.zeros((mc["heads"], 64)), f_b=np.linspace(5.5, 7.0, mc["heads"]), i_b=np.zeros(mc["heads"]))
    m, _, _ = made("slow_" + which, dtype, max_batch=128, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 420, seed=9)
    want = seq_oracle.run_sogavik(cfg, t, toks)
    for at in (64, 128, 200):
        r = rows(seq_oracle.run_sogavik(cfg, t, toks, pair_kw={"right_kw": {"lose_at": at}}), want, range(len(toks)))
        assert max(r[:at]) < 1e-9 and np.median(r[at:at + 200]) > 0.1, at
    for sizes in ([420], [64], [1], [200, 1, 1, 2, 70]):
        assert max(rows(run_portions(m, toks, sizes), want, range(len(toks)))) < (1e-3 if dtype == "float32" else 2 * TOL[dtype]), sizes


@pytest.mark.parametrize("which", ["scan", "chunked"])
def test_one_written_token_far_back(made, which):
    """the mark opens the input gate by e^9, everything else writes e^-3: hundreds of tokens later the memory still answers with the mark's value, and the running maximum that it
    set is the one every later token's weights are relative to"""
    mc = SM(3, 10, 14, 12.0) if which == "scan" else SM(3, 32, 16, 12.0)
    H, d, dv, W = mc["heads"], mc["dim"], mc["vdim"], 64
    i = np.zeros((H, W))
    i[:, 0] = 2.0
    cfg, t = memory_alone(mc, W, 3, f=np.zeros((H, W)), f_b=np.full(H, 9.0), i=i, i_b=np.full(H, -3.0))
    rng = np.random.default_rng(1)
    mark_embedding(t, cfg, rng)
    t = bf16(t)
    m, _, _ = made("written_" + which, "float32", max_batch=128, cfg=cfg, tensors=t)
    for mark in (0, 1, 63, 64, 100):
        toks = tokens_for(cfg, 400, seed=40 + mark, lo=1)
        toks[mark] = 0
        want = seq_oracle.run_sogavik(cfg, t, toks)
        r = rows(seq_oracle.run_sogavik(cfg, t, toks, pair_kw={"right_kw": {"lose_at": mark + 1}}), want, range(len(toks)))
        assert max(r[:mark + 1]) < 1e-9 and np.median(r[mark + 200:]) > 0.1, mark
        for sizes in ([400], [1], [64], [mark + 1, 2, 130]):
            assert max(rows(run_portions(m, toks, sizes), want, range(len(toks)))) < 1e-3, (mark, sizes)


def test_gates_at_both_ends_side_by_side(made):
    """log input gates from -29 to 29 and forget gates from one part in e^29 to all of it, head by head and moving: nothing overflows or vanishes, and the chunked memory agrees
    with the scan; where little was written the floor of the denominator decides"""
    mc = SM(8, 32, 32, 30.0)
    cfg, t = memory_alone(mc, 64, 7, i_b=np.linspace(-40.0, 60.0, 8), f_b=np.linspace(9.0, -40.0, 8)[[0, 7, 1, 6, 2, 5, 3, 4]])
    t["l0.mix.right.i"], t["l0.mix.right.f"] = t["l0.mix.right.i"] * 4.0, t["l0.mix.right.f"] * 4.0
    m, _, _ = made("gates", "float32", max_batch=256, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 256, seed=11)
    want = seq_oracle.run_sogavik(cfg, t, toks)
    assert np.isfinite(want).all()
    for sizes in ([256], [1], [100, 3]):
        assert err(run_portions(m, toks, sizes), want) < TOL["float32"], sizes
    cfg, t = memory_alone(SM(4, 16, 16, 30.0), 64, 8, i_b=np.full(4, -6.0))
    m, _, _ = made("floor", "float32", max_batch=64, cfg=cfg, tensors=t)
    want = seq_oracle.run_sogavik(cfg, t, toks[:100])
    assert err(seq_oracle.run_sogavik(cfg, t, toks[:100], pair_kw={"right_kw": {"use_floor": False}}), want) > 0.02
    for sizes in ([64], [1], [40, 2]):
        assert err(run_portions(m, toks[:100], sizes), want) < TOL["float32"], sizes


@pytest.mark.parametrize("side", [5, 64])
def test_the_tokens_own_input_decides(made, side):
    """a model whose layers' token inputs outweigh the rest: portions of every size, single tokens and the captured greedy step all read the present token's row at their own
    layer's place"""
    cfg = SC(64, 30, [SL(SA(2, 1, 8, 8, 0.3, 6, 4)), SL(SA(2, 2, 8, 8, 0.3, 6, 8), SM(2, 16, 8, 5.0)), SL(SA(1, 1, 8, 8, 0.3, 6, 2), moe=(3, 2, 16))], side=side, eps=1e-5)
    t = synth.seq_tensors(cfg, 8)
    for i in range(3):
        t[f"l{i}.side.norm"] = t[f"l{i}.side.norm"] * 6.0
    t = bf16(t)
    m, _, _ = made("side%d" % side, "float32", max_batch=16, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 40, seed=2)
    want = seq_oracle.run_sogavik(cfg, t, toks)
    shifted = dict(t, **{"side.embed": np.roll(t["side.embed"], side, axis=1)})
    assert min(rows(seq_oracle.run_sogavik(cfg, shifted, toks), want, range(40))) > 0.1
    for sizes in ([40], [1], [2], [8, 1, 5]):
        assert err(run_portions(m, toks, sizes), want) < TOL["float32"], sizes
    ids = m.generate(toks[:7], 12)
    full = np.concatenate([toks[:7], ids])
    want = seq_oracle.run_sogavik(cfg, t, full[:-1])
    assert all(want[6 + i].max() - want[6 + i][tok] < 1e-4 * (want.max() - want.min()) for i, tok in enumerate(ids))


def test_logits_far_apart_at_the_router(made):
    """router logits hundreds apart: the choice is among logits (their soft-max over all experts would be 0 for every one but the first), the weights those of the chosen ones"""
    cfg = SC(40, 30, [SL(SA(2, 1, 8, 8, 0.3, 6, 4), moe=(6, 3, 16))], side=None, eps=1e-5)
    t = synth.seq_tensors(cfg, 2)
    t["l0.mlp.router"] = t["l0.mlp.router"] * 0.5
    t["l0.mlp.router.b"] = np.float32([0.0, -150.0, -300.0, -450.0, -600.0, 150.0])
    t = bf16(t)
    m, _, _ = made("router", "float32", max_batch=32, cfg=cfg, tensors=t)
    toks = tokens_for(cfg, 40, seed=2)
    want = seq_oracle.run_sogavik(cfg, t, toks)
    for sizes in ([40], [1], [9]):
        assert err(run_portions(m, toks, sizes), want) < TOL["float32"], sizes


def test_long_decoding_keeps_the_caches(made):
    m, cfg, t = made("aligned", "float32", max_batch=16)
    toks = tokens_for(cfg, 260, seed=6)
    want = seq_oracle.run_sogavik(cfg, t, toks)
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
    want = seq_oracle.run_sogavik(cfg, t, full[:-1])
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
    """mode bit 1 keeps the per-key attention, the token-by-token scan and the 64 x 64 mat-mul (also for the experts' grouped products): the faster forms of a portion and of a
    single token must give the same logits (fp32: up to the order of sums)"""
    m, cfg, t = made(name, dtype, max_batch=128)
    toks = tokens_for(cfg, 250, seed=9)
    cuts = ([128], [1], [70, 1, 1, 1, 9])
    fast = [run_portions(m, toks, sizes) for sizes in cuts]
    m.set_mode(2)
    plain = [run_portions(m, toks, sizes) for sizes in cuts]
    m.set_mode(0)
    want = seq_oracle.run_sogavik(cfg, t, toks)
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


def test_a_window_wider_than_the_context_fills_it_and_no_more(ctx, tmp_path):
    cfg = SC(40, 50, [SL(SA(3, 1, 10, 6, 0.3, 500, 4)), SL(SA(2, 1, 16, 6, 0.3, 21, 4), SM(2, 7, 5, 5.0))], side=3, eps=1e-5)
    t = synth.write_seq_model_dir(str(tmp_path), cfg, 0)
    m = seqmodel.load_model(ctx, str(tmp_path), dtype="float32", max_batch=8, n_slots=1, max_context=20)
    toks = tokens_for(cfg, 20)
    s = m.acquire()
    got = [m.forward(s, toks[:18], np.arange(18))]
    with pytest.raises(hip.PSHipError):
        m.forward(s, [1, 2, 3])
    got.append(m.forward(s, toks[18:], [0, 1]))
    m.release(s)
    assert err(np.concatenate(got), seq_oracle.run_sogavik(cfg, t, toks)) < TOL["float32"]
    m.close()
