"""Whole stacks of attention / linear-attention layers on the GPU against the plain statement: whole prompts, portions of any
size, token by token, recorded decoding, loops, slots used again, generation through the scheduler, command line and trace."""
import io
import json

import numpy as np
import pytest

import mixer_models as M
from oracle import mixer_stack as O

pytestmark = pytest.mark.gpu

# error of the logits (mean taken off, rms) over their spread
F32_TOL, BF16_TOL = 2e-5, 4e-2


@pytest.fixture(scope="module")
def ai(pkg):
    import local_ai_amd
    return local_ai_amd


CONFIGS = {
    "both": lambda: M.config(97, 48, [M.attention(4, 2, 12, 20, mlp=M.dense(56)), M.lightning(3, 16, 24, mlp=M.moe(5, 2, 40)),
                                      M.attention(2, 2, 24, 16, mlp=M.moe(6, 3, 24)), M.lightning(2, 40, 12)], {"start": 1, "stop": 3, "times": 2}),
    "loop_all": lambda: M.config(61, 64, [M.lightning(2, 8, 16, [0.9, 1.0], mlp=M.dense(32)), M.attention(3, 1, 32, 40, diff=0.5)],
                                 {"start": 0, "stop": 2, "times": 3}, eps=1e-3),
    "ragged": lambda: M.config(51, 30, [M.attention(3, 3, 5, 7, scale=0.6, mlp=M.moe(4, 1, 19)), M.lightning(1, 9, 11, mlp=M.dense(13))]),
    "attention_only": lambda: M.config(200, 128, [M.attention(8, 2, 64, 128, mlp=M.dense(96)), M.attention(2, 1, 128, 64, mlp=None)]),
    "lightning_only": lambda: M.config(77, 72, [M.lightning(4, 72, 136, mlp=M.moe(3, 3, 48)), M.lightning(5, 33, 40, mlp=M.dense(200))],
                                       {"start": 1, "stop": 2, "times": 1}),
    # norms behind the branches
    "latent_and_states": lambda: M.vifivik(90, 80, [M.latent(5, 24, 8, 40, 48, ff=72), M.retention(3, 40, 24, ff=56), M.latent(5, 24, 8, 40, 48, kv_from=0, ff=40),
                                                    M.mamba2(6, 24, 20, 2, 4, 2, ff=64), M.latent(6, 16, 12, 24, 96)]),
    "latent_shared": lambda: M.vifivik(64, 96, [M.mamba2(2, 48, 32, 1, 3, 1), M.latent(8, 32, 32, 64, 160, base=500.0, ff=48),
                                                M.latent(3, 56, 32, 24, 160, base=500.0, kv_from=1, scale=0.3), M.latent(4, 16, 32, 16, 160, base=500.0, kv_from=1, ff=32)],
                                       eps=1e-3, cap=5.0),
    # (enough values per branch that none of them happens to vanish, where the norm behind it would amplify rounding)
    "latent_ragged": lambda: M.vifivik(51, 30, [M.latent(3, 5, 6, 7, 11, ff=13), M.retention(3, 9, 11), M.mamba2(3, 7, 5, 3, 2, 1, ff=9), M.latent(5, 1, 2, 9, 13)]),
    "latent_wide": lambda: M.vifivik(72, 128, [M.latent(3, 128, 64, 128, 512, ff=96), M.latent(16, 72, 20, 136, 264), M.latent(1, 200, 40, 48, 64)]),
    "latent_beyond_the_tiles": lambda: M.vifivik(40, 64, [M.latent(2, 40, 72, 24, 96), M.latent(2, 264, 16, 300, 640, ff=24)]),
    "states_only": lambda: M.vifivik(77, 72, [M.mamba2(6, 20, 130, 3, 5, 2, ff=40), M.mamba2(2, 64, 300, 1, 1, 2), M.retention(2, 128, 64, [1.0, 0.25], ff=64),
                                              M.mamba2(8, 128, 64, 8, 4, 8), M.retention(4, 33, 72)]),
    "wide_heads": lambda: M.config(40, 64, [M.attention(2, 1, 160, 320), M.lightning(2, 288, 24)]),
}


def build(ai, gpu, name, dtype="float32", max_tokens=512, **options):
    ctx, K = gpu
    cfg = CONFIGS[name]()
    t = M.weights(cfg, seed=sum(map(ord, name)))
    m = ai.stack_pipeline.StackPipeline(ctx, K, ai.registry.read_config(cfg), M.Tensors(t), max_tokens,
                                        ai.F32 if dtype == "float32" else ai.BF16, **options)
    return cfg, M.plain_weights(t), m


def check(got, want, dtype, what):
    d = got - want
    d = d - d.mean(1, keepdims=True)
    e = np.sqrt((d ** 2).mean(1)) / want.std()
    tol = F32_TOL if dtype == "float32" else BF16_TOL
    assert np.isfinite(got).all() and e.max() <= tol, f"{what}: {e.max():.3g} at {int(e.argmax())} of {len(e)}"


def feed(m, tokens, cuts):
    """Logits of every token, the tokens cut into portions."""
    s, out, at = m.new_sequence(), [], 0
    for c in cuts:
        out.append(m.step(s, tokens[at:at + c], list(range(c))))
        at += c
    assert at == len(tokens) and s.position == at
    m.end_sequence(s)
    return np.concatenate(out)


def cuts_of(n, pattern):
    out, i = [], 0
    while sum(out) < n:
        out.append(min(pattern[i % len(pattern)], n - sum(out)))
        i += 1
    return out


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_portions_and_decoding_agree_with_the_plain_statement(ai, gpu, name, dtype):
    cfg, w, m = build(ai, gpu, name, dtype, max_rows=160)          # the longest prompt takes two passes
    tokens = [int(t) for t in np.random.default_rng(5).integers(0, cfg["vocab"], 201)]
    want = O.forward(cfg, w, tokens)
    for what, cuts in (("whole", [201]), ("token by token", [1] * 201), ("portions", cuts_of(201, [37, 2, 64, 3, 17, 33])), ("twos", cuts_of(201, [2])),
                       ("prompt, then decoding", [101] + [1] * 100), ("a long portion after decoding", [1] * 5 + [170, 1, 1, 24])):
        print(f"{name} {dtype} {what}", flush=True)
        check(feed(m, tokens, cuts), want, dtype, f"{name} {what}")


@pytest.mark.parametrize("name", ["both", "loop_all", "latent_and_states", "latent_shared"])
def test_residual_stream_after_every_layer_run(ai, gpu, name):
    cfg, w, m = build(ai, gpu, name)
    tokens = [int(t) for t in np.random.default_rng(6).integers(0, cfg["vocab"], 23)]
    want = []
    O.forward(cfg, w, tokens, residuals=want)
    for cuts in ([23], [1] * 23, [2, 17, 4]):
        got = [[] for _ in m.runs]

        def observe(i, x, rows):
            m.ctx.synchronize()
            got[i].append(x.as_array(np.float32, rows * cfg["width"]).reshape(rows, -1))
        m.observe = observe
        feed_s, at = m.new_sequence(), 0
        for c in cuts:
            m.step(feed_s, tokens[at:at + c])
            at += c
        m.end_sequence(feed_s)
        for i, (a, b) in enumerate(zip(got, want)):
            assert np.abs(np.concatenate(a) - b).max() <= 3e-5 * np.abs(b).max(), f"{cuts} run {i}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_token_decides_through_the_caches(ai, gpu, dtype):
    """One layer whose scores single out the one key that matches the query's token, hundreds of positions back and at block
    edges: the head's output is the value of that position, in a prompt, in portions and decoded."""
    ctx, K = gpu
    V, W = 40, 96
    cfg = M.config(V, W, [M.attention(1, 1, 32, 32, scale=1.0, diff=0.0)])
    t = {n: np.zeros_like(x) for n, x in M.weights(cfg, 3).items()}
    g = np.random.default_rng(8)
    keys, vals = np.linalg.qr(g.standard_normal((32, 32)))[0], g.standard_normal((32, 16))
    vals *= 3.0 / np.linalg.norm(vals, axis=1, keepdims=True)
    e = np.zeros((V, W))
    e[:32, :32], e[:32, 32:48] = keys, vals
    e[32:, 64:] = keys[:8]                            # token 32 + i asks for the key of token i; it has none itself
    t["embed"] = M.bf16_bits(e)
    for n in ("l0.norm1", "final.norm"):
        t[n] = M.bf16_bits(np.ones(W))
    q, k = np.zeros((64, W)), np.zeros((64, W))
    q[:32, 64:], k[:32, :32] = np.eye(32) * 4, np.eye(32) * 4
    t["l0.mix.q"], t["l0.mix.k"] = M.bf16_bits(q), M.bf16_bits(k)
    v = np.zeros((32, W))
    v[:16, 32:48] = np.eye(16)
    t["l0.mix.v"] = M.bf16_bits(v)
    t["l0.mix.lq2"] = M.bf16_bits(np.ones(32))
    t["l0.mix.lk2"] = M.bf16_bits(-np.full(32, 5.0 / 32))
    t["l0.mix.lq1"], t["l0.mix.lk1"] = t["l0.mix.lq2"], t["l0.mix.lk2"]      # lambda = exp(-5) - exp(-5): the first map alone
    o = np.zeros((W, 32))
    o[48:64, :16] = np.eye(16) * 3
    t["l0.mix.o"] = M.bf16_bits(o)
    head = np.zeros((V, W))
    head[:32, 48:64] = vals
    t["head"] = M.bf16_bits(head)
    m = ai.stack_pipeline.StackPipeline(ctx, K, ai.registry.read_config(cfg), M.Tensors(t), 1024, ai.F32 if dtype == "float32" else ai.BF16)
    w = M.plain_weights(t)
    places = [0, 1, 31, 32, 33, 63, 64, 500]
    tokens = [9] * 900
    for i, p in enumerate(places):
        tokens[p] = i
    tokens += [32 + i for i in range(8)]
    want = O.forward(cfg, w, tokens)
    assert [int(r[:32].argmax()) for r in want[900:]] == list(range(8)) and np.abs(want[900:]).max() > 1
    for cuts in ([908], [900] + [1] * 8, cuts_of(908, [64, 37, 2])):
        s, at, got = m.new_sequence(), 0, []
        for c in cuts:
            wanted = [i for i in range(c) if at + i >= 900]
            got.append(m.step(s, tokens[at:at + c], wanted))
            at += c
        m.end_sequence(s)
        got = np.concatenate(got)
        assert [int(r[:32].argmax()) for r in got] == list(range(8)), cuts[:3]
        check(got, want[900:], dtype, f"far token {cuts[:3]}")


@pytest.mark.parametrize("sink", [None, 25.0])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_token_decides_through_the_latent_cache(ai, gpu, dtype, sink):
    """As above through latents, in a layer of its own and in one that reads its cache.  With a large sink, which takes nearly all
    of every softmax, the favourite's share stays in the right proportion to it."""
    ctx, K = gpu
    V, W, R = 40, 160, 64
    layers = [M.latent(1, 32, 2, 32, R, scale=1.0), M.latent(1, 32, 2, 32, R, scale=1.0, kv_from=0)]
    cfg = M.vifivik(V, W, layers, cap=30.0)
    t = {n: np.zeros_like(x) for n, x in M.weights(cfg, 3).items()}
    g = np.random.default_rng(8)
    keys = np.linalg.qr(g.standard_normal((32, 32)))[0]
    e = np.zeros((V, W))
    e[:32, :32] = keys * 6                            # the latent's first half; the second half is the value
    e[:32, 32:64] = np.eye(32) * 6
    e[32:, 64:96] = keys[:8] * 6                      # token 32 + i asks for the key of token i
    t["embed"] = M.bf16_bits(e)
    for n in ("l0.norm1", "l1.norm1"):
        t[n] = M.bf16_bits(np.full(W, 0.5))
    t["final.norm"] = M.bf16_bits(np.ones(W))
    for i in range(2):
        p = f"l{i}.mix."
        q = np.zeros((34, W))
        q[:32, 64:96] = np.eye(32)
        t[p + "q"] = M.bf16_bits(q)
        uk, uv = np.zeros((32, R)), np.zeros((32, R))
        uk[:, :32], uv[:, 32:] = np.eye(32), np.eye(32)
        t[p + "uk"], t[p + "uv"] = M.bf16_bits(uk), M.bf16_bits(uv)
        t[p + "sink"] = M.bf16_bits(np.array([-20.0 if sink is None else sink]))
        o = np.zeros((W, 32))
        o[96 + 32 * i:128 + 32 * i] = np.eye(32)
        t[p + "o"] = M.bf16_bits(o)
    dkv = np.zeros((R + 2, W))
    dkv[:R, :R] = np.eye(R)
    t["l0.mix.dkv"], t["l0.mix.dkv.norm"] = M.bf16_bits(dkv), M.bf16_bits(np.ones(R))
    head = np.zeros((V, W))
    head[:32, 96:128], head[:32, 128:160] = np.eye(32) * 3, np.eye(32) * 3
    t["head"] = M.bf16_bits(head)
    m = ai.stack_pipeline.StackPipeline(ctx, K, ai.registry.read_config(cfg), M.Tensors(t), 1024, ai.F32 if dtype == "float32" else ai.BF16)
    w = M.plain_weights(t)
    places = [0, 1, 31, 32, 33, 63, 64, 500]
    tokens = [9] * 900
    for i, p in enumerate(places):
        tokens[p] = i
    tokens += [32 + i for i in range(8)]
    want = O.forward(cfg, w, tokens)
    assert [int(r[:32].argmax()) for r in want[900:]] == list(range(8)) and np.abs(want[900:]).max() > 1
    for cuts in ([908], [900] + [1] * 8, [898, 2] + [3, 5], cuts_of(908, [64, 37, 2, 66])):
        s, at, got = m.new_sequence(), 0, []
        for c in cuts:
            wanted = [i for i in range(c) if at + i >= 900]
            got.append(m.step(s, tokens[at:at + c], wanted))
            at += c
        m.end_sequence(s)
        got = np.concatenate([x for x in got if len(x)])
        assert [int(r[:32].argmax()) for r in got] == list(range(8)), cuts[:3]
        check(got, want[900:], dtype, f"far token {cuts[:3]}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_first_tokens_reach_the_last_through_the_states(ai, gpu, dtype):
    """State layers alone, with decays near one: exchanging the very first token moves the last logits, by the plain statement's
    amount, whether the tokens between were a prompt, portions or decoded."""
    ctx, K = gpu
    cfg = M.vifivik(30, 64, [M.retention(2, 32, 32, [1.0, 0.9999]), M.mamba2(2, 32, 32)])
    t = M.weights(cfg, 4)
    t["l1.mix.dt_bias"], t["l1.mix.A_log"] = M.bf16_bits(np.array([-4.0, -2.0])), M.bf16_bits(np.array([-6.0, -7.0]))
    m = ai.stack_pipeline.StackPipeline(ctx, K, ai.registry.read_config(cfg), M.Tensors(t), 400, ai.F32 if dtype == "float32" else ai.BF16)
    w, tokens = M.plain_weights(t), [int(x) for x in np.random.default_rng(3).integers(0, 30, 300)]
    other = [(tokens[0] + 1) % 30] + tokens[1:]
    a, b = O.forward(cfg, w, tokens), O.forward(cfg, w, other)
    assert np.abs(a[-1] - b[-1]).max() > 0.01 * a.std()
    for cuts in ([300], [1] * 300, cuts_of(300, [2, 65, 17])):
        check(feed(m, tokens, cuts), a, dtype, f"{cuts[:3]}")
        check(feed(m, other, cuts), b, dtype, f"{cuts[:3]}")


@pytest.mark.parametrize("name", ["both", "latent_and_states"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_slots_used_again_and_interleaved_sequences(ai, gpu, name, dtype):
    """A long sequence, then shorter ones in the same slot; three live sequences that take turns of unequal size."""
    cfg, w, m = build(ai, gpu, name, dtype, max_tokens=300, max_sequences=3)
    g = np.random.default_rng(9)
    seqs = [[int(t) for t in g.integers(0, cfg["vocab"], n)] for n in (290, 3, 77, 1, 150)]
    want = [O.forward(cfg, w, t) for t in seqs]
    for t, x in zip(seqs, want):
        check(feed(m, t, cuts_of(len(t), [100, 1, 1, 1])), x, dtype, f"{len(t)} tokens")
    live = {i: [m.new_sequence(), 0, []] for i in (0, 2, 4)}
    while live:
        for i in list(live):
            s, at, got = live[i]
            c = min(int(g.choice([1, 1, 2, 29])), len(seqs[i]) - at)
            got.append(m.step(s, seqs[i][at:at + c], list(range(c))))
            live[i][1] = at + c
            if at + c == len(seqs[i]):
                check(np.concatenate(got), want[i], dtype, f"interleaved {i}")
                m.end_sequence(s)
                del live[i]
    assert m.slots.available() == 3


@pytest.mark.parametrize("name,n,capacity", [("both", 120, 400), ("latent_and_states", 60, 63), ("latent_wide", 60, 63)])
def test_recorded_decoding_equals_unrecorded_bit_for_bit(ai, gpu, name, n, capacity):
    """The recorded step is replayed between other sequences' prompts, which also make the scratch buffers move.  (A recorded step
    splits a latent cache by its capacity, an unrecorded one by its position: so short a cache neither splits.)"""
    cfg, _, m = build(ai, gpu, name, "bfloat16", max_tokens=capacity, max_sequences=2)
    _, _, plain = build(ai, gpu, name, "bfloat16", max_tokens=capacity, max_sequences=2, graphs=False)
    g = np.random.default_rng(10)
    tokens = [int(t) for t in g.integers(0, cfg["vocab"], n)]

    def run(model, disturb):
        s, out = model.new_sequence(), []
        for i, t in enumerate(tokens):
            out.append(model.step(s, [t], [0])[0])
            if disturb and i in (1, 5, 6, 40):
                o = model.new_sequence()
                model.step(o, tokens[:10 * (i + 1) % n + 2], [0, 1])
                model.step(o, [3], [0])
                model.end_sequence(o)
        recorded = s.graph is not None
        model.end_sequence(s)
        return np.stack(out), recorded
    a, rec_a = run(m, True)
    b, rec_b = run(plain, False)
    assert rec_a and not rec_b and np.array_equal(a, b)


@pytest.mark.parametrize("name", ["loop_all", "latent_and_states"])
def test_long_decoding(ai, gpu, name):
    cfg, w, m = build(ai, gpu, name, max_tokens=700)
    tokens = [int(t) for t in np.random.default_rng(11).integers(0, cfg["vocab"], 640)]
    want = O.forward(cfg, w, tokens)
    check(feed(m, tokens, [1] * 640), want, "float32", "640 decoded tokens")


def test_wanted_places_order_and_bounds(ai, gpu):
    cfg, w, m = build(ai, gpu, "ragged", max_tokens=40)
    tokens = [int(t) for t in np.random.default_rng(12).integers(0, cfg["vocab"], 20)]
    want = O.forward(cfg, w, tokens)
    s = m.new_sequence()
    got = m.step(s, tokens[:12], [11, 0, 5, 5])
    check(got, want[[11, 0, 5, 5]], "float32", "order")
    assert m.step(s, tokens[12:15]).shape == (0, cfg["vocab"])
    check(m.step(s, tokens[15:], [4]), want[[19]], "float32", "after a step without wanted places")
    for bad in (([], []), ([1], [1]), ([cfg["vocab"]], []), ([1] * 21, [])):
        with pytest.raises(ai.InvalidArgument):
            m.step(s, *bad)
    assert s.position == 20
    m.end_sequence(s)


def greedy_of(cfg, w, prompt, n):
    mem, out = {}, []
    logits = O.forward(cfg, w, prompt, mem)[-1]
    for _ in range(n):
        out.append(int(logits.argmax()))
        logits = O.forward(cfg, w, [out[-1]], mem)[-1]
    return out


@pytest.mark.parametrize("name", ["both", "latent_and_states", "latent_shared"])
@pytest.mark.parametrize("portion", [5, 512])
def test_greedy_generation_through_the_scheduler(ai, gpu, name, portion):
    cfg, w, m = build(ai, gpu, name, max_tokens=120, max_sequences=2)
    g, gen = np.random.default_rng(13), ai.generation
    prompts = [[int(t) for t in g.integers(0, cfg["vocab"], n)] for n in (4, 33, 1, 70)]
    sch = gen.Scheduler(m, portion)
    reqs = [sch.submit(gen.Request(p, 20 + 5 * i)) for i, p in enumerate(prompts)]
    sch.run()
    for i, (r, p) in enumerate(zip(reqs, prompts)):
        assert r.tokens == greedy_of(cfg, w, p, 20 + 5 * i), i
    # sampling from the host with temperature 0 over the same logits, without the device's own choice
    r = sch.submit(gen.Request(prompts[1], 12, gen.Sampler(temperature=1e-6, top_k=1)))
    sch.run()
    assert r.tokens == reqs[1].tokens[:12]


@pytest.mark.parametrize("name", ["both", "latent_and_states"])
def test_command_line_and_trace_from_a_model_folder(ai, gpu, tmp_path, capsys, monkeypatch, name):
    from local_ai_amd import cli, trace
    cfg = CONFIGS[name]()
    t = M.weights(cfg, 21)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    ai.safetensors.write(str(tmp_path / "model.safetensors"), t)
    w = M.plain_weights(t)
    assert cli.main(["generate", "--model", str(tmp_path), "--dtype", "float32", "--prompt", "3,1,4", "--prompt", "7", "--max-new-tokens", "6"]) == 0
    lines = capsys.readouterr().out.split()
    assert [[int(x) for x in l.split(",")] for l in lines[-2:]] == [greedy_of(cfg, w, [3, 1, 4], 6), greedy_of(cfg, w, [7], 6)]
    toks = [int(x) for x in np.random.default_rng(1).integers(0, cfg["vocab"], 50)]
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:40], "want": [3, 39]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[40:], "want": [9]}], "end": ["x"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(map(json.dumps, steps))))
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"]) == 0
    assert capsys.readouterr().out.split("\n")[:2] == ["done 0", "done 1"]
    want = O.forward(cfg, w, toks)
    check(np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, -1), want[[3, 39]], "float32", "step 0")
    check(np.fromfile(tmp_path / "1.f32", "<f4").reshape(1, -1), want[[49]], "float32", "step 1")
    with pytest.raises(ai.gguf.InvalidFormat):
        cfg["width"] = 40
        (tmp_path / "config.json").write_text(json.dumps(cfg))
        ai.registry.load_model(str(tmp_path), 16)


def test_the_quantized_pipeline_serves_through_the_same_scheduler(ai, gpu):
    """A DecodePipeline behind the same calls: greedy tokens equal those of its own prefill and decode calls."""
    ctx, K = gpu
    P = ai.pipeline
    cfg = P.Gemma4QATConfig(vocab_size=640, hidden_size=512, num_hidden_layers=2, num_attention_heads=4, num_key_value_heads=1, head_dim=128,
                            global_head_dim=256, sliding_window=16, layer_types=["sliding_attention", "full_attention"])
    pipe = P.DecodePipeline.from_host(ctx, K, cfg, ai.synth.decode_model_tensors(cfg, ai.synth.rng(5), [512, 512]), 256, max_batch=16)
    prompt = [5, 17, 600, 3, 9, 44]
    got = ai.generation.generate(ai.generation.PipelineSequences(pipe), prompt, 5)
    pipe.reset()
    pipe.write_logits(pipe.prefill_prompt(prompt))
    pipe.position = len(prompt)
    want = [int(pipe.logits().argmax())]
    for _ in range(4):
        pipe.decode_step(want[-1])
        want.append(int(pipe.logits().argmax()))
    assert got == want
