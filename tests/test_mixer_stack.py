"""CPU checks of the stack of attention / linear-attention layers: the plain statement against closed forms, configuration
and registry, the weight file reader, the sampler and the scheduler."""
import json
import struct

import numpy as np
import pytest

import mixer_models as M
from oracle import mixer_stack as O


@pytest.fixture(scope="module")
def ai(pkg):
    import local_ai_amd
    return local_ai_amd


# ---- the plain statement ----------------------------------------------------------------------------------------------
def test_recurrence_is_the_decayed_sum_and_carries_its_state():
    g = np.random.default_rng(1)
    q, k, v = g.standard_normal((9, 2, 3)), g.standard_normal((9, 2, 3)), g.standard_normal((9, 2, 4))
    d = np.array([0.7, 1.0])
    o, s = O.lightning_recurrence(q, k, v, d)
    for t in range(9):
        for h in range(2):
            want = sum(d[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            assert np.allclose(o[t, h], want)
    o1, s1 = O.lightning_recurrence(q[:4], k[:4], v[:4], d)
    o2, s2 = O.lightning_recurrence(q[4:], k[4:], v[4:], d, s1)
    assert np.allclose(np.concatenate([o1, o2]), o) and np.allclose(s2, s)


def test_differential_mixer_reduces_to_one_map_and_sees_no_future():
    g = np.random.default_rng(2)
    w = {n: g.standard_normal(s) for n, s in (("q", (2 * 2 * 3, 5)), ("k", (2 * 3, 5)), ("v", (4, 5)), ("o", (5, 8)))}
    w.update({"q.b": g.standard_normal(12), "k.b": g.standard_normal(6), "v.b": g.standard_normal(4)})
    w.update({n: np.zeros(3) for n in ("lq1", "lk1", "lq2", "lk2")})
    h = g.standard_normal((6, 5))
    y, _ = O.differential_mixer(h, w, 2, 1, 3, 4, 0.5, 0.0, 1e-6)      # lambda = 1 - 1 + 0
    q = (h @ w["q"].T + w["q.b"]).reshape(6, 2, 2, 3)
    k, v = (h @ w["k"].T + w["k.b"]).reshape(6, 2, 3), h @ w["v"].T + w["v.b"]
    o = np.stack([O.unit_rms(O.causal_softmax_attention(q[:, i, 0], k[:, 0], v, 0.5, 0), 1e-6) for i in range(2)], 1)
    assert np.allclose(y, o.reshape(6, 8) @ w["o"].T)
    h2 = h.copy()
    h2[4:] += 1.0
    assert np.allclose(O.differential_mixer(h2, w, 2, 1, 3, 4, 0.5, 0.0, 1e-6)[0][:4], y[:4])
    head, past = O.differential_mixer(h[:2], w, 2, 1, 3, 4, 0.5, 0.3, 1e-6)
    tail, _ = O.differential_mixer(h[2:], w, 2, 1, 3, 4, 0.5, 0.3, 1e-6, past)
    whole, _ = O.differential_mixer(h, w, 2, 1, 3, 4, 0.5, 0.3, 1e-6)
    assert np.allclose(np.concatenate([head, tail]), whole)


def test_router_takes_the_largest_and_weights_the_input():
    router = np.array([[1.0, 0.0], [0.0, 1.0], [-1.0, 0.0]])
    ids, wt = O.route(np.array([[2.0, 1.0]]), router, 2)
    assert ids.tolist() == [[0, 1]] and np.allclose(wt, [[O.sigmoid(2.0), O.sigmoid(1.0)]])
    eye = np.eye(2)
    y = O.moe_ff(np.array([[2.0, 1.0]]), router, [eye] * 3, [eye] * 3, 1)
    assert np.allclose(y, [[(2 * wt[0, 0]) ** 2, wt[0, 0] ** 2]])      # inside the square


def test_loop_order():
    assert O.layer_runs(4, {"start": 1, "stop": 3, "times": 2}) == [(0, 0), (1, 0), (2, 0), (1, 1), (2, 1), (3, 0)]
    assert O.layer_runs(2, None) == [(0, 0), (1, 0)]


# ---- configuration, registry, files ------------------------------------------------------------------------------------
def _small():
    return M.config(23, 16, [M.attention(2, 1, 4, 6, mlp=M.dense(12)), M.lightning(2, 4, 5, mlp=M.moe(3, 2, 7)), M.lightning(1, 3, 2)],
                    {"start": 1, "stop": 3, "times": 2})


def test_registry_reads_the_configuration(ai):
    c = ai.registry.read_config(_small())
    assert (c.vocab, c.width, c.eps) == (23, 16, 1e-5) and "Komirax" in ai.registry.ARCHITECTURES
    a, b, d = c.layers
    assert a.mixer == ai.mixers.AttentionSpec(2, 1, 4, 6, 0.5, maps=2, diff=0.2, bias=True) and a.ff == ai.mixers.DenseSpec(12)
    assert b.mixer.decay == pytest.approx([0.5, 0.995]) and b.ff == ai.mixers.MoeSpec(3, 2, 7) and d.ff is None
    assert [(i, bool(p)) for i, p in c.runs()] == [(0, False), (1, False), (2, False), (1, True), (2, False)]
    plain = ai.registry.read_config({**_small(), "loop": None})
    assert [i for i, _ in plain.runs()] == [0, 1, 2]
    with pytest.raises(ai.InvalidArgument, match="unknown architecture"):
        ai.registry.read_config({"architecture": "None such"})
    broken = _small()
    del broken["layers"][1]["mixer"]["decay"]
    with pytest.raises(ai.InvalidArgument, match="decay"):
        ai.registry.read_config(broken)
    with pytest.raises(ai.InvalidArgument):
        ai.stack_pipeline.StackConfig(8, 8, 1e-6, c.layers, ai.stack_pipeline.Loop(2, 5, 2)).runs()


def _vifivik():
    return M.vifivik(23, 16, [M.latent(2, 4, 6, 5, 8, base=100.0, ff=12), M.retention(2, 4, 5, [0.5, 0.75]), M.mamba2(4, 3, 5, 2, 3, 2, ff=7),
                              M.latent(3, 2, 6, 7, 8, base=100.0, kv_from=0)], cap=9.0)


def test_registry_reads_a_stack_with_norms_behind_the_branches(ai):
    X, c = ai.mixers, ai.registry.read_config(_vifivik())
    c.check()
    assert c.layer is X.OutputNormLayer and c.softcap == 9.0 and c.loop is None and (c.vocab, c.width, c.eps) == (23, 16, 1e-5)
    assert c.layers[0] == X.LayerSpec(X.LatentAttentionSpec(2, 4, 6, 5, 8, 100.0, 10 ** -0.5), X.GatedSpec(12))
    assert c.layers[1] == X.LayerSpec(X.LinearAttentionSpec(2, 4, 5, [0.5, 0.75], ai.ACT_NONE, 0.5, ai.ACT_SILU, True))
    assert c.layers[2] == X.LayerSpec(X.SelectiveSpec(4, 3, 5, 2, 3, 2), X.GatedSpec(7)) and c.layers[3].mixer.kv_from == 0

    def broken(change):
        d = _vifivik()
        change(d)
        with pytest.raises(ai.InvalidArgument):
            ai.registry.read_config(d).check()
    broken(lambda d: d["layers"][3]["mixer"].update(kv_from=1))        # no latent layer
    broken(lambda d: d["layers"][3]["mixer"].update(kv_from=3))        # not an earlier one
    broken(lambda d: d["layers"][3]["mixer"].update(kv_rank=9))
    broken(lambda d: d["layers"][3]["mixer"]["rot"].update(base=7.0))
    broken(lambda d: d["layers"][0]["mixer"]["rot"].update(dims=4))
    broken(lambda d: d["layers"][0].update(type="attention"))
    broken(lambda d: d["layers"][0]["mlp"].update(kind="moe"))
    broken(lambda d: d["layers"][2]["mixer"].pop("state"))
    broken(lambda d: d.update(logit_softcap=0.0))


# ---- the plain statement of Vifivik's mechanisms ------------------------------------------------------------------------
def test_rotation_keeps_lengths_and_depends_on_the_distance():
    g = np.random.default_rng(1)
    q, k = g.standard_normal(8), g.standard_normal(8)

    def at(x, p):
        return O.rotate_pairs(x[None], [p], 50.0)[0]
    assert np.allclose(at(q, 0), q) and np.isclose(at(q, 17) @ at(q, 17), q @ q)
    assert np.isclose(at(q, 9) @ at(k, 4), at(q, 105) @ at(k, 100)) and not np.isclose(at(q, 9) @ at(k, 4), at(q, 9) @ at(k, 5))
    assert np.allclose(at(np.array([1.0, 0, 0, 0]), 2), [np.cos(2), np.sin(2), 0, 0])       # the pair is (0, 1), the angle counts up


def test_sink_takes_its_share_once():
    g = np.random.default_rng(2)
    q, k, v = g.standard_normal((5, 3)), g.standard_normal((5, 3)), g.standard_normal((5, 4))
    plain, sunk = O.causal_softmax_attention(q, k, v, 0.7, 0), O.sink_softmax_attention(q, k, v, 0.7, 1.3, 0)
    for i in range(5):
        z = np.exp(0.7 * (k[:i + 1] @ q[i])).sum()
        assert np.allclose(sunk[i], plain[i] * z / (z + np.exp(1.3)))
    assert np.allclose(O.sink_softmax_attention(q, k, v, 0.7, -100.0, 0), plain)


def test_latent_mixer_is_the_same_in_the_latent_space_and_in_portions():
    """Queries through the key projection and outputs through the value projection give what keys and values of every head give."""
    g = np.random.default_rng(3)
    H, d, e, n, r, W, T = 2, 3, 4, 5, 6, 7, 9
    w = {k: g.standard_normal(s) for k, s in (("q", (H * (d + e), W)), ("dkv", (r + e, W)), ("dkv.norm", (r,)), ("uk", (H * d, r)), ("uv", (H * n, r)),
                                              ("sink", (H,)), ("g", (H, W)), ("o", (W, H * n)))}
    h = g.standard_normal((T, W))
    c, kr = O.latent_rows(h, w, r, 30.0, 1e-5, 0)
    y = O.latent_mixer(h, w, H, d, e, n, 30.0, 0.4, c, kr, 0)
    q = (h @ w["q"].T).reshape(T, H, d + e)
    o = []
    for i in range(H):
        ql = np.concatenate([q[:, i, :d] @ w["uk"].reshape(H, d, r)[i], O.rotate_pairs(q[:, i, d:], range(T), 30.0)], axis=1)
        ol = O.sink_softmax_attention(ql, np.concatenate([c, kr], 1), c, 0.4, w["sink"][i], 0)
        o.append(O.sigmoid(h @ w["g"][i])[:, None] * (ol @ w["uv"].reshape(H, n, r)[i].T))
    assert np.allclose(np.concatenate(o, 1) @ w["o"].T, y)
    c2, kr2 = O.latent_rows(h[4:], w, r, 30.0, 1e-5, 4)
    assert np.allclose(c2, c[4:]) and np.allclose(kr2, kr[4:])
    assert np.allclose(O.latent_mixer(h[4:], w, H, d, e, n, 30.0, 0.4, c, kr, 4), y[4:])


def test_selective_recurrence_is_the_decayed_sum():
    g = np.random.default_rng(4)
    T, H, G, N, e = 7, 4, 2, 3, 2
    x, B, C, dt = g.standard_normal((T, H, e)), g.standard_normal((T, G, N)), g.standard_normal((T, G, N)), g.random((T, H))
    a_log, D = g.standard_normal(H), g.standard_normal(H)
    y, S = O.selective_recurrence(x, B, C, dt, a_log, D)
    for t in range(T):
        for h in range(H):
            want = D[h] * x[t, h]
            for s in range(t + 1):
                want = want + np.exp(-np.exp(a_log[h]) * dt[s + 1:t + 1, h].sum()) * dt[s, h] * (B[s, h // 2] @ C[t, h // 2]) * x[s, h]
            assert np.allclose(y[t, h], want)
    y1, S1 = O.selective_recurrence(x[:3], B[:3], C[:3], dt[:3], a_log, D)
    y2, S2 = O.selective_recurrence(x[3:], B[3:], C[3:], dt[3:], a_log, D, S1)
    assert np.allclose(np.concatenate([y1, y2]), y) and np.allclose(S2, S)


@pytest.mark.parametrize("taps", [1, 2, 4])
def test_causal_convolution_and_grouped_norm(taps):
    g = np.random.default_rng(5)
    x, w, b = g.standard_normal((6, 3)), g.standard_normal((3, taps)), g.standard_normal(3)
    y, past = O.causal_conv(x, np.zeros((taps - 1, 3)), w, b)
    for c in range(3):
        assert np.allclose(y[:, c], b[c] + np.convolve(x[:, c], w[c, ::-1])[:6])
    y1, p1 = O.causal_conv(x[:1], np.zeros((taps - 1, 3)), w, b)
    y2, p2 = O.causal_conv(x[1:], p1, w, b)
    assert np.allclose(np.concatenate([y1, y2]), y) and np.allclose(p2, past)
    v, z = g.standard_normal((2, 6)), g.standard_normal((2, 6))
    u = v * z / (1 + np.exp(-z))
    got = O.gated_group_norm(v, z, np.arange(6.0), 2, 0.0)
    assert np.allclose(got[:, :3], u[:, :3] / np.sqrt((u[:, :3] ** 2).mean(1, keepdims=True)) * np.arange(3.0))
    assert np.allclose(got[:, 3:], u[:, 3:] / np.sqrt((u[:, 3:] ** 2).mean(1, keepdims=True)) * np.arange(3.0, 6.0))


def test_capped_logits_and_portions_of_a_small_stack():
    cfg = _vifivik()
    w = M.plain_weights(M.weights(cfg, 6))
    tokens = [3, 1, 4, 1, 5, 9, 2, 6]
    whole = O.forward(cfg, w, tokens)
    assert np.abs(whole).max() < 9.0
    mem = {}
    parts = [O.forward(cfg, w, p, mem) for p in (tokens[:3], tokens[3:4], tokens[4:])]
    assert np.allclose(np.concatenate(parts), whole)
    assert np.allclose(O.softcap(np.array([1e-3, 50.0]), 9.0), [1e-3, 9.0], atol=1e-3)


def test_difference_lambda_matches_the_plain_statement(ai):
    g = np.random.default_rng(3)
    w = {n: g.standard_normal(10) * 0.3 for n in ("lq1", "lk1", "lq2", "lk2")}
    assert ai.mixers.difference_lambda(w["lq1"], w["lk1"], w["lq2"], w["lk2"], 0.35) == pytest.approx(O.diff_lambda(w, 0.35), rel=1e-5)


def test_safetensors_round_trip_and_rejections(ai, tmp_path):
    st = ai.safetensors
    p = str(tmp_path / "a.safetensors")
    f = np.arange(6, dtype=np.float32).reshape(2, 3) / 3
    st.write(p, {"f": f, "b": M.bf16_bits(f), "i": np.array([1, -2], np.int32)})
    t = st.SafetensorsFile(p)
    assert np.array_equal(t.f32("f"), f) and np.array_equal(t.bf16("b"), M.bf16_bits(f)) and np.array_equal(t.bf16("f"), M.bf16_bits(f))
    assert np.array_equal(t.f32("b"), M.bf16_values(M.bf16_bits(f))) and t.raw("i")[1].tolist() == [1, -2]
    assert t.shape("f") == (2, 3) and "f" in t and "x" not in t
    for bad in (lambda: t.bf16("x"), lambda: t.f32("f", (3, 2))):
        with pytest.raises(ai.gguf.InvalidFormat):
            bad()
    x = np.array([1.0, 1.00390625, 1.01171875, np.nan, -0.0], np.float32)      # ties go to even
    assert np.array_equal(st.round_to_bf16(x)[:3], [0x3F80, 0x3F80, 0x3F82]) and np.isnan(M.bf16_values(st.round_to_bf16(x))[3])
    q = tmp_path / "b.safetensors"
    q.write_bytes(struct.pack("<Q", 1 << 40) + b"{}")
    with pytest.raises(ai.gguf.InvalidFormat):
        st.SafetensorsFile(str(q))
    with pytest.raises(ai.Io):
        st.SafetensorsFile(str(tmp_path / "missing"))


# ---- sampler and scheduler ---------------------------------------------------------------------------------------------
def test_sampler(ai):
    S = ai.generation.Sampler
    z = np.array([0.0, 3.0, 3.0, 1.0])
    assert S().pick(z) == 1
    assert {S(temperature=1.0, top_k=1, seed=i).pick(z) for i in range(5)} == {1}
    assert {S(temperature=1.0, top_k=2, seed=i).pick(z) for i in range(30)} == {1, 2}
    assert {S(temperature=1.0, top_p=0.5, seed=i).pick(z) for i in range(30)} <= {1, 2}
    a, b = S(temperature=2.0, seed=7), S(temperature=2.0, seed=7)
    assert [a.pick(z) for _ in range(20)] == [b.pick(z) for _ in range(20)]
    n = [S(temperature=1.0, seed=i).pick(z) for i in range(400)]
    p = np.exp(z) / np.exp(z).sum()
    assert abs(n.count(3) / 400 - p[3]) < 0.05 and abs(n.count(1) / 400 - p[1]) < 0.1


class _Counting:
    """Next token = (sum of everything seen) mod 97; records the portions."""
    vocab_size = 97

    def __init__(self, pkg, slots):
        outer = self

        class Slot:
            def __init__(self):
                self.sum, self.n = 0, 0

            def reset(self):
                self.sum, self.n = 0, 0
        self.slots, self.calls, self.max_tokens = pkg.kv_cache.SlotPool(Slot, slots), [], 40

    def new_sequence(self):
        return self.slots.acquire()

    def end_sequence(self, s):
        self.slots.release(s)

    def step(self, s, tokens, want=()):
        self.calls.append(len(tokens))
        out = np.zeros((len(want), 97), np.float32)
        for i, t in enumerate(tokens):
            s.sum += t
            for j, p in enumerate(want):
                if p == i:
                    out[j, s.sum % 97] = 1
        s.n += len(tokens)
        return out


def _counted(prompt, n):
    total, out = sum(prompt), []
    for _ in range(n):
        out.append(total % 97)
        total += out[-1]
    return out


@pytest.mark.parametrize("slots", [1, 2, 5])
def test_scheduler_shares_slots_and_keeps_requests_apart(ai, slots):
    g = ai.generation
    m = _Counting(ai, slots)
    sch = g.Scheduler(m, portion=4)
    prompts = [[1, 2, 3], list(range(11)), [5], [9] * 8]
    reqs = [sch.submit(g.Request(p, 5 + i)) for i, p in enumerate(prompts)]
    sch.run()
    for i, (r, p) in enumerate(zip(reqs, prompts)):
        assert r.done and r.tokens == _counted(p, 5 + i)
    assert m.slots.available() == slots and max(m.calls) == 4
    stop = _counted([1, 2, 3], 3)[2]
    assert g.generate(m, [1, 2, 3], 9, stop_tokens=[stop]) == _counted([1, 2, 3], 3)
    assert g.generate(m, [1], 0) == []
    for bad in (g.Request([], 3), g.Request([1] * 30, 20)):
        with pytest.raises(ai.InvalidArgument):
            sch.submit(bad)


def test_slot_pool(ai):
    m = _Counting(ai, 2)
    a, b = m.new_sequence(), m.new_sequence()
    with pytest.raises(ai.InvalidArgument):
        m.new_sequence()
    a.sum = 5
    m.end_sequence(a)
    assert m.new_sequence() is a and a.sum == 0
    with pytest.raises(ai.InvalidArgument):
        m.slots.release(object())


def test_trace_replay_orders_and_files(ai, tmp_path):
    from local_ai_amd import trace
    m = _Counting(ai, 3)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": [5, 7, 9], "want": [2, 0]}, {"id": "b", "tokens": [4], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": [1], "want": [0]}], "end": ["b", "a"]},
             {"step": 2, "entries": [{"id": "a", "tokens": [3], "want": []}], "end": ["a"]}]
    said = []
    trace.replay(m, [json.dumps(s) for s in steps] + ["\n"], str(tmp_path), said.append)
    assert said == ["done 0", "done 1", "done 2"] and m.slots.available() == 3
    a = np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, 97)
    assert a.argmax(1).tolist() == [21, 5] and np.fromfile(tmp_path / "1.f32", "<f4").argmax() == 5
    assert not (tmp_path / "2.f32").exists()
