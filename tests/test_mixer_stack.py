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
