"""The kernels for models with bf16 weights, each against plain f64 arithmetic: products by segments in every form, norms,
softmax attention with one and two maps over block caches, linear attention (recurrent and chunked), mixture of experts."""
import numpy as np
import pytest

import mixer_models as M
from oracle import mixer_stack as O

pytestmark = pytest.mark.gpu

F32_TOL, BF16_TOL = 2e-5, 1.2e-2      # of the largest wanted value


@pytest.fixture(scope="module")
def ai(pkg):
    import local_ai_amd
    return local_ai_amd


def upload(ai, ctx, x, dtype):
    return ai.Buffer.from_slice(ctx, M.bf16_bits(x) if dtype == ai.BF16 else np.asarray(x, np.float32))


def download(ai, buf, count, dtype):
    return M.bf16_values(buf.as_array(np.uint16, count)) if dtype == ai.BF16 else buf.as_array(np.float32, count)


def empty(ai, ctx, count, dtype):
    return ai.Buffer.empty(ctx, count * (2 if dtype == ai.BF16 else 4))


def stored(x, ai, dtype):
    return M.rounded(x) if dtype == ai.BF16 else np.asarray(x, np.float32).astype(np.float64)


def close(got, want, tol, what=""):
    err = np.abs(got - want).max() / max(np.abs(want).max(), 1e-9)
    assert np.isfinite(got).all() and err <= tol, f"{what}: {err:.3g}"


ACTS = [lambda z: z, O.silu, O.gelu_tanh, O.relu_squared, O.sigmoid]


def block_order():
    """Place of each of a value block's 32 positions."""
    return np.array([((p >> 2) & 3) * 8 + ((p >> 4) & 1) * 4 + (p & 3) for p in range(32)])


def values_from_cache(flat, cols):
    """[positions, cols] from [block][cols][32]."""
    b = flat.reshape(-1, cols, 32)[:, :, block_order()]
    return b.transpose(0, 2, 1).reshape(-1, cols)


# ---- products ----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("m,k,n", [(1, 64, 48), (2, 256, 200), (31, 72, 33), (33, 40, 70), (64, 520, 130), (65, 64, 64), (129, 200, 257),
                                   (300, 136, 2052), (7, 60, 45), (140, 7, 9), (2100, 128, 2048),
                                   (1, 4104, 300), (1, 5000, 17), (1, 8192, 70), (1, 16384, 9), (1, 20008, 5), (1, 16, 270000), (600, 2048, 1100)])
def test_linear_rows(ai, gpu, dtype, m, k, n):
    ctx, K = gpu
    dt = ai.BF16 if dtype == "bf16" else ai.F32
    g = np.random.default_rng(m + k + n)
    x, w, b = stored(g.standard_normal((m, k)), ai, dt), M.rounded(g.standard_normal((n, k)) / np.sqrt(k)), g.standard_normal(n).astype(np.float32)
    want = x @ w.T + b
    print(f"linear {dtype} {m} {k} {n}", flush=True)
    xb, L = upload(ai, ctx, x, dt), ai.linear_weight
    act = (m + n) % 5
    lin = L.StackedLinear(ctx, [M.bf16_bits(w)], [L.Segment(n, act)], [b])
    out, res = empty(ai, ctx, m * n, ai.F32), upload(ai, ctx, np.ones((m, n)), ai.F32)
    batch = ai.CommandBatch(ctx)
    lin.rows_into(batch, K, xb, dt, m, [out], ai.F32)
    lin.rows_add_into(batch, K, xb, dt, m, res)
    batch.commit_and_wait()
    close(download(ai, out, m * n, ai.F32).reshape(m, n), ACTS[act](want), F32_TOL, "f32 output")
    close(download(ai, res, m * n, ai.F32).reshape(m, n), ACTS[act](want) + 1, F32_TOL, "residual")
    if m == 1:
        v = empty(ai, ctx, n, ai.F32)
        K.linear_vector_into(batch, xb, dt, lin.weight, lin.bias, k, lin.segments, [v], ai.F32)
        batch.commit_and_wait()
        close(download(ai, v, n, ai.F32), ACTS[act](want)[0], F32_TOL, "vector")


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("m,pos,width,heads,dim,pad,vdim,vpad", [(5, 30, 64, 3, 20, 32, 12, 32), (1, 31, 64, 3, 20, 32, 12, 32), (70, 1, 40, 2, 32, 32, 64, 64),
                                                                 (1, 32, 520, 1, 5, 32, 33, 64), (33, 63, 36, 2, 24, 32, 40, 64), (40, 100, 64, 2, 16, 32, 32, 32)])
def test_segments_write_caches_at_the_position(ai, gpu, dtype, m, pos, width, heads, dim, pad, vdim, vpad):
    """Three segments: plain rows, padded heads at the position, value blocks at the position; rows past the end are dropped."""
    ctx, K = gpu
    dt = ai.BF16 if dtype == "bf16" else ai.F32
    g, L, cap = np.random.default_rng(pos + m), ai.linear_weight, 128
    ws = [M.rounded(g.standard_normal((heads * d, width)) / np.sqrt(width)) for d in (dim, dim, vdim)]
    x = stored(g.standard_normal((m, width)), ai, dt)
    b = [g.standard_normal(w.shape[0]).astype(np.float32) for w in ws]
    lin = L.StackedLinear(ctx, [M.bf16_bits(w) for w in ws],
                          [L.Segment(heads * dim, ai.ACT_SILU, dim, pad), L.Segment(heads * dim, 0, dim, pad, ai.ROWS_AT_POSITION),
                           L.Segment(heads * vdim, 0, vdim, vpad, ai.BLOCKS_AT_POSITION)], b)
    q, k, v = empty(ai, ctx, m * heads * pad, dt), empty(ai, ctx, cap * heads * pad, dt), empty(ai, ctx, cap * heads * vpad, dt)
    p = ai.Buffer.from_slice(ctx, np.array([pos], np.uint32))
    print(f"segments {dtype} {m} {pos}", flush=True)
    batch = ai.CommandBatch(ctx)
    lin.rows_into(batch, K, upload(ai, ctx, x, dt), dt, m, [q, k, v], dt, p)
    batch.commit_and_wait()

    def check():
        tol = BF16_TOL if dt == ai.BF16 else F32_TOL
        got = download(ai, q, m * heads * pad, dt).reshape(m, heads, pad)
        close(got[:, :, :dim], O.silu(x @ ws[0].T + b[0]).reshape(m, heads, dim), tol, "q")
        assert not got[:, :, dim:].any()
        stay = min(m, cap - pos)
        got = download(ai, k, cap * heads * pad, dt).reshape(cap, heads, pad)
        close(got[pos:pos + stay, :, :dim], (x @ ws[1].T + b[1]).reshape(m, heads, dim)[:stay], tol, "k")
        assert not got[:pos].any() and not got[pos + stay:].any() and not got[:, :, dim:].any()
        got = values_from_cache(download(ai, v, cap * heads * vpad, dt), heads * vpad).reshape(cap, heads, vpad)
        close(got[pos:pos + stay, :, :vdim], (x @ ws[2].T + b[2]).reshape(m, heads, vdim)[:stay], tol, "v")
        assert not got[:pos].any() and not got[pos + stay:].any() and not got[:, :, vdim:].any()
    check()
    if m == 1:
        for t in (q, k, v):
            t.fill_zero()
        K.linear_vector_into(batch, upload(ai, ctx, x, dt), dt, lin.weight, lin.bias, width, lin.segments, [q, k, v], dt, False, p)
        batch.commit_and_wait()
        check()


@pytest.mark.parametrize("k,n", [(64, 40), (60, 33), (512, 130), (1000, 64), (1536, 20), (4096, 70), (9000, 12), (2501, 9)])
def test_linear_vector_stages(ai, gpu, k, n):
    """The norm (with an addition and a stored sum) and the gated norm in front of a one-row product."""
    ctx, K = gpu
    g, L, eps = np.random.default_rng(k), ai.linear_weight, 1e-3
    w = M.rounded(g.standard_normal((n, k)) / np.sqrt(k))
    x, add, nw, gate = (stored(g.standard_normal(k), ai, ai.F32) for _ in range(4))
    lin = L.StackedLinear(ctx, [M.bf16_bits(w)], [L.Segment(n)])
    xb, ab, nb = (upload(ai, ctx, t, ai.F32) for t in (x, add, nw))
    print(f"vector stages {k} {n}", flush=True)
    batch = ai.CommandBatch(ctx)
    outs = [empty(ai, ctx, n, ai.F32) for _ in range(4)]
    kept = empty(ai, ctx, k, ai.F32)
    lin.normed_vector_into(batch, K, xb, nb, eps, [outs[0]], ai.F32)
    lin.normed_vector_into(batch, K, xb, nb, eps, [outs[1]], ai.F32, None, ab, kept)
    for i, dt in ((2, ai.F32), (3, ai.BF16)):
        K.linear_gated_vector_into(batch, xb, upload(ai, ctx, gate, dt), dt, nb, eps, lin.weight, None, k, lin.segments, [outs[i]], ai.F32)
    batch.commit_and_wait()
    got = [download(ai, o, n, ai.F32) for o in outs]
    close(got[0], w @ (O.unit_rms(x, eps) * nw), F32_TOL)
    close(got[1], w @ (O.unit_rms(x + add, eps) * nw), F32_TOL)
    close(download(ai, kept, k, ai.F32), x + add, F32_TOL)
    close(got[2], w @ (O.unit_rms(x, eps) * nw * O.sigmoid(gate)), F32_TOL)
    close(got[3], w @ (O.unit_rms(x, eps) * nw * O.sigmoid(M.rounded(gate))), F32_TOL)
    with pytest.raises(ai.InvalidArgument):          # the sum must not go where the other workgroups still read
        lin.normed_vector_into(batch, K, xb, nb, eps, [outs[0]], ai.F32, None, ab, xb)


@pytest.mark.parametrize("rows,dim", [(1, 64), (5, 100), (3, 1024), (2, 4096), (4, 5000), (70, 33)])
def test_row_norms_and_gather(ai, gpu, rows, dim):
    ctx, K = gpu
    g, eps = np.random.default_rng(dim), 1e-4
    x, add, gate = (stored(g.standard_normal((rows, dim)), ai, ai.F32) for _ in range(3))
    w = stored(g.standard_normal(dim), ai, ai.F32)
    xb, ab, wb = upload(ai, ctx, x, ai.F32), upload(ai, ctx, add, ai.F32), upload(ai, ctx, w, ai.F32)
    batch = ai.CommandBatch(ctx)
    print(f"norms {rows} {dim}", flush=True)
    for dt, tol in ((ai.F32, F32_TOL), (ai.BF16, BF16_TOL)):
        out, kept, picked = empty(ai, ctx, rows * dim, dt), empty(ai, ctx, rows * dim, ai.F32), empty(ai, ctx, 3 * dim, dt)
        K.norm_rows_f32_into(batch, xb, ab, wb, kept, None, out, dt, dim, rows, eps)
        pick = [rows - 1, 0, rows // 2]
        K.norm_rows_f32_into(batch, xb, None, wb, None, ai.Buffer.from_slice(ctx, np.array(pick, np.uint32)), picked, dt, dim, 3, eps)
        gated = empty(ai, ctx, rows * dim, dt)
        K.gated_norm_rows_into(batch, xb, upload(ai, ctx, gate, dt), wb, gated, dt, dim, rows, eps)
        batch.commit_and_wait()
        close(download(ai, out, rows * dim, dt).reshape(rows, dim), O.unit_rms(x + add, eps) * w, tol)
        close(download(ai, kept, rows * dim, ai.F32).reshape(rows, dim), x + add, F32_TOL)
        close(download(ai, picked, 3 * dim, dt).reshape(3, dim), (O.unit_rms(x, eps) * w)[pick], tol)
        close(download(ai, gated, rows * dim, dt).reshape(rows, dim), O.unit_rms(x, eps) * w * O.sigmoid(stored(gate, ai, dt)), tol)
    table = g.standard_normal((9, dim))
    idx = np.array([8, 0, 3, 200], np.uint32)
    out = empty(ai, ctx, 4 * dim, ai.F32)
    K.embed_rows_bf16_into(batch, upload(ai, ctx, table, ai.BF16), 9, dim, ai.Buffer.from_slice(ctx, idx), 4, out)
    z = x.astype(np.float32)
    z[0, dim // 2] = z[0, dim - 1] = 9.0
    best, pos = ai.Buffer.empty(ctx, 4 * rows), ai.Buffer.from_slice(ctx, np.array([5], np.uint32))
    K.argmax_rows_f32_into(batch, ai.Buffer.from_slice(ctx, z), best, rows, dim)
    K.advance_position_into(batch, pos, 7)
    batch.commit_and_wait()
    assert np.array_equal(download(ai, out, 4 * dim, ai.F32).reshape(4, dim), M.rounded(table)[[8, 0, 3, 8]])
    assert best.as_array(np.uint32).tolist() == z.argmax(1).tolist() and pos.as_array(np.uint32, 1)[0] == 12


# ---- softmax attention -------------------------------------------------------------------------------------------------
def attention_case(ai, gpu, dtype, maps, heads, kv_heads, dim, vdim, start, rows, cap, seed=0, spike=None, stale=False, lam=0.4, out_scale=0.7):
    """Caches filled as the projections fill them.  `spike` = (row, key): one key that takes nearly all of a row's weight."""
    ctx, K = gpu
    dt = ai.BF16 if dtype == "bf16" else ai.F32
    g, eps, scale = np.random.default_rng(seed + start + rows + dim), 1e-5, dim ** -0.5
    L, dq, dv = start + rows, K.attention_padded_dim(dim), K.attention_padded_vdim(vdim)
    q, k, v = (stored(g.standard_normal(s), ai, dt) for s in ((rows, heads, maps, dim), (L, kv_heads, maps, dim), (L, kv_heads, vdim)))
    if spike is not None:
        row, key = spike
        u = np.sign(g.standard_normal(dim))
        k[key] = stored(u * 5.0, ai, dt)
        q[row] = stored(u * 14.0 / np.sqrt(dim), ai, dt)
    fill = 3.0 if stale else 0.0                      # what an earlier, longer sequence would have left behind
    kc, vc, qp = np.full((cap, kv_heads, maps, dq), fill), np.full((cap, kv_heads, dv), fill), np.zeros((rows, heads, maps, dq))
    kc[:, :, :, dim:] = vc[:, :, vdim:] = 0.0
    kc[:L, :, :, :dim], vc[:L, :, :vdim], qp[..., :dim] = k, v, q
    blocks = np.zeros((cap // 32, kv_heads * dv, 32))
    blocks[:, :, block_order()] = vc.reshape(cap // 32, 32, kv_heads * dv).transpose(0, 2, 1)
    out, pos = empty(ai, ctx, rows * heads * vdim, dt), ai.Buffer.from_slice(ctx, np.array([start], np.uint32))
    print(f"attention {dtype} maps {maps} heads {heads}/{kv_heads} dim {dim} vdim {vdim} start {start} rows {rows}", flush=True)
    batch = ai.CommandBatch(ctx)
    K.attention_rows_into(batch, upload(ai, ctx, qp, dt), upload(ai, ctx, kc, dt), upload(ai, ctx, blocks, dt), out, dt, pos, start, rows, heads,
                          kv_heads, maps, dim, vdim, cap, scale, lam, out_scale, eps)
    batch.commit_and_wait()
    got = download(ai, out, rows * heads * vdim, dt).reshape(rows, heads, vdim)
    want = np.zeros((rows, heads, vdim))
    for h in range(heads):
        j = h // (heads // kv_heads)
        a = [O.causal_softmax_attention(q[:, h, m], k[:, j, m], v[:, j], scale, start) for m in range(maps)]
        want[:, h] = a[0] if maps == 1 else O.unit_rms(a[0] - lam * a[1], eps) * out_scale
    # over a thousand random keys the difference of the two averages is small and its norm enlarges the rounding of both sums about thirtyfold
    close(got, want, BF16_TOL if dt == ai.BF16 else F32_TOL if maps == 1 else 1e-4, "attention")
    if spike is not None and maps == 1:
        close(got[spike[0]].reshape(kv_heads, -1, vdim), v[spike[1]][:, None].repeat(heads // kv_heads, 1), 0.03, "the far key's value")
    return got


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("maps", [1, 2])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(3, 3, 32, 64), (6, 2, 24, 40), (8, 1, 64, 128), (3, 3, 8, 16), (4, 2, 128, 256), (5, 1, 20, 33), (34, 2, 16, 24)])
@pytest.mark.parametrize("start,rows", [(0, 1), (31, 1), (32, 2), (95, 34), (0, 97), (63, 190)])
def test_attention_shapes(ai, gpu, dtype, maps, heads, kv_heads, dim, vdim, start, rows):
    attention_case(ai, gpu, dtype, maps, heads, kv_heads, dim, vdim, start, rows, 256)


@pytest.mark.parametrize("dim,vdim", [(32, 32), (32, 128), (32, 256), (64, 32), (64, 64), (64, 256), (128, 32), (128, 64), (128, 128), (128, 256), (136, 64), (48, 300)])
@pytest.mark.parametrize("rows", [1, 150])
@pytest.mark.parametrize("maps", [1, 2])
def test_attention_every_head_size(ai, gpu, maps, dim, vdim, rows):
    attention_case(ai, gpu, "bf16", maps, 4, 2, dim, vdim, 70, rows, 256)


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("rows", [1, 3, 300])
@pytest.mark.parametrize("key", [0, 1, 31, 32, 33, 511, 1000, 1023])
def test_attention_finds_one_key_far_away(ai, gpu, dtype, rows, key):
    attention_case(ai, gpu, dtype, 1, 4, 2, 32, 64, 1023, rows, 1344, spike=(rows - 1, key))
    attention_case(ai, gpu, dtype, 2, 4, 2, 32, 64, 1023, rows, 1344, spike=(0, key))


@pytest.mark.parametrize("rows", [1, 40, 200])
def test_attention_ignores_what_lies_behind_the_last_position(ai, gpu, rows):
    """Stale rows and block entries past the last position (a slot that is used again) must not change a bit."""
    a = attention_case(ai, gpu, "bf16", 2, 4, 2, 32, 64, 45, rows, 320)
    b = attention_case(ai, gpu, "bf16", 2, 4, 2, 32, 64, 45, rows, 320, stale=True)
    assert np.array_equal(a, b)


def test_attention_long_context_splits(ai, gpu):
    for rows in (1, 5):
        attention_case(ai, gpu, "bf16", 2, 2, 1, 32, 32, 9000, rows, 9056, spike=(0, 37))


def test_attention_rejects(ai, gpu):
    ctx, K = gpu
    b, batch = ai.Buffer.empty(ctx, 1 << 16), ai.CommandBatch(ctx)
    for args in ((5, 1, 3, 2, 1, 32, 32, 32), (31, 2, 2, 2, 1, 32, 32, 32), (0, 1, 2, 2, 3, 32, 32, 32), (0, 1, 2, 2, 1, 32, 32, 40)):
        with pytest.raises(ai.InvalidArgument):
            K.attention_rows_into(batch, b, b, b, b, ai.BF16, b, *args, 1.0)
    assert batch.dispatch_count() == 0


# ---- linear attention --------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("heads,dim,vdim", [(4, 32, 48), (3, 20, 33), (2, 64, 128), (1, 128, 80), (2, 200, 48), (2, 8, 100)])
@pytest.mark.parametrize("cuts", [[1, 1, 1], [16, 2], [64], [17, 65, 130], [63, 1, 64], [300]])
def test_linear_attention_forms(ai, gpu, heads, dim, vdim, cuts):
    """Recurrent in both types and chunked, in portions: the outputs, and the state after every portion."""
    ctx, K = gpu
    g, T = np.random.default_rng(dim + sum(cuts)), sum(cuts)
    decay = np.array([0.9995, 0.3, 1.0, 0.0][:heads])
    dq = K.linear_attention_padded_dim(dim)
    q, k, v = (M.rounded(g.standard_normal(s)) for s in ((T, heads, dim), (T, heads, dim), (T, heads, vdim)))
    q[-1] = M.rounded(k[0] * 3)                      # the last row asks for the first
    for dt, chunked in ((ai.F32, False), (ai.BF16, False), (ai.BF16, True)):
        print(f"linear attention {heads} {dim} {vdim} {cuts} dtype {dt} chunked {chunked}", flush=True)
        state = ai.Buffer.empty(ctx, heads * vdim * dq * 4)
        db = ai.Buffer.from_slice(ctx, decay.astype(np.float32))
        pw = ai.Buffer.from_slice(ctx, (decay[:, None] ** np.arange(65)).astype(np.float32))
        s, at = None, 0
        for n in cuts:
            part = slice(at, at + n)
            qp, kp = np.full((n, heads, dq), 2.0), np.full((n, heads, dq), 2.0)      # the padding's content must not matter
            qp[..., :dim], kp[..., :dim] = q[part], k[part]
            qb, kb, vb = upload(ai, ctx, qp, dt), upload(ai, ctx, kp, dt), upload(ai, ctx, v[part], dt)
            out = empty(ai, ctx, n * heads * vdim, ai.F32)
            batch = ai.CommandBatch(ctx)
            if chunked:
                work = ai.Buffer.empty(ctx, K.linear_attention_workspace_bytes(n, heads, dim, vdim))
                K.linear_attention_chunked_into(batch, qb, kb, vb, state, pw, work, out, n, heads, dim, vdim)
            else:
                K.linear_attention_recurrent_into(batch, qb, kb, vb, dt, state, db, out, n, heads, dim, vdim)
            batch.commit_and_wait()
            want, s = O.lightning_recurrence(q[part], k[part], v[part], decay, s)
            close(download(ai, out, n * heads * vdim, ai.F32).reshape(n, heads, vdim), want, F32_TOL, f"rows {part}")
            got = state.as_array(np.float32).reshape(heads, vdim, dq)
            close(got[:, :, :dim].transpose(0, 2, 1), s, F32_TOL, f"state after {at + n}")
            at += n


# ---- mixture of experts ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("rows,experts,top,width,ff", [(2, 5, 2, 64, 48), (7, 3, 3, 40, 33), (65, 11, 1, 64, 88), (300, 4, 2, 64, 72), (600, 2, 1, 32, 40),
                                                       (33, 70, 8, 32, 16), (130, 130, 3, 24, 24), (5, 1, 1, 60, 20), (90, 6, 2, 136, 257),
                                                       (3, 300, 4, 24, 16), (2, 4, 3, 4104, 40), (2, 6, 3, 64, 1500)])
def test_mixture_of_experts(ai, gpu, dtype, rows, experts, top, width, ff):
    ctx, K = gpu
    dt = ai.BF16 if dtype == "bf16" else ai.F32
    g = np.random.default_rng(rows + experts)
    x = stored(g.standard_normal((rows, width)), ai, dt)
    ups, downs = (M.rounded(g.standard_normal(s) / np.sqrt(s[2])) for s in ((experts, ff, width), (experts, width, ff)))
    logits = (g.permuted(np.tile(np.arange(experts), (rows, 1)), axis=1) * 0.37 - 1.0).astype(np.float32)
    if experts > 4:
        logits[:, 4] = -50.0                          # an expert that nobody takes
    res = g.standard_normal((rows, width)).astype(np.float32)
    order = np.argsort(-logits, axis=1, kind="stable")[:, :top]
    want, single = res.astype(np.float64), np.zeros((rows, width))
    for t in range(rows):
        for e in order[t]:
            single[t] += downs[e] @ O.relu_squared(ups[e] @ (O.sigmoid(float(logits[t, e])) * x[t]))
    want = want + single
    print(f"experts {dtype} {rows} {experts} {top} {width} {ff}", flush=True)
    plan = ai.Buffer.empty(ctx, 4 * K.moe_plan_words(rows, experts, top))
    up, down = (ai.Buffer.from_slice(ctx, M.bf16_bits(w)) for w in (ups, downs))
    hidden, slots, rb = empty(ai, ctx, rows * top * ff, dt), empty(ai, ctx, rows * top * width, ai.F32), upload(ai, ctx, res, ai.F32)
    lb = ai.Buffer.from_slice(ctx, logits)
    batch = ai.CommandBatch(ctx)
    K.moe_route_into(batch, lb, plan, rows, experts, top)
    K.moe_up_into(batch, upload(ai, ctx, x, dt), dt, plan, up, hidden, rows, experts, top, width, ff, ai.ACT_RELU_SQUARED)
    K.moe_down_into(batch, hidden, dt, plan, down, slots, rb, rows, experts, top, width, ff)
    batch.commit_and_wait()
    assert np.array_equal(plan.as_array(np.uint32, rows * top).reshape(rows, top), order)
    tol = F32_TOL if dt == ai.F32 else BF16_TOL
    close(download(ai, rb, rows * width, ai.F32).reshape(rows, width), want, tol, "residual")
    # one row through the form that selects and norms by itself
    nw, eps = stored(1 + 0.1 * g.standard_normal(width), ai, ai.F32), 1e-5
    h = O.unit_rms(x[0], eps) * nw
    one = sum(downs[e] @ O.relu_squared(ups[e] @ (O.sigmoid(float(logits[0, e])) * h)) for e in order[0])
    rb0, hid = upload(ai, ctx, res[0], ai.F32), empty(ai, ctx, top * ff, ai.F32)
    K.moe_vector_up_into(batch, upload(ai, ctx, x[0], ai.F32), upload(ai, ctx, nw, ai.F32), eps, lb, up, hid, experts, top, width, ff, ai.ACT_RELU_SQUARED)
    K.moe_vector_down_into(batch, hid, lb, down, rb0, experts, top, width, ff)
    batch.commit_and_wait()
    close(download(ai, rb0, width, ai.F32), res[0] + one, F32_TOL, "one row")


def test_equal_scores_go_to_the_lower_expert(ai, gpu):
    ctx, K = gpu
    logits = np.zeros((3, 9), np.float32)
    logits[1, 6] = logits[1, 2] = 1.0
    plan, batch = ai.Buffer.empty(ctx, 4 * K.moe_plan_words(3, 9, 2)), ai.CommandBatch(ctx)
    K.moe_route_into(batch, ai.Buffer.from_slice(ctx, logits), plan, 3, 9, 2)
    batch.commit_and_wait()
    assert plan.as_array(np.uint32, 6).reshape(3, 2).tolist() == [[0, 1], [2, 6], [0, 1]]
