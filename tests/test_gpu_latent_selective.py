"""The kernels of latent attention, of the selective state space and of norms behind the branches, each against plain f64
arithmetic."""
import numpy as np
import pytest

import mixer_models as M
from oracle import mixer_stack as O
from test_gpu_mixers import BF16_TOL, F32_TOL, close, download, empty, stored, upload, values_from_cache

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def ai(pkg):
    import local_ai_amd
    return local_ai_amd


def f32(ai, ctx, x):
    return ai.Buffer.from_slice(ctx, np.ascontiguousarray(x, np.float32))


# ---- latent attention ------------------------------------------------------------------------------------------------------
def cache_rows(K, latent, rot):
    """Cache rows as the kernels keep them, zeros in the padding."""
    T, r = latent.shape
    out = np.zeros((T, K.latent_row(r, rot.shape[1])))
    out[:, :r], out[:, K.latent_padded_rank(r):K.latent_padded_rank(r) + rot.shape[1]] = latent, rot
    return out


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("heads,rank,rot", [(1, 3, 2), (5, 48, 8), (3, 130, 64), (2, 512, 20), (2, 70, 72)])
@pytest.mark.parametrize("start,rows", [(0, 1), (31, 3), (1000, 70)])
def test_latent_prepare(ai, gpu, dtype, heads, rank, rot, start, rows):
    ctx, K = gpu
    dt, g = ai.BF16 if dtype == "bf16" else ai.F32, np.random.default_rng(rank + rows)
    capacity, row, dv = (start + rows + 31) // 32 * 32, K.latent_row(rank, rot), K.latent_padded_rank(rank)
    q, down, w = (g.standard_normal(s).astype(np.float32) for s in ((rows, heads, rot), (rows, rank + rot), (rank,)))
    base, dim = 700.0, 5
    freq = f32(ai, ctx, base ** (-2.0 * np.arange(rot // 2) / rot))
    pos, qb, db, wb = ai.Buffer.from_slice(ctx, np.array([start], np.uint32)), f32(ai, ctx, q), f32(ai, ctx, down), f32(ai, ctx, w)
    cache, ql, qe = empty(ai, ctx, capacity * row, dt), upload(ai, ctx, np.full((rows, heads, row), 7.0), ai.F32), upload(ai, ctx, np.full((rows, heads, dim + rot + 3), 7.0), dt)
    batch = ai.CommandBatch(ctx)
    K.latent_prepare_into(batch, qb, db, wb, freq, pos, ql, ai.F32, cache, dt, rows, heads, rank, rot, row, dv, rank, capacity, 1e-4)
    K.latent_prepare_into(batch, qb, None, None, freq, pos, qe, dt, cache, dt, rows, heads, rank, rot, dim + rot + 3, dim, dim, capacity, 1e-4)
    batch.commit_and_wait()
    where, tol = range(start, start + rows), BF16_TOL if dt == ai.BF16 else 1e-4      # (a 32-bit angle at position 1000)
    want = cache_rows(K, O.unit_rms(down[:, :rank].astype(np.float64), 1e-4) * w, O.rotate_pairs(down[:, rank:].astype(np.float64), where, base))
    got = download(ai, cache, capacity * row, dt).reshape(capacity, row)
    close(got[start:start + rows], want, tol, "cache rows")
    assert not got[:start].any() and not got[start + rows:].any()
    turned = O.rotate_pairs(q.astype(np.float64), where, base)
    got = download(ai, ql, rows * heads * row, ai.F32).reshape(rows, heads, row)
    close(got[..., dv:dv + rot], turned, 1e-4, "queries")
    assert (got[..., :rank] == 7).all() and not got[..., rank:dv].any() and not got[..., dv + rot:].any()
    got = download(ai, qe, rows * heads * (dim + rot + 3), dt).reshape(rows, heads, dim + rot + 3)
    close(got[..., dim:dim + rot], turned, tol, "queries behind unrotated columns")
    assert (got[..., :dim] == 7).all() and not got[..., dim + rot:].any()


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("rows,heads,n,k,ld", [(1, 1, 1, 1, 1), (1, 5, 96, 128, 100), (3, 4, 33, 40, 40), (17, 2, 16, 520, 16), (64, 3, 50, 11, 64)])
def test_head_linear(ai, gpu, dtype, rows, heads, n, k, ld):
    ctx, K = gpu
    dt, g = ai.BF16 if dtype == "bf16" else ai.F32, np.random.default_rng(n + k)
    x, w = stored(g.standard_normal((rows, heads, k)), ai, dt), M.rounded(g.standard_normal((heads, n, k)))
    want = np.stack([x[:, h] @ w[h].T for h in range(heads)], 1)
    xb, wb, batch = upload(ai, ctx, x, dt), ai.Buffer.from_slice(ctx, M.bf16_bits(w)), ai.CommandBatch(ctx)
    for out in {ai.F32, dt}:
        y = upload(ai, ctx, np.full((rows, heads, ld), 5.0), out)
        K.head_linear_into(batch, xb, dt, wb, y, out, rows, heads, n, k, ld)
        batch.commit_and_wait()
        got = download(ai, y, rows * heads * ld, out).reshape(rows, heads, ld)
        close(got[..., :n], want, F32_TOL if out == ai.F32 else BF16_TOL)
        assert (got[..., n:] == 5).all()


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("heads,dim,rot,vdim,rank", [(1, 5, 2, 3, 7), (3, 40, 16, 24, 96), (2, 128, 64, 128, 256)])
def test_latent_expand(ai, gpu, dtype, heads, dim, rot, vdim, rank):
    ctx, K = gpu
    dt, g, T = ai.BF16 if dtype == "bf16" else ai.F32, np.random.default_rng(rank), 96
    c, kr = stored(g.standard_normal((T, rank)), ai, dt), stored(g.standard_normal((T, rot)), ai, dt)
    uk, uv = (M.rounded(g.standard_normal((heads * n, rank)) / np.sqrt(rank)) for n in (dim, vdim))
    dq, dv = K.attention_padded_dim(dim + rot), K.attention_padded_vdim(vdim)
    keys, values = empty(ai, ctx, T * heads * dq, dt), empty(ai, ctx, T * heads * dv, dt)
    batch = ai.CommandBatch(ctx)
    K.latent_expand_into(batch, upload(ai, ctx, cache_rows(K, c, kr), dt), dt, ai.Buffer.from_slice(ctx, M.bf16_bits(np.concatenate([uk, uv]))), keys, values, T,
                         heads, dim, rot, vdim, rank)
    batch.commit_and_wait()
    tol = F32_TOL if dt == ai.F32 else BF16_TOL
    got = download(ai, keys, T * heads * dq, dt).reshape(T, heads, dq)
    close(got[..., :dim], (c @ uk.T).reshape(T, heads, dim), tol, "keys")
    assert np.array_equal(got[..., dim:dim + rot], np.repeat(kr[:, None], heads, 1).astype(np.float32))
    close(values_from_cache(download(ai, values, T * heads * dv, dt), heads * dv).reshape(T, heads, dv)[..., :vdim], (c @ uv.T).reshape(T, heads, vdim), tol, "values")


def latent_case(ai, gpu, dtype, heads, rank, rot, start, rows, capacity, spike=None, stale=False, sink=0.5):
    """`spike` (row, key): that row's queries match that key far better than any other."""
    ctx, K = gpu
    dt, g, T = ai.BF16 if dtype == "bf16" else ai.F32, np.random.default_rng(heads + rank + start + rows), start + rows
    c, kr = stored(g.standard_normal((T, rank)), ai, dt), stored(g.standard_normal((T, rot)), ai, dt)
    q, scale = g.standard_normal((rows, heads, rank + rot)), 1.0 / np.sqrt(rank + rot)
    if spike:
        q[spike[0]] = np.concatenate([c[spike[1]], kr[spike[1]]]) * (12.0 / np.sqrt(rank + rot)) * np.linspace(1, 2, heads)[:, None]
        scale = 1.0
    sinks, gates = np.linspace(-2, sink, heads), g.standard_normal((rows, heads))
    q, sinks, gates = (x.astype(np.float32).astype(np.float64) for x in (q, sinks, gates))
    want = np.stack([O.sink_softmax_attention(q[:, h], np.concatenate([c, kr], 1), c, scale, sinks[h], start) for h in range(heads)], 1) * O.sigmoid(gates)[..., None]
    row, dv = K.latent_row(rank, rot), K.latent_padded_rank(rank)
    cache = np.zeros((capacity, row))
    cache[:T] = cache_rows(K, c, kr)
    if stale:
        cache[T:] = np.random.default_rng(1).standard_normal((capacity - T, row)) * 50
    qp = np.zeros((rows, heads, row))
    qp[..., :rank], qp[..., dv:dv + rot] = q[..., :rank], q[..., rank:]
    out, pos, batch = empty(ai, ctx, rows * heads * rank, dt), ai.Buffer.from_slice(ctx, np.array([start], np.uint32)), ai.CommandBatch(ctx)
    print(f"latent {dtype} {heads} {rank} {rot} {start} {rows} {capacity} {spike}", flush=True)
    K.latent_attention_rows_into(batch, f32(ai, ctx, qp), upload(ai, ctx, cache, dt), out, dt, pos, start, rows, heads, rank, rot, capacity, scale, f32(ai, ctx, sinks),
                                 f32(ai, ctx, gates))
    batch.commit_and_wait()
    got = download(ai, out, rows * heads * rank, dt).reshape(rows, heads, rank)
    close(got, want, F32_TOL if dt == ai.F32 else BF16_TOL, "output")
    return got


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("rows,heads,dim,rank,rot,own", [(1, 1, 3, 5, 2, True), (1, 6, 64, 128, 16, False), (1, 16, 128, 512, 64, True), (40, 3, 40, 96, 20, True)])
def test_latent_queries_equal_the_two_steps(ai, gpu, dtype, rows, heads, dim, rank, rot, own):
    ctx, K = gpu
    dt, g = ai.BF16 if dtype == "bf16" else ai.F32, np.random.default_rng(rank)
    row, dv, start = K.latent_row(rank, rot), K.latent_padded_rank(rank), 17
    q, uk = upload(ai, ctx, g.standard_normal((rows, heads, dim)), dt), ai.Buffer.from_slice(ctx, M.bf16_bits(g.standard_normal((heads, rank, dim))))
    qr, down, nw = f32(ai, ctx, g.standard_normal((rows, heads, rot))), f32(ai, ctx, g.standard_normal((rows, rank + rot))) if own else None, f32(ai, ctx, g.standard_normal(rank))
    freq, pos, batch = f32(ai, ctx, 30.0 ** -np.arange(rot // 2)), ai.Buffer.from_slice(ctx, np.array([start], np.uint32)), ai.CommandBatch(ctx)
    caches, outs = [empty(ai, ctx, 64 * row, dt) for _ in range(2)], [empty(ai, ctx, rows * heads * row, ai.F32) for _ in range(2)]
    K.latent_prepare_into(batch, qr, down, nw, freq, pos, outs[0], ai.F32, caches[0], dt, rows, heads, rank, rot, row, dv, rank, 64, 1e-5)
    K.head_linear_into(batch, q, dt, uk, outs[0], ai.F32, rows, heads, rank, dim, row)
    K.latent_queries_into(batch, q, uk, qr, down, nw, freq, pos, outs[1], caches[1], dt, rows, heads, dim, rank, rot, 64, 1e-5)
    batch.commit_and_wait()
    for a, b, t in ((*caches, dt), (*outs, ai.F32)):
        n = 64 * row if a is caches[0] else rows * heads * row
        assert np.array_equal(download(ai, a, n, t), download(ai, b, n, t))
    assert own == bool(download(ai, caches[1], 64 * row, dt).any())


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("heads,rank,rot", [(1, 3, 2), (5, 64, 8), (3, 100, 64), (16, 160, 32), (17, 512, 64), (2, 300, 20), (2, 70, 72), (2, 600, 16)])
@pytest.mark.parametrize("start,rows", [(0, 1), (31, 1), (32, 2), (95, 34), (0, 64), (600, 1)])
def test_latent_attention_shapes(ai, gpu, dtype, heads, rank, rot, start, rows):
    latent_case(ai, gpu, dtype, heads, rank, rot, start, rows, 640)


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("rank", [40, 128, 512])
@pytest.mark.parametrize("key", [0, 1, 15, 16, 31, 32, 33, 511, 1000, 1023])
def test_latent_attention_finds_one_key_far_away(ai, gpu, dtype, rank, key):
    latent_case(ai, gpu, dtype, 4, rank, 16, 1023, 1, 1344, spike=(0, key))
    latent_case(ai, gpu, dtype, 4, rank, 16, 1020, 6, 1344, spike=(4, key))


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
def test_a_large_sink_leaves_the_rest_its_small_share(ai, gpu, dtype):
    for rows in (1, 7):
        latent_case(ai, gpu, dtype, 3, 64, 8, 300, rows, 320, sink=30.0)
        latent_case(ai, gpu, dtype, 3, 64, 8, 0, rows, 320, sink=100.0)


def test_latent_attention_ignores_what_lies_behind_the_last_position(ai, gpu):
    for rank, rows in ((128, 1), (512, 1), (64, 40)):
        a = latent_case(ai, gpu, "bf16", 4, rank, 32, 45, rows, 320)
        assert np.array_equal(a, latent_case(ai, gpu, "bf16", 4, rank, 32, 45, rows, 320, stale=True))


def test_latent_attention_long_context_splits(ai, gpu):
    for rows in (1, 5):
        latent_case(ai, gpu, "bf16", 2, 128, 16, 9000, rows, 9056, spike=(0, 37))


def test_latent_attention_rejects(ai, gpu):
    ctx, K = gpu
    b, batch = ai.Buffer.empty(ctx, 1 << 16), ai.CommandBatch(ctx)
    for args in ((31, 2, 2, 32, 8, 32), (0, 1, 0, 32, 8, 32), (0, 1, 2, 2000, 8, 32), (0, 1, 2, 32, 8, 40), (0, 1, 2, 512, 64, 64000)):
        with pytest.raises(ai.InvalidArgument):
            K.latent_attention_rows_into(batch, b, b, b, ai.BF16, b, *args, 1.0)
    assert batch.dispatch_count() == 0


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(2, 2, 56, 24), (3, 1, 160, 128), (2, 2, 192, 128), (2, 1, 250, 256), (1, 1, 264, 40)])
@pytest.mark.parametrize("start,rows", [(0, 1), (40, 3), (0, 97), (130, 190), (3000, 66)])
def test_softmax_attention_with_sink_and_gate(ai, gpu, dtype, heads, kv_heads, dim, vdim, start, rows):
    ctx, K = gpu
    dt, g, T = ai.BF16 if dtype == "bf16" else ai.F32, np.random.default_rng(dim + rows), start + rows
    cap, dq, dv = (T + 31) // 32 * 32, K.attention_padded_dim(dim), K.attention_padded_vdim(vdim)
    q, k, v = (stored(g.standard_normal(s), ai, dt) for s in ((rows, heads, dim), (T, kv_heads, dim), (T, kv_heads, vdim)))
    sinks, gates = np.linspace(-1, 3, heads).astype(np.float32), g.standard_normal((rows, heads)).astype(np.float32)
    want = np.stack([O.sink_softmax_attention(q[:, h], k[:, h // (heads // kv_heads)], v[:, h // (heads // kv_heads)], dim ** -0.5, float(sinks[h]), start)
                     for h in range(heads)], 1) * O.sigmoid(gates.astype(np.float64))[..., None]
    qp, kp, vp = np.zeros((rows, heads, dq)), np.zeros((cap, kv_heads, dq)), np.zeros((cap, kv_heads * dv))
    qp[..., :dim], kp[:T, :, :dim] = q, k
    vp.reshape(cap, kv_heads, dv)[:T, :, :vdim] = v
    blocks = np.zeros((cap // 32, kv_heads * dv, 32))
    from test_gpu_mixers import block_order
    blocks[:, :, block_order()] = vp.reshape(cap // 32, 32, kv_heads * dv).transpose(0, 2, 1)
    out, pos, batch = empty(ai, ctx, rows * heads * vdim, dt), ai.Buffer.from_slice(ctx, np.array([start], np.uint32)), ai.CommandBatch(ctx)
    print(f"attention with sink {dtype} {heads} {kv_heads} {dim} {vdim} {start} {rows}", flush=True)
    K.attention_rows_into(batch, upload(ai, ctx, qp, dt), upload(ai, ctx, kp, dt), upload(ai, ctx, blocks, dt), out, dt, pos, start, rows, heads, kv_heads, 1, dim, vdim,
                          cap, dim ** -0.5, sink=f32(ai, ctx, sinks), gate=f32(ai, ctx, gates))
    batch.commit_and_wait()
    close(download(ai, out, rows * heads * vdim, dt).reshape(rows, heads, vdim), want, F32_TOL if dt == ai.F32 else BF16_TOL)


# ---- selective state space --------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("heads,vdim,state,groups,taps", [(1, 3, 5, 1, 1), (4, 24, 20, 2, 4), (3, 33, 64, 3, 2), (2, 64, 128, 1, 3), (6, 16, 130, 2, 6), (2, 20, 300, 1, 4), (2, 8, 12, 1, 20)])
@pytest.mark.parametrize("cuts", [[1, 1, 1, 1, 1], [2, 2, 1, 2], [17, 1, 65, 2, 130], [63, 1, 64, 1], [200]])
def test_selective_state_space(ai, gpu, heads, vdim, state, groups, taps, cuts):
    """The kernels from the projections to the recurrence's output, in portions, and the states left behind: all f32, and bf16
    through the chunked and the recurrent form.  One row goes through the fused step in f32."""
    ctx, K = gpu
    g, T = np.random.default_rng(state + sum(cuts)), sum(cuts)
    inner, n = heads * vdim, groups * state
    ch, dq = inner + 2 * n, K.linear_attention_padded_dim(state)
    w, bias = g.standard_normal((ch, taps)).astype(np.float32).astype(np.float64), g.standard_normal(ch).astype(np.float32).astype(np.float64)
    dt_bias, a_log, D = np.linspace(-6, 1, heads), np.linspace(2.5, -3, heads), g.standard_normal(heads)
    dt_bias, a_log, D = (v.astype(np.float32).astype(np.float64) for v in (dt_bias, a_log, D))
    dt_raw = g.standard_normal((T, heads)).astype(np.float32)
    wb, bb = f32(ai, ctx, w.T), f32(ai, ctx, bias)
    head_args = [f32(ai, ctx, v) for v in (dt_bias, a_log, D)]
    for dt, chunked in ((ai.F32, False), (ai.BF16, False), (ai.BF16, True)):
        if chunked and state > 256:
            continue
        print(f"selective {heads} {vdim} {state} {groups} {taps} {cuts} dtype {dt} chunked {chunked}", flush=True)
        u = stored(g.standard_normal((T, ch)), ai, dt)
        ring, memory = ai.Buffer.empty(ctx, taps * ch * 4), ai.Buffer.empty(ctx, heads * vdim * dq * 4)
        past, S, at = np.zeros((taps - 1, ch)), None, 0
        for rows in cuts:
            part = slice(at, at + rows)
            pos, batch = ai.Buffer.from_slice(ctx, np.array([at], np.uint32)), ai.CommandBatch(ctx)
            o, db = empty(ai, ctx, rows * inner, ai.F32), f32(ai, ctx, dt_raw[part])
            c, past = O.causal_conv(u[part], past, w, bias)
            c = O.silu(c)
            if rows == 1:
                K.selective_step_into(batch, f32(ai, ctx, u[part]), ring, wb, bb, pos, db, *head_args, memory, o, heads, vdim, groups, state, taps)
            else:
                x, B, C = (upload(ai, ctx, np.full(s, 9.0), dt) for s in ((rows, inner), (rows, groups, dq), (rows, groups, dq)))
                K.selective_conv_into(batch, upload(ai, ctx, u[part], dt), dt, ring, wb, bb, pos, x, B, C, rows, heads, vdim, groups, state, taps)
                if chunked:
                    steps, work = ai.Buffer.empty(ctx, K.selective_steps_bytes(rows, heads)), ai.Buffer.empty(ctx, K.linear_attention_workspace_bytes(rows, heads, state, vdim))
                    K.selective_chunked_into(batch, x, B, C, db, *head_args, memory, steps, work, o, rows, heads, vdim, groups, state)
                else:
                    K.selective_recurrent_into(batch, x, B, C, dt, db, *head_args, memory, o, rows, heads, vdim, groups, state)
            batch.commit_and_wait()
            if rows > 1:
                got = [download(ai, x, rows * inner, dt)] + [download(ai, b, rows * groups * dq, dt).reshape(rows, groups, dq) for b in (B, C)]
                close(np.concatenate([got[0].reshape(rows, -1)] + [b[..., :state].reshape(rows, -1) for b in got[1:]], 1), c, F32_TOL if dt == ai.F32 else BF16_TOL, "convolution")
                assert not any(b[..., state:].any() for b in got[1:])
                if dt == ai.BF16:                    # the recurrence is judged on what it was given
                    c = np.concatenate([got[0].reshape(rows, -1)] + [b[..., :state].reshape(rows, -1) for b in got[1:]], 1).astype(np.float64)
            y, S = O.selective_recurrence(c[:, :inner].reshape(rows, heads, vdim), c[:, inner:inner + n].reshape(rows, groups, state), c[:, inner + n:].reshape(rows, groups, state),
                                          O.softplus(dt_raw[part].astype(np.float64) + dt_bias), a_log, D, S)
            close(download(ai, o, rows * inner, ai.F32).reshape(rows, heads, vdim), y, F32_TOL, f"rows {part}")
            close(memory.as_array(np.float32).reshape(heads, vdim, dq)[..., :state].transpose(0, 2, 1), S, F32_TOL, f"state after {at + rows}")
            at += rows
            kept = ring.as_array(np.float32).reshape(taps, ch)
            for p in range(max(0, at - taps + 1), at):
                assert np.array_equal(kept[p % taps], u[p].astype(np.float32)), p


# ---- linear attention with scaled keys ----------------------------------------------------------------------------------------
def test_linear_attention_scale(ai, gpu):
    ctx, K = gpu
    g, H, d, e, T = np.random.default_rng(1), 2, 32, 40, 100
    q, k, v = (M.rounded(g.standard_normal(s)) for s in ((T, H, d), (T, H, d), (T, H, e)))
    decay = np.array([0.9, 0.99])
    want, _ = O.lightning_recurrence(q, k * 0.3, v, decay)
    qb, kb, vb = (upload(ai, ctx, x, ai.BF16) for x in (q, k, v))
    pw, db = f32(ai, ctx, decay[:, None] ** np.arange(65)), f32(ai, ctx, decay)
    batch, outs, states = ai.CommandBatch(ctx), [empty(ai, ctx, T * H * e, ai.F32) for _ in range(2)], [ai.Buffer.empty(ctx, H * e * d * 4) for _ in range(2)]
    work = ai.Buffer.empty(ctx, K.linear_attention_workspace_bytes(T, H, d, e))
    K.linear_attention_chunked_into(batch, qb, kb, vb, states[0], pw, work, outs[0], T, H, d, e, 0.3)
    K.linear_attention_recurrent_into(batch, qb, kb, vb, ai.BF16, states[1], db, outs[1], T, H, d, e, 0.3)
    batch.commit_and_wait()
    for o in outs:
        close(download(ai, o, T * H * e, ai.F32).reshape(T, H, e), want, F32_TOL)


# ---- norms with gates, norms behind the branches, gated products ------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("dim,group", [(6, 3), (64, 8), (96, 32), (288, 144), (512, 64), (1024, 1024), (1536, 512), (4096, 1024), (2048, 16), (5000, 1250), (1200, 48), (4104, 4104)])
@pytest.mark.parametrize("weight,act,first", [(True, "silu", True), (False, "silu", False), (True, "sigmoid", False)])
def test_gated_norm_in_parts(ai, gpu, dtype, dim, group, weight, act, first):
    ctx, K = gpu
    dt, g, eps, rows = ai.BF16 if dtype == "bf16" else ai.F32, np.random.default_rng(dim + group), 1e-3, 3
    x, z, w = g.standard_normal((rows, dim)).astype(np.float32), stored(g.standard_normal((rows, dim)), ai, dt), g.standard_normal(dim).astype(np.float32)
    x[1] *= np.repeat(np.linspace(0.05, 20, dim // group), group)           # parts of very different size
    f, code = (O.silu, ai.ACT_SILU) if act == "silu" else (O.sigmoid, ai.ACT_SIGMOID)
    u = x.astype(np.float64)
    u = O.unit_rms((u * f(z) if first else u).reshape(rows, -1, group), eps).reshape(rows, dim) * (w if weight else 1.0) * (1.0 if first else f(z))
    xb, zb, wb, out, batch = f32(ai, ctx, x), upload(ai, ctx, z, dt), f32(ai, ctx, w) if weight else None, empty(ai, ctx, rows * dim, dt), ai.CommandBatch(ctx)
    K.gated_norm_rows_into(batch, xb, zb, wb, out, dt, dim, rows, eps, group, code, first)
    batch.commit_and_wait()
    tol = F32_TOL if dt == ai.F32 else BF16_TOL
    close(download(ai, out, rows * dim, dt).reshape(rows, dim), u, tol)
    assert K.gated_vector_fits(dim, group) == (group == dim or (dim <= 4096 and group % 8 == 0 and (group % 512 == 0 or group // 8 in (1, 2, 4, 8, 16, 32))))
    m = M.rounded(g.standard_normal((20, dim)) / np.sqrt(dim))
    lin, y = ai.linear_weight.StackedLinear(ctx, [M.bf16_bits(m)], [ai.linear_weight.Segment(20)]), empty(ai, ctx, 20, ai.F32)
    for i in range(rows):
        xi, zi = f32(ai, ctx, x[i]), upload(ai, ctx, z[i], dt)

        def product():
            K.linear_gated_vector_into(batch, xi, zi, dt, wb, eps, lin.weight, None, dim, lin.segments, [y], ai.F32, group=group, gate_act=code, gate_first=first)
        if not K.gated_vector_fits(dim, group):
            with pytest.raises(ai.InvalidArgument):
                product()
            continue
        product()
        batch.commit_and_wait()
        close(download(ai, y, 20, ai.F32), u[i] @ m.T, F32_TOL, f"product of row {i}")


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("dim", [30, 64, 320, 1000, 4096, 4100, 5001])
def test_norm_behind_a_branch(ai, gpu, dtype, dim):
    ctx, K = gpu
    dt, g, eps, rows = ai.BF16 if dtype == "bf16" else ai.F32, np.random.default_rng(dim), 1e-4, 5
    x, y, w = (g.standard_normal(s).astype(np.float32) for s in ((rows, dim), (rows, dim), (dim,)))
    want = x + O.unit_rms(y.astype(np.float64), eps) * w
    xb, yb, wb, out, batch = f32(ai, ctx, x), f32(ai, ctx, y), f32(ai, ctx, w), empty(ai, ctx, rows * dim, dt), ai.CommandBatch(ctx)
    m = M.rounded(g.standard_normal((37, dim)) / np.sqrt(dim))
    lin, L = ai.linear_weight.StackedLinear(ctx, [M.bf16_bits(m)], [ai.linear_weight.Segment(37)]), ai.linear_weight
    p, s = empty(ai, ctx, 37, ai.F32), empty(ai, ctx, dim, ai.F32)
    lin.residual_vector_into(batch, K, xb, yb, s, wb, eps, [p], ai.F32)
    batch.commit_and_wait()
    close(download(ai, p, 37, ai.F32), want[0] @ m.T, F32_TOL, "product")
    close(download(ai, s, dim, ai.F32), want[0], F32_TOL, "stream")
    with pytest.raises(ai.InvalidArgument):
        lin.residual_vector_into(batch, K, xb, yb, xb, wb, eps, [p], ai.F32)
    K.residual_rows_into(batch, xb, None, None, None, out, dt, dim, rows, eps)
    batch.commit_and_wait()
    assert np.array_equal(download(ai, out, rows * dim, dt).reshape(rows, dim), stored(x, ai, dt).astype(np.float32))
    K.residual_rows_into(batch, xb, yb, wb, xb, out, dt, dim, rows, eps)
    batch.commit_and_wait()
    close(download(ai, xb, rows * dim, ai.F32).reshape(rows, dim), want, F32_TOL, "rows")
    close(download(ai, out, rows * dim, dt).reshape(rows, dim), want, F32_TOL if dt == ai.F32 else BF16_TOL, "copy")


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("m,k,n", [(2, 64, 24), (65, 40, 33), (130, 128, 256), (7, 13, 5), (300, 512, 1000)])
def test_gate_and_up_in_one_product(ai, gpu, dtype, m, k, n):
    ctx, K = gpu
    dt, g, L = ai.BF16 if dtype == "bf16" else ai.F32, np.random.default_rng(m + n), ai.linear_weight
    x, a, b = stored(g.standard_normal((m, k)), ai, dt), *(M.rounded(g.standard_normal((n, k)) / np.sqrt(k)) for _ in range(2))
    want = O.silu(x @ a.T) * (x @ b.T)
    both = M.bf16_bits(np.stack([a, b], 1).reshape(2 * n, k))
    lin, h, batch = L.StackedLinear(ctx, [both], [L.Segment(2 * n, ai.ACT_SILU_PAIRS)]), empty(ai, ctx, m * n, dt), ai.CommandBatch(ctx)
    lin.rows_into(batch, K, upload(ai, ctx, x, dt), dt, m, [h], dt)
    batch.commit_and_wait()
    close(download(ai, h, m * n, dt).reshape(m, n), want, F32_TOL if dt == ai.F32 else BF16_TOL)


@pytest.mark.parametrize("dtype", ["bf16", "f32"])
@pytest.mark.parametrize("k,n", [(64, 1), (13, 5), (512, 33), (2048, 3000), (4096, 70), (4100, 40), (5000, 1500), (16384, 9), (20008, 17)])
def test_gate_and_up_of_one_row(ai, gpu, dtype, k, n):
    ctx, K = gpu
    g, L, dt = np.random.default_rng(n), ai.linear_weight, ai.BF16 if dtype == "bf16" else ai.F32
    x, a, b = stored(g.standard_normal(k), ai, dt), *(M.rounded(g.standard_normal((n, k)) / np.sqrt(k)) for _ in range(2))
    y, w, s = g.standard_normal(k).astype(np.float32), np.ones(k, np.float32), empty(ai, ctx, k, ai.F32)
    lin = L.StackedLinear(ctx, [M.bf16_bits(np.stack([a, b], 1).reshape(2 * n, k))], [L.Segment(2 * n, ai.ACT_SILU_PAIRS)])
    outs, batch = [empty(ai, ctx, n, ai.F32), empty(ai, ctx, n, ai.BF16), empty(ai, ctx, n, ai.F32)], ai.CommandBatch(ctx)
    xb = upload(ai, ctx, x, dt)
    lin.vector_into(batch, K, xb, dt, [outs[0]], ai.F32)
    lin.vector_into(batch, K, xb, dt, [outs[1]], ai.BF16)
    lin.residual_vector_into(batch, K, f32(ai, ctx, x), f32(ai, ctx, y), s, f32(ai, ctx, w), 1e-5, [outs[2]], ai.F32)
    batch.commit_and_wait()
    want = O.silu(a @ x) * (b @ x)
    close(download(ai, outs[0], n, ai.F32), want, F32_TOL)
    close(download(ai, outs[1], n, ai.BF16), want, BF16_TOL)
    x = x + O.unit_rms(y.astype(np.float64), 1e-5)
    close(download(ai, outs[2], n, ai.F32), O.silu(a @ x) * (b @ x), F32_TOL, "behind a normed branch")


def test_pairs_stand_alone_in_a_product_of_one_row(ai, gpu):
    ctx, K = gpu
    L, b, batch = ai.linear_weight, ai.Buffer.empty(ctx, 4096), ai.CommandBatch(ctx)
    with pytest.raises(ai.InvalidArgument):
        K.linear_vector_into(batch, b, ai.F32, b, None, 8, L.Segments([L.Segment(8, ai.ACT_SILU_PAIRS), L.Segment(8)]), [b, b], ai.F32)
    with pytest.raises(ai.InvalidArgument):
        K.linear_vector_into(batch, b, ai.F32, b, None, 8, L.Segments([L.Segment(7, ai.ACT_SILU_PAIRS)]), [b], ai.F32)


def test_destinations_of_mixed_types(ai, gpu):
    """bf16 and f32 destinations of one product, with padded heads."""
    ctx, K = gpu
    g, L = np.random.default_rng(2), ai.linear_weight
    for m, heads in ((1, 3), (5, 3), (70, 8)):
        x, w = M.rounded(g.standard_normal((m, 64))), M.rounded(g.standard_normal((heads * 12 + 20, 64)) / 8)
        lin = L.StackedLinear(ctx, [M.bf16_bits(w[:heads * 12]), M.bf16_bits(w[heads * 12:])], [L.Segment(heads * 12, head=12, padded=16), L.Segment(20, layout=ai.ROWS_F32)])
        a, b, batch = empty(ai, ctx, m * heads * 16, ai.BF16), empty(ai, ctx, m * 20, ai.F32), ai.CommandBatch(ctx)
        xb = upload(ai, ctx, x, ai.BF16)
        if m == 1:
            lin.vector_into(batch, K, xb, ai.BF16, [a, b], ai.BF16)
        else:
            lin.rows_into(batch, K, xb, ai.BF16, m, [a, b], ai.BF16)
        batch.commit_and_wait()
        want = x @ w.T
        close(download(ai, a, m * heads * 16, ai.BF16).reshape(m, heads, 16)[..., :12], want[:, :heads * 12].reshape(m, heads, 12), BF16_TOL)
        close(download(ai, b, m * 20, ai.F32).reshape(m, 20), want[:, heads * 12:], F32_TOL)


def test_softcap(ai, gpu):
    ctx, K = gpu
    x = np.linspace(-200, 200, 1037).astype(np.float32)
    b, batch = f32(ai, ctx, x), ai.CommandBatch(ctx)
    K.softcap_f32_into(batch, b, x.size, 15.5)
    batch.commit_and_wait()
    close(download(ai, b, x.size, ai.F32), O.softcap(x.astype(np.float64), 15.5), 1e-6)
    with pytest.raises(ai.InvalidArgument):
        K.softcap_f32_into(batch, b, x.size, 0.0)
