"""Napadra on the GPU: every kernel against a plain evaluation, and the model through the engine's own scheduler, cache, state
and step function against oracle/napadra_oracle.py."""
import copy
import math
import types

import pytest
import torch

from napadra_util import CONFIGS, LIMIT, Reference, attn, config, distance, make_model, mlstm, run_cut, session, tokens
from oracle import napadra_oracle as O

pytestmark = [pytest.mark.gpu, pytest.mark.timeout(120)]
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def g(seed):
    return torch.Generator().manual_seed(seed)


def dev(t, dtype=None):
    return t.to("cuda", dtype) if dtype else t.to("cuda")


def i32(x):
    return torch.as_tensor(x, dtype=torch.int32, device="cuda")


def padc(t, n):
    return torch.nn.functional.pad(t, (0, n - t.shape[-1]))


# ---- kernels --------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("M,N,K", [(1, 40, 72), (1, 1032, 264), (3, 104, 264), (16, 64, 64), (40, 520, 96), (100, 264, 136), (200, 72, 128), (300, 512, 1024)])
def test_gated_glu(dtype, M, N, K):
    from nanovllm import hip_ops
    dt = DT[dtype]
    x, w = torch.randn(M, K, generator=g(1)).to(dt), (torch.randn(2 * N, K, generator=g(2)) * 1.5 * K ** -0.5).to(dt)
    z = x.double() @ w.double().T
    for limit in (0.8, 1.9, 50.0):     # the clamps cut most, some, none of the values
        y = hip_ops.gated_glu(dev(x), dev(w), limit)
        assert y.dtype == dt
        tol = 2e-5 if dtype == "float32" else 1e-2
        assert torch.allclose(y.cpu().double(), O.clamped_glu(z[:, :N], z[:, N:], limit), rtol=tol, atol=tol), limit


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [72, 75, 1040])
def test_embed_rows_with_positions(dtype, width):
    from nanovllm import hip_ops
    wp = hip_ops.round8(width)
    table = torch.randn(50, width, generator=g(1)).to(DT[dtype])
    ids, pos = torch.tensor([3, 49, 0, 3, 17, 9]), [0, 1, 77, 4095, 1000003, -1]
    i = torch.arange(wp // 2, dtype=torch.float64)
    x = hip_ops.embed_rows(dev(ids), dev(table), wp, pos=i32(pos), freq=dev(10000.0 ** (-2 * i / width))).cpu()
    for r, p in enumerate(pos[:5]):
        want = torch.tensor([(math.sin if j % 2 == 0 else math.cos)(p * 10000.0 ** (-2 * (j // 2) / width)) for j in range(width)]).double()
        assert torch.allclose(x[r, :width].double(), table[ids[r]].double() + want, atol=1e-6, rtol=1e-6), p
    assert torch.all(x[:, width:] == 0) and torch.isfinite(x).all()


def _portions(plan):
    """Steps of (sequence, length) -> the step's metadata."""
    at, par, steps = {}, {}, []
    for step in plan:
        pos, seq_of, qs, sin, sout = [], [], [0], [], []
        for s, (seq, n) in enumerate(step):
            a, p = at.get(seq, 0), par.get(seq, 0)
            pos += range(a, a + n)
            seq_of += [s] * n
            qs.append(qs[-1] + n)
            sin.append(2 * seq + p)
            sout.append(2 * seq + 1 - p)
            at[seq], par[seq] = a + n, 1 - p
        steps.append((step, types.SimpleNamespace(pos=i32(pos), seq_of=i32(seq_of), q_start=i32(qs), state_in=i32(sin), state_out=i32(sout))))
    return steps


PLANS = [[[(0, 700), (1, 41), (2, 9)]],
         [[(0, 530), (1, 1)], [(1, 1), (0, 2), (2, 1)], [(1, 1), (2, 2)], [(0, 168), (2, 6), (1, 38)]],
         [[(2, 1)], [(2, 1), (1, 17)], [(1, 24), (2, 1)], [(2, 1)], [(2, 5), (0, 1)], [(0, 699)]]]


@pytest.mark.parametrize("width,S", [(64, 1), (76, 2), (200, 3), (1032, 4), (72, 5), (64, 6), (2056, 2), (40, 8), (136, 7), (8200, 2), (4104, 4)])
@pytest.mark.parametrize("y_kind", ["none", "bf16", "f32"])
def test_stream_norm(width, S, y_kind):
    from nanovllm import hip_ops
    wp, eps, gain = hip_ops.round8(width), 1e-4, 1.7
    L = {0: 700, 1: 41, 2: 9} if width < 4000 else {0: 40, 1: 17, 2: 9}
    plans = PLANS if width < 4000 else [[[(0, 40), (1, 17), (2, 9)]], [[(0, 1), (2, 2)], [(2, 7), (0, 38), (1, 1)], [(1, 16), (0, 1)]]]
    x = {s: torch.randn(n, S, width, generator=g(s)) for s, n in L.items()}
    y = {s: torch.randn(n, width, generator=g(10 + s)).to(torch.bfloat16).float() for s, n in L.items()}
    ys, sh = 1 + 0.3 * torch.randn(width, generator=g(20)), torch.randn(width, generator=g(21))
    mix, wo, wi = (torch.randn(*s, generator=g(22 + i)) for i, s in enumerate(((S, S), (S,), (S,))))
    mo = torch.cat([mix.flatten(), wo])
    ref_x, ref_h, plain_h = {}, {}, {}
    for s in L:
        ref_x[s] = x[s].double() if y_kind == "none" else O.spread(x[s].double(), mix.double(), wo.double(), ys.double() * y[s].double())
        plain_h[s] = O.unit_rms(O.collapse(ref_x[s], wi.double()), eps) * gain
        ref_h[s] = O.token_shift(plain_h[s], sh.double())
    form = dict(y_scale=dev(padc(ys, wp)), mix_out=dev(mo), w_in=dev(wi), gain=gain, act_dtype=torch.float32)
    outs = []
    for plan in plans:
        state = torch.full((6, wp), float("nan"), device="cuda")
        at, got_h, got_x = {s: 0 for s in L}, {s: [] for s in L}, {s: [] for s in L}
        for step, meta in _portions(plan):
            cut = lambda t: torch.cat([padc(t[s][at[s]: at[s] + n], wp) for s, n in step])  # noqa: E731
            yk = {"none": None, "bf16": dev(cut(y), torch.bfloat16), "f32": dev(cut(y))}[y_kind]
            xs = dev(cut(x))
            xo, h = hip_ops.stream_norm(xs, S, width, eps, y=yk, shift=dev(padc(sh, wp)), state=state, meta=meta, **form)
            if len(plan) == 1:      # without the shift; gathered rows; streams alone
                xo2, h2 = hip_ops.stream_norm(xs, S, width, eps, y=yk, **form)
                assert torch.allclose(h2[:, :width].cpu().double(), torch.cat([plain_h[s] for s, _ in step]), rtol=1e-5, atol=2e-5)
                rows = i32([5, 0, 5, 11])
                h3 = hip_ops.stream_norm(xs, S, width, eps, y=yk, rows=rows, **form)[1]
                assert torch.equal(h3, h2[rows.long()])
                if yk is not None:
                    assert torch.equal(hip_ops.stream_norm(xs, S, width, eps, y=yk, y_scale=form["y_scale"], mix_out=form["mix_out"])[0], xo)
                one = xs[:, 0].contiguous()   # a row that stands for all streams
                a, b = (hip_ops.stream_norm(t, S, width, eps, y=yk, **form)[1] for t in (one, one[:, None].expand(-1, S, -1).contiguous()))
                assert torch.equal(a, b)
            assert torch.all(h[:, width:] == 0)
            r = 0
            for s, n in step:
                got_h[s].append(h[r: r + n, :width].cpu())
                got_x[s].append(xo[r: r + n, :, :width].cpu())
                r, at[s] = r + n, at[s] + n
        got_h = {s: torch.cat(v) for s, v in got_h.items()}
        for s in L:
            n = got_h[s].shape[0]
            assert torch.allclose(got_h[s].double(), ref_h[s][:n], rtol=1e-5, atol=3e-5), s
            assert torch.allclose(torch.cat(got_x[s]).double(), ref_x[s][:n], rtol=1e-5, atol=2e-5)
        outs.append(got_h)
    for s in L:   # however the sequence was cut: beyond the order of a row's sum nothing may differ
        for o in outs[1:]:
            assert torch.allclose(o[s], outs[0][s][: o[s].shape[0]], rtol=1e-6, atol=2e-6)


def _paged(rows, G, bs, n_blocks, perm):
    """[T, G, d] of several sequences scattered over the blocks `perm`; unused memory is NaN."""
    cache = torch.full((n_blocks, G, bs, rows[0].shape[2]), float("nan"))
    bt = torch.full((len(rows), max(-(-r.shape[0] // bs) for r in rows)), -1, dtype=torch.int32)
    it = iter(perm)
    for s, r in enumerate(rows):
        for b in range(-(-r.shape[0] // bs)):
            bt[s, b] = next(it)
            part = r[b * bs: (b + 1) * bs]
            cache[bt[s, b], :, : part.shape[0]] = part.transpose(0, 1)
    return cache, bt


def _visible(n, window, chunk):
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    v = j <= i
    if window:
        v &= i - j < window
    if chunk:
        v &= i // chunk == j // chunk
    return v


def _attn_case(H, G, dk, dv, window, chunk, bs, lens, n_q, dtype):
    """Random q, k, v with keys that stand out just inside and outside the edges of the last row, at a page border, and far back."""
    R = H // G
    k = [torch.randn(n, G, dk, generator=g(s)) * 0.7 for s, n in enumerate(lens)]
    v = [torch.randn(n, G, dv, generator=g(50 + s)) for s, n in enumerate(lens)]
    q = [torch.randn(m, H, dk, generator=g(90 + s)) * 0.7 for s, m in enumerate(n_q)]
    for s, n in enumerate(lens):
        p = n - 1
        lo = max(p - window + 1 if window else 0, p - p % chunk if chunk else 0)
        for h, j in ((0, lo), (H - 1, lo - 1), (H // 2, (p // bs) * bs - 1), (H // 3, 0)):
            if 0 <= j < n:
                k[s][j, h // R] = q[s][-1, h] / q[s][-1, h].norm() ** 2 * (25 + 0.6 * (p - j))
    c = lambda ts: [t.to(DT[dtype]).float() for t in ts]  # noqa: E731
    return c(q), c(k), c(v)


def _attn_reference(q, k, v, window, chunk, scale, slope, sink):
    n, m = k.shape[0], q.shape[0]
    H, G = q.shape[1], k.shape[1]
    vis = _visible(n, window, chunk)[n - m:]
    dist = (torch.arange(n - m, n)[:, None] - torch.arange(n)[None, :]).double()
    out = torch.empty(m, H, v.shape[2], dtype=torch.float64)
    for h in range(H):
        s = (q[:, h].double() @ k[:, h // (H // G)].double().T) * scale - (slope[h].double() if slope is not None else 0.0) * dist
        a = O.sink_softmax(s, vis, sink[h].double() if sink is not None else torch.tensor(-1e30).double())
        out[:, h] = a @ v[:, h // (H // G)].double()
    return out


FORMS = [(6, 2, 24, 40, 0, 50, 64), (4, 4, 128, 128, 0, 200, 64), (3, 1, 136, 200, 0, 1, 64), (16, 1, 64, 256, 70, 0, 128), (2, 2, 200, 64, 0, 64, 64),
         (20, 1, 256, 256, 0, 333, 64), (8, 2, 64, 64, 100, 0, 192), (5, 5, 8, 8, 0, 0, 64), (4, 2, 256, 128, 0, 96, 64)]


@pytest.mark.parametrize("H,G,dk,dv,window,chunk,bs", FORMS)
@pytest.mark.parametrize("kind", ["decode1", "decode1_split", "decode5", "decode1_new", "decode5_new", "prefill", "plain", "plain_f32"])
def test_group_attention(H, G, dk, dv, window, chunk, bs, kind):
    """Every form over pages in disorder, with NaNs wherever nothing was stored; with bias and sink, and without."""
    from nanovllm import hip_ops
    dtype = "float32" if kind == "plain_f32" else "bfloat16"
    dt, span = DT[dtype], max(window, chunk, 90)
    if kind.startswith("decode1"):
        lens, n_q = [1, span + 1, 2 * span, span + 37, 321], [1] * 5
    elif kind.startswith("decode5"):
        lens, n_q = [5, span + 2, 2 * span + 1, 2, 130], [5, 5, 3, 2, 4]
    else:
        lens, n_q = [300, span + 60, 2 * span + 129, 2, 64], [300, 60, 129, 2, 64]
    q, k, v = _attn_case(H, G, dk, dv, window, chunk, bs, lens, n_q, dtype)
    perm = torch.randperm(40, generator=g(7)).tolist()
    kc, bt = _paged(k, G, bs, 40, perm)
    vc, _ = _paged(v, G, bs, 40, perm)
    T = sum(n_q)
    pos = i32(torch.cat([torch.arange(n - m, n) for n, m in zip(lens, n_q)]))
    seq_of = i32(torch.arange(len(lens)).repeat_interleave(torch.tensor(n_q)))
    qr = torch.cat(q).reshape(T, H * dk)
    qs = [0]
    for m in n_q:
        qs.append(qs[-1] + m)
    for slope, sink in ((torch.tensor([O.slope(h, H) for h in range(H)]), torch.randn(H, generator=g(5)) * 2), (None, torch.randn(H, generator=g(5)) * 2), (None, None)):
        out = torch.full((T, H * dv), float("nan"), dtype=dt, device="cuda")
        form = (H, window, chunk, 0.9, dev(slope) if slope is not None else None, dev(sink) if sink is not None else None)
        args = (dev(qr, dt), dev(kc, dt), dev(vc, dt), i32(bt))
        new = None
        if kind.endswith("_new"):   # the step's own keys and values are not in the cache yet: it must hold them afterwards
            rows = torch.cat([torch.cat([t[s][lens[s] - n_q[s]:].reshape(n_q[s], -1) for s in range(len(lens))]) for t in (k, v)], 1)
            slots = torch.cat([bt[s, torch.arange(n - m, n) // bs] * bs + torch.arange(n - m, n) % bs for s, (n, m) in enumerate(zip(lens, n_q))])
            for c in args[1:3]:
                c[dev(slots) // bs, :, dev(slots) % bs] = float("nan")
            rows = dev(rows, dt)
            new = (rows[:, : G * dk], rows[:, G * dk:], i32(qs), i32(slots))
        if kind == "prefill":
            tiles = [(s, o) for s, n in enumerate(n_q) for o in range(0, n, hip_ops.group_attn_tile_rows(H, G))]
            wide = torch.full((3 + bt.shape[0], bt.shape[1]), -1, dtype=torch.int32)
            wide[3:] = bt       # portions whose block tables are not the first rows
            hip_ops.group_attn_prefill(*args[:3], i32(wide), 3, i32(qs), pos, i32([t[0] for t in tiles]), i32([t[1] for t in tiles]), *form, out)
        elif kind.startswith("plain"):
            hip_ops.group_attn_plain(*args, pos, seq_of, *form, out)
        else:
            per = max(1, min(max(n_q), hip_ops.GROUP_ATTN_ROWS // (H // G)))   # (five rows of a portion may be several tiles)
            tok = [qs[s] + o for s, n in enumerate(n_q) for o in range(0, n, per)]
            cnt = [min(per, n - o) for n in n_q for o in range(0, n, per)]
            hip_ops.group_attn_decode(*args, pos, seq_of, i32(tok), i32(cnt), per, *form, out, num_splits=7 if kind == "decode1_split" else 1, new=new)
            if new is not None:
                assert torch.equal(args[1].nan_to_num(), dev(kc, dt).nan_to_num()) and torch.equal(args[2].nan_to_num(), dev(vc, dt).nan_to_num())
        got = out.cpu().double().view(T, H, dv)
        for s in range(len(lens)):
            ref = _attn_reference(q[s], k[s], v[s], window, chunk, 0.9, slope, sink)
            err = (got[qs[s]: qs[s + 1]] - ref).abs().max()
            assert err < (4e-5 if dtype == "float32" else 3e-2), (s, float(err), slope is not None, sink is not None)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_group_kv_store(dtype):
    from nanovllm import hip_ops
    G, dk, dv, bs, T = 3, 24, 40, 64, 70
    x = torch.randn(T, 16 + G * dk + 8 + G * dv, generator=g(1)).to(DT[dtype])
    kc, vc = torch.zeros(4, G, bs, dk, dtype=DT[dtype], device="cuda"), torch.zeros(4, G, bs, dv, dtype=DT[dtype], device="cuda")
    slots = torch.randperm(4 * bs, generator=g(2))[:T].tolist()
    slots[5] = -1
    hip_ops.group_kv_store(dev(x), 16, 16 + G * dk + 8, i32(slots), kc, vc)
    ek, ev = torch.zeros_like(kc).cpu(), torch.zeros_like(vc).cpu()
    for r, s in enumerate(slots):
        if s >= 0:
            ek[s // bs, :, s % bs] = x[r, 16: 16 + G * dk].view(G, dk)
            ev[s // bs, :, s % bs] = x[r, -G * dv:].view(G, dv)
    assert torch.equal(kc.cpu(), ek) and torch.equal(vc.cpu(), ev)


@pytest.mark.parametrize("H,dim,vdim,cap", [(3, 20, 44, 9.0), (2, 64, 64, 15.0), (2, 72, 136, 4.0), (1, 128, 256, 9.0), (2, 256, 72, 9.0), (1, 200, 200, 30.0), (1, 8, 328, 9.0), (1, 264, 16, 9.0)])
@pytest.mark.parametrize("form", ["recurrent_f32", "recurrent_bf16", "chunkwise"])
def test_matrix_memory(H, dim, vdim, cap, form):
    """Portions of several sequences in all sizes, slots in disorder, their state NaN until it is written.  Gates near both ends of
    their range: a memory that forgets within a token, and one that keeps its first tokens for hundreds."""
    from nanovllm import hip_ops
    if form == "chunkwise" and dim > hip_ops.MEMORY_CHUNK_MAX_DIM:
        pytest.skip("keys beyond the chunkwise kernel: such layers always go token by token")
    f32, eps, width = form == "recurrent_f32", 1e-5, 40
    dt, dimp, vdimp = torch.float32 if f32 else torch.bfloat16, hip_ops.round8(dim), hip_ops.round8(vdim)
    L = {0: 700, 1: 41, 2: 9} if form == "chunkwise" else {0: 90, 1: 41, 2: 9}
    rnd = lambda i, *s: torch.randn(*s, generator=g(i))  # noqa: E731
    r16 = lambda t: t.to(dt).float()  # noqa: E731
    q, k, v, gt = ({s: r16(rnd(100 * i + s, n, H, d) * sc) for s, n in L.items()} for i, (d, sc) in enumerate(((dim, 1), (dim, 1), (vdim, 1), (vdim, 1))))
    h = {s: r16(rnd(400 + s, n, width)) for s, n in L.items()}
    wif, bif, norm = r16(rnd(500, 2 * H, width) * 0.4), torch.cat([rnd(501, H), 6 * rnd(502, H)]), 1 + 0.2 * rnd(503, H * vdim)
    if H == 1:
        bif[1] = 30.0        # hardly forgets
    ref = {}
    for s in L:
        z = h[s].double() @ wif.double().T + bif.double()
        i, f = O.soft_cap(z[:, :H], cap), O.log_sigmoid(O.soft_cap(z[:, H:], cap))
        o = torch.stack([O.unit_rms(O.mlstm_cell(q[s][:, a].double() * dim ** -0.5, k[s][:, a].double(), v[s][:, a].double(), i[:, a], f[:, a]), eps) for a in range(H)], 1)
        ref[s] = o.reshape(len(o), -1) * norm.double() * torch.sigmoid(gt[s].reshape(len(o), -1).double())
    x = {s: torch.cat([padc(t[s], p).reshape(L[s], -1) for t, p in ((q, dimp), (k, dimp), (v, vdimp), (gt, vdimp))], 1) for s in L}
    plans = PLANS if form == "chunkwise" else [[[(0, 90), (1, 41), (2, 9)]], [[(2, 1), (0, 63)], [(0, 1), (1, 2)], [(1, 39), (2, 7), (0, 26)], [(2, 1)]]]
    normp = padc(norm.view(H, vdim), vdimp).reshape(-1)
    for plan in plans:
        state = tuple(torch.full((6, H, *s), float("nan"), device="cuda") for s in ((dimp, vdimp), (dimp,), ()))
        at, got = {s: 0 for s in L}, {s: [] for s in L}
        for step, meta in _portions(plan):
            cut = lambda t: torch.cat([t[s][at[s]: at[s] + n] for s, n in step])  # noqa: E731
            xs, T = dev(cut(x), dt), sum(n for _, n in step)
            y = torch.full((T, H * vdimp), float("nan"), dtype=dt, device="cuda")
            rows = (xs, dev(cut(h), dt), dev(wif, dt), dev(bif), dev(normp), y)
            rest = (state, meta.pos, meta.q_start, meta.state_in, meta.state_out, H, dim, vdim, cap, eps)
            if form == "chunkwise":
                tiles = [(s, o) for s, (_, n) in enumerate(step) for o in range(0, n, 128)]
                hip_ops.memory_chunkwise(*rows, *rest[:5], i32([t[0] for t in tiles]), i32([t[1] for t in tiles]), *rest[5:])
            else:
                hip_ops.memory_recurrent(*rows, *rest)
            y, r = y.cpu().double().view(T, H, vdimp), 0
            assert torch.all(y[..., vdim:] == 0)
            for s, n in step:
                got[s].append(y[r: r + n, :, :vdim].reshape(n, -1))
                r, at[s] = r + n, at[s] + n
        for s in L:
            o = torch.cat(got[s])
            err = (o - ref[s][: o.shape[0]]).abs().max()
            assert err < (1e-4 if f32 else 4e-2), (s, float(err))
            if not f32:   # rounding of the output alone, not of anything inside the recurrence
                rel = (o - ref[s][: o.shape[0]]).pow(2).mean().sqrt() / ref[s].pow(2).mean().sqrt()
                assert rel < (4e-3 if form == "chunkwise" else 2.5e-3), (s, float(rel))


# ---- the model through the engine -------------------------------------------------------------------------------------------
@pytest.fixture(scope="module", params=list(CONFIGS))
def model(request, tmp_path_factory):
    path = tmp_path_factory.mktemp(request.param)
    cfg, t = make_model(path, request.param, seed=len(request.param))
    toks = tokens(cfg, 420, 3)
    return types.SimpleNamespace(name=request.param, path=path, cfg=cfg, t=t, toks=toks, ref=Reference(cfg, t, toks))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers(model, dtype):
    """The sum of the streams after every layer of one prompt."""
    from nanovllm.engine.sequence import Sequence
    from nanovllm.engine.step_batch import build_step
    ref = []
    O.forward(model.cfg, model.t, model.toks[:150], layers_out=ref)
    with session(model.path, dtype, 192) as s:
        r, sch = s.engine.model_runner, s.scheduler
        seq = Sequence(model.toks[:150])
        host, on_device, _ = build_step([sch.feed(seq, 150, [])], r.model, r.block_size)
        tap = []
        with torch.inference_mode():
            r.model(on_device(r._to_device(host)), residual_tap=tap)
        assert len(tap) == len(ref) == len(model.cfg["layers"])
        moved = [[], [], []]
        for k in range(3):
            O.forward(model.cfg, model.t, model.toks[:150], layers_out=moved[k], noise=k)
        for i, (a, b) in enumerate(zip(tap, ref)):
            limit = LIMIT[dtype] if dtype == "float32" else max(LIMIT[dtype], 4 * max(distance(m[i], b) for m in moved))
            assert distance(a.cpu(), b) < limit, f"layer {i}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_against_cuts(model, dtype):
    """A whole prompt, portions of many sizes down to two tokens, token-by-token decoding: the same logits, at every position.
    Pages and slots are used again by every run."""
    with session(model.path, dtype, 448) as s:
        for cuts in ([420], [200, 1], [37, 64, 2, 2, 3, 130, 5, 1, 1, 40], [1, 2, 2, 17, 64, 1, 1, 96, 2, 33], [129], [16], [17]):
            model.ref.check(run_cut(s, model.toks, cuts), dtype, cuts)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_batches(model, dtype):
    """Up to four live requests, portions beside single tokens, requests that pause, end and make room for others."""
    ref = {n: Reference(model.cfg, model.t, model.toks[o: o + n]) for n, o in ((1, 5), (23, 11), (150, 100), (97, 200), (260, 0), (61, 300))}
    off = {1: 5, 23: 11, 150: 100, 97: 200, 260: 0, 61: 300}
    plan = [{260: 90, 23: 2}, {260: 1, 23: 1, 150: 80}, {150: 2, 97: 64}, {260: 130, 150: 1, 97: 1, 23: 20}, {1: 1, 260: 2, 150: 40, 97: 30},
            {61: 50, 260: 1, 150: 1, 97: 2}, {61: 1, 260: 36}, {61: 10, 150: 26}]
    at, got = {n: 0 for n in ref}, {n: [] for n in ref}
    with session(model.path, dtype, 640, eager=False) as s:
        for step in plan:
            entries, end = [], []
            for n, k in step.items():
                entries.append({"id": n, "tokens": model.toks[off[n] + at[n]: off[n] + at[n] + k], "want": list(range(k))})
                at[n] += k
                if at[n] == n:
                    end.append(n)
            out, r = s.step(entries, end), 0
            for n, k in step.items():
                got[n].append(out[r: r + k])
                r += k
        bm = s.scheduler.block_manager
        assert len(bm.free_block_ids) + sum(b >= 0 for q in s.live.values() for b in q.block_table) == 10
    for n in ref:
        ref[n].check(torch.cat(got[n]), dtype, n)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_graphs_and_eager(dtype, tmp_path):
    """Hundreds of decoded tokens: chunk edges pass over decoded tokens and page borders, pages behind the chunk are given back;
    the captured step replays between other work and equals the eager one."""
    cfg = config(64, 96, 2, [attn(4, 2, 16, 24, 70, 72), mlstm(2, 24, 16, 40), attn(4, 2, 16, 24, 5, None, kv_from=0)], 0.5)
    cfg, t = make_model(tmp_path, cfg, 1)
    toks = tokens(cfg, 330, 2)
    ref = Reference(cfg, t, toks)
    outs = []
    for eager in (True, False):
        with session(tmp_path, dtype, 192, eager=eager) as s:   # fewer pages than tokens: 330 tokens need the pages behind the chunk
            outs.append(run_cut(s, toks, [9, 1]))
            assert s.engine.model_runner.step_graphs if not eager else True
    ref.check(outs[0], dtype)
    assert torch.equal(outs[0], outs[1])


def test_far_and_edge_keys_show(tmp_path):
    """One attention layer, long chunk: a query that stands out for ONE far key (its first token), for the first key of its chunk and for
    the one in front of it.  Through prefill and through decoding, against the plain evaluation, where leaving the key
    out moves the logits far."""
    cfg = config(64, 64, 1, [attn(2, 1, 64, 64, 192, None, scale=1.0)], 1.0)
    t = O.random_tensors(cfg, 4)
    t["l0.shift"].zero_()
    t["l0.mix.q"], t["l0.mix.k"] = t["l0.mix.q"] * 0.1, t["l0.mix.k"] * 0.1
    # one input direction marks a key, one a query; both meet in the first coordinate of every head
    mark_k, mark_q = t["embed"].float()[60], t["embed"].float()[61]
    t["embed"][60], t["embed"][61] = (mark_k * 0).to(torch.bfloat16), (mark_q * 0).to(torch.bfloat16)
    t["embed"][60, 40], t["embed"][61, 41] = 60.0, 60.0
    t["l0.mix.q"][0, 41], t["l0.mix.q"][64, 41], t["l0.mix.k"][0, 40] = 4.0, 4.0, 8.0
    O.write_model(str(tmp_path), cfg, t)
    base = [int(x) % 60 for x in tokens(cfg, 400, 9)]
    for key, query in ((0, 191), (192, 383), (191, 192), (192, 192 + 64), (0, 128), (255, 256)):
        toks = list(base)
        toks[key], toks[query] = 60, 61
        ref = Reference(cfg, t, toks)
        if key // 192 == query // 192 and key + 1 != query:
            without = list(base)
            without[query] = 61
            assert distance(O.forward(cfg, t, without)[query: query + 1], ref.logits[query: query + 1]) > 0.1, (key, query)
        for dtype in ("float32", "bfloat16"):
            with session(tmp_path, dtype, 448) as s:
                ref.check(run_cut(s, toks, [400]), dtype, (key, query))
                ref.check(run_cut(s, toks, [query - 1, 1, 1, 2, 30]), dtype, (key, query))


def test_tiny_changes_show(model):
    """Faults planted in the plain evaluation are far outside the limit the other tests use: a chunk one token longer or shorter, a
    sink left out, a lost shift, a stream matrix transposed, a borrowed cache taken from the wrong place, a gate without its cap."""
    ref, T = model.ref.logits[:200], 200
    toks = model.toks[:T]

    def differs(cfg, t):
        return distance(O.forward(cfg, t, toks), ref) > 10 * LIMIT["float32"]

    for i, e in enumerate(model.cfg["layers"]):
        for d in (-1, 1) if e["type"] == "attention" else ():
            c = copy.deepcopy(model.cfg)
            c["layers"][i]["mixer"]["mask"]["size"] += d
            if 0 < c["layers"][i]["mixer"]["mask"]["size"] < T - 10:
                assert differs(c, model.t), (i, d)
        if e["type"] == "mlstm":
            c = copy.deepcopy(model.cfg)
            c["layers"][i]["mixer"]["gate_cap"] *= 1.5
            assert differs(c, model.t), i
        edits = [("shift", lambda v: v * 0), ("ls1", lambda v: v * 0 + 1), ("norm1", lambda v: v * 1.05), ("mix.sink", lambda v: v - 30),
                 ("mix.norm", lambda v: v.flip(0)), ("mix.i.b", lambda v: v + 0.3), ("hc1.out", lambda v: v * 1.05)]
        if model.cfg["streams"] > 1:
            edits.append(("hc1.mix", lambda v: v.T))
        for name, edit in edits:
            if f"l{i}.{name}" in model.t:
                t = dict(model.t)
                t[f"l{i}.{name}"] = edit(t[f"l{i}.{name}"].float()).to(torch.bfloat16)
                assert differs(model.cfg, t), (i, name)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_generate(model, dtype):
    """Greedy generation through LLM.generate: own scheduler with a token budget smaller than the prompts, more requests than
    state slots, preemption for want of pages.  A token may differ from the plain evaluation's only within its rounding."""
    from nanovllm import LLM, SamplingParams
    prompts = [tokens(model.cfg, n, 50 + n) for n in (3, 130, 61, 200, 1, 77)]
    llm = LLM(str(model.path), dtype=dtype, max_num_seqs=3, max_num_batched_tokens=96, max_model_len=512, num_kvcache_blocks=7)
    try:
        out = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True), use_tqdm=False)
        assert len(llm.scheduler.block_manager.free_block_ids) == 7 and len(llm.scheduler.state_manager.free_slots) == 3
    finally:
        llm.exit()
    torch.cuda.empty_cache()
    for p, o in zip(prompts, out):
        got = o["token_ids"]
        assert len(got) == 12
        lg = O.forward(model.cfg, model.t, p + got[:-1])[len(p) - 1:]
        gap = lg.max(-1).values - lg.gather(1, torch.tensor(got)[:, None])[:, 0]
        assert float(gap.max()) <= 6 * LIMIT[dtype] * float(lg.pow(2).mean().sqrt()), gap


@pytest.mark.parametrize("name", ["odd", "memory"])
def test_memory_sized_pool_and_sampling(tmp_path, name):
    """Without a given pool the engine sizes it by memory (or, without attention, by the sequences it may hold); temperatures above zero
    sample."""
    from nanovllm import LLM, SamplingParams
    cfg, t = make_model(tmp_path, name, 5)
    llm = LLM(str(tmp_path), max_num_seqs=5, max_num_batched_tokens=256, max_model_len=256, gpu_memory_utilization=0.05)
    try:
        assert llm.config.num_kvcache_blocks >= (1000 if name == "odd" else 20)
        a, b = (llm.generate([tokens(cfg, 20, 1)], SamplingParams(temperature=x, max_tokens=24, ignore_eos=True), use_tqdm=False)[0]["token_ids"]
                for x in (0.0, 50.0))
        assert len(a) == len(b) == 24 and a != b
    finally:
        llm.exit()
    torch.cuda.empty_cache()
