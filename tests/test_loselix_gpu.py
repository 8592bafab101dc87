"""Loselix on the GPU: every kernel against a plain evaluation, and the model through the engine's own scheduler, cache and step function
against oracle/loselix_oracle.py."""
import copy
import math
import types

import pytest
import torch

from loselix_util import CONFIGS, LIMIT, Reference, config, distance, gated, make_model, run_cut, session, sigmoid, tokens, two_maps
from oracle import loselix_oracle as O

pytestmark = [pytest.mark.gpu, pytest.mark.timeout(120)]
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def g(seed):
    return torch.Generator().manual_seed(seed)


def dev(t, dtype=None):
    return t.to("cuda", dtype) if dtype else t.to("cuda")


def i32(x):
    return torch.as_tensor(x, dtype=torch.int32, device="cuda")


def close(a, b, tol):
    return torch.allclose(a.cpu().double(), b.double(), rtol=tol, atol=tol)


# ---- kernels --------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("M,N,K", [(1, 40, 72), (1, 1032, 264), (3, 104, 264), (16, 64, 64), (40, 520, 96), (200, 72, 128), (300, 512, 1024)])
def test_columns_of_a_joint_projection(dtype, M, N, K):
    """Square of relu, plain columns, sigmoid, in one projection, into a part of wider rows."""
    from nanovllm import hip_ops
    dt, tol = DT[dtype], 2e-5 if dtype == "float32" else 1.5e-2
    x, w = torch.randn(M, K, generator=g(1)).to(dt), (torch.randn(N, K, generator=g(2)) * 1.5 * K ** -0.5).to(dt)
    z = x.double() @ w.double().T
    for a, b in ((0, 8), (8, 24), (24, N), (N, N), (16, 1 << 24), (0, 0)):
        want = torch.cat([O.relu_squared(z[:, :a]), z[:, a: b], O.sigmoid(z[:, min(max(a, b), N):])], 1)
        rows = torch.full((M, N + 24), 7.0, dtype=dt, device="cuda")
        hip_ops.linear_act(dev(x), dev(w), act=(hip_ops.ACT_RELU2_GATE, float(a), float(b)), out=rows[:, 16: 16 + N])
        assert close(rows[:, 16: 16 + N], want, tol), (a, b)
        assert torch.all(rows[:, :16] == 7) and torch.all(rows[:, 16 + N:] == 7)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [72, 75, 520, 1040, 2056, 4100, 8200])
def test_residual_norm(dtype, width):
    from nanovllm import hip_ops
    dt, wp, eps, tol = DT[dtype], hip_ops.round8(width), 1e-3, 2e-5 if dtype == "float32" else 1e-2
    pad = lambda t: torch.nn.functional.pad(t, (0, wp - width))  # noqa: E731
    for T in (1, 5, 41) if width < 8000 else (3,):
        x, y, gain = pad(torch.randn(T, width, generator=g(1))), pad(torch.randn(T, width, generator=g(2)) * 2), pad(1 + 0.2 * torch.randn(width, generator=g(3)))
        table, ids = pad(torch.randn(30, width, generator=g(4))).to(dt), torch.randint(0, 30, (T,), generator=g(5))
        slabs, rows = torch.randn(3, T, wp, generator=g(6)), torch.randint(0, T, (7,), generator=g(7))
        slabs[..., width:] = 0
        dy = dev(y, dt)
        for xx in (x, None):
            for kind in ("none", "rows", "f32", "slabs"):
                for emb in (False, True):
                    if xx is None and not emb:
                        continue
                    yk = {"none": None, "rows": dy, "f32": dev(y), "slabs": hip_ops.PartialSum(dev(slabs))}[kind]
                    s = torch.zeros(T, wp, dtype=torch.float64) if xx is None else xx.double()
                    s = s + {"none": 0, "rows": dy.cpu().double(), "f32": y.double(), "slabs": slabs.double().sum(0)}[kind] + (table[ids].double() if emb else 0)
                    n = O.norm_plain(s[:, :width], gain[:width].double(), eps)
                    args = dict(y=yk, embed=(dev(ids), dev(table)) if emb else None, act_dtype=dt)
                    xd = dev(xx) if xx is not None else None
                    xo, h = hip_ops.residual_norm(xd, width, wp, eps, g=dev(gain), **args)
                    assert xo.dtype == torch.float32 and h.dtype == dt and close(xo, s, 2e-6) and close(h[:, :width], n, tol) and torch.all(h[:, width:] == 0), (T, kind, emb)
                    assert torch.equal(hip_ops.residual_norm(xd, width, wp, eps, **args)[0], xo)
                    if xx is not None:
                        none, hr = hip_ops.residual_norm(xd, width, wp, eps, g=dev(gain), rows=i32(rows), keep_x=False, **args)
                        assert none is None and torch.equal(hr, h[dev(rows)])


def test_residual_norm_many_rows():
    """The form for long prompts (the residual past the caches) gives what the one for few rows does."""
    from nanovllm import hip_ops
    for w in (64, 1000, 1400, 3000):
        x, y, gain = torch.randn(2100, w, device="cuda"), torch.randn(2100, w, device="cuda").to(torch.bfloat16), torch.rand(w, device="cuda")
        a = hip_ops.residual_norm(x, w, w, 1e-5, y=y, g=gain)
        b = [hip_ops.residual_norm(x[i: i + 700], w, w, 1e-5, y=y[i: i + 700], g=gain) for i in (0, 700, 1400)]
        for k in (0, 1):
            assert torch.allclose(a[k].float(), torch.cat([p[k] for p in b]).float(), rtol=1e-6 if k == 0 else 1e-2, atol=1e-6)


@pytest.mark.parametrize("M,N,K", [(97, 264, 1024), (128, 2048, 4096), (200, 520, 2048), (300, 1032, 8192), (500, 64, 1536)])
def test_slices_of_k(M, N, K):
    """Partial sums of a projection of some hundred rows, out of a part of wider rows: as many slices as the chip has room for, and given numbers."""
    from nanovllm import hip_ops
    rows = torch.randn(M, K + 72, generator=g(1)).to(torch.bfloat16)
    w = (torch.randn(N, K, generator=g(2)) * K ** -0.5).to(torch.bfloat16)
    want = rows[:, 8: 8 + K].double() @ w.double().T
    assert hip_ops.gemm_slices(M, N, K) > 1 and hip_ops.gemm_slices(40, N, K) == 1 and hip_ops.gemm_slices(M, N, K + 8) == 1 and hip_ops.gemm_slices(16384, 4096, K) == 1
    for ns in {hip_ops.gemm_slices(M, N, K), 2, 4, 8}:
        part = hip_ops.gemm_bf16_partial(dev(rows)[:, 8: 8 + K], dev(w), ns).part
        assert part.shape == (ns, M, N) and close(part.sum(0), want, 1e-4), ns
        k = K // ns
        assert close(part[1], rows[:, 8 + k: 8 + 2 * k].double() @ w[:, k: 2 * k].double().T, 1e-4)


def test_rotation_far_positions():
    from nanovllm.layers.rotary_embedding import HalfRotary
    rot = HalfRotary(40, 20, 500000.0)
    rot.prepare(torch.device("cuda", 0))
    pos = [0, 1, 4095, 1000003, 200000001, -1]
    cs = rot.table(i32(pos)).cpu().double()
    for r, p in enumerate(pos[:5]):
        a = torch.tensor([p * 500000.0 ** (-2 * i / 20) for i in range(10)], dtype=torch.float64)
        assert torch.allclose(cs[r, :, 0], torch.cos(a), atol=3e-7) and torch.allclose(cs[r, :, 1], torch.sin(a), atol=3e-7)
    tables = {}
    assert rot.shared_table(i32(pos), tables) is HalfRotary(40, 20, 500000.0).shared_table(i32(pos), tables)


def _slots(T, bs, n_blocks):
    s = torch.randperm(n_blocks * bs, generator=g(3))[:T]
    s[T // 2] = -1
    return s


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,maps,dm,dv,dims", [(6, 2, 1, 24, 40, 4), (4, 4, 2, 32, 16, 32), (8, 1, 1, 128, 128, 64), (2, 2, 2, 40, 8, 14), (3, 1, 1, 8, 72, 2), (5, 5, 2, 64, 64, 48)])
@pytest.mark.parametrize("T", [1, 37, 2111])
def test_group_rotate_store(dtype, H, G, maps, dm, dv, dims, T):
    from nanovllm import hip_ops
    from nanovllm.layers.rotary_embedding import HalfRotary
    dt, bs = DT[dtype], 64
    nb = -(-T // bs) + 2
    q_off, k_off, v_off = 8, 16 + H * maps * dm, 16 + (H + G) * maps * dm + 24
    x = torch.randn(T, v_off + G * dv + 16, generator=g(1)).to(dt)
    rot = HalfRotary(dm, dims, 300.0)
    rot.prepare(torch.device("cuda", 0))
    pos, slots = torch.randint(0, 5000, (T,), generator=g(2)), _slots(T, bs, nb)
    kc, vc = (torch.zeros(nb, G, bs, d, dtype=dt, device="cuda") for d in (maps * dm, dv))
    xd = dev(x).clone()
    hip_ops.group_rotate_store(xd, q_off, k_off, v_off, H, maps, dims, rot.table(i32(pos)), i32(slots), kc, vc)

    def turned(t):     # [T, heads, dm], row by row at its own position
        a = pos.double()[:, None, None] * torch.tensor([300.0 ** (-2 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
        u, v = t[..., : dims // 2].double(), t[..., dims // 2: dims].double()
        return torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin(), t[..., dims:].double()], -1)

    tol = 1e-5 if dtype == "float32" else 1.6e-2
    q = x[:, q_off: q_off + H * maps * dm].view(T, H * maps, dm)
    got = xd.cpu()
    assert close(got[:, q_off: q_off + H * maps * dm].view(T, H * maps, dm), turned(q), tol)
    rest = torch.ones(x.shape[1], dtype=torch.bool)
    for h in range(H * maps):
        rest[q_off + h * dm: q_off + h * dm + dims] = False
    assert torch.equal(got[:, rest], x[:, rest])     # nothing but the queries' rotated columns changes
    k = turned(x[:, k_off: k_off + G * maps * dm].view(T, G * maps, dm)).view(T, G, maps * dm)
    v = x[:, v_off: v_off + G * dv].view(T, G, dv)
    ok = slots >= 0
    ek, ev = torch.zeros(kc.shape, dtype=torch.float64), torch.zeros(vc.shape, dtype=dt)
    ek[slots[ok] // bs, :, slots[ok] % bs], ev[slots[ok] // bs, :, slots[ok] % bs] = k[ok], v[ok]
    assert close(kc, ek, tol) and torch.equal(vc.cpu(), ev)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,dim", [(6, 2, 20), (4, 4, 128), (70, 1, 40), (40, 4, 128), (3, 3, 264), (70, 10, 128)])
@pytest.mark.parametrize("first,count", [(0, None), (1, 1)])
def test_group_norm_store(dtype, H, G, dim, first, count):
    """Norms over the whole projection; the raw keys (all heads, or one of them) and 1 / rms of the whole key row are kept."""
    from nanovllm import hip_ops
    if first + (count or G) > G:
        pytest.skip("one key head")
    dt, bs, T, nb, dp, eps = DT[dtype], 64, 45, 3, hip_ops.round8(dim), 1e-2
    n_kept = count or G
    pad = lambda t: torch.nn.functional.pad(t, (0, dp - dim)).reshape(T, -1)  # noqa: E731
    q, k = (torch.randn(T, n, dim, generator=g(i)).to(dt) * (1 + torch.arange(T).view(-1, 1, 1) % 5).to(dt) for i, n in ((1, H), (2, G)))
    x = torch.cat([torch.ones(T, 8).to(dt), pad(q), torch.ones(T, 16).to(dt), pad(k), torch.ones(T, 8).to(dt)], 1)
    q_off, k_off = 8, 24 + H * dp
    gain = torch.nn.functional.pad(1 + 0.3 * torch.randn(H, dim, generator=g(4)), (0, dp - dim)).reshape(-1)
    pos, slots = torch.randint(0, 700, (T,), generator=g(5)), _slots(T, bs, nb)
    for coef, every in ((0.0, 0), (0.6, 1), (0.3, 50)):
        cache, ks = torch.zeros(nb, n_kept, bs, dp, dtype=dt, device="cuda"), torch.zeros(nb, bs, device="cuda")
        xd = dev(x).clone()
        hip_ops.group_norm_store(xd, q_off, k_off, dev(gain), H * dim, G * dp, G * dim, first, eps, i32(pos), i32(slots), cache, ks, (coef, every))
        temp = 1 + coef * torch.log((pos + 1).div(max(every, 1), rounding_mode="floor").double() + 1) if every else torch.ones(T).double()
        want = O.unit_rms(q.double().reshape(T, -1), eps).view(T, H, dim) * gain.view(H, dp)[:, :dim].double() * temp[:, None, None]
        got = xd.cpu()
        assert close(got[:, q_off: q_off + H * dp].view(T, H, dp)[..., :dim], want, 2e-5 if dtype == "float32" else 2e-2)
        keep = torch.ones(x.shape[1], dtype=torch.bool)
        keep[q_off: q_off + H * dp] = False
        assert torch.equal(got[:, keep], x[:, keep])
        ok = slots >= 0
        ek, es = torch.zeros(cache.shape, dtype=dt), torch.zeros(nb, bs, dtype=torch.float64)
        ek[slots[ok] // bs, :, slots[ok] % bs] = torch.nn.functional.pad(k, (0, dp - dim))[ok][:, first: first + n_kept]
        es[slots[ok] // bs, slots[ok] % bs] = 1 / torch.sqrt(k.double().reshape(T, -1).pow(2).mean(-1) + eps)[ok]
        assert torch.equal(cache.cpu(), ek) and close(ks, es, 1e-6)


def _paged(rows, G, bs, n_blocks, perm, fill=float("nan")):
    """[T, G, d] of several sequences scattered over the blocks `perm`; unused memory is NaN."""
    cache = torch.full((n_blocks, G, bs, rows[0].shape[2]), fill)
    bt = torch.full((len(rows), max(-(-r.shape[0] // bs) for r in rows)), -1, dtype=torch.int32)
    it = iter(perm)
    for s, r in enumerate(rows):
        for b in range(-(-r.shape[0] // bs)):
            bt[s, b] = next(it)
            part = r[b * bs: (b + 1) * bs]
            cache[bt[s, b], :, : part.shape[0]] = part.transpose(0, 1)
    return cache, bt


FORMS = [("two_maps", 6, 2, 24, 40, 64), ("two_maps", 4, 4, 64, 128, 64), ("two_maps", 12, 1, 128, 256, 128), ("two_maps", 2, 2, 8, 8, 64), ("two_maps", 5, 1, 72, 64, 192),
         ("two_maps", 3, 1, 32, 200, 64), ("two_maps_70", 6, 2, 24, 40, 64), ("two_maps_70", 4, 1, 64, 128, 64), ("two_maps_0", 4, 2, 40, 72, 64),
         ("sigmoid", 6, 2, 24, 24, 64), ("sigmoid", 20, 1, 128, 128, 64), ("sigmoid", 3, 3, 200, 200, 128), ("sigmoid", 8, 2, 64, 64, 64),
         ("softmax", 6, 3, 40, 72, 64), ("softmax", 17, 1, 128, 64, 64)]


@pytest.mark.parametrize("form,H,G,dim,dv,bs", FORMS)
@pytest.mark.parametrize("kind", ["decode1", "decode1_split", "decode5", "prefill", "plain", "plain_f32"])
def test_group_attention_forms(form, H, G, dim, dv, bs, kind):
    """Two maps with a soft cap that scores come near, a high one, none; sigmoid weights over keys that are the values, a softmax without sinks; gates per head, per column, none.  Pages in
    disorder, NaNs wherever nothing was stored; single keys that stand out: the first one, those at page borders, the row's own."""
    from nanovllm import hip_ops
    dtype = "float32" if kind == "plain_f32" else "bfloat16"
    form, cap = (form[:8], float(form[9:] or 20)) if form.startswith("two_maps") else (form, 0.0)
    dt, R, maps = DT[dtype], H // G, 2 if form == "two_maps" else 1
    r = lambda t: t.to(dt).float()  # noqa: E731
    if kind.startswith("decode1"):
        lens, n_q = [1, 65, 128, 257, 321], [1] * 5
    elif kind == "decode5":
        lens, n_q = [5, 66, 129, 2, 130], [5, 5, 3, 2, 4]
    else:
        lens, n_q = [300, 190, 257, 2, 64], [300, 60, 129, 2, 64]
    k = [torch.randn(n, G, maps, dim, generator=g(s)) * 0.7 for s, n in enumerate(lens)]
    v = [torch.randn(n, G, dv, generator=g(50 + s)) for s, n in enumerate(lens)]
    q = [torch.randn(m, H, maps, dim, generator=g(90 + s)) * 0.7 for s, m in enumerate(n_q)]
    scale, lam, post, eps = 0.9, 0.4, 0.6, 1e-3
    for s, n in enumerate(lens):
        for h, j in ((0, 0), (H - 1, (n - 1) // 64 * 64), (H // 2, (n - 1) // 64 * 64 - 1), (H // 3, n - 1)):
            if 0 <= j < n:
                for m in range(maps):
                    a = q[s][-1, h, m]
                    k[s][j, h // R, m] = a / a.norm() ** 2 * (18 + 3 * m)
    q, k, v = [r(t) for t in q], [r(t) for t in k], [r(t) for t in v]
    ks = [0.5 + torch.rand(n, 1, 1, generator=g(30 + s)) for s, n in enumerate(lens)]
    if form == "sigmoid":
        v = [t[:, :, 0] for t in k]
    perm = torch.randperm(40, generator=g(7)).tolist()
    kc, bt = _paged([t.reshape(t.shape[0], G, maps * dim) for t in k], G, bs, 40, perm)
    vc, _ = _paged(v, G, bs, 40, perm)
    sc, _ = _paged(ks, 1, bs, 40, perm)
    T, bias = sum(n_q), -2 + torch.randn(H, generator=g(5))
    pos = i32(torch.cat([torch.arange(n - m, n) for n, m in zip(lens, n_q)]))
    seq_of = i32(torch.arange(len(lens)).repeat_interleave(torch.tensor(n_q)))
    qs = [0]
    for m in n_q:
        qs.append(qs[-1] + m)
    dq, dk = dev(torch.cat(q).reshape(T, -1), dt), dev(kc, dt)
    dvc = dk if form == "sigmoid" else dev(vc, dt)
    gates = torch.rand(T, H * dv + 8, generator=g(11)).to(dt)
    for gate in (None, "head", "column"):
        parts = hip_ops.GroupParts(maps=maps, gate=None if gate is None else dev(gates), gate_cols=gate == "column")
        if form == "two_maps":
            parts.cap, parts.lam, parts.post, parts.eps, parts.vn = cap, lam, post, eps, dv
        if form == "sigmoid":
            parts.sigmoid, parts.bias, parts.kscale = True, dev(bias), dev(sc).view(40, bs)
        wide = torch.full((T, H * dv + 16), float("nan"), dtype=dt, device="cuda")
        out = wide[:, 8: 8 + H * dv]
        args, shape = (dq, dk, dvc, i32(bt)), (H, 0, 0, scale, None, None)
        if kind == "prefill":
            tiles = [(s, o) for s, n in enumerate(n_q) for o in range(0, n, hip_ops.group_attn_tile_rows(H, G, maps))]
            tables = torch.full((3 + bt.shape[0], bt.shape[1]), -1, dtype=torch.int32)
            tables[3:] = bt       # portions whose block tables are not the first rows
            hip_ops.group_attn_prefill(*args[:3], i32(tables), 3, i32(qs), pos, i32([t[0] for t in tiles]), i32([t[1] for t in tiles]), *shape, out, parts=parts)
        elif kind.startswith("plain"):
            hip_ops.group_attn_plain(*args, pos, seq_of, *shape, out, parts=parts)
        else:
            per = max(1, min(max(n_q), hip_ops.group_attn_rows(maps) // R))
            tok = [qs[s] + o for s, n in enumerate(n_q) for o in range(0, n, per)]
            cnt = [min(per, n - o) for n in n_q for o in range(0, n, per)]
            hip_ops.group_attn_decode(*args, pos, seq_of, i32(tok), i32(cnt), per, *shape, out, num_splits=7 if kind == "decode1_split" else 1, parts=parts)
        assert torch.isnan(wide[:, :8]).all() and torch.isnan(wide[:, 8 + H * dv:]).all()
        got = out.cpu().double().view(T, H, dv)
        for s, n in enumerate(lens):
            m0, visible = n_q[s], O.causal(n)[n - n_q[s]:]
            for h in range(H):
                res = []
                for m in range(maps):
                    z = (q[s][:, h, m].double() @ k[s][:, h // R, m].double().T) * scale
                    if form == "sigmoid":
                        a = O.sigmoid(z * ks[s][:, 0, 0].double() + bias[h].double()) * visible
                    else:
                        z = (O.soft_cap(z, cap) if cap else z).masked_fill(~visible, -math.inf)
                        a = torch.softmax(z, -1)
                    res.append(a @ v[s][:, h // R].double())
                want = res[0] if maps == 1 else O.unit_rms(res[0] - lam * res[1], eps) * post
                gt = gates[qs[s]: qs[s] + m0].double()
                want = want * (1 if gate is None else gt[:, h: h + 1] if gate == "head" else gt[:, h * dv: (h + 1) * dv])
                size = max(1.0, float(want.abs().max()))
                err = float((got[qs[s]: qs[s] + m0, h] - want).abs().max()) / size
                assert err < (5e-5 if dtype == "float32" else 3e-2), (gate, s, h, err)


# ---- the model through the engine -------------------------------------------------------------------------------------------
@pytest.fixture(scope="module", params=list(CONFIGS))
def model(request, tmp_path_factory):
    path = tmp_path_factory.mktemp(request.param)
    cfg, t = make_model(path, request.param, seed=len(request.param))
    toks = tokens(cfg, 420, 3)
    return types.SimpleNamespace(name=request.param, path=path, cfg=cfg, t=t, toks=toks, ref=Reference(cfg, t, toks))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers(model, dtype):
    """The residual stream after every layer run of one prompt."""
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
        assert len(tap) == len(ref) == len(O.layer_order(model.cfg))
        moved = [[], [], []]
        for k in range(3):
            O.forward(model.cfg, model.t, model.toks[:150], layers_out=moved[k], noise=k)
        for i, (a, b) in enumerate(zip(tap, ref)):
            limit = LIMIT[dtype] if dtype == "float32" else max(LIMIT[dtype], 4 * max(distance(m[i], b) for m in moved))
            assert distance(a.cpu(), b) < limit, f"layer run {i}"


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
    """Hundreds of decoded tokens over page borders; the captured step replays between other work and gives what the eager one does (in bf16 up to
    the rounding of another number of key splits)."""
    cfg = config(64, 96, [gated(4, 2, 16, 24, 40, dims=16), sigmoid(4, 2, 24, 72), two_maps(4, 2, 16, 24, None, dims=8)], (0, 2, 2))
    cfg, t = make_model(tmp_path, cfg, 1)
    toks = tokens(cfg, 330, 2)
    ref = Reference(cfg, t, toks)
    outs = []
    for eager in (True, False):
        with session(tmp_path, dtype, 384, eager=eager) as s:
            outs.append(run_cut(s, toks, [9, 1]))
            assert s.engine.model_runner.step_graphs if not eager else True
        ref.check(outs[-1], dtype, eager)
    if dtype == "float32":
        assert torch.equal(outs[0], outs[1])


@pytest.mark.parametrize("kind", ["two_maps", "gated", "sigmoid"])
def test_far_keys_show(tmp_path, kind):
    """One attention layer and a query that stands out for ONE key: the first token, keys at page borders, far and near ones.  Through prefill and
    through decoding, against the plain evaluation, where leaving the key out moves the logits far."""
    layer = {"two_maps": two_maps(2, 1, 64, 64, None, dims=8, cap=50.0, scale=1.0), "gated": gated(2, 1, 64, 64, None, dims=8, scale=1.0), "sigmoid": sigmoid(2, 1, 64, None, scale=0.2)}[kind]
    cfg = config(64, 64, [layer])
    t = O.random_tensors(cfg, 4)
    for w in ("q", "k"):
        t[f"l0.mix.{w}"] = t[f"l0.mix.{w}"] * 0.1
    # one input direction marks a key, one a query; both meet in a column of every head that does not turn
    t["embed"][60], t["embed"][61] = torch.zeros(64), torch.zeros(64)
    t["embed"][:, 40:42] = 0
    t["embed"][60, 40], t["embed"][61, 41] = 9.0, 9.0
    t["l0.norm1"] = torch.ones_like(t["l0.norm1"])
    t["l0.mix.q"].view(-1, 64, 64)[:, 30, 41], t["l0.mix.k"].view(-1, 64, 64)[:, 30, 40] = 0.9, 0.9
    if kind == "sigmoid":
        t["l0.mix.pb"] = torch.full((2,), -9.0, dtype=torch.bfloat16)
    O.write_model(str(tmp_path), cfg, t)
    base = [int(x) % 60 for x in tokens(cfg, 400, 9)]
    for key, query in ((0, 399), (63, 64), (64, 383), (127, 257), (0, 128), (255, 256), (319, 398)):
        toks = list(base)
        toks[key], toks[query] = 60, 61
        ref = Reference(cfg, t, toks)
        without = list(base)
        without[query] = 61
        assert distance(O.forward(cfg, t, without)[query: query + 1], ref.logits[query: query + 1]) > 0.1, (key, query)
        for dtype in ("float32", "bfloat16"):
            with session(tmp_path, dtype, 448) as s:
                ref.check(run_cut(s, toks, [400]), dtype, (key, query))
                ref.check(run_cut(s, toks, [query - 1 if query > 1 else 1, 1, 1, 2, 30]), dtype, (key, query))


def test_tiny_changes_show(model):
    """Faults planted in the plain evaluation are far outside the limit the other tests use."""
    ref, T = model.ref.logits[:120], 120
    toks = model.toks[:T]

    def differs(cfg, t):
        return distance(O.forward(cfg, t, toks), ref) > 10 * LIMIT["float32"]

    def edited(i, path, f):
        c = copy.deepcopy(model.cfg)
        m = c["layers"][i]["mixer"]
        for k in path[:-1]:
            m = m[k]
        m[path[-1]] = f(m[path[-1]])
        return c

    for i, e in enumerate(model.cfg["layers"]):
        changes = [(("scale",), lambda v: v * 1.02)]
        if "rot" in e["mixer"] and e["mixer"]["rot"]["dims"] > 2:
            changes += [(("rot", "dims"), lambda v: v - 2), (("rot", "base"), lambda v: v * 1.5)]
        if e["type"] == "attention":
            changes += [(("diff",), lambda v: v + 0.02), (("softcap",), lambda v: v * 0.9)]
        if e["type"] == "attention_3":
            changes += [(("q_temp", "coef"), lambda v: v * 1.2), (("q_temp", "every"), lambda v: v + 1)]
        for path, f in changes:
            assert differs(edited(i, path, f), model.t), (i, path)
        edits = [("norm1", lambda v: v * 1.05), ("mix.lq1", lambda v: v * 0), ("mix.lk2", lambda v: v + 0.5), ("mix.pb", lambda v: v + 0.1), ("mix.g", lambda v: v * 0),
                 ("mix.q.norm", lambda v: v.flip(0)), ("mix.k.norm", lambda v: v.flip(0))]
        for name, edit in edits:
            if f"l{i}.{name}" in model.t:
                t = dict(model.t)
                t[f"l{i}.{name}"] = edit(t[f"l{i}.{name}"].float()).to(torch.bfloat16)
                assert differs(model.cfg, t), (i, name)
    if model.cfg["loop"] and model.cfg["loop"]["times"] > 1:
        for k, d in (("times", -1), ("times", 1)):
            c = copy.deepcopy(model.cfg)
            c["loop"][k] += d
            assert differs(c, model.t), k


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


def test_memory_sized_pool_and_sampling(tmp_path):
    """Without a given pool the engine sizes it by memory; temperatures above zero sample."""
    from nanovllm import LLM, SamplingParams
    cfg, t = make_model(tmp_path, "odd", 5)
    free = torch.cuda.mem_get_info()
    used = 1 - free[0] / free[1]
    llm = LLM(str(tmp_path), max_num_seqs=5, max_num_batched_tokens=256, max_model_len=256, gpu_memory_utilization=min(0.9, used + 0.05))
    try:
        assert llm.config.num_kvcache_blocks >= 1000
        a, b = (llm.generate([tokens(cfg, 20, 1)], SamplingParams(temperature=x, max_tokens=24, ignore_eos=True), use_tqdm=False)[0]["token_ids"]
                for x in (0.0, 50.0))
        assert len(a) == len(b) == 24 and a != b
    finally:
        llm.exit()
    torch.cuda.empty_cache()
