"""Dafolorn on the GPU: every kernel against a plain evaluation, and the model through the engine's own scheduler, cache, state
and step function against oracle/dafolorn_oracle.py."""
import types

import pytest
import torch

from dafolorn_util import CONFIGS, LIMIT, config, distance, layer, make_model, run_cut, session, tokens
from oracle import dafolorn_oracle as O

pytestmark = [pytest.mark.gpu, pytest.mark.timeout(120)]
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def g(seed):
    return torch.Generator().manual_seed(seed)


def dev(t, dtype=None):
    return t.to("cuda", dtype) if dtype else t.to("cuda")


def i32(x):
    return torch.as_tensor(x, dtype=torch.int32, device="cuda")


# ---- kernels --------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("M,N,K", [(1, 40, 72), (3, 104, 264), (40, 520, 96), (100, 264, 136), (200, 72, 128), (300, 512, 1024)])
def test_linear_act(dtype, M, N, K):
    from nanovllm import hip_ops
    dt = DT[dtype]
    x, w, b = torch.randn(M, K, generator=g(1)).to(dt), (torch.randn(N, K, generator=g(2)) * K ** -0.5).to(dt), torch.randn(N, generator=g(3)).to(dt)
    z = x.double() @ w.double().T + b.double()
    p, q = torch.tensor(0.3).double(), torch.tensor(-0.8).double()
    xi = (hip_ops.ACT_XIELU, float(O.softplus(p)), float(0.5 + O.softplus(q)))
    for act, ref in ((hip_ops.NO_ACT, z), (xi, O.xielu(z, p, q)), ((hip_ops.ACT_SOFTCAP, 1.5, 0.0), O.soft_cap(z, 1.5))):
        for f32 in (False, True):
            y = hip_ops.linear_act(dev(x), dev(w), dev(b), act, out_f32=f32)
            tol = 2e-5 if y.dtype == torch.float32 else 1e-2
            assert torch.allclose(y.cpu().double(), ref, rtol=tol, atol=tol), (act[0], f32)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [72, 76, 1040])
def test_embed_rows(dtype, width):
    from nanovllm import hip_ops
    wp = hip_ops.round8(width)
    table = torch.randn(50, width, generator=g(1)).to(DT[dtype])
    ids = torch.tensor([3, 49, 0, 3, 17])
    cat = torch.full((5, 2 * wp), 7.0, dtype=DT[dtype], device="cuda")
    x = hip_ops.embed_rows(dev(ids), dev(table), wp, cat[:, wp:]).cpu()
    assert torch.equal(x[:, :width], table[ids].float()) and torch.all(x[:, width:] == 0)
    assert torch.equal(cat[:, wp:].cpu().float(), x) and torch.all(cat[:, :wp] == 7)


def _portions(lens_per_step):
    """Steps of (sequence, start, length) -> metadata of glm_seq_norm."""
    at, par, steps = {}, {}, []
    for step in lens_per_step:
        pos, seq_of, qs, sin, sout = [], [], [0], [], []
        for s, (seq, n) in enumerate(step):
            a = at.get(seq, 0)
            pos += range(a, a + n)
            seq_of += [s] * n
            qs.append(qs[-1] + n)
            p = par.get(seq, 0)
            sin.append(2 * seq + p)
            sout.append(2 * seq + 1 - p)
            at[seq], par[seq] = a + n, 1 - p
        steps.append((step, types.SimpleNamespace(pos=i32(pos), seq_of=i32(seq_of), q_start=i32(qs), state_in=i32(sin), state_out=i32(sout))))
    return steps


@pytest.mark.parametrize("width,taps", [(64, 2), (76, 3), (200, 4), (1032, 5), (72, 8), (64, 13)])
@pytest.mark.parametrize("y_kind", ["none", "bf16", "f32", "slabs"])
def test_seq_norm(width, taps, y_kind):
    from nanovllm import hip_ops
    wp, tp, eps = hip_ops.round8(width), hip_ops.seq_norm_taps(taps), 1e-5
    L = {0: 700, 1: 41, 2: 9}
    pad = lambda t: torch.nn.functional.pad(t, (0, wp - width))  # noqa: E731
    x = {s: torch.randn(n, width, generator=g(s)) for s, n in L.items()}
    y = {s: torch.randn(n, width, generator=g(10 + s)).to(torch.bfloat16).float() for s, n in L.items()}
    gp, gq = 1 + 0.2 * torch.randn(width, generator=g(20)), 1 + 0.2 * torch.randn(width, generator=g(21))
    cw = torch.randn(width, taps, generator=g(22)).to(torch.bfloat16).float()
    conv = torch.zeros(tp, wp)
    conv[tp - taps:, :width] = cw.T
    ref_x = {s: (x[s].double() + O.unit_rms(y[s].double(), eps) * gp.double()) if y_kind != "none" else x[s].double() for s in L}
    ref_h = {s: O.canon(O.unit_rms(ref_x[s], eps) * gq.double(), cw.double()) for s in L}
    plans = [[[(0, 700), (1, 41), (2, 9)]],
             [[(0, 530), (1, 1)], [(1, 1), (0, 2), (2, 1)], [(1, 1), (2, 2)], [(0, 168), (2, 6), (1, 38)]],
             [[(2, 1)], [(2, 1), (1, 17)], [(1, 24), (2, 1)], [(2, 1)], [(2, 5), (0, 1)], [(0, 699)]]]
    outs = []
    for plan in plans:
        state = torch.full((6, max(tp - 1, 1), wp), float("nan"), device="cuda")
        at, got_h, got_x = {s: 0 for s in L}, {s: [] for s in L}, {s: [] for s in L}
        for step, meta in _portions(plan):
            cut = lambda t: torch.cat([pad(t[s][at[s]: at[s] + n]) for s, n in step])  # noqa: E731
            xs, ys = dev(cut(x)), cut(y)
            yk = {"none": None, "bf16": dev(ys, torch.bfloat16), "f32": dev(ys),
                  "slabs": hip_ops.PartialSum(dev(torch.stack([ys * 0.25, ys * 0.75])))}[y_kind]
            xo, h = hip_ops.seq_norm(xs, width, eps, y=yk, g_post=dev(pad(gp)), g_pre=dev(pad(gq)), conv=(dev(conv, torch.bfloat16), state), meta=meta,
                                     act_dtype=torch.float32)
            assert torch.all(h[:, width:] == 0)
            r = 0
            for s, n in step:
                got_h[s].append(h[r: r + n, :width].cpu())
                got_x[s].append(xo[r: r + n, :width].cpu())
                r, at[s] = r + n, at[s] + n
        got_h = {s: torch.cat(v) for s, v in got_h.items()}
        for s in L:
            n = got_h[s].shape[0]
            assert torch.allclose(got_h[s].double(), ref_h[s][:n], rtol=1e-5, atol=2e-5), s
            assert torch.allclose(torch.cat(got_x[s]).double(), ref_x[s][:n], rtol=1e-5, atol=1e-5)
        outs.append(got_h)
    for s in L:   # however the sequence was cut: beyond the order of a row's sum nothing may differ
        for o in outs[1:]:
            assert torch.allclose(o[s], outs[0][s][: o[s].shape[0]], rtol=1e-6, atol=2e-6)


def _paged(rows, bs, n_blocks, seed):
    """Latent rows of several sequences scattered over pages; unused memory is NaN."""
    perm = torch.randperm(n_blocks, generator=g(seed)).tolist()
    cache = torch.full((n_blocks, bs, rows[0].shape[1]), float("nan"))
    width = max(-(-r.shape[0] // bs) for r in rows)
    bt = torch.full((len(rows), width), -1, dtype=torch.int32)
    for s, r in enumerate(rows):
        for b in range(-(-r.shape[0] // bs)):
            bt[s, b] = perm.pop()
            part = r[b * bs: (b + 1) * bs]
            cache[bt[s, b], : part.shape[0]] = part
    return cache, bt


def _standout(q, c, t, h, j, gain=40.0):
    """Make key j the one that row (t, h) sees, if it sees it: its score stands out by `gain`."""
    c[j] = q[t, h] / q[t, h].norm() ** 2 * gain


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,rank,vdim,window,bs", [(6, 40, 24, 50, 64), (1, 264, 72, 1, 32), (2, 64, 16, 100, 32), (32, 512, 128, 300, 64), (70, 24, 8, 33, 256),
                                                   (16, 1000, 40, 64, 64), (40, 576, 16, 129, 64)])
@pytest.mark.parametrize("n_q,splits", [(1, 0), (1, 1), (1, 5), (2, 0), (37, 3)])
def test_latent_attn(dtype, H, rank, vdim, window, bs, n_q, splits):
    from nanovllm import hip_ops
    dt, rp, S = DT[dtype], hip_ops.round8(rank), 4
    lens = [n_q, window + n_q + 70, window + n_q, 2 * bs + n_q]
    c = [torch.zeros(n, rp) for n in lens]
    for s, n in enumerate(lens):
        c[s][:, :rank] = torch.randn(n, rank, generator=g(s))
    q = torch.zeros(S, n_q, H, rp)
    q[..., :rank] = torch.randn(S, n_q, H, rank, generator=g(9)) * 0.5
    # a key just inside and one just outside the window of a row each, one at a page border
    for s, n in enumerate(lens):
        p = n - 1
        for h, j in ((0, p - window + 1), (H - 1, p - window), (H // 2, (p // bs) * bs)):
            if 0 <= j < n and (h == 0 or H > 2):
                _standout(q[s], c[s], n_q - 1, h, j)
    q, c = q.to(dt), [x.to(dt) for x in c]
    wuv = (torch.randn(H, vdim, rp, generator=g(5)) * rank ** -0.5).to(dt)
    wuv[..., rank:] = 0
    sink = torch.randn(H, generator=g(6)) * 2
    cache, bt = _paged([x.float() for x in c], bs, 64 if bs < 256 else 16, 7)
    pos = torch.cat([torch.arange(n - n_q, n) for n in lens])
    seq_of = torch.arange(S).repeat_interleave(n_q)
    tpt = min(hip_ops.latent_tokens_per_tile(rp, H), n_q)
    tok = [s * n_q + k for s in range(S) for k in range(0, n_q, tpt)]
    cnt = [min(tpt, n_q - k) for s in range(S) for k in range(0, n_q, tpt)]
    out = torch.full((S * n_q, H * vdim), float("nan"), dtype=dt, device="cuda")
    hip_ops.latent_attn(dev(q.reshape(S * n_q, H, rp)), dev(cache, dt), i32(tok), i32(cnt), tpt, i32(pos), i32(seq_of), i32(bt), window, 1.0,
                        dev(sink), dev(wuv), out, num_splits=splits)
    got = out.cpu().double().view(S, n_q, H, vdim)
    for s, n in enumerate(lens):
        vis = O.window_mask(n, window)[n - n_q:]
        for h in range(0, H, max(1, H // 5)):
            a = O.sink_softmax(q[s, :, h].double() @ c[s].double().T, vis, sink[h].double())
            ref = a @ c[s].double() @ wuv[h].double().T
            tol = 5e-5 if dtype == "float32" else 2e-2
            err = (got[s, :, h] - ref).abs().max() / max(1.0, float(ref.abs().max()))
            assert err < tol, (s, h, float(err))


@pytest.mark.parametrize("H,dk,dv,window", [(3, 24, 40, 50), (2, 128, 128, 200), (1, 136, 200, 1), (4, 64, 256, 64), (2, 200, 64, 1000), (2, 256, 256, 129)])
def test_window_attn_prefill(H, dk, dv, window):
    from nanovllm import hip_ops
    lens, hist = [300, 2, 129, 64], [0, min(window - 1, 77), window - 1, min(3, window - 1)]
    ks = [0]
    for n, h in zip(lens, hist):
        ks.append(ks[-1] + n + h)
    qs = [0]
    for n in lens:
        qs.append(qs[-1] + n)
    q = torch.randn(qs[-1], H, dk, generator=g(1)) * 0.7
    k, v = torch.randn(ks[-1], H, dk, generator=g(2)) * 0.7, torch.randn(ks[-1], H, dv, generator=g(3))
    for s in range(len(lens)):   # keys that stand out: just inside the window of the last row, just outside, the first key
        i = hist[s] + lens[s] - 1
        for h, j in ((0, i - window + 1), (H - 1, i - window), (H - 1, 0)):
            if 0 <= j:
                k[ks[s] + j, h] = q[qs[s + 1] - 1, h] / q[qs[s + 1] - 1, h].norm() ** 2 * 30
    q, k, v = (t.to(torch.bfloat16) for t in (q, k, v))
    sink = torch.randn(H, generator=g(4)) * 2
    tiles = [(s, o) for s, n in enumerate(lens) for o in range(0, n, 128)]
    kv = torch.cat([k.reshape(ks[-1], -1), v.reshape(ks[-1], -1)], 1).cuda()
    out = torch.full((qs[-1], H * dv), float("nan"), dtype=torch.bfloat16, device="cuda")
    hip_ops.window_attn_prefill(dev(q.reshape(qs[-1], -1)), kv[:, : H * dk], kv[:, H * dk:], out, i32(qs), i32(ks), i32([t[0] for t in tiles]),
                                i32([t[1] for t in tiles]), H, dk, dv, window, 1.0, dev(sink))
    got = out.cpu().double().view(-1, H, dv)
    for s, n in enumerate(lens):
        vis = O.window_mask(n + hist[s], window)[hist[s]:]
        for h in range(H):
            a = O.sink_softmax(q[qs[s]: qs[s + 1], h].double() @ k[ks[s]: ks[s + 1], h].double().T, vis, sink[h].double())
            ref = a @ v[ks[s]: ks[s + 1], h].double()
            assert (got[qs[s]: qs[s + 1], h] - ref).abs().max() < 4e-2, (s, h)


# ---- the model through the engine -------------------------------------------------------------------------------------------
@pytest.fixture(scope="module", params=list(CONFIGS))
def model(request, tmp_path_factory):
    path = tmp_path_factory.mktemp(request.param)
    cfg, t = make_model(path, request.param, seed=len(request.param))
    toks = tokens(cfg, 420, 3)
    return types.SimpleNamespace(name=request.param, path=path, cfg=cfg, t=t, toks=toks, ref=O.forward(cfg, t, toks))


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
        assert len(tap) == len(ref) == len(r.model.runs)
        for i, (a, b) in enumerate(zip(tap, ref)):
            assert distance(a.cpu(), b) < LIMIT[dtype], f"layer run {i}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_against_cuts(model, dtype):
    """A whole prompt, portions of many sizes down to two tokens, token-by-token decoding: the same logits, at every position.
    Pages and slots are used again by every run."""
    with session(model.path, dtype, 448) as s:
        for cuts in ([420], [200, 1], [37, 64, 2, 2, 3, 130, 5, 1, 1, 40], [1, 2, 2, 17, 64, 1, 1, 96, 2, 33], [129]):
            assert distance(run_cut(s, model.toks, cuts), model.ref) < LIMIT[dtype], cuts


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_batches(model, dtype):
    """Up to four live requests, portions beside single tokens, requests that pause, end and make room for others."""
    ref = {n: O.forward(model.cfg, model.t, model.toks[o: o + n]) for n, o in ((1, 5), (23, 11), (150, 100), (97, 200), (260, 0), (61, 300))}
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
        o = torch.cat(got[n])
        assert distance(o, ref[n][: o.shape[0]]) < LIMIT[dtype], n


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_graphs_and_eager(dtype, tmp_path):
    """Hundreds of decoded tokens: windows pass over decoded tokens and page borders, pages behind the windows are given back;
    the captured step replays between other work and equals the eager one."""
    cfg = config(64, 96, 4, [layer(4, 16, 24, 40, 70, 72), layer(3, 24, 16, 56, 5, 72)], (0, 2, 2), 10.0)
    cfg, t = make_model(tmp_path, cfg, 1)
    toks = tokens(cfg, 330, 2)
    ref = O.forward(cfg, t, toks)
    outs = []
    for eager in (True, False):
        with session(tmp_path, dtype, 192, eager=eager) as s:   # fewer pages than tokens: 330 tokens need the windows' trimming
            outs.append(run_cut(s, toks, [9, 1]))
            assert s.engine.model_runner.step_graphs if not eager else True
    assert distance(outs[0], ref) < LIMIT[dtype] and distance(outs[1], ref) < LIMIT[dtype]
    assert torch.equal(outs[0], outs[1])


def test_tiny_changes_show(model):
    """A window one token longer or shorter, a sink left out, a lost convolution input, a missing pass vector: planted in the
    plain evaluation, each is far outside the limit the other tests use."""
    import copy
    ref = model.ref[:200]
    for i in range(len(model.cfg["layers"])):
        for d in (-1, 1):
            c = copy.deepcopy(model.cfg)
            c["layers"][i]["mixer"]["mask"]["size"] += d
            if 0 < c["layers"][i]["mixer"]["mask"]["size"] < 190:
                assert distance(O.forward(c, model.t, model.toks[:200]), ref) > 10 * LIMIT["float32"], (i, d)
    for name, edit in (("l0.mix.sink", lambda v: v - 30), ("l0.canon1", lambda v: torch.cat([torch.zeros_like(v[:, :1]), v[:, 1:]], 1)),
                       ("l0.mlp.act", lambda v: v.flip(0))):
        t = dict(model.t)
        t[name] = edit(t[name])
        assert distance(O.forward(model.cfg, t, model.toks[:200]), ref) > 10 * LIMIT["float32"], name


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
    cfg, t = make_model(tmp_path, "tail", 5)
    llm = LLM(str(tmp_path), max_num_seqs=5, max_num_batched_tokens=256, max_model_len=256, gpu_memory_utilization=0.05)
    try:
        assert llm.config.num_kvcache_blocks > 1000
        a, b = (llm.generate([tokens(cfg, 20, 1)], SamplingParams(temperature=x, max_tokens=24, ignore_eos=True), use_tqdm=False)[0]["token_ids"]
                for x in (0.0, 50.0))
        assert len(a) == len(b) == 24 and a != b
    finally:
        llm.exit()
    torch.cuda.empty_cache()
