"""`python bench.py --design loselix`: prefill and decode throughput of the Loselix design at layer sizes of real models (random
weights), beside GLM-4-MoE's dense layers at equal size (same width, heads, head size, key/value heads, parameters of the feed-forward,
layer runs, vocabulary), and the time of every kernel of both against its roofline (HBM 8 TB/s, bf16 MFMA 2.5 PFLOP/s).  Prints one JSON
line per size and mode."""
from __future__ import annotations

import json
from dataclasses import replace

import torch

from bench_dafolorn import MODES, SIZES as GLM_SIZES, gemm_cost, glm_kernels, glm_model, glm_step, graph_of, kernel_table, time_us

SIZES = {size: (w, heads, heads // 4, dim, ff, vocab) for size, (w, heads, dim, _, _, ff, vocab) in GLM_SIZES.items()}
KINDS = {"attention": "differential", "attention_2": "softmax", "attention_3": "sigmoid"}
LOOP = {"start": 3, "stop": 6, "times": 2}


def loselix_config(width, heads, kv, dim, ff, vocab):
    """Twice the three kinds of attention; the second three run twice: nine layer runs, three of each kind."""
    base = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5}
    kinds = [{"type": "attention", "mixer": dict(base, dim=dim // 2, scale=(dim // 2) ** -0.5, rot={"base": 1e4, "dims": dim // 4}, diff=0.6, softcap=40.0)},
             {"type": "attention_2", "mixer": dict(base, rot={"base": 1e4, "dims": dim // 2})},
             {"type": "attention_3", "mixer": dict(base, q_temp={"coef": 0.3, "every": 1024})}]
    return {"architecture": "Loselix", "width": width, "vocab": vocab, "norm": {"eps": 1e-5}, "loop": LOOP, "layers": [dict(k, mlp={"kind": "dense", "ff": ff}) for k in kinds * 2]}


def random_fetch(cfg, dev):
    g = torch.Generator(device=dev).manual_seed(1)

    def n(*shape, std, mean=0.0):
        return torch.randn(shape, generator=g, device=dev, dtype=torch.float32).mul_(std).add_(mean).to(torch.bfloat16)

    w = cfg.hidden_size

    def fetch(prefix):
        if prefix in ("embed", "head"):
            return {prefix: n(cfg.vocab_size, w, std=0.7 if prefix == "embed" else w ** -0.5)}
        if prefix == "final.norm":
            return {prefix: n(w, std=0.1, mean=1.0)}
        s = cfg.layers[int(prefix[1:])]
        H, G, d, v, f, m = s.heads, s.kv_heads, s.dim, s.vdim, s.ff, 2 if s.type == "attention" else 1
        t = {"norm1": n(w, std=0.1, mean=1.0), "mix.q": n(H * m * d, w, std=w ** -0.5), "mix.k": n(G * m * d, w, std=w ** -0.5), "mix.o": n(w, H * v, std=(H * v) ** -0.5),
             "mlp.up": n(f, w, std=w ** -0.5), "mlp.down": n(w, f, std=f ** -0.5)}
        if s.type != "attention_3":
            t["mix.v"] = n(G * v, w, std=w ** -0.5)
        if s.type == "attention":
            t.update({f"mix.{k}": n(d, std=0.1) for k in ("lq1", "lk1", "lq2", "lk2")})
        elif s.type == "attention_2":
            t["mix.g"] = n(H, w, std=w ** -0.5)
        else:
            t.update({"mix.q.norm": n(H * d, std=0.1, mean=1.0), "mix.k.norm": n(G * d, std=0.1, mean=1.0), "mix.pb": n(H, std=0.3, mean=-7.0), "mix.g": n(H * v, w, std=w ** -0.5)})
        return {f"{prefix}.{k}": x for k, x in t.items()}

    return fetch


def loselix_model(size, dev):
    from nanovllm.models.loselix.config import read_config
    from nanovllm.models.loselix.model import LoselixForCausalLM
    cfg = read_config(loselix_config(*SIZES[size]))
    with torch.device(dev):
        m = LoselixForCausalLM(cfg)
        m.load_from(random_fetch(cfg, dev))
    return m


def loselix_step(m, mode, B, n, dev):
    """(device batch of one step, tokens per step) over caches filled with unit-rms values."""
    from nanovllm.engine.step_batch import Chunk, build_step
    bs = 64
    per = -(-n // bs)
    m.allocate(B * per, bs, B, dev)
    for layer in m.layers:
        for kc, vc, ks in layer.mixer.caches:
            kc.normal_(), vc.normal_()
            if ks is not None:
                ks.fill_(1.0)
    perm = torch.randperm(B * per, generator=torch.Generator().manual_seed(2)).view(B, per).tolist()
    if mode == "decode":
        chunks = [Chunk([7 + b], n - 1, perm[b], 2 * b, 2 * b + 1, [0]) for b in range(B)]
        host, on_device, _ = build_step(chunks, m, bs, pad_rows=B, table_width=per)
    else:
        toks = torch.randint(0, m.config.vocab_size, (B, n), generator=torch.Generator().manual_seed(3)).tolist()
        chunks = [Chunk(toks[b], 0, perm[b], 2 * b, 2 * b + 1, [n - 1]) for b in range(B)]
        host, on_device, _ = build_step(chunks, m, bs)
    return on_device(torch.from_numpy(host).to(dev)), (B if mode == "decode" else B * n)


def kind_kernels(m, meta, mode, B, n, kind, h):
    """Projections, rows and attention of the layers of one kind."""
    from nanovllm import hip_ops as ops
    name, T, w, out = KINDS[kind], meta.ids.numel(), m.config.hidden_size, {}
    pairs = B * (n * (n + 1) // 2 if mode != "decode" else n)
    S = [l for l in m.layers if l.spec.type == kind]
    b, a = S[0].block, S[0].mixer
    k = b.attp + b.ffp
    H, G, dk, dv = a.heads, a.kv_heads, a.dk, a.vdimp
    rows = torch.randn(T, b.attp + b.in_proj.N, device=h.device).to(torch.bfloat16)
    out[f"gemm up|qkv|g ({name})"] = ([lambda l=l: l.block.in_proj(h, act=l.block.act, out=rows[:, b.attp:]) for l in S], *gemm_cost(T, b.in_proj.N, w))
    ns = b.slices(T)
    if ns > 1:
        out[f"gemm o|down ({name})"] = ([lambda l=l: ops.gemm_bf16_partial(rows[:, :k], l.block.out_proj.weight, ns) for l in S], *gemm_cost(T, w, k))
    else:
        out[f"gemm o|down ({name})"] = ([lambda l=l: l.block.out_proj(rows[:, :k]) for l in S], *gemm_cost(T, w, k))
    xr = rows[:, k:]
    if kind == "attention_3":
        f = lambda l: ops.group_norm_store(xr, 0, a.k_off, l.mixer.gain, H * a.dim, G * dk, G * a.dim, 0, 1e-5, meta.pos, meta.slots, l.mixer.caches[0][0], l.mixer.caches[0][2], a.temperature)  # noqa: E731
        out["norm + store (sigmoid)"] = ([lambda l=l: f(l) for l in S], 2 * T * (2 * H * dk + 2 * G * dk), 0)
        kv_bytes = 2 * G * dk + 4
    else:
        cs, rot = a.rot.table(meta.pos), a.rot
        f = lambda l: ops.group_rotate_store(xr, 0, a.k_off, a.v_off, H, a.maps, rot.dims, cs, meta.slots, *l.mixer.caches[0][:2])  # noqa: E731
        out[f"rotate + store ({name})"] = ([lambda l=l: f(l) for l in S], 2 * T * (2 * H * a.maps * rot.dims + 2 * G * (dk + dv)) + 4 * T * rot.dims, 0)
        kv_bytes = 2 * G * (dk + dv)

    def attend(l):
        mx = l.mixer
        kc, vc, ks = mx.caches[0]
        parts = replace(mx.parts, kscale=ks, gate=xr[:, a.g_off:] if a.gate else None)
        q, o = xr[:, : a.k_off], rows[:, : a.heads * a.vdimp]
        if mode == "decode":
            per = min(a.tokens_per_tile, meta.max_short)
            ops.group_attn_decode(q, kc, vc, meta.block_tables, meta.pos, meta.seq_of, *meta.tiles[per], per, a.heads, 0, 0, a.scale, None, None, o, parts=parts)
        else:
            ops.group_attn_prefill(q, kc, vc, meta.block_tables, meta.n_short, meta.long_q_start, meta.pos, *meta.chunk_tiles[0, a.tile_rows], a.heads, 0, 0, a.scale, None, None, o,
                                   parts=parts)

    fl = 2 * pairs * H * a.maps * (a.dimp + dv)
    by = B * n * kv_bytes + 2 * T * H * (dk + dv)
    out[f"attention ({name})"] = ([lambda l=l: attend(l) for l in S], by, fl)
    return out


def repeated(ops):
    """The layers of a kind over again until a graph holds nine launches like the ones beside it (a replay's own cost is shared by them)."""
    return {k: (fns * -(-9 // len(fns)), *cost) for k, (fns, *cost) in ops.items()}


def loselix_kernels(m, meta, mode, B, n):
    from nanovllm import hip_ops as ops
    cfg = m.config
    T, w, wp, dev, bf = meta.ids.numel(), cfg.hidden_size, cfg.padded_width, meta.ids.device, torch.bfloat16
    rnd = lambda *s: torch.randn(*s, device=dev).to(bf)  # noqa: E731
    x, h, y = torch.randn(T, wp, device=dev), rnd(T, wp), rnd(T, wp)
    ns = m.layers[0].block.slices(T)
    if ns > 1:
        y = ops.PartialSum(torch.randn(ns, T, wp, device=dev))
    yb = 2 if ns == 1 else 4 * ns
    L, out = list(m.layers), {}

    def norm(y, **kw):
        return [lambda l=l: ops.residual_norm(x, w, wp, 1e-5, y=y, g=l.g, **kw) for l in L]

    out["residual_norm"] = (norm(y), T * w * (4 + yb + 4 + 2), 0)
    out["residual_norm (embedding added)"] = (norm(y, embed=(meta.ids, m.embed)), T * w * (4 + yb + 2 + 4 + 2), 0)
    for kind in KINDS:
        out.update(kind_kernels(m, meta, mode, B, n, kind, h))
    return out


@torch.inference_mode()
def run(args) -> None:
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(0)
    from nanovllm import hip_ops
    from nanovllm.utils.context import reset_context
    hip_ops.load_library()
    for size in (args.design_sizes.split(",") if args.design_sizes else SIZES):
        m = loselix_model(size, dev)
        runs = len(m.runs)
        glm, gcfg = glm_model(size, runs, dev)
        for name, (mode, B, n) in MODES.items():
            rec = {"design": "loselix", "size": size, "mode": name, "layer_runs": runs, "dtype": "bf16", "data": "synthetic"}
            reps = args.steps if mode == "decode" else max(2, args.steps // 4)
            meta, toks = loselix_step(m, mode, B, n, dev)
            step = graph_of(lambda: torch.argmax(m(meta), -1)).replay if mode == "decode" else (lambda: torch.argmax(m(meta), -1))
            us = time_us(step, reps, args.warmup)
            rec["loselix"] = {"tokens_per_s": round(toks / us * 1e6, 1), "ms_per_step": round(us / 1e3, 3),
                              "kernels": kernel_table(repeated(loselix_kernels(m, meta, mode, B, n)), reps) if not args.no_extras else {}}
            del step, meta
            ids, pos = glm_step(glm, gcfg, mode, B, n, dev)
            body = lambda: torch.argmax(glm.compute_logits(glm(ids, pos)), -1)  # noqa: E731
            step = graph_of(body).replay if mode == "decode" else body
            us = time_us(step, reps, args.warmup)
            rec["glm4_dense"] = {"tokens_per_s": round(toks / us * 1e6, 1), "ms_per_step": round(us / 1e3, 3),
                                 "kernels": kernel_table(glm_kernels(glm, gcfg, mode, B, n, pos), reps) if not args.no_extras else {}}
            del step
            reset_context()
            torch.cuda.empty_cache()
            print(json.dumps(rec), flush=True)
        del m, glm
        torch.cuda.empty_cache()
