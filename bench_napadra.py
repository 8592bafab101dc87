"""`python bench.py --design napadra`: prefill and decode throughput of the Napadra design at layer sizes of real models (random
weights), beside GLM-4-MoE's dense layers at equal size (same width, heads, head size, key/value heads, parameters of the feed-forward,
layers, vocabulary), and the time of every kernel of both against its roofline (HBM 8 TB/s, bf16 MFMA 2.5 PFLOP/s).  Prints one JSON line
per size and mode."""
from __future__ import annotations

import json

import torch

from bench_dafolorn import MODES, gemm_cost, glm_kernels, glm_model, glm_step, graph_of, kernel_table, time_us

SIZES = {
    # width, heads, key/value heads, head size, chunk, feed-forward, vocabulary; memory heads, key size, value size
    "2k": (2048, 16, 4, 128, 1024, 4096, 32768, 8, 128, 256),
    "4k": (4096, 32, 8, 128, 4096, 8192, 32768, 16, 128, 256),
}
LAYERS = 8


def napadra_config(width, heads, kv, dim, chunk, ff, vocab, mheads, mdim, mvdim):
    """Two groups of: two attention layers, one that borrows the second one's cache, one matrix memory."""
    mlp = {"kind": "dense", "ff": ff, "limit": 7.0}

    def attn(kv_from=None):
        m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "mask": {"size": chunk}, "scale": dim ** -0.5}
        return {"type": "attention", "mixer": m if kv_from is None else dict(m, kv_from=kv_from), "mlp": mlp}

    mem = {"type": "mlstm", "mixer": {"heads": mheads, "dim": mdim, "vdim": mvdim, "gate_cap": 15.0}, "mlp": mlp}
    layers = [x for i in range(0, LAYERS, 4) for x in (attn(), attn(), attn(i + 1), mem)]
    return {"architecture": "Napadra", "width": width, "vocab": vocab, "streams": 2, "residual_mult": 0.5, "norm": {"eps": 1e-5}, "layers": layers}


def random_fetch(cfg, dev):
    g = torch.Generator(device=dev).manual_seed(1)

    def n(*shape, std, mean=0.0):
        return torch.randn(shape, generator=g, device=dev, dtype=torch.float32).mul_(std).add_(mean).to(torch.bfloat16)

    w, S = cfg.hidden_size, cfg.streams

    def fetch(prefix):
        if prefix in ("embed", "head"):
            return {prefix: n(cfg.vocab_size, w, std=0.7 if prefix == "embed" else w ** -0.5)}
        if prefix == "final.norm":
            return {prefix: n(std=0.1, mean=1.0)}
        s = cfg.layers[int(prefix[1:])]
        H, d, v, f = s.heads, s.dim, s.vdim, s.ff
        t = {"shift": n(w, std=0.3), "mix.q": n(H * d, w, std=w ** -0.5), "mix.o": n(w, H * v, std=(H * v) ** -0.5),
             "mlp.gate": n(f, w, std=w ** -0.5), "mlp.up": n(f, w, std=w ** -0.5), "mlp.down": n(w, f, std=f ** -0.5)}
        for q in (1, 2):
            t.update({f"norm{q}": n(std=0.1, mean=1.0), f"ls{q}": n(w, std=0.2, mean=1.0), f"hc{q}.in": n(S, std=0.2, mean=0.5),
                      f"hc{q}.out": n(S, std=0.2, mean=1.0), f"hc{q}.mix": n(S, S, std=0.1) + torch.eye(S, device=dev, dtype=torch.bfloat16)})
        if s.type == "attention":
            t["mix.sink"] = n(H, std=1.0)
            if s.kv_from is None:
                t.update({"mix.k": n(s.kv_heads * d, w, std=w ** -0.5), "mix.v": n(s.kv_heads * v, w, std=w ** -0.5)})
        else:
            t.update({"mix.k": n(H * d, w, std=w ** -0.5), "mix.v": n(H * v, w, std=w ** -0.5), "mix.g": n(H * v, w, std=w ** -0.5), "mix.norm": n(H * v, std=0.1, mean=1.0),
                      "mix.i": n(H, w, std=w ** -0.5), "mix.i.b": n(H, std=1.0), "mix.f": n(H, w, std=w ** -0.5), "mix.f.b": n(H, std=1.0, mean=4.0)})
        return {f"{prefix}.{k}": x for k, x in t.items()}

    return fetch


def napadra_model(size, dev):
    from nanovllm.models.napadra.config import read_config
    from nanovllm.models.napadra.model import NapadraForCausalLM
    cfg = read_config(napadra_config(*SIZES[size]))
    with torch.device(dev):
        m = NapadraForCausalLM(cfg)
        m.load_from(random_fetch(cfg, dev))
    return m


def napadra_step(m, mode, B, n, dev):
    """(device batch of one step, tokens per step) over caches and states filled with unit-rms values."""
    from nanovllm.engine.step_batch import Chunk, build_step
    bs = 64
    per = -(-n // bs)
    m.allocate(B * per, bs, B, dev)
    for layer in m.layers:
        for t in (getattr(layer.mixer, "k_cache", None), getattr(layer.mixer, "v_cache", None), layer.sub1.state, *(getattr(layer.mixer, "state", None) or ())):
            if t is not None:
                t.normal_()
    perm = torch.randperm(B * per, generator=torch.Generator().manual_seed(2)).view(B, per).tolist()
    if mode == "decode":
        chunks = [Chunk([7 + b], n - 1, perm[b], 2 * b, 2 * b + 1, [0]) for b in range(B)]
        host, on_device, _ = build_step(chunks, m, bs, pad_rows=B, table_width=per)
    else:
        toks = torch.randint(0, m.config.vocab_size, (B, n), generator=torch.Generator().manual_seed(3)).tolist()
        chunks = [Chunk(toks[b], 0, perm[b], 2 * b, 2 * b + 1, [n - 1]) for b in range(B)]
        host, on_device, _ = build_step(chunks, m, bs)
    return on_device(torch.from_numpy(host).to(dev)), (B if mode == "decode" else B * n)


def napadra_kernels(m, meta, mode, B, n):
    from nanovllm import hip_ops as ops
    cfg = m.config
    T, w, S, dev, bf = meta.ids.numel(), cfg.hidden_size, cfg.streams, meta.ids.device, torch.bfloat16
    rnd = lambda *s: torch.randn(*s, device=dev).to(bf)  # noqa: E731
    att = [layer for layer in m.layers if layer.spec.type == "attention"]
    own, mem, L = [layer for layer in att if layer.mixer.own_kv], [layer for layer in m.layers if layer.spec.type == "mlstm"], list(m.layers)
    a, e = att[0].mixer, mem[0].mixer
    x, h, y = torch.randn(T, S, w, device=dev), rnd(T, w), rnd(T, w)
    act, o = rnd(T, cfg.layers[0].ff), rnd(T, a.heads * a.vdimp)
    out = {}
    nb = T * w * (8 * S + 2 + 2)
    out["stream_norm (feed-forward)"] = ([lambda l=l: l.sub2.enter(x, l.sub1, y, meta, bf) for l in L], nb, 0)
    out["stream_norm (mixer, token shift)"] = ([lambda l=l: l.sub1.enter(x, l.sub2, y, meta, bf) for l in L], nb, 0)

    def gemm(name, lins, inp):
        out[name] = ([lambda p=p: p(inp) for p in lins], *gemm_cost(T, lins[0].N, lins[0].K))

    gemm("gemm qkv", [l.mixer.qkv_proj for l in own], h)
    gemm("gemm o", [l.mixer.o_proj for l in att], o)
    ff, K = cfg.layers[0].ff, w
    out["gemm gate|up + clamped unit"] = ([lambda l=l: ops.gated_glu(h, l.mlp.gate_up.weight, l.mlp.limit) for l in L], 2 * (2 * ff * K + T * K + T * ff), 4 * T * ff * K)
    gemm("gemm down", [l.mlp.down for l in L], act)
    qkv = rnd(T, a.qkv_proj.N)
    H, G, d, nq = a.heads, a.kv_heads, a.dimp, a.heads * a.dimp
    if mode != "decode":
        out["kv store"] = ([lambda l=l: ops.group_kv_store(qkv, nq, nq + G * d, meta.slots, l.mixer.k_cache, l.mixer.v_cache) for l in own], 2 * 2 * T * 2 * G * d, 0)
    form = lambda l: (H, 0, l.mixer.chunk, l.mixer.scale, l.mixer.slope, l.mixer.sink, o)  # noqa: E731
    pairs = sum(i % a.chunk + 1 for i in (range(n) if mode != "decode" else (n - 1,)))
    if mode == "decode":
        tok, cnt = meta.tiles[1]
        new = (qkv[:, nq: nq + G * d], qkv[:, nq + G * d:], meta.q_start, meta.slots)
        out["attention (store, merge)"] = (
            [lambda l=l: ops.group_attn_decode(qkv[:, :nq], l.mixer.k_cache, l.mixer.v_cache, meta.block_tables, meta.pos, meta.seq_of, tok, cnt, 1, *form(l), new=new) for l in own],
            2 * B * pairs * 2 * G * d, 4 * B * pairs * H * d)
    else:
        out["attention"] = (
            [lambda l=l: ops.group_attn_prefill(qkv[:, :nq], l.mixer.k_cache, l.mixer.v_cache, meta.block_tables, meta.n_short, meta.long_q_start, meta.pos,
                                                *meta.chunk_tiles[a.chunk, a.tile_rows], *form(l)) for l in own],
            2 * T * (2 * H + 2 * G) * d, 4 * B * pairs * H * d)
    gemm("gemm memory q|k|v|g", [l.mixer.in_proj for l in mem], h)
    gemm("gemm memory o", [l.mixer.o_proj for l in mem], rnd(T, e.heads * e.vdimp))
    mx, my = rnd(T, e.in_proj.N), rnd(T, e.heads * e.vdimp)
    mh, md, mv = e.heads, e.dimp, e.vdimp
    rest = lambda l: (l.mixer.state, meta.pos, meta.q_start, meta.state_in, meta.state_out, mh, e.dim, e.vdim, e.cap, e.eps)  # noqa: E731
    io = 2 * T * mh * (2 * md + 3 * mv)
    if mode == "decode":
        out["memory recurrent"] = (
            [lambda l=l: ops.memory_recurrent(mx, h, l.mixer.gates.weight[: 2 * mh], l.mixer.gate_bias, l.mixer.norm, my, *rest(l)) for l in mem],
            io + 8 * B * mh * (md * mv + md), 0)
    else:
        tiles = (meta.long_tile_seq, meta.long_tile_off)
        out["memory gates + chunkwise + output"] = (
            [lambda l=l: ops.memory_chunkwise(mx, h, l.mixer.gates.weight[: 2 * mh], l.mixer.gate_bias, l.mixer.norm, my, *rest(l)[:5], *tiles, *rest(l)[5:]) for l in mem],
            io + 2 * T * w, 0)
    return out


@torch.inference_mode()
def run(args) -> None:
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(0)
    from nanovllm import hip_ops
    from nanovllm.utils.context import reset_context
    hip_ops.load_library()
    for size in (args.design_sizes.split(",") if args.design_sizes else SIZES):
        m = napadra_model(size, dev)
        glm, gcfg = glm_model(size, LAYERS, dev)
        for name, (mode, B, n) in MODES.items():
            rec = {"design": "napadra", "size": size, "mode": name, "layers": LAYERS, "dtype": "bf16", "data": "synthetic"}
            reps = args.steps if mode == "decode" else max(2, args.steps // 4)
            meta, toks = napadra_step(m, mode, B, n, dev)
            step = graph_of(lambda: torch.argmax(m(meta), -1)).replay if mode == "decode" else (lambda: torch.argmax(m(meta), -1))
            us = time_us(step, reps, args.warmup)
            rec["napadra"] = {"tokens_per_s": round(toks / us * 1e6, 1), "ms_per_step": round(us / 1e3, 3),
                              "kernels": kernel_table(napadra_kernels(m, meta, mode, B, n), reps) if not args.no_extras else {}}
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
