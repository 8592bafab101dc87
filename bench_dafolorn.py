"""`python bench.py --design dafolorn`: prefill and decode throughput of the Dafolorn design at layer sizes of real models
(random weights), beside GLM-4-MoE's dense layers at equal size (same width, heads, head size, parameters of the feed-forward,
layer runs, vocabulary), and the time of every kernel of both against its roofline (HBM 8 TB/s, bf16 MFMA 2.5 PFLOP/s).
Prints one JSON line per size and mode."""
from __future__ import annotations

import json
import types

import torch

HBM, MFMA = 8.0e12, 2.5e15
SIZES = {
    # (width, heads, head size, latent, window, feed-forward, vocabulary)
    "2k": (2048, 16, 128, 256, 1024, 6144, 32768),
    "4k": (4096, 32, 128, 512, 4096, 12288, 32768),
}
MODES = {"prefill_4x4096": ("prefill", 4, 4096), "decode_b32_ctx4096": ("decode", 32, 4096), "decode_b128_ctx4096": ("decode", 128, 4096),
         "decode_b1_ctx4096": ("decode", 1, 4096)}


def dafolorn_config(width, heads, dim, rank, window, ff, vocab):
    """Six layers, the middle two three times: ten layer runs."""
    one = {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": dim, "kv_rank": rank, "mask": {"size": window},
           "scale": dim ** -0.5}, "mlp": {"kind": "dense", "ff": ff}}
    return {"architecture": "Dafolorn", "width": width, "vocab": vocab, "canon": {"taps": 4}, "norm": {"eps": 1e-5}, "layers": [one] * 6,
            "loop": {"start": 2, "stop": 4, "times": 3}, "logit_softcap": 30.0}


def glm_config(width, heads, dim, ff, vocab, layers, max_pos):
    return types.SimpleNamespace(
        hidden_size=width, num_attention_heads=heads, num_key_value_heads=heads // 4, head_dim=dim, attention_bias=True, use_qk_norm=False,
        partial_rotary_factor=0.5, rope_theta=1e6, rope_scaling=None, max_position_embeddings=max_pos, rms_norm_eps=1e-5,
        n_routed_experts=None, intermediate_size=ff * 2 // 3, first_k_dense_replace=layers, hidden_act="silu", vocab_size=vocab,
        num_hidden_layers=layers, num_layers_to_load=layers, tie_word_embeddings=False, torch_dtype=torch.bfloat16)


def random_fetch(cfg, dev):
    g = torch.Generator(device=dev).manual_seed(1)

    def n(*shape, std):
        return torch.randn(*shape, generator=g, device=dev, dtype=torch.float32).mul_(std).to(torch.bfloat16)

    w, taps = cfg.hidden_size, cfg.conv_taps

    def fetch(prefix):
        if prefix == "embed":
            return {prefix: n(cfg.vocab_size, w, std=0.7)}
        if prefix == "final.norm":
            return {prefix: n(w, std=0.1)}
        if prefix == "loop.in":
            return {prefix: n(w, 2 * w, std=(2 * w) ** -0.5)}
        if prefix == "loop.step":
            return {prefix: n(cfg.loop.times, w, std=0.3)}
        s = cfg.layers[int(prefix[1:])]
        H, d, v, r, f = s.heads, s.dim, s.vdim, s.kv_rank, s.ff
        t = {"norm1": n(w, std=0.1), "norm1b": n(w, std=0.1), "norm2": n(w, std=0.1), "norm2b": n(w, std=0.1),
             "canon1": n(w, taps, std=0.3), "canon2": n(w, taps, std=0.3), "mix.q": n(H * d, w, std=w ** -0.5), "mix.dkv": n(r, w, std=w ** -0.5),
             "mix.dkv.norm": n(r, std=0.1) + 1, "mix.uk": n(H * d, r, std=r ** -0.5), "mix.uv": n(H * v, r, std=r ** -0.5), "mix.sink": n(H, std=1.0),
             "mix.o": n(w, H * v, std=(H * v) ** -0.5), "mlp.up": n(f, w, std=w ** -0.5), "mlp.down": n(w, f, std=f ** -0.5), "mlp.act": n(2, std=0.5)}
        return {f"{prefix}.{k}": x for k, x in t.items()}

    return fetch


def graph_of(fn):
    fn()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        fn()
    torch.cuda.synchronize()
    return g


def time_us(run, reps, warm=3):
    for _ in range(warm):
        run()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    torch.cuda.synchronize()
    a.record()
    for _ in range(reps):
        run()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / reps * 1e3


def kernel_table(ops, reps):
    """ops: {name: (one closure per layer, bytes, flops)} of ONE launch -> time and share of the roofline that binds."""
    out = {}
    for name, (fns, nbytes, flops) in ops.items():
        g = graph_of(lambda: [f() for f in fns])
        us = time_us(g.replay, reps) / len(fns)
        floor = max(nbytes / HBM, flops / MFMA)
        out[name] = {"us": round(us, 2), "bound": "hbm" if nbytes / HBM >= flops / MFMA else "mfma", "of_roofline": round(floor * 1e6 / us, 3)}
    return out


def gemm_cost(M, N, K):
    return 2 * (N * K + M * K + M * N), 2 * M * N * K


# ---- Dafolorn ---------------------------------------------------------------------------------------------------------------
def dafolorn_model(size, dev):
    from nanovllm.models.dafolorn.config import read_config
    from nanovllm.models.dafolorn.model import DafolornForCausalLM
    w, heads, dim, rank, window, ff, vocab = SIZES[size]
    cfg = read_config(dafolorn_config(w, heads, dim, rank, window, ff, vocab))
    with torch.device(dev):
        m = DafolornForCausalLM(cfg)
        m.load_from(random_fetch(cfg, dev))
    return m


def dafolorn_step(m, mode, B, n, dev):
    """(device batch of one step, tokens per step) over a cache filled with unit-rms rows."""
    from nanovllm.engine.step_batch import Chunk, build_step
    bs = 64
    per = -(-n // bs)
    m.allocate(B * per, bs, B, dev)
    for layer in m.layers:
        for c in layer.mixer.caches:
            c.normal_()
        for e in layer.entries():
            for s in e.state:
                s.normal_()
    perm = torch.randperm(B * per, generator=torch.Generator().manual_seed(2)).view(B, per).tolist()
    if mode == "decode":
        chunks = [Chunk([7 + b], n - 1, perm[b], 2 * b, 2 * b + 1, [0]) for b in range(B)]
        host, on_device, _ = build_step(chunks, m, bs, pad_rows=B, table_width=per)
    else:
        toks = torch.randint(0, m.config.vocab_size, (B, n), generator=torch.Generator().manual_seed(3)).tolist()
        chunks = [Chunk(toks[b], 0, perm[b], 2 * b, 2 * b + 1, [n - 1]) for b in range(B)]
        host, on_device, _ = build_step(chunks, m, bs)
    return on_device(torch.from_numpy(host).to(dev)), (B if mode == "decode" else B * n)


def dafolorn_kernels(m, meta, mode, B, n):
    from nanovllm import hip_ops as ops
    cfg, s0 = m.config, m.config.layers[0]
    T, w, H, d, v, r, f, W = meta.ids.numel(), cfg.hidden_size, s0.heads, s0.dim, s0.vdim, s0.kv_rank, s0.ff, s0.window
    dev, bf = meta.ids.device, torch.bfloat16
    rnd = lambda *s: torch.randn(*s, device=dev).to(bf)  # noqa: E731
    x, h, act, att, y = torch.randn(T, w, device=dev), rnd(T, w), rnd(T, f), rnd(T, H * v), rnd(T, w)
    qc = rnd(T, H * d + r)
    L = list(m.layers)
    out = {}
    out["seq_norm"] = ([lambda e=layer.entry2, g=layer.g_post1: e(x, y, g, meta, 0, bf) for layer in L], T * w * (4 + 4 + 2 + 2), 0)
    for name, lin, inp, act_ in (("gemm q|latent", lambda l: l.mixer.qc_proj, h, None), ("gemm o", lambda l: l.mixer.o_proj, att, None),
                                 ("gemm up + xielu", lambda l: l.mlp.up, h, 1), ("gemm down", lambda l: l.mlp.down, act, None)):
        lins = [lin(layer) for layer in L]
        out[name] = ([lambda p=p, i=inp, a=(layer.mlp.act if act_ else ops.NO_ACT): p(i, act=a) for p, layer in zip(lins, L)],
                     *gemm_cost(T, lins[0].N, lins[0].K))
    if mode == "decode":
        keys = min(W, n)
        tok, cnt = meta.tiles[1]
        qa = rnd(T, H, r)
        o2 = torch.empty(T, H * v, dtype=bf, device=dev)
        out["latent prepare (norm, store, W_uk q)"] = (
            [lambda mx=layer.mixer: ops.latent_prepare(qc, H * d, H, d, r, mx.c_gain, mx.eps, meta.slots, mx.caches[0], T, mx.wukt) for layer in L],
            2 * (H * d * r + T * (H * d + 2 * r + H * r)), 2 * T * H * d * r)
        out["latent attention + merge, W_uv"] = (
            [lambda mx=layer.mixer: ops.latent_attn(qa, mx.caches[0], tok, cnt, 1, meta.pos, meta.seq_of, meta.block_tables, W, mx.scale, mx.sink,
                                                    mx.wuv, o2) for layer in L],
            2 * (B * keys * r + H * v * r + T * H * (r + v)), 2 * T * H * (2 * keys * r + r * v))
    else:
        win = meta.windows[W]
        c = rnd(win.rows, r)
        kv = rnd(win.rows, H * (d + v))
        o2 = torch.empty(T, H * v, dtype=bf, device=dev)
        pairs = B * sum(min(i + 1, W) for i in range(n))
        out["latent prepare (norm, store)"] = (
            [lambda mx=layer.mixer: ops.latent_prepare(qc, H * d, H, d, r, mx.c_gain, mx.eps, meta.slots, mx.caches[0], 0, mx.wukt, win.crow, win.rows)
             for layer in L], 2 * T * r * 3, 0)
        out["gemm expand k|v"] = ([lambda p=layer.mixer.expand: p(c) for layer in L], *gemm_cost(win.rows, L[0].mixer.expand.N, L[0].mixer.expand.K))
        out["window attention"] = (
            [lambda mx=layer.mixer: ops.window_attn_prefill(qc[:, : H * d], kv[:, : H * d], kv[:, H * d:], o2, meta.long_q_start, win.k_start,
                                                            meta.long_tile_seq, meta.long_tile_off, H, d, v, W, mx.scale, mx.sink) for layer in L],
            2 * (T * H * (d + v) + win.rows * H * (d + v)), 2 * pairs * H * (d + v))
    return out


# ---- GLM-4-MoE dense layers ---------------------------------------------------------------------------------------------------
def glm_model(size, layers, dev):
    from nanovllm.models.glm4_moe.model import Glm4MoeForCausalLM
    w, heads, dim, _, _, ff, vocab = SIZES[size]
    cfg = glm_config(w, heads, dim, ff, vocab, layers, 8192)
    old = torch.get_default_dtype()
    torch.set_default_dtype(torch.bfloat16)
    try:
        with torch.device(dev):
            m = Glm4MoeForCausalLM(cfg)
    finally:
        torch.set_default_dtype(old)
    g = torch.Generator(device=dev).manual_seed(1)
    for name, p in m.named_parameters():
        p.data.normal_(0.0, 0.02, generator=g)
        if "norm" in name:
            p.data.add_(1.0)
    return m, cfg


def glm_step(m, cfg, mode, B, n, dev):
    from nanovllm.utils.context import set_context
    bs, nkv = 256, cfg.num_key_value_heads
    per = -(-n // bs)
    kv = torch.empty(2, cfg.num_hidden_layers, B * per, bs, nkv, cfg.head_dim, device=dev, dtype=torch.bfloat16).normal_()
    for i, a in enumerate([x for x in m.modules() if hasattr(x, "k_cache")]):
        a.k_cache, a.v_cache = kv[0, i], kv[1, i]
    perm = torch.randperm(B * per, generator=torch.Generator().manual_seed(2)).view(B, per)
    bt = perm.to(torch.int32).to(dev)
    if mode == "decode":
        pos = torch.full((B,), n - 1, dtype=torch.int64, device=dev)
        slots = (bt[:, (n - 1) // bs] * bs + (n - 1) % bs).to(torch.int32)
        set_context(False, slot_mapping=slots, context_lens=torch.full((B,), n, dtype=torch.int32, device=dev), block_tables=bt)
        ids = torch.randint(0, cfg.vocab_size, (B,), device=dev)
    else:
        pos = torch.arange(n, device=dev).repeat(B)
        slots = (bt.long().repeat_interleave(bs, 1)[:, :n] * bs + torch.arange(n, device=dev) % bs).reshape(-1).to(torch.int32)
        cu = (torch.arange(B + 1, device=dev) * n).to(torch.int32)
        set_context(True, cu, cu, n, n, slots, None, None)
        ids = torch.randint(0, cfg.vocab_size, (B * n,), device=dev)
    return ids, pos


def glm_kernels(m, cfg, mode, B, n, pos):
    from nanovllm import hip_ops as ops
    from nanovllm.utils.context import get_context
    ctx = get_context()
    w, nh, nkv, hd, I = cfg.hidden_size, cfg.num_attention_heads, cfg.num_key_value_heads, cfg.head_dim, cfg.intermediate_size
    T, dev, bf = pos.numel(), pos.device, torch.bfloat16
    rnd = lambda *s: torch.randn(*s, device=dev).to(bf)  # noqa: E731
    h, res, att, act, qkv = rnd(T, w), rnd(T, w), rnd(T, nh * hd), rnd(T, I), rnd(T, (nh + 2 * nkv) * hd)
    L = list(m.model.layers)
    out = {"add_rmsnorm": ([lambda l=l: l.post_attention_layernorm(h, res) for l in L], T * w * 8, 0)}
    qp = lambda l: l.self_attn.qkv_proj  # noqa: E731
    N = (nh + 2 * nkv) * hd
    if mode == "decode":
        out["gemm qkv"] = ([lambda l=l: qp(l)(h) for l in L], *gemm_cost(T, N, w))
        out["paged attention (rotary, store)"] = (
            [lambda a=l.self_attn: ops.paged_attn_decode_qkv(qkv, nh, nkv, hd, pos, a.rotary_emb.cos_sin_cache, a.rotary_emb.rotary_dim, ctx.slot_mapping,
                                                             a.attn.k_cache, a.attn.v_cache, ctx.context_lens, ctx.block_tables, a.attn.scale) for l in L],
            2 * B * n * nkv * hd * 2, 4 * B * n * nh * hd)
    else:
        k, v = rnd(T, nkv, hd), rnd(T, nkv, hd)
        q = att.view(T, nh, hd)
        out["gemm qkv + rotary + store"] = (
            [lambda a=l.self_attn: ops.gemm_qkv_rope_store(h, a.qkv_proj.weight.data, a.qkv_proj.bias.data, nh, nkv, hd, pos, a.rotary_emb.cos_sin_cache,
                                                           a.rotary_emb.rotary_dim, a.attn.k_cache, a.attn.v_cache, ctx.slot_mapping, True) for l in L],
            *gemm_cost(T, N, w))
        out["varlen attention"] = (
            [lambda a=l.self_attn: ops.varlen_attn_prefill(q, k, v, ctx.cu_seqlens_q, ctx.cu_seqlens_k, n, a.attn.scale) for l in L],
            2 * T * (2 * nh + 2 * nkv) * hd, 4 * B * (n * (n + 1) // 2) * nh * hd)
    out["gemm o"] = ([lambda l=l: l.self_attn.o_proj(att) for l in L], *gemm_cost(T, w, nh * hd))
    out["gemm gate|up + silu"] = ([lambda l=l: ops.grouped_gemm_gateup_silu(h, l.mlp.gate_up_proj.weight.data.unsqueeze(0), None, None, T) for l in L],
                                  2 * (2 * I * w + T * w + T * I), 2 * T * 2 * I * w)
    out["gemm down"] = ([lambda l=l: ops.grouped_gemm_down(act, l.mlp.down_proj.weight.data.unsqueeze(0), None, None, 0) for l in L],
                        *gemm_cost(T, w, I))
    return out


@torch.inference_mode()
def run(args) -> None:
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(0)
    from nanovllm import hip_ops
    from nanovllm.utils.context import reset_context
    hip_ops.load_library()
    for size in (args.design_sizes.split(",") if args.design_sizes else SIZES):
        m = dafolorn_model(size, dev)
        runs = len(m.runs)
        glm, gcfg = glm_model(size, runs, dev)
        for name, (mode, B, n) in MODES.items():
            rec = {"design": "dafolorn", "size": size, "mode": name, "layer_runs": runs, "dtype": "bf16", "data": "synthetic"}
            reps = args.steps if mode == "decode" else max(2, args.steps // 4)
            meta, toks = dafolorn_step(m, mode, B, n, dev)
            step = graph_of(lambda: torch.argmax(m(meta), -1)).replay if mode == "decode" else (lambda: torch.argmax(m(meta), -1))
            us = time_us(step, reps, args.warmup)
            rec["dafolorn"] = {"tokens_per_s": round(toks / us * 1e6, 1), "ms_per_step": round(us / 1e3, 3),
                               "kernels": kernel_table(dafolorn_kernels(m, meta, mode, B, n), reps) if not args.no_extras else {}}
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
