"""`python bench.py --design gulozen`: prefill and decode throughput of the Gulozen design at layer sizes of real models (random
weights), beside GLM-4-MoE's own layers at equal size (same width, heads, head size, experts, experts per token, size of an expert, layers,
vocabulary; GLM's shared expert comes on top), and the time of every kernel of both against its roofline (HBM 8 TB/s, bf16 MFMA 2.5 PFLOP/s).
Prints one JSON line per size and mode."""
from __future__ import annotations

import json
import types

import torch

from bench_dafolorn import MODES, gemm_cost, glm_kernels, glm_step, graph_of, kernel_table, time_us

SIZES = {
    # width, heads, unrotated, rotated and value columns of a head, query latent, latent, experts, per token, size of an expert, vocabulary; heads and
    # head size of the linear attention
    "2k": (2048, 16, 128, 64, 128, 768, 512, 64, 6, 1024, 32768, 16, 128),
    "4k": (4096, 32, 128, 64, 128, 1536, 512, 64, 8, 1408, 32768, 32, 128),
}
LAYERS, GROUPS, TAPS = 8, 4, 4


def gulozen_config(width, heads, dim, rot, vdim, q_rank, kv_rank, experts, top, ff, vocab, lheads, ldim):
    """Twice: three layers of latent attention, one of linear attention; all with experts."""
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    att = {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": (dim + rot) ** -0.5,
        "rot": {"base": 10000.0, "dims": rot, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}}
    lin = {"type": "lightning", "mlp": mlp, "mixer": {"heads": lheads, "dim": ldim, "vdim": ldim, "decay": [1 - 2.0 ** -(2 + 8 * h / lheads) for h in range(lheads)]}}
    return {"architecture": "Gulozen", "width": width, "vocab": vocab, "norm": {"eps": 1e-5, "groups": GROUPS}, "canon": {"taps": TAPS}, "embedding": {"scale": 4.0},
            "layers": [att, att, att, lin] * (LAYERS // 4)}


def random_fetch(cfg, dev):
    g = torch.Generator(device=dev).manual_seed(1)

    def n(*shape, std, mean=0.0):
        return torch.randn(shape, generator=g, device=dev, dtype=torch.float32).mul_(std).add_(mean).to(torch.bfloat16)

    w = cfg.hidden_size

    def fetch(prefix):
        if prefix in ("embed", "head"):
            return {prefix: n(cfg.vocab_size, w, std=0.25 if prefix == "embed" else w ** -0.5)}
        if prefix == "final.norm":
            return {prefix: n(w, std=0.1, mean=1.0)}
        i = int(prefix[1:])
        s = cfg.layers[i]
        H, d, v = s.heads, s.dim, s.vdim
        t = {"norm1": n(w, std=0.1, mean=1.0), "norm2": n(w, std=0.1, mean=1.0), "canon1": n(w, TAPS, std=0.3), "dwa": n(i + 2, std=0.3), "mix.g": n(H * v, w, std=w ** -0.5),
             "mix.o": n(w, H * v, std=(H * v) ** -0.5), "mlp.router": n(s.experts, w, std=w ** -0.5)}
        if s.type == "lightning":
            t.update({"mix.q": n(H * d, w, std=w ** -0.5), "mix.k": n(H * d, w, std=w ** -0.5), "mix.v": n(H * v, w, std=w ** -0.5), "mix.norm": n(H * v, std=0.1, mean=1.0)})
        else:
            q, r, rd = s.q_rank, s.kv_rank, s.rot_dim
            t.update({"mix.dq": n(q, w, std=w ** -0.5), "mix.dq.norm": n(q, std=0.1, mean=1.0), "mix.uq": n(H * (d + rd), q, std=q ** -0.5), "mix.dkv": n(r + rd, w, std=w ** -0.5),
                      "mix.dkv.norm": n(r, std=0.1, mean=1.0), "mix.uk": n(H * d, r, std=r ** -0.5), "mix.uv": n(H * v, r, std=r ** -0.5), "mix.sink": n(H, std=1.0)})
        for e in range(s.experts):
            t.update({f"mlp.e{e}.gate": n(s.ff, w, std=w ** -0.5), f"mlp.e{e}.up": n(s.ff, w, std=w ** -0.5), f"mlp.e{e}.down": n(w, s.ff, std=s.ff ** -0.5)})
        return {f"{prefix}.{k}": x for k, x in t.items()}

    return fetch


def gulozen_model(size, dev):
    from nanovllm.models.gulozen.config import read_config
    from nanovllm.models.gulozen.model import GulozenForCausalLM
    cfg = read_config(gulozen_config(*SIZES[size]))
    with torch.device(dev):
        m = GulozenForCausalLM(cfg)
        m.load_from(random_fetch(cfg, dev))
    return m


def gulozen_step(m, mode, B, n, dev):
    """(device batch of one step, tokens per step) over caches and states filled with unit-rms values."""
    from nanovllm.engine.step_batch import Chunk, build_step
    bs = 64
    per = -(-n // bs)
    m.allocate(B * per, bs, B, dev)
    for layer in m.layers:
        for t in (layer.taps.state, getattr(layer.mixer, "state", None), *getattr(layer.mixer, "caches", ())):
            if t is not None:
                t.normal_()
    perm = torch.randperm(B * per, generator=torch.Generator().manual_seed(2)).view(B, per).tolist()
    if mode == "decode":
        chunks = [Chunk([7 + 13 * b], n - 1, perm[b], 2 * b, 2 * b + 1, [0]) for b in range(B)]
        host, on_device, _ = build_step(chunks, m, bs, pad_rows=B, table_width=per)
    else:
        toks = torch.randint(0, m.config.vocab_size, (B, n), generator=torch.Generator().manual_seed(3)).tolist()
        chunks = [Chunk(toks[b], 0, perm[b], 2 * b, 2 * b + 1, [n - 1]) for b in range(B)]
        host, on_device, _ = build_step(chunks, m, bs)
    return on_device(torch.from_numpy(host).to(dev)), (B if mode == "decode" else B * n)


def expert_kernels(h, mlps, experts, top, I, shared, tag=""):
    """Grouped projections over a random routing with distinct experts per token; `mlps`: (w13, w2) per layer."""
    from nanovllm import hip_ops as ops
    T, w = h.shape
    dev = h.device
    idx = torch.stack([torch.randperm(experts, device=dev)[:top] for _ in range(min(T, 512))]).repeat(-(-T // 512), 1)[:T].contiguous()
    idx = idx.sort(-1).values
    wts = torch.full((T, top), 1.0 / top, dtype=torch.bfloat16, device=dev)
    offs, tok, scale, _ = ops.moe_align(idx, wts if shared else None, experts, shared)
    used = int((torch.bincount(idx.reshape(-1), minlength=experts) > 0).sum()) + int(shared)
    R = tok.numel()
    act = torch.randn(R, I, device=dev).to(torch.bfloat16)
    return {f"experts gate|up{tag}": ([lambda w13=w13: ops.grouped_gemm_gateup_silu(h, w13, offs, tok, R, max_rows_per_group=T) for w13, _ in mlps],
                                      2 * (used * 2 * I * w + T * w + R * I), 4 * R * I * w),
            f"experts down{tag}": ([lambda w2=w2: ops.grouped_gemm_down(act, w2, offs, scale, experts if shared else 0, max_rows_per_group=T) for _, w2 in mlps],
                                   2 * (used * I * w + R * I + R * w), 2 * R * I * w)}


def gulozen_kernels(m, meta, mode, B, n):
    from nanovllm import hip_ops as ops
    cfg, res = m.config, m.residual
    T, w, dev, bf = meta.ids.numel(), cfg.hidden_size, meta.ids.device, torch.bfloat16
    rnd = lambda *s: torch.randn(*s, device=dev).to(bf)  # noqa: E731
    att, lin, L = [l for l in m.layers if l.spec.type == "latent_attention"], [l for l in m.layers if l.spec.type == "lightning"], list(m.layers)
    a, e, s0 = att[0].mixer, lin[0].mixer, cfg.layers[0]
    planes, x, h, y = torch.randn(LAYERS, T, w, device=dev), torch.randn(T, w, device=dev), rnd(T, w), rnd(T, w)
    out = {}
    top = s0.top
    rows = ops.ExpertRows(rnd(T * top, w), torch.randperm(T * top, device=dev).to(torch.int32), torch.rand(T, top, device=dev))
    out["depth_norm (inside a layer)"] = ([lambda l=l: res.inside(x, y, l.g_post1) for l in L], T * w * (4 + 2 + 4 + 2), 0)
    out["depth_norm (experts, average, convolution)"] = (
        [lambda i=i: res.behind(i, planes, x, rows, L[i].g_post2, L[i + 1].taps, meta) for i in range(LAYERS - 1)],
        T * w * (4 + 2 * top + 4 + 4 + 2) + T * w * 4 * sum(range(1, LAYERS)) / (LAYERS - 1), 0)

    def gemm(name, lins, inp, act=ops.NO_ACT):
        out[name] = ([lambda p=p: p(inp, act=act) for p in lins], *gemm_cost(T, lins[0].N, lins[0].K))

    H, hd, r, rc = a.heads, a.dimp + a.rotp, a.rp, a.rc
    gemm("gemm latents|gate", [l.mixer.qc_proj for l in att], h, a.act)
    gemm("gemm q from its latent", [l.mixer.uq_proj for l in att], rnd(T, a.uq_proj.K))
    gemm("gemm o", [l.mixer.o_proj for l in att], rnd(T, H * a.vdimp))
    qc, q, o = rnd(T, a.qc_proj.N), rnd(T, H * hd), torch.empty(T, H * a.vdimp, dtype=bf, device=dev)
    gate = qc[:, a.g_off:]
    cs = a.rot.table(meta.pos)
    query = (0, a.q_rank, a.cq_gain)
    if mode == "decode":
        tok, cnt = meta.tiles[1]
        qa = rnd(T, H, rc)
        out["latent rows (norms, rotation, store)"] = (
            [lambda x=l.mixer: ops.latent_rows(qc, x.c_off, x.rank, x.c_gain, cs, x.eps, meta.slots, x.caches[0], query) for l in att], 2 * T * 2 * (rc + a.c_off), 0)
        out["absorb"] = ([lambda x=l.mixer: ops.latent_absorb(q, H, x.dimp, cs, x.wukt, x.rotp) for l in att],
                         2 * (H * a.dimp * r + T * H * (hd + rc)), 2 * T * H * a.dimp * r)
        out["latent attention + merge, W_uv"] = (
            [lambda x=l.mixer: ops.latent_attn(qa, x.caches[0], tok, cnt, 1, meta.pos, meta.seq_of, meta.block_tables, x.window, x.scale, x.sink, x.wuv, o, gate=gate) for l in att],
            2 * (B * n * rc + H * a.vdimp * r + T * H * (rc + 2 * a.vdimp)), 2 * T * H * (n * (rc + r) + r * a.vdimp))
    else:
        win = meta.windows[a.window]
        c = rnd(win.rows, rc)
        kv = rnd(win.rows, a.expand.N)
        nk = H * a.dimp
        pairs = B * (n * (n + 1) // 2)
        out["latent rows (norms, rotation, store)"] = (
            [lambda x=l.mixer: ops.latent_rows(qc, x.c_off, x.rank, x.c_gain, cs, x.eps, meta.slots, x.caches[0], query, win.crow, win.rows) for l in att],
            2 * T * (3 * rc + 2 * a.c_off), 0)
        out["gemm expand k|v"] = ([lambda p=l.mixer.expand: p(c[:, :r]) for l in att], *gemm_cost(win.rows, a.expand.N, a.expand.K))
        out["attention"] = (
            [lambda x=l.mixer: ops.window_attn_prefill(q, kv[:, :nk], kv[:, nk:], o, meta.long_q_start, win.k_start, meta.long_tile_seq, meta.long_tile_off, H, hd, x.vdimp, x.window,
                                                       x.scale, x.sink, kr=c[:, r:], cs=cs, gate=gate) for l in att],
            2 * T * H * (hd + 2 * a.vdimp) + 2 * win.rows * (a.expand.N + a.rotp), 2 * pairs * H * (hd + a.vdimp))
    gemm("gemm memory q|k|v|g", [l.mixer.in_proj for l in lin], h, (ops.ACT_SILU_GATE, float(e.g_off), 0.0))
    mh, md, mv = e.heads, e.dimp, e.vdimp
    gemm("gemm memory o", [l.mixer.o_proj for l in lin], rnd(T, mh * mv))
    mx, my = rnd(T, e.in_proj.N), torch.empty(T, mh * mv, dtype=bf, device=dev)
    io = 2 * T * mh * (2 * md + 3 * mv)
    rest = lambda l: (l.mixer.state, meta.pos, meta.q_start, meta.state_in, meta.state_out, mh, md, mv)  # noqa: E731

    def memory(l):
        f = ops.linear_recurrent if mode == "decode" else ops.linear_chunkwise
        ops.row_norm_gate(f(mx, l.mixer.decay if mode == "decode" else l.mixer.powers, *rest(l)), mx[:, e.g_off:], l.mixer.norm, mh * l.mixer.vdim, l.mixer.eps, my)

    out["memory " + ("recurrent" if mode == "decode" else "chunkwise") + " + norm"] = ([lambda l=l: memory(l) for l in lin], io + 8 * B * mh * md * mv, 0)
    E = s0.experts
    out["gemm router"] = ([lambda l=l: l.mlp.router(h, out_f32=True) for l in L], 2 * (E * w + T * w + 2 * T * E), 2 * T * E * w)
    lg = torch.randn(T, E, device=dev)
    if mode == "decode":
        out["select + align"] = ([lambda: ops.softmax_router_align(lg, E, top) for l in L], 4 * T * E, 0)
    else:
        out["select"] = ([lambda: ops.softmax_router(lg, E, top) for l in L], 4 * T * E + 12 * T * top, 0)
    out.update(expert_kernels(h, [(l.mlp.w13, l.mlp.w2) for l in L], E, top, m.layers[0].mlp.ffp, False))
    return out



# ---- GLM-4-MoE's own layers -----------------------------------------------------------------------------------------------------
def glm_moe_model(size, dev):
    from nanovllm.models.glm4_moe.model import Glm4MoeForCausalLM
    w, heads, dim, _, _, _, _, experts, top, ff, vocab = SIZES[size][:11]
    cfg = types.SimpleNamespace(
        hidden_size=w, num_attention_heads=heads, num_key_value_heads=heads // 4, head_dim=dim, attention_bias=True, use_qk_norm=False, partial_rotary_factor=0.5,
        rope_theta=1e6, rope_scaling=None, max_position_embeddings=8192, rms_norm_eps=1e-5, n_routed_experts=experts, num_experts_per_tok=top, moe_intermediate_size=ff,
        intermediate_size=ff, n_group=1, topk_group=1, routed_scaling_factor=1.0, n_shared_experts=1, first_k_dense_replace=0, hidden_act="silu", vocab_size=vocab,
        num_hidden_layers=LAYERS, num_layers_to_load=LAYERS, tie_word_embeddings=False, torch_dtype=torch.bfloat16)
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


def glm_moe_kernels(m, cfg, mode, B, n, pos):
    """The attention half as beside the other designs, and the block of experts (shared one included)."""
    from nanovllm import hip_ops as ops
    L = list(m.model.layers)
    moes = [l.mlp for l in L]
    out = glm_kernels(m, cfg, mode, B, n, pos)     # (its dense feed-forwards are never run)
    out.pop("gemm gate|up + silu"), out.pop("gemm down")
    T, w = pos.numel(), cfg.hidden_size
    h = torch.randn(T, w, device=pos.device).to(torch.bfloat16)
    out.update(expert_kernels(h, [x._stacked() for x in moes], cfg.n_routed_experts, cfg.num_experts_per_tok, cfg.moe_intermediate_size, True))
    E = cfg.n_routed_experts
    if ops.router_by_gemm(T, E):
        out["gemm router"] = ([lambda x=x: ops.gemm_bf16(h, x.gate.weight.data) for x in moes], 2 * (E * w + T * w + T * E), 2 * T * E * w)
    return out


@torch.inference_mode()
def run(args) -> None:
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(0)
    from nanovllm import hip_ops
    from nanovllm.utils.context import reset_context
    hip_ops.load_library()
    for size in (args.design_sizes.split(",") if args.design_sizes else SIZES):
        m = gulozen_model(size, dev)
        glm, gcfg = glm_moe_model(size, dev)
        for name, (mode, B, n) in MODES.items():
            rec = {"design": "gulozen", "size": size, "mode": name, "layers": LAYERS, "dtype": "bf16", "data": "synthetic"}
            reps = args.steps if mode == "decode" else max(2, args.steps // 4)
            meta, toks = gulozen_step(m, mode, B, n, dev)
            step = graph_of(lambda: torch.argmax(m(meta), -1)).replay if mode == "decode" else (lambda: torch.argmax(m(meta), -1))
            us = time_us(step, reps, args.warmup)
            rec["gulozen"] = {"tokens_per_s": round(toks / us * 1e6, 1), "ms_per_step": round(us / 1e3, 3),
                              "kernels": kernel_table(gulozen_kernels(m, meta, mode, B, n), reps) if not args.no_extras else {}}
            del step, meta
            ids, pos = glm_step(glm, gcfg, mode, B, n, dev)
            body = lambda: torch.argmax(glm.compute_logits(glm(ids, pos)), -1)  # noqa: E731
            step = graph_of(body).replay if mode == "decode" else body
            us = time_us(step, reps, args.warmup)
            rec["glm4_moe"] = {"tokens_per_s": round(toks / us * 1e6, 1), "ms_per_step": round(us / 1e3, 3),
                               "kernels": kernel_table(glm_moe_kernels(glm, gcfg, mode, B, n, pos), reps) if not args.no_extras else {}}
            del step
            reset_context()
            torch.cuda.empty_cache()
            print(json.dumps(rec), flush=True)
        del m, glm
        torch.cuda.empty_cache()
