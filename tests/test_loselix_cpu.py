"""Loselix without a GPU: configuration and registry, layouts of the joint projections, tensor-parallel slices, and the plain evaluation's
mechanisms against values worked out by hand."""
import copy
import math
import types

import pytest
import torch

from loselix_util import CONFIGS, config, gated, make_model, sigmoid, two_maps
from oracle import loselix_oracle as O

D = torch.float64


def t64(x):
    return torch.tensor(x, dtype=D)


def sg(z):
    return 1 / (1 + math.exp(-z))


# ---- mechanisms of the plain evaluation ------------------------------------------------------------------------------------
def test_rotation_by_hand():
    """Column i turns with column i + dims / 2; columns behind dims stay."""
    x = t64([[1.0, 2.0, 3.0, 4.0, 5.0, 6.0]]).repeat(3, 1)
    got = O.rotate_half(x, {"base": 100.0, "dims": 4})
    for p in range(3):
        for i, f in enumerate((1.0, 0.1)):
            u, v, a = float(x[p, i]), float(x[p, i + 2]), p * f
            assert abs(got[p, i] - (u * math.cos(a) - v * math.sin(a))) < 1e-12 and abs(got[p, i + 2] - (v * math.cos(a) + u * math.sin(a))) < 1e-12
        assert got[p, 4:].tolist() == [5.0, 6.0]
    from nanovllm.layers.rotary_embedding import HalfRotary
    assert HalfRotary(6, 4, 100.0).freq == (1.0, 0.1) and HalfRotary(6, 4, 100.0).pairs == 2 and HalfRotary(6, 4, 100.0).key == HalfRotary(9, 4, 100.0).key
    for bad in ((8, 10), (8, 3), (8, 0)):
        with pytest.raises(ValueError, match="rotation"):
            HalfRotary(*bad, 100.0)


def test_temperature_by_hand():
    got = O.query_temperature(7, {"coef": 0.5, "every": 3}, D)
    assert torch.allclose(got, t64([1, 1] + [1 + 0.5 * math.log(2)] * 3 + [1 + 0.5 * math.log(3)] * 2))
    assert torch.allclose(O.query_temperature(3, {"coef": 2.0, "every": 1}, D), t64([1 + 2 * math.log(n) for n in (2, 3, 4)]))


def test_two_maps_by_hand():
    """One head of one column per map that does not turn (position 0 and 1 with a tiny frequency), values of two columns."""
    W = O.Weights({"q": torch.tensor([[1.0], [0.0], [2.0], [0.0]]), "k": torch.tensor([[3.0], [0.0], [1.0], [0.0]]), "v": torch.tensor([[1.0], [2.0]]), "o": torch.eye(2),
                   "lq1": torch.tensor([0.5, 1.0]), "lk1": torch.tensor([0.2, 0.3]), "lq2": torch.tensor([1.0, 0.0]), "lk2": torch.tensor([-0.7, 9.0])})
    spec = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 0.25, "softcap": 2.0, "diff": 0.3, "rot": {"base": 1e30, "dims": 2}}
    spec["rot"]["base"] = 1.0          # (the frequency is one: the pair turns by the position)
    h = t64([[2.0], [-3.0]])
    lam = math.exp(0.1 + 0.3) - math.exp(-0.7) + 0.3
    assert abs(O.map_weight(W, "", 0.3) - lam) < 1e-6
    from nanovllm.layers.group_attention import map_weight
    assert abs(map_weight(W.t, 0.3) - lam) < 1e-6
    c = math.cos(1.0)                  # query at 1, key at 0: the product of first columns times cos 1
    res = []
    for a, b in ((1.0, 3.0), (2.0, 1.0)):
        s = [2 * math.tanh(a * -3 * b * 2 * c * 0.25 / 2), 2 * math.tanh(a * -3 * b * -3 * 0.25 / 2)]
        e = [math.exp(z) for z in s]
        res.append([(e[0] * 2 * m + e[1] * -3 * m) / sum(e) for m in (1, 2)])
    d = [x - lam * y for x, y in zip(*res)]
    r = math.sqrt((d[0] ** 2 + d[1] ** 2) / 2 + 1e-3)
    got = O.differential(h, W, "", spec, 1e-3, O.Project())
    assert torch.allclose(got[1], t64([0.7 * d[0] / r, 0.7 * d[1] / r]))


def test_sigmoid_attention_by_hand():
    """Norms over both heads at once, one key head for two query heads, weights that are not normalised, values that are the raw keys."""
    W = O.Weights({"q": torch.tensor([[3.0], [4.0]]), "k": torch.tensor([[2.0]]), "q.norm": torch.tensor([1.0, 2.0]), "k.norm": torch.tensor([1.5]), "pb": torch.tensor([-1.0, 0.5]),
                   "g": torch.tensor([[0.1], [0.2]]), "o": torch.eye(2)})
    spec = {"heads": 2, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 0.5, "q_temp": {"coef": 1.0, "every": 2}}
    h = t64([[1.0], [-2.0]])
    got = O.sigmoid_attention(h, W, "", spec, 0.25, O.Project())
    kn = [1.5 * 2 / math.sqrt(4 + 0.25), 1.5 * -4 / math.sqrt(16 + 0.25)]
    rq, temp = math.sqrt((36 + 64) / 2 + 0.25), 1 + math.log(2)
    for i, (a, gain, pb, gate) in enumerate(((-6.0, 1.0, -1.0, 0.1), (-8.0, 2.0, 0.5, 0.2))):
        q = a / rq * gain * temp
        want = sum(sg(q * kn[j] * 0.5 + pb) * raw for j, raw in enumerate((2.0, -4.0))) * sg(gate * -2.0)
        assert abs(got[1, i] - want) < 1e-7


def test_gated_heads_by_hand():
    W = O.Weights({"q": torch.tensor([[1.0], [0.0], [0.5], [0.0]]), "k": torch.tensor([[1.0], [0.0]]), "v": torch.tensor([[2.0]]), "g": torch.tensor([[1.0], [-1.0]]), "o": torch.eye(2)})
    spec = {"heads": 2, "kv_heads": 1, "dim": 2, "vdim": 1, "scale": 0.7, "rot": {"base": 1.0, "dims": 2}}
    got = O.gated_heads(t64([[1.0], [3.0]]), W, "", spec, 1e-5, O.Project())
    for i, (a, gt) in enumerate(((1.0, 3.0), (0.5, -3.0))):
        e = [math.exp(a * 3 * 1 * math.cos(1.0) * 0.7), math.exp(a * 3 * 3 * 0.7)]
        assert abs(got[1, i] - (e[0] * 2 + e[1] * 6) / sum(e) * sg(gt)) < 1e-7


def test_layer_and_loop_by_hand():
    """Both sublayers read one norm; the embedding comes in again ahead of every pass but the first."""
    assert O.layer_order(CONFIGS["odd"]) == [(0, False), (1, False), (2, False), (1, True), (2, False)]
    assert O.layer_order(CONFIGS["tall"]) == [(i, t > 0 and i == 0) for t in range(3) for i in range(3)]
    assert O.layer_order(CONFIGS["wide"]) == [(0, False), (1, False), (2, False)]
    cfg = config(8, 9, [gated(1, 1, 4, 4, 8), sigmoid(1, 1, 4)], (0, 2, 3))
    t = O.random_tensors(cfg, 1)
    t["l0.mix.o"], t["l1.mix.o"] = torch.zeros_like(t["l0.mix.o"]), torch.zeros_like(t["l1.mix.o"])
    layers = []
    O.forward(cfg, t, [3, 5], layers_out=layers)
    e = t["embed"][[3, 5]].double()
    x = e
    for p in range(3):
        x = x + e if p else x
        h = O.norm_plain(x, t["l0.norm1"].double(), 1e-5)
        x = x + (torch.clamp(h @ t["l0.mlp.up"].double().T, min=0) ** 2) @ t["l0.mlp.down"].double().T
        assert torch.allclose(layers[2 * p], x) and torch.allclose(layers[2 * p + 1], x)


# ---- configuration and registry -----------------------------------------------------------------------------------------------
def test_registry_and_config(tmp_path):
    from nanovllm.config import Config
    from nanovllm.engine.key_reach import EVERYTHING
    from nanovllm.models.layer_loop import layer_runs, run_indices
    from nanovllm.models.loselix.config import read_config
    from nanovllm.models.registry import find_model
    assert find_model({"architecture": "Loselix"}).name == "loselix" and find_model({"architecture": "Gulozen"}).name == "gulozen"
    make_model(tmp_path, "odd")
    c = Config(str(tmp_path), dtype="float32", max_model_len=100000, max_num_batched_tokens=64)
    hf = c.hf_config
    assert c.kvcache_block_size == 64 and hf.torch_dtype == torch.float32 and hf.key_reach.windows == (EVERYTHING,) and hf.key_reach.first_visible(5000) == 0
    a, b, e = hf.layers
    assert (a.type, a.heads, a.kv_heads, a.dim, a.vdim, a.ff, a.rot_dims, a.diff, a.softcap) == ("attention", 4, 2, 20, 12, 100, 6, 0.7, 9.0)
    assert (b.type, b.ff, b.temp_coef, b.temp_every) == ("attention_3", 0, 0.7, 7) and (e.rot_dims, e.rot_base, e.vdim) == (12, 10000.0, 28)
    assert layer_runs(hf) == [(0, None), (1, 0), (2, None), (1, 1), (2, None)] and run_indices(hf) == ([0, 0, 0, 1, 1], [1, 2, 2])
    assert read_config(CONFIGS["wide"]).loop is None and read_config(CONFIGS["wide"]).rms_norm_eps == 1e-3
    without = {k: v for k, v in CONFIGS["wide"].items() if k != "loop"}
    assert read_config(without).loop is None
    with pytest.raises(ValueError):
        Config(str(tmp_path), dtype="float16")


@pytest.mark.parametrize("edit,match", [
    (lambda c: c["layers"][1].update(type="mystery"), "mystery"), (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "sparse"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(sections=[1, 2]), "sections"), (lambda c: c["layers"][0]["mixer"].update(softcap=0), "soft cap"),
    (lambda c: c["layers"][1]["mixer"].update(vdim=24), "keys of 20 columns that are values of 24"), (lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=0), "every 0"),
    (lambda c: c["layers"][2]["mixer"].update(kv_heads=2), "group up"), (lambda c: c["loop"].update(stop=4), "does not fit"), (lambda c: c["layers"][2]["mlp"].update(ff=0), "positive")])
def test_what_the_design_does_not_have_is_refused(edit, match):
    from nanovllm.models.loselix.config import read_config
    c = copy.deepcopy(CONFIGS["odd"])
    edit(c)
    with pytest.raises((NotImplementedError, ValueError), match=match):
        read_config(c)


def test_loader_reports_missing_tensors(tmp_path):
    from nanovllm.models.loselix.config import read_config
    from nanovllm.models.loselix.model import LoselixForCausalLM
    cfg, t = make_model(tmp_path, "odd")
    LoselixForCausalLM(read_config(cfg)).load_weights(str(tmp_path))
    for name in ("l0.mix.lq2", "l1.mix.pb", "l1.mix.q.norm", "l2.mix.g", "l0.mlp.up"):
        O.write_model(str(tmp_path / name), cfg, {k: v for k, v in t.items() if k != name})
        with pytest.raises(KeyError, match=name.split(".")[-1]):
            LoselixForCausalLM(read_config(cfg)).load_weights(str(tmp_path / name))


def test_cache_sizes_and_tiles():
    """Keys that are values are kept once, with one number per token; every pass of the loop has its own cache."""
    from nanovllm.models.loselix.config import read_config
    from nanovllm.models.loselix.model import LoselixForCausalLM
    m = LoselixForCausalLM(read_config(CONFIGS["odd"]))
    m.dtype = torch.bfloat16
    one = [2 * 2 * (2 * 24 + 16), 3 * 24 * 2 + 4, 2 * (16 + 32)]
    assert [layer.mixer.cache_bytes_per_token() for layer in m.layers] == [one[0], 2 * one[1], 2 * one[2]]
    assert m.cache_bytes_per_token() == one[0] + 2 * one[1] + 2 * one[2] and m.state_bytes_per_slot() == 0
    m.allocate(3, 64, 2, "cpu")
    caches = [c for layer in m.layers for c in layer.mixer.caches]
    assert len(caches) == 5 and len({c[0].data_ptr() for c in caches}) == 5
    assert sum(sum(t.numel() * t.element_size() for t in {id(x): x for x in c if x is not None}.values()) for c in caches) == 3 * 64 * m.cache_bytes_per_token()
    assert m.tile_sizes == [4, 5, 8] and m.chunk_tiles == [(0, 64), (0, 128)]
    assert not any(layer.mixer.tiled for layer in LoselixForCausalLM(read_config(dict(CONFIGS["huge"], layers=CONFIGS["huge"]["layers"][:2], loop=None))).layers)


# ---- tensor parallelism -----------------------------------------------------------------------------------------------------------
def test_tensor_parallel_slices_add_up(monkeypatch):
    """Two ranks' heads and feed-forward columns, evaluated in plain arithmetic over the loaded (padded, sliced) joint projections: the sum
    over the ranks is what the whole model's layer adds to the residual."""
    from nanovllm.layers import group_attention, parallel_block
    from nanovllm.models.loselix.config import read_config
    from nanovllm.models.loselix.model import make_mixer
    cfg = config(40, 64, [two_maps(4, 2, 12, 20, 44), gated(8, 4, 12, 20, 24, dims=8), sigmoid(6, 2, 20, None, 0.7, 5)])
    t = {k: v.float() for k, v in O.random_tensors(cfg, 3).items()}
    T = 21
    h = torch.randn(T, 40, generator=torch.Generator().manual_seed(1))
    W, hd, hf = O.Weights(t), h.double(), read_config(cfg)
    hf.torch_dtype = torch.float32
    part = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p)}  # noqa: E731
    for i, e in enumerate(cfg["layers"]):
        spec, p, got = e["mixer"], f"l{i}.", 0.0
        want = O.MIXERS[e["type"]](hd, W, p + "mix.", spec, 1e-5, O.Project())
        if e["mlp"]:
            want = want + O.relu_squared(hd @ W[p + "mlp.up"].T) @ W[p + "mlp.down"].T
        for rank in range(2):
            grp = types.SimpleNamespace(world_size=2, rank=rank)
            for mod in (group_attention, parallel_block):
                monkeypatch.setattr(mod, "get_tp_group", lambda: grp)
            mx = make_mixer(hf, hf.layers[i], 1)
            b = parallel_block.ParallelBlock(40, mx, hf.layers[i].ff, torch.float32)
            b.load(part(p + "mix."), part(p + "mlp."), "cpu")
            z = (h @ b.in_proj.weight.T).double()
            unit, x = torch.clamp(z[:, : b.ffp], min=0) ** 2, z[:, b.ffp:]
            if mx.gate or b.ff:
                assert b.act[1:] == (b.ffp, b.ffp + mx.g_off if mx.gate else 1 << 24)
            H, G, d, R = mx.heads, mx.kv_heads, mx.dimp, mx.heads // mx.kv_heads
            out = torch.zeros(T, H, mx.vdimp, dtype=D)
            if e["type"] == "attention_3":
                q, k = x[:, : mx.k_off].view(T, mx.q_heads, d), x[:, mx.k_off: mx.g_off].view(T, mx.k_heads, d)
                rms = lambda v, n: torch.sqrt(v.reshape(T, -1).pow(2).sum(-1) / n + 1e-5)[:, None, None]  # noqa: E731
                q = q / rms(q, mx.q_heads * 20) * mx.gain.view(mx.q_heads, d) * O.query_temperature(T, spec["q_temp"], D)[:, None, None]
                ks = 1 / rms(k, mx.k_heads * 20)[:, 0, 0]
                for j in range(H):
                    kj = k[:, rank * G + j // R]
                    out[:, j] = O.sigmoid_weights((q[:, rank * H + j] @ kj.T) * ks * mx.scale, mx.parts.bias[j].double()) @ kj
                gate = O.sigmoid(x[:, mx.g_off:]).view(T, H, -1)
            else:
                q, k = (O.rotate_half(x[:, a: c].reshape(T, -1, d), spec["rot"]) for a, c in ((0, mx.k_off), (mx.k_off, mx.v_off)))
                v = x[:, mx.v_off: mx.v_off + G * mx.vdimp].view(T, G, -1)
                for j in range(H):
                    if mx.maps == 2:
                        a = [O.causal_softmax(O.soft_cap(q[:, 2 * j + m] @ k[:, 2 * (j // R) + m].T * mx.scale, mx.cap)) @ v[:, j // R] for m in (0, 1)]
                        o = a[0] - mx.parts.lam * a[1]
                        out[:, j] = mx.parts.post * o / torch.sqrt(o.pow(2).sum(-1, keepdim=True) / mx.parts.vn + 1e-5)
                    else:
                        out[:, j] = O.causal_softmax(q[:, j] @ k[:, j // R].T * mx.scale) @ v[:, j // R]
                gate = O.sigmoid(x[:, mx.g_off: mx.g_off + H])[..., None] if mx.gate else 1.0
            got = got + torch.cat([(out * gate).reshape(T, -1), unit], 1) @ b.out_proj.weight.double().T
        assert torch.allclose(got[:, :40], want, atol=3e-5, rtol=1e-4), e["type"]
    for args in ((30, 4, 2, 8, 8), (30, 12, 3, 8, 8)):
        monkeypatch.setattr(group_attention, "get_tp_group", lambda: types.SimpleNamespace(world_size=8, rank=0))
        with pytest.raises(ValueError, match="do not split"):
            group_attention.GroupAttention(*args, 0.3, torch.float32, joint=True)


def test_parts_that_do_not_go_together():
    from nanovllm.layers.group_attention import GroupAttention
    for bad in (dict(sigmoid_kv=True, cap=3.0), dict(sigmoid_kv=True, diff=0.1), dict(sigmoid_kv=True, own_kv=False)):
        with pytest.raises(ValueError, match="go together"):
            GroupAttention(32, 4, 2, 8, 8, 0.3, torch.bfloat16, joint=True, **bad)
    assert not GroupAttention(32, 4, 2, 8, 8, 0.3, torch.bfloat16, joint=True, cap=3.0).tiled and GroupAttention(32, 4, 2, 8, 8, 0.3, torch.bfloat16, joint=True, cap=3.0, diff=0.2).tiled
