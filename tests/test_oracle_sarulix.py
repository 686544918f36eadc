"""The plain Sarulix implementation against what its equations fix, and the parts of the framework's
Sarulix code that need no GPU."""

import json
import math

import pytest
import torch
import torch.nn.functional as F

import sarulix_helpers as H
from astrai_amd.extension import _mix
from astrai_amd.model import MixerCache, SarulixConfig, SarulixLM, architecture_of, architectures, load_checkpoint
from astrai_amd.model.mixers import BlockDiagonal, PackedLinear, Rows, ShortConv, heads_of
from oracle import sarulix_oracle as S

F64 = torch.float64


def gen(seed=1):
    return torch.Generator().manual_seed(seed)


def randn(g, *size):
    return torch.randn(*size, generator=g, dtype=F64)


# ---------------------------------------------------------------- the plain implementation


def test_activations_and_norms():
    z = torch.linspace(-12, 12, 97, dtype=F64)
    assert torch.allclose(S.gelu_tanh(z), F.gelu(z, approximate="tanh"))
    assert torch.allclose(S.softplus(z), F.softplus(z)) and torch.allclose(S.sigmoid(z), torch.sigmoid(z))
    x = torch.tensor([[3.0, -1.0, 2.0, 0.0]], dtype=F64)
    assert torch.allclose(S.rms(x, 0.5), x / math.sqrt(14 / 4 + 0.5))
    assert torch.allclose(S.unit(x), x / math.sqrt(14 + 1e-6))


def test_sink_is_a_key_of_score_zero_without_a_value():
    s = torch.tensor([[-3.0, 0.5, float("-inf"), 2.0], [-900.0, -950.0, -901.0, -980.0], [900.0, 3.0, 2.0, 1.0]], dtype=F64)
    want = torch.softmax(torch.cat([s, torch.zeros(3, 1, dtype=F64)], -1), -1)[:, :4]
    assert torch.allclose(S.softmax_with_sink(s), want)


def test_attention_core_of_a_group():
    g = gen()
    q, k, v = randn(g, 5, 4, 6), randn(g, 5, 2, 6), randn(g, 5, 2, 3)
    out = S.attention_core(q, k, v, 0.3, 1.7)
    for h in range(4):
        for i in range(5):
            e = [math.exp(1.7 * math.tanh(0.3 * float(q[i, h] @ k[j, h // 2]) / 1.7)) for j in range(i + 1)]
            want = sum(x * v[j, h // 2] for j, x in enumerate(e)) / (1 + sum(e))
            assert torch.allclose(out[i, h], want)


def test_rotation_pairs_halves_and_leaves_the_rest():
    x = randn(gen(), 3, 2, 10)
    y = S.rotate_half(x, torch.arange(3), 6, 50.0)
    assert torch.equal(y[..., 6:], x[..., 6:]) and torch.equal(y[0], x[0])
    for i in range(3):
        a = 2 * 50.0 ** (-2 * i / 6)
        u, v = x[2, :, i], x[2, :, i + 3]
        assert torch.allclose(y[2, :, i], u * math.cos(a) - v * math.sin(a))
        assert torch.allclose(y[2, :, i + 3], v * math.cos(a) + u * math.sin(a))


def test_short_conv_looks_back_only():
    x, w = randn(gen(), 6, 2), randn(gen(2), 2, 3)
    y = S.short_conv(x, w)
    assert torch.allclose(y[0], x[0] * w[:, 2])
    assert torch.allclose(y[4], x[2] * w[:, 0] + x[3] * w[:, 1] + x[4] * w[:, 2])
    assert torch.allclose(S.short_conv(x, w[:, :1]), x * w[:, 0])


def test_linear_unit_is_a_decayed_sum_and_can_be_cut():
    g = gen()
    u, r, i, lam = randn(g, 9, 4), torch.rand(9, 4, dtype=F64), torch.rand(9, 4, dtype=F64), randn(g, 4)
    out, state = S.linear_unit_scan(u, r, i, lam)
    a = torch.exp(-8 * r * F.softplus(lam))
    want = sum(a[j + 1:].prod(0) * torch.sqrt(1 - a[j] ** 2) * i[j] * u[j] for j in range(9))
    assert torch.allclose(out[-1], want) and torch.equal(state, out[-1])
    x, s = S.linear_unit_scan(u[:4], r[:4], i[:4], lam)
    y, s = S.linear_unit_scan(u[4:], r[4:], i[4:], lam, s)
    assert torch.allclose(torch.cat([x, y]), out) and torch.allclose(s, state)


def test_delta_rule_replaces_what_a_key_held():
    """With unit keys, no decay and beta = 1 a write leaves exactly its value under its key."""
    g = gen()
    k, v, q = S.unit(randn(g, 7, 1, 5)), randn(g, 7, 1, 3), randn(g, 7, 1, 5)
    one = torch.ones(7, 1, 5, dtype=F64)
    out, s = S.delta_scan(q, k, v, one, one[..., 0])
    assert torch.allclose(s[0].T @ k[-1, 0], v[-1, 0], atol=1e-5) and torch.allclose(out[-1, 0], s[0].T @ q[-1, 0])
    # decays act on the rows of the key channels, before the read that the write corrects
    dec = torch.rand(2, 1, 5, dtype=F64, generator=g)
    beta = torch.tensor([[0.3], [0.8]], dtype=F64)
    out, s2 = S.delta_scan(q[:2], k[:2], v[:2], dec, beta)
    s1 = torch.outer(k[0, 0], 0.3 * v[0, 0])
    d1 = dec[1, 0][:, None] * s1
    want = d1 + torch.outer(k[1, 0], 0.8 * (v[1, 0] - d1.T @ k[1, 0]))
    assert torch.allclose(s2[0], want) and torch.allclose(out[1, 0], want.T @ q[1, 0])


def test_layer_order():
    cfg = H.mixed()
    want = [(0, None)] + [(i, t if i == 1 else None) for t in range(3) for i in (1, 2, 3)] + [(4, None), (5, None)]
    assert S.layer_order(cfg) == want
    got = SarulixConfig.from_dict(cfg).order()
    assert [(i, t if begins else None) for i, t, begins in got] == want
    assert [t for _, t, _ in got] == [0, 0, 0, 0, 1, 1, 1, 2, 2, 2, 0, 0]
    none = SarulixConfig.from_dict(H.mixed(loop=(0, 0, 0)))
    assert none.order() == [(i, 0, False) for i in range(6)]
    assert SarulixConfig.from_dict(H.mixed(loop=(0, 6, 1))).order() == [(i, 0, i == 0) for i in range(6)]


def test_loop_of_the_plain_implementation_by_hand():
    """One layer run twice: what enters each pass, spelled out."""
    cfg = H.config([H.rglru(width=24, blocks=2)], width=20, vocab=11, loop=(0, 1, 2))
    w = {k: t.double() for k, t in H.tensors(cfg).items()}
    ids = torch.tensor([3, 1, 7])
    x = x0 = w["embed"][ids] * 2.5
    for t in range(2):
        x = x @ w["loop.in"][:, :20].T + x0 @ w["loop.in"][:, 20:].T + w["loop.step"][t]
        x = x + S.rglru(S.rms(x, 1e-2) * (1 + w["l0.norm1"]), w, "l0.mix.", cfg["layers"][0]["mixer"])
    want = S.rms(x, 1e-2) * (1 + w["final.norm"]) @ w["head"].T * 0.4
    layers = []
    assert torch.allclose(S.forward(cfg, w, ids, layers_out=layers), want) and len(layers) == 2


# ---------------------------------------------------------------- configuration and weights


def test_registry_and_configuration():
    assert "Sarulix" in architectures()
    cfg = H.mixed()
    arch = architecture_of(cfg)
    made = arch.configure(cfg, H.tensors(cfg, ranks=(12, 20)))
    assert arch.model_class is SarulixLM and made.loop == (1, 4, 3) and made.ranks == {0: (12, 20), 3: (12, 20)}
    assert made.embedding_scale == 2.5 and made.logit_scale == 0.4 and made.eps == 1e-2
    for loop in ((2, 2, 1), (0, 7, 1), (-1, 2, 1), (0, 2, 0)):
        with pytest.raises(ValueError, match="loop"):
            SarulixConfig.from_dict(dict(cfg, loop=dict(zip(("start", "stop", "times"), loop))))
    assert SarulixConfig.from_dict(dict(cfg, loop=None)).loop == (0, 0, 0)


def test_bad_layers_are_refused():
    def build(layer):
        return SarulixLM(SarulixConfig.from_dict(H.config([layer])))
    with pytest.raises(ValueError, match="unknown mixer"):
        build(dict(H.rglru(), type="other"))
    with pytest.raises(ValueError, match="equal blocks"):
        build(H.rglru(width=90, blocks=4))
    with pytest.raises(ValueError, match="share"):
        build(H.attention(heads=5, kv_heads=2))
    with pytest.raises(ValueError, match="share"):
        build(H.delta(heads=3, kv_heads=2))
    with pytest.raises(ValueError, match="rotation over 26 of 24"):
        build(H.attention(dim=24, rot=26))
    with pytest.raises(ValueError, match="feed-forward"):
        build(dict(H.rglru(), mlp={"kind": "sparse", "ff": 8}))


def test_weights_arrive_where_they_belong():
    cfg = H.mixed()
    w = H.tensors(cfg, 3)
    model = SarulixLM(architecture_of(cfg).configure(cfg, w)).load_tensors(w)
    x = torch.randn(4, 88, generator=gen().manual_seed(2))
    a = model.layers[2].mix
    got = a.in_proj(x)
    want = x @ w["l2.mix.k"].float().T + w["l2.mix.k.b"].float()
    off = a.in_proj.offset["k"]
    got_k = got[:, off:off + 96].reshape(4, 3, 32)
    assert torch.allclose(got_k[..., :24].reshape(4, 72), want, atol=1e-5) and got_k[..., 24:].count_nonzero() == 0
    assert torch.equal(a.q_norm.weight[:24], w["l2.mix.q.norm"].float())
    r = model.layers[1].mix
    assert torch.allclose(r.coef.weight.reshape(3, 32)[:, :30].reshape(-1),
                          (-8 * F.softplus(w["l1.mix.lam"].double())).float())
    assert torch.equal(r.conv.weight.reshape(4, 3, 32)[..., :30].reshape(4, 90), w["l1.mix.conv"].float().T)
    assert torch.equal(r.r.weight[1, :30, :30], w["l1.mix.ra"][1].float())
    d = model.layers[3].mix
    assert torch.allclose(d.decay.weight, w["l3.mix.A_log"].double().exp().float())
    assert torch.allclose(model.layers[0].norm1.weight, 1 + w["l0.norm1"].float())
    assert torch.allclose(model.final_norm.weight, (1 + w["final.norm"].float()) * 0.4)
    x0 = torch.randn(4, 88, generator=gen().manual_seed(4))
    both = F.linear(x, model.loop_in.weight[:88]) + F.linear(x0, model.loop_in.weight[model.loop_in.offset["b"]:])[:, :88]
    assert torch.allclose(both, torch.cat([x, x0], 1) @ w["loop.in"].float().T, atol=1e-5)
    # what kernels read in fp32 stays so in a bf16 model
    model.to(torch.bfloat16)
    assert r.coef.weight.dtype == r.conv.weight.dtype == d.dt_bias.weight.dtype == torch.float32
    assert r.r.weight.dtype == model.loop_in.weight.dtype == torch.bfloat16


def test_checkpoint_errors_name_the_tensor(tmp_path):
    import safetensors.torch as st
    cfg = H.mixed()
    (tmp_path / "config.json").write_text(json.dumps(cfg))

    def load(**change):
        w = {k: t for k, t in {**H.tensors(cfg), **change}.items() if t is not None}
        st.save_file(w, str(tmp_path / "model.safetensors"))
        return load_checkpoint(str(tmp_path), "cpu", torch.float32)

    model = load()
    assert isinstance(model, SarulixLM) and model.layers[0].mix.a2.inputs.size == 12
    with pytest.raises(ValueError, match="l2.mix.o.b is missing"):
        load(**{"l2.mix.o.b": None})
    with pytest.raises(ValueError, match="l0.mix.g1 is missing"):
        load(**{"l0.mix.g1": None})
    with pytest.raises(ValueError, match="loop.step has shape"):
        load(**{"loop.step": torch.zeros(2, 88)})
    with pytest.raises(ValueError, match="unexpected .*stray"):
        load(stray=torch.zeros(1))


def test_packed_biases_block_matrices_and_taps():
    lin = PackedLinear(Rows("h", 1, ((6, 6),)), [heads_of("q", 2, 3), heads_of("g", 1, 5)], biased=("q",))
    assert lin.expected() == {"q": (6, 6), "g": (5, 6), "q.b": (6,)}
    lin.reset_parameters()
    lin.assign("q.b", torch.arange(6.0) + 1)
    assert lin.bias.reshape(3, 32)[:, :3].tolist() == [[1, 2, 3], [4, 5, 6], [0, 0, 0]] and lin.bias.count_nonzero() == 6
    block = BlockDiagonal(heads_of("u", 2, 3))
    block.assign(torch.arange(18.0).reshape(2, 3, 3), torch.arange(6.0).reshape(2, 3))
    block.finalize(True)
    assert block.weight.shape == (2, 32, 32) and torch.equal(block.transposed[1, :3, :3], torch.arange(9.0, 18).reshape(3, 3).T)
    conv = ShortConv([heads_of("q", 1, 2), heads_of("v", 1, 1)], 3)
    conv.assign([torch.tensor([[1.0, 2, 3], [4, 5, 6]]), torch.tensor([[7.0, 8, 9]])])
    assert conv.weight.shape == (3, 64) and conv.weight[:, 0].tolist() == [1, 2, 3] and conv.weight[:, 32].tolist() == [7, 8, 9]
    assert conv.weight[:, 1].tolist() == [4, 5, 6] and conv.bias is None


def test_every_pass_has_its_own_cache():
    model = SarulixLM(SarulixConfig.from_dict(H.mixed()))
    cache = model.new_cache(2, 10)
    assert isinstance(cache, MixerCache)
    assert sorted(cache.rows) == [(2, 0), (2, 1), (2, 2), (4, 0)]
    assert sorted(cache.state) == sorted(cache.ring) == [(0, 0), (1, 0), (1, 1), (1, 2), (3, 0), (3, 1), (3, 2), (5, 0)]
    assert cache.rows[2, 1].shape == (2, 10, 3 * (32 + 64)) and cache.ring[3, 0].shape == (2, 1 + 8, 2 * 32 + 3 * 96)
    assert cache.state[0, 0].shape == (2, 4, 64, 32) and cache.state[1, 0].shape == (2, 96)
    cache.state[1, 2].fill_(1.0)
    cache.advance(3)
    cache.reset()
    assert cache.tokens == 0 and cache.state[1, 2].count_nonzero() == 0


def test_launch_plans():
    s = _mix.GqaShape(16, 4, 128, 128, 128, 0.1)
    assert _mix.gqa_rows_nsplit(s, 32, 1, 1024) == 4 and _mix.gqa_rows_nsplit(s, 1, 1, 200) == 1
    assert _mix.gqa_rows_nsplit(s, 1, 1, 1 << 20) == _mix.MAX_SPLIT
    assert _mix.rglru_nseg(32, 8, 256, 512) == 1 and _mix.rglru_nseg(1, 1, 64, 100) == 1
    assert _mix.rglru_nseg(1, 8, 256, 4096) > 1 and _mix.ring_rows(4) == 3 + _mix.RING_STEPS


# ---------------------------------------------------------------- the C ABI without a GPU


def test_mix_registry_names():
    from astrai_amd.extension import KERNEL_NAMES, get_module, is_available
    for name in ("grouped_attention", "gated_recurrence", "delta_rule"):
        assert name in KERNEL_NAMES and is_available(name)
    assert get_module("delta_rule").delta_chunk is _mix.delta_chunk


def test_arguments_are_validated_before_anything_is_launched():
    """16 stands for an aligned non-null pointer that is never dereferenced."""
    lib = _mix.load()
    assert lib is not None, _mix.load_error()
    P, N = 16, None

    def err():
        return lib.astrai_mix_last_error().decode()

    norm = lambda y, ldy, u, ldu, w=8, d=0: lib.astrai_mix_sum_norm(y, ldy, N, 4, 1.0, N, u, ldu, N, P, N, P, 4, w, 1e-6, 0, d, N)
    assert norm(N, 8, N, 0) == 1 and "null" in err()
    assert norm(P, 7, N, 0) == 1 and "bad size" in err()
    assert norm(P, 8, P, 4) == 1 and "bad size" in err()
    assert norm(8, 8, N, 0) == 1 and "aligned" in err()
    assert norm(P, 8, N, 0, d=5) == 1 and "dtype" in err()
    assert lib.astrai_mix_act_mul(P, P, 4, 16, 2, 0, N) == 1 and "activation" in err()
    assert lib.astrai_mix_head_gated_rms_norm(P, P, 64, P, P, 4, 3, 32, 32, 1e-6, 0, N) == 1
    ap = lambda k, v, half, h=4, kh=2, dim=24, dk=32: lib.astrai_mix_gqa_append(
        P, 320, k, v, P, 64, half, P, P, P, P, 1, 8, 64, h, kh, dk, 32, dim, 1e-6, 0, N)
    assert ap(128, 192, 13) == 1 and "bad columns" in err()
    assert ap(100, 192, 8) == 1 and "bad columns" in err()
    assert ap(128, 192, 8, kh=3) == 1 and "bad heads" in err()
    assert ap(128, 192, 8, dk=40) == 1 and "multiples of 32" in err()
    pre = lambda start, g, dk=32, scale=0.5: lib.astrai_mix_gqa_prefill(P, 640, g, P, P, 1, 30, 64, start, 4, 2, dk, 32, 9, scale, 5.0, 1, N)
    assert pre(35, 192) == 1 and "tokens" in err()
    assert pre(0, 600) == 1 and "gate" in err()
    assert pre(0, 192, dk=160) == 2 and pre(0, 192, scale=1e-6) == 2
    rows = lambda nsplit, dk=32: lib.astrai_mix_gqa_rows(P, 1280, -1, P, P, P, P, 1, 2, 64, 4, 2, dk, 32, 9, 0.5, 0.0, 0, nsplit, N)
    assert rows(65) == 1 and "nsplit" in err()
    assert rows(1, 288) == 2
    assert not _mix.gqa_rows_supported(_mix.GqaShape(4, 2, 288, 32, 288, 0.5), 64)
    assert lib.astrai_mix_gqa_rows_general(P, 8192, -1, P, P, P, 1, 2, 64, 4, 2, 1056, 32, 9, 0.5, 0.0, 0, 1, N) == 2
    assert lib.astrai_mix_conv(P, 64, 8, 60, P, N, 4, P, P, P, 1, 5, 0, 1, 0, N) == 1 and "columns" in err()
    assert lib.astrai_mix_conv(P, 64, 0, 64, P, N, 0, P, P, P, 1, 5, 0, 1, 0, N) == 1 and "taps" in err()
    ch = lambda bp, nseg, scratch: lib.astrai_mix_rglru_chunk(P, P, 4096, 0, P, P, P, P, P, P, scratch, P, 1, 300, 2, bp, nseg, N)
    assert ch(40, 1, N) == 1 and ch(64, 2, N) == 1 and ch(64, 400, P) == 1 and ch(1056, 1, N) == 2
    st = lambda seq: lib.astrai_mix_rglru_step(P, 256, 0, 128, P, P, 4, P, P, P, P, P, P, P, P, P, 1, seq, 2, 64, N)
    assert st(9) == 2 and "tokens" in err()
    de = lambda qkv, seq, dp=32, vp=32, ldg=128: lib.astrai_mix_delta_step(
        qkv, P, 8192, 0, 320, P, 3, P, P, P, P, P, P, ldg, P, P, P, 1, seq, 4, 2, dp, vp, 24, 0.2, 1e-6, 0, N)
    assert de(N, 9) == 2 and de(P, 9, vp=288, ldg=2048) == 2 and de(P, 9, dp=512, vp=256, ldg=2048) == 2
    assert de(P, 9, ldg=96) == 1 and "gate" in err()
    assert lib.astrai_mix_delta_chunk(P, P, 8192, 320, P, P, P, P, P, P, 1, 40, 4, 2, 288, 32, 0.2, N) == 2
    assert lib.astrai_mix_delta_image_bytes(288) == 0 and lib.astrai_mix_delta_image_bytes(128) == 27 * 1024
    assert not _mix.delta_step_supported(_mix.DeltaShape(4, 2, 512, 256, 200, 0.2))
    assert _mix.delta_step_supported(_mix.DeltaShape(4, 2, 256, 256, 200, 0.2))
