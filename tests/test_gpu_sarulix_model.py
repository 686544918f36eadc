"""Sarulix models through the framework's forward, caches and greedy generation, against the plain
implementation in float64."""

import json
import os

import pytest
import torch

import sarulix_helpers as H
from astrai_amd.model import RequestCaches, SarulixLM, architecture_of, greedy_generate, load_checkpoint
from oracle import sarulix_oracle as S
from sarulix_helpers import relative_rms as worst_rms

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
# the worst token's error; that of all tokens together stays below a third of it
TOL = {torch.float32: 2e-5, torch.bfloat16: 6e-2}
DTYPES = [torch.float32, torch.bfloat16]


def relative_rms(got, want):
    """The worst row's relative error, or three times that of all rows if this is larger."""
    d, w = got.double().cpu() - want.double().cpu(), want.double().cpu()
    return max(worst_rms(got, want), 3 * (d.pow(2).mean() / w.pow(2).mean()).sqrt().item())


def build(cfg, weights, dtype):
    config = architecture_of(cfg).configure(cfg, weights)
    with torch.device(DEV):
        model = SarulixLM(config).to(dtype).eval()
    return model.load_tensors(weights)


def tokens(cfg, n, seed=0, batch=1):
    return torch.randint(0, cfg["vocab"], (batch, n), generator=torch.Generator().manual_seed(seed))


def run(model, ids, cuts, cache=None):
    """Logits [batch, n, vocab] of the tokens given in portions."""
    cache = cache or model.new_cache(ids.size(0), ids.size(1))
    out, lo = [], cache.tokens
    for c in cuts:
        out.append(model(ids[:, lo:lo + c].to(DEV), cache)["logits"].float().cpu())
        cache.advance(c)
        lo += c
    return torch.cat(out, 1)


@pytest.fixture(scope="module", params=DTYPES, ids=["fp32", "bf16"])
def mixed(request):
    cfg = H.mixed()
    w = H.tensors(cfg, 1)
    return cfg, w, build(cfg, w, request.param), request.param


def test_layers_against_the_plain_implementation(mixed):
    cfg, w, model, dtype = mixed
    ids, want, got = tokens(cfg, 70), [], []
    S.forward(cfg, w, ids[0], layers_out=want)
    model(ids.to(DEV), residuals=got)
    assert len(got) == len(want) == 12
    for k, (a, b) in enumerate(zip(got, want)):
        print("layer run", k, dtype, relative_rms(a[0], b), flush=True)
        assert relative_rms(a[0], b) < TOL[dtype], k


@pytest.mark.parametrize("layer", [H.attention(), H.rglru(ff=30), H.delta(), H.attention(heads=3, kv_heads=1, rot=24)],
                         ids=["attention", "rglru", "delta", "shared"])
def test_each_mixer_alone(layer):
    cfg = H.config([layer])
    w = H.tensors(cfg, 4)
    ids = tokens(cfg, 90, 4)
    want = S.forward(cfg, w, ids[0])
    for dtype in DTYPES:
        model = build(cfg, w, dtype)
        for cuts in ([90], [1] * 90, [40, 2, 17, 9, 8, 14]):
            err = relative_rms(run(model, ids, cuts)[0], want)
            print("mixer", layer["type"], dtype, cuts[:2], err, flush=True)
            assert err < TOL[dtype]


@pytest.mark.parametrize("cuts", [[150], [1] * 150, [2] * 75, [110, 3, 2, 35], [64, 64, 22], [17, 100, 33], [149, 1], [8, 9, 16, 117]],
                         ids=lambda c: f"{len(c)}x{c[0]}")
def test_portions(mixed, cuts):
    cfg, w, model, dtype = mixed
    ids = tokens(cfg, 150, 3)
    assert relative_rms(run(model, ids, cuts)[0], S.forward(cfg, w, ids[0])) < TOL[dtype]


@pytest.mark.parametrize("loop", [(0, 0, 0), (0, 6, 2), (0, 1, 1), (5, 6, 4), (2, 5, 1)], ids=str)
def test_loops(loop):
    cfg = H.mixed(loop=loop)
    w = H.tensors(cfg, 7)
    ids = tokens(cfg, 60, 7)
    want = S.forward(cfg, w, ids[0])
    for dtype in DTYPES:
        model = build(cfg, w, dtype)
        for cuts in ([60], [30, 1, 1, 2, 26]):
            print("loop", loop, dtype, cuts[:2], flush=True)
            assert relative_rms(run(model, ids, cuts)[0], want) < TOL[dtype]


def test_batch_of_sequences_equals_each_alone(mixed):
    cfg, w, model, dtype = mixed
    ids = tokens(cfg, 90, 4, batch=3)
    got = run(model, ids, [60, 20, 1, 1, 8])
    for b in range(3):
        assert relative_rms(got[b], S.forward(cfg, w, ids[b])) < TOL[dtype]
        alone = run(model, ids[b:b + 1], [60, 20, 1, 1, 8])
        assert relative_rms(got[b], alone[0]) < TOL[dtype] / 3


def test_cache_used_again(mixed):
    cfg, w, model, dtype = mixed
    pool = RequestCaches(lambda: model.new_cache(1, 130))
    first, second, other = tokens(cfg, 130, 5), tokens(cfg, 77, 6), tokens(cfg, 40, 7)
    a = run(model, first, [100, 1, 29], pool.of("a"))
    b1 = run(model, other[:, :20], [20], pool.of("b"))     # alive while "a" ends and "c" takes its place
    held = pool.of("a")
    pool.end("a")
    assert pool.of("c") is held
    c = run(model, second, [1, 2, 47, 2, 25], pool.of("c"))
    b2 = run(model, other, [15, 5], pool.of("b"))
    assert relative_rms(a[0], S.forward(cfg, w, first[0])) < TOL[dtype]
    assert relative_rms(c[0], S.forward(cfg, w, second[0])) < TOL[dtype]
    assert relative_rms(torch.cat([b1, b2], 1)[0], S.forward(cfg, w, other[0])) < TOL[dtype]
    with pytest.raises(ValueError, match="do not fit"):
        model(tokens(cfg, 100).to(DEV), pool.of("c"))


def test_long_decoding(mixed):
    cfg, w, model, dtype = mixed
    ids = tokens(cfg, 500, 8)
    got = run(model, ids, [40] + [1] * 460)
    print('long decoding', dtype, relative_rms(got[0], S.forward(cfg, w, ids[0])), flush=True)
    assert relative_rms(got[0], S.forward(cfg, w, ids[0])) < TOL[dtype]


@pytest.mark.parametrize("kind", ["attention", "rglru", "delta"])
def test_a_far_token_is_heard(kind):
    """Another token near the start changes no logits before its place and the plain implementation's logits far
    after it, by the same amount, in prompts and in decoding."""
    layer = {"attention": H.attention(), "rglru": H.rglru(), "delta": H.delta()}[kind]
    cfg = H.config([layer])
    w = H.tensors(cfg, 2)
    if kind == "rglru":
        w["l0.mix.ra.b"][:] = -8.0       # hardly any decay
        w["l0.mix.ra"] *= 0
    elif kind == "delta":
        w["l0.mix.A_log"][:] = -7.0
        w["l0.mix.b"] *= 4
    else:
        w["l0.mix.q.norm"] *= 2          # sharper attention
        w["l0.mix.k.norm"] *= 2
    n, place = 700, 5
    a = tokens(cfg, n, 9)
    b = a.clone()
    b[0, place] = (b[0, place] + 1) % cfg["vocab"]
    want = S.forward(cfg, w, a[0]) - S.forward(cfg, w, b[0])
    assert want[-50:].norm() > 1e-3
    model = build(cfg, w, torch.float32)
    for cuts in ([n], [300] + [1] * 60 + [340], [place + 1, n - place - 41] + [8] * 5):
        print("far", kind, cuts[:2], flush=True)
        diff = run(model, a, cuts)[0] - run(model, b, cuts)[0]
        assert torch.equal(diff[:place], torch.zeros_like(diff[:place]))
        assert (diff[-50:].double() - want[-50:]).norm() < 0.02 * want[-50:].norm()


def test_other_sizes():
    """Sizes with their own corners: width and feed-forward not multiples of anything, one head, one block, one tap,
    no padding at all, heads and blocks larger than the matrix-core kernels take, equal ranks and ranks of 1."""
    cases = [
        (H.config([H.attention(1, 1, 32, 32, 32, ff=33), H.rglru(32, 1, 1, ff=7), H.delta(1, 1, 32, 32, 1)], width=37,
                  vocab=59, scale=1.0, logit_scale=1.0, loop=(1, 3, 2)), (1, 1)),
        (H.config([H.attention(4, 1, 160, 72, 8), H.rglru(2100, 2, 5), H.delta(2, 1, 200, 136, 6), H.attention(9, 3, 12, 140, 6)],
                  width=130, loop=(0, 2, 2)), (33, 33)),
        (H.config([H.delta(5, 5, 7, 9, 2), H.rglru(50, 10, 3), H.attention(2, 2, 130, 260, 128, ff=None)], width=64,
                  vocab=1030), (64, 3)),
    ]
    for i, (cfg, ranks) in enumerate(cases):
        w = H.tensors(cfg, 20 + i, ranks=ranks)
        ids = tokens(cfg, 140, i)
        want = S.forward(cfg, w, ids[0])
        for dtype in DTYPES:
            model = build(cfg, w, dtype)
            for cuts in ([140], [70, 2, 1, 1, 66]):
                err = relative_rms(run(model, ids, cuts)[0], want)
                print("sizes", i, dtype, cuts[:2], err, flush=True)
                assert err < TOL[dtype] * 1.5


def test_logits_of_chosen_places(mixed):
    cfg, w, model, dtype = mixed
    ids = tokens(cfg, 50, 2).to(DEV)
    full = model(ids)["logits"][0]
    some = model(ids, logits_at=torch.tensor([49, 3], device=DEV))["logits"][0]
    assert some.shape == (2, cfg["vocab"]) and relative_rms(some, full[[49, 3]]) < TOL[dtype] / 3
    assert model(ids, logits_at=torch.empty(0, dtype=torch.long, device=DEV))["logits"].shape == (1, 0, cfg["vocab"])


def test_greedy_generation_follows_the_plain_argmax():
    """Every token that generation picks is the plain implementation's choice for the tokens before it."""
    cfg = H.mixed()
    w = H.tensors(cfg, 1)
    prompt = tokens(cfg, 45, 11, batch=2)
    model = build(cfg, w, torch.float32)
    out = greedy_generate(model, prompt.to(DEV), 40).cpu()
    for b in range(2):
        seq = torch.cat([prompt[b], out[b]])
        assert torch.equal(S.forward(cfg, w, seq)[44:-1].argmax(-1), out[b])


def test_generation_with_a_replayed_graph_equals_eager():
    """Several replays, each step's token equal to the eager one (same kernels, same order of sums)."""
    cfg = H.mixed()
    w = H.tensors(cfg, 1)
    for dtype in DTYPES:
        model = build(cfg, w, dtype)
        prompt = tokens(cfg, 70, 12, batch=2).to(DEV)
        eager = greedy_generate(model, prompt, 60)
        for _ in range(2):
            assert torch.equal(greedy_generate(model, prompt, 60, use_graph=True), eager)
            torch.cuda.synchronize()


def test_graph_replay_logits_equal_eager_step_by_step(mixed):
    cfg, w, model, dtype = mixed
    ids = tokens(cfg, 60, 13).to(DEV)
    cache, ref = model.new_cache(1, 60), model.new_cache(1, 60)
    for c in (cache, ref):
        model(ids[:, :30], c)
        c.advance(30)
    tok, pos = ids[:, 30:31].clone(), torch.tensor([30], device=DEV)
    s = torch.cuda.Stream()
    s.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(s):
        warm = model.new_cache(1, 60)
        model(tok, warm, pos)
    torch.cuda.current_stream().wait_stream(s)
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        out = model(tok, cache, pos)["logits"]
    for i in range(30, 60):
        tok.copy_(ids[:, i:i + 1])
        pos.fill_(i)
        graph.replay()
        got = out.clone()
        cache.advance(1)
        want = model(ids[:, i:i + 1], ref)["logits"]
        ref.advance(1)
        torch.cuda.synchronize()
        assert torch.equal(got, want), i


def test_trace_replay(tmp_path):
    """A schedule of portions through the trace runner, from a checkpoint directory."""
    import safetensors.torch as st

    from astrai_amd.trace import replay

    cfg = H.mixed()
    w = H.tensors(cfg, 1)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    st.save_file(w, str(tmp_path / "model.safetensors"))
    for dtype in DTYPES:
        model = load_checkpoint(str(tmp_path), DEV, dtype)
        caches = RequestCaches(lambda: model.new_cache(1, 64))
        step = 0
        for name, n, cuts in (("a", 60, (40, 2, 18)), ("b", 33, (33,))):
            ids = tokens(cfg, n, n)[0]
            want, lo = S.forward(cfg, w, ids), 0
            for c in cuts:
                places = [0, c - 1] if c != 2 else []
                replay(model, caches, {"step": step, "entries": [{"id": name, "tokens": ids[lo:lo + c].tolist(),
                                                                  "want": places}],
                                       "end": [name] if lo + c == n else []}, str(tmp_path))
                path = tmp_path / f"{step}.f32"
                assert path.exists() == bool(places)
                if places:
                    rows = torch.frombuffer(bytearray(path.read_bytes()), dtype=torch.float32).reshape(len(places), -1)
                    assert relative_rms(rows, want[[lo + p for p in places]]) < TOL[dtype]
                    os.unlink(path)
                lo, step = lo + c, step + 1
