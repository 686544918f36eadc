"""Lugitar models through the framework's forward, caches and greedy generation, against the plain
implementation in float64."""

import json
import os

import pytest
import torch

import lugitar_helpers as H
from astrai_amd.model import LugitarConfig, LugitarLM, RequestCaches, greedy_generate, load_checkpoint
from lugitar_helpers import relative_rms
from oracle import lugitar_oracle as L

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
TOL = {torch.float32: 1e-5, torch.bfloat16: 3e-2}
DTYPES = [torch.float32, torch.bfloat16]


def build(cfg, weights, dtype):
    with torch.device(DEV):
        model = LugitarLM(LugitarConfig.from_dict(cfg)).to(dtype).eval()
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


def test_layers_against_the_plain_implementation():
    cfg = H.mixed()
    w = H.tensors(cfg, 1)
    ids = tokens(cfg, 70)
    for dtype in DTYPES:
        for depth in range(1, len(cfg["layers"]) + 1):
            part = dict(cfg, layers=cfg["layers"][:depth])
            ww = {k: t for k, t in w.items() if not k.startswith("l") or int(k[1:k.index(".")]) < depth}
            want = []
            L.forward(part, ww, ids[0], layers_out=want)
            got = build(part, ww, dtype)(ids.to(DEV))["residual"][0]
            print("layers", dtype, depth, relative_rms(got, want[-1]), flush=True)
            assert relative_rms(got, want[-1]) < TOL[dtype], depth


@pytest.mark.parametrize("cuts", [[150], [1] * 150, [2] * 75, [110, 3, 2, 35], [64, 64, 22], [17, 100, 33], [149, 1]],
                         ids=lambda c: f"{len(c)}x{c[0]}")
def test_portions(mixed, cuts):
    cfg, w, model, dtype = mixed
    ids = tokens(cfg, 150, 3)
    want = L.forward(cfg, w, ids[0])
    assert relative_rms(run(model, ids, cuts)[0], want) < TOL[dtype]


def test_batch_of_sequences_equals_each_alone(mixed):
    cfg, w, model, dtype = mixed
    ids = tokens(cfg, 90, 4, batch=3)
    got = run(model, ids, [60, 20, 1, 1, 8])
    for b in range(3):
        assert relative_rms(got[b], L.forward(cfg, w, ids[b])) < TOL[dtype]
        alone = run(model, ids[b:b + 1], [60, 20, 1, 1, 8])
        assert relative_rms(got[b], alone[0]) < TOL[dtype] / 3


def test_cache_used_again(mixed):
    cfg, w, model, dtype = mixed
    pool = RequestCaches(lambda: model.new_cache(1, 130))
    first, second = tokens(cfg, 130, 5), tokens(cfg, 77, 6)
    other = tokens(cfg, 40, 7)
    a = run(model, first, [100, 1, 29], pool.of("a"))
    b1 = run(model, other[:, :20], [20], pool.of("b"))     # alive while "a" ends and "c" takes its place
    held = pool.of("a")
    pool.end("a")
    assert pool.of("c") is held
    c = run(model, second, [50, 2, 25], pool.of("c"))
    b2 = run(model, other, [15, 5], pool.of("b"))
    assert relative_rms(a[0], L.forward(cfg, w, first[0])) < TOL[dtype]
    assert relative_rms(c[0], L.forward(cfg, w, second[0])) < TOL[dtype]
    assert relative_rms(torch.cat([b1, b2], 1)[0], L.forward(cfg, w, other[0])) < TOL[dtype]
    with pytest.raises(ValueError, match="do not fit"):
        model(tokens(cfg, 100).to(DEV), pool.of("c"))


def test_long_decoding(mixed):
    cfg, w, model, dtype = mixed
    ids = tokens(cfg, 700, 8)
    got = run(model, ids, [40] + [1] * 660)
    assert relative_rms(got[0], L.forward(cfg, w, ids[0])) < TOL[dtype]


@pytest.mark.parametrize("window", [1, 2, 33, 128])
def test_a_token_is_heard_until_the_window_ends(window):
    """Another token at one place changes the logits of exactly the places whose window reaches it, whether those
    are part of the prompt or decoded."""
    cfg = H.config([H.latent(window=window)])
    w = H.tensors(cfg, 2)
    place, n = 40, 40 + window + 6
    a = tokens(cfg, n, 9)
    b = a.clone()
    b[0, place] = (b[0, place] + 1) % cfg["vocab"]
    for dtype in DTYPES:
        model = build(cfg, w, dtype)
        for cuts in ([n], [place + 1] + [1] * (n - place - 1), [place] + [2] * ((n - place) // 2) + [1] * ((n - place) % 2)):
            print("window", window, dtype, cuts[:3], flush=True)
            la, lb = run(model, a, cuts)[0], run(model, b, cuts)[0]
            changed = (la != lb).any(-1)
            want = torch.zeros(n, dtype=torch.bool)
            want[place:place + window] = True
            assert torch.equal(changed, want)


def test_a_far_token_is_kept_by_the_recurrence():
    cfg = H.config([H.lightning(decay=(0.3, 0.9, 0.9999))])
    w = H.tensors(cfg, 2)
    n = 900
    a = tokens(cfg, n, 9)
    b = a.clone()
    b[0, 5] = (b[0, 5] + 1) % cfg["vocab"]
    want = L.forward(cfg, w, a[0]) - L.forward(cfg, w, b[0])
    model = build(cfg, w, torch.float32)
    for cuts in ([n], [300] + [1] * 60 + [540]):
        diff = run(model, a, cuts)[0] - run(model, b, cuts)[0]
        assert torch.equal(diff[:5], torch.zeros_like(diff[:5]))
        assert want[-1].norm() > 1e-3 and (diff[-1].double() - want[-1]).norm() < 0.02 * want[-1].norm()


def test_other_sizes():
    """Sizes with their own corners: width and feed-forward not multiples of anything, one head, no padding at all,
    latents larger than the matrix-core kernels take, no window, no scaling, a residual factor of 1."""
    cases = [
        H.config([H.latent(heads=1, dim=32, rot_dim=32, vdim=32, kv_rank=32, ff=33), H.lightning(1, 32, 32, (1.0,), 7)],
                 width=37, vocab=59, mult=1.0),
        H.config([H.latent(heads=2, dim=160, rot_dim=72, vdim=136, kv_rank=100, window=70),
                  H.latent(heads=9, dim=12, rot_dim=72, vdim=20, kv_rank=100, kv_from=0, window=71,
                           rot=H.rotation(72, scaling=H.YARN)),
                  H.lightning(2, 288, 40, (0.9, 0.99))], width=130),
        H.config([H.latent(heads=2, dim=16, rot_dim=6, vdim=24, kv_rank=1100, rot=H.rotation(6, 1e4), window=None,
                           ff=None), H.lightning(ff=None)], width=64, vocab=1030),
    ]
    for i, cfg in enumerate(cases):
        w = H.tensors(cfg, 20 + i)
        ids = tokens(cfg, 140, i)
        want = L.forward(cfg, w, ids[0])
        for dtype in DTYPES:
            model = build(cfg, w, dtype)
            for cuts in ([140], [70, 2, 1, 1, 66]):
                print("sizes", i, dtype, cuts[:2], flush=True)
                err = relative_rms(run(model, ids, cuts)[0], want)
                print("   ", err, flush=True)
                assert err < TOL[dtype] * 1.5


def test_logits_of_chosen_places(mixed):
    cfg, w, model, dtype = mixed
    ids = tokens(cfg, 50, 2).to(DEV)
    full = model(ids)["logits"][0]
    some = model(ids, logits_at=torch.tensor([49, 3], device=DEV))["logits"][0]
    assert some.shape == (2, cfg["vocab"])
    assert relative_rms(some, full[[49, 3]]) < 1e-6 or dtype == torch.bfloat16 and relative_rms(some, full[[49, 3]]) < 1e-2
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
        logits = L.forward(cfg, w, seq)[44:-1]
        assert torch.equal(logits.argmax(-1), out[b])


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
            want, lo = L.forward(cfg, w, ids), 0
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
