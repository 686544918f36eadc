"""Every kernel of libastrai_mix.so against the plain implementation in float64 on the same inputs."""

import pytest
import torch

from astrai_amd.extension import _mix
from astrai_amd.extension._mix import LatentShape, pad_to
from astrai_amd.model.mixers import Rotation
from lugitar_helpers import YARN, relative_rms, rotation
from oracle import lugitar_oracle as L

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
# the worst token's rms error over the rms of all; bf16 rounds latents, absorbed queries, keys, values, outputs
TOL = {torch.float32: 1e-5, torch.bfloat16: 2e-2}
DTYPES = [torch.float32, torch.bfloat16]


def randn(g, *size, dtype=torch.float32, std=1.0):
    return (torch.randn(*size, generator=g) * std).to(dtype)


def log(*what):
    print(*what, flush=True)


# ---------------------------------------------------------------- row operations


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [1, 72, 101, 1024, 1028, 3000, 8192, 9000])
def test_residual_and_embed_norm(width, dtype):
    log("residual_norm", width, dtype)
    g = torch.Generator().manual_seed(width)
    n, eps, mult = 7, 1e-3, 0.37
    y = randn(g, n, width, dtype=dtype) + 2.0          # a mean that has to be taken off
    x = randn(g, n, width, std=3.0)
    w1, w2 = randn(g, width) + 1, randn(g, width) + 1
    xd = x.to(DEV)
    h = _mix.residual_norm(y.to(DEV), xd, w1.to(DEV), w2.to(DEV), mult, eps)
    want = x.double() + mult * L.layer_norm(y.double(), w1.double(), eps)
    assert relative_rms(xd, want) < 1e-6
    if width > 1:
        assert relative_rms(h, L.layer_norm(want, w2.double(), eps)) < TOL[dtype]
    table = randn(g, 11, width, dtype=dtype)
    tokens = torch.tensor([3, 0, 10, 3])
    x2, h2 = _mix.embed_norm(table.to(DEV), tokens.to(DEV), w2.to(DEV), eps)
    assert torch.equal(x2.cpu(), table[tokens].float())
    if width > 1:
        assert relative_rms(h2, L.layer_norm(table[tokens].double(), w2.double(), eps)) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_silu_mul_and_gated_rms_norm(dtype):
    g = torch.Generator().manual_seed(5)
    for n, ff in ((1, 8), (5, 72), (300, 1000)):
        log("silu_mul", n, ff, dtype)
        gu = randn(g, n, 2 * ff, dtype=dtype, std=3.0)
        want = L.silu(gu[:, :ff].double()) * gu[:, ff:].double()
        assert relative_rms(_mix.silu_mul(gu.to(DEV)), want) < TOL[dtype]
    for n, width, count in ((1, 32, 17), (6, 96, 96), (9, 2080, 2000)):
        log("gated_rms_norm", n, width, count, dtype)
        o = randn(g, n, width, dtype=dtype, std=5.0)
        o[:, count:] = 0
        proj, w = randn(g, n, width + 40, dtype=dtype), randn(g, width) + 1
        got = _mix.gated_rms_norm(o.to(DEV), proj.to(DEV), 8, w.to(DEV), count, 1e-2)
        od = o.double()
        want = od / torch.sqrt(od[:, :count].pow(2).mean(-1, keepdim=True) + 1e-2) * w.double()
        want = want * torch.sigmoid(proj[:, 8:8 + width].double())
        assert relative_rms(got, want) < TOL[dtype]


def test_silu_at_the_ends():
    z = torch.tensor([[-200.0, -90.0, -30.0, 0.0, 30.0, 90.0, 200.0, 1.0] + [1.0] * 8])
    for dtype in DTYPES:
        y = _mix.silu_mul(z.to(dtype).to(DEV)).cpu().float()
        assert torch.isfinite(y).all() and y[0, :3].abs().max() < 1e-9 and y[0, 6] == 200.0


# ---------------------------------------------------------------- latent attention

# heads, dim, rot_dim, vdim, kv_rank: padding of every part, several tile sizes, one head, more rows than a tile
SHAPES = [(3, 24, 8, 40, 56), (1, 32, 32, 32, 32), (5, 64, 40, 96, 200), (2, 128, 64, 128, 512), (20, 40, 16, 64, 96)]


class Case:
    """A layer's projections with padded head sizes, random or prepared, and its cache."""

    def __init__(self, shape, window, dtype, n, batch=1, seed=0, scale=None, max_len=None):
        self.heads, self.dim, self.rd, self.vd, self.rank = shape
        self.s = LatentShape(self.heads, pad_to(self.dim), pad_to(self.rd), pad_to(self.rank), pad_to(self.vd),
                             self.rank, _mix.UNBOUNDED if window is None else window,
                             scale or (self.dim + self.rd) ** -0.5)
        self.dtype, self.n, self.batch, self.window = dtype, n, batch, window
        g = torch.Generator().manual_seed(seed)
        s = self.s
        self.q = randn(g, batch, n, self.heads, self.dim + self.rd, dtype=dtype)
        self.dkv = randn(g, batch, n, self.rank + self.rd, dtype=dtype)
        self.gate = randn(g, batch, n, self.heads, dtype=dtype)
        self.norm = randn(g, self.rank) * 0.2 + 1
        self.uk = randn(g, self.heads, self.dim, self.rank, dtype=dtype, std=self.rank ** -0.5)
        self.uv = randn(g, self.heads, self.vd, self.rank, dtype=dtype, std=self.rank ** -0.5)
        self.rot = rotation(self.rd, scaling=YARN)
        self.max_len = max_len or n + 5
        self.eps = 1e-5
        self.gcols = pad_to(self.heads, 8)
        # stale rows of a former sequence must not matter
        self.cache = torch.full((batch, self.max_len, s.cache_cols), 7.0, dtype=dtype, device=DEV)
        self.table = Rotation.from_dict(self.rot).table(self.max_len).to(DEV)
        self.norm_p = torch.cat([self.norm, torch.ones(s.rp - self.rank)]).to(DEV)
        self.pack()

    def pack(self):
        s = self.s
        uk = torch.zeros(self.heads, s.dn, s.rp, dtype=self.dtype)
        uk[:, :self.dim, :self.rank] = self.uk
        uv = torch.zeros(self.heads, s.vp, s.rp, dtype=self.dtype)
        uv[:, :self.vd, :self.rank] = self.uv
        self.w_ukv = torch.cat([uk, uv], 1).reshape(-1, s.rp).contiguous().to(DEV)
        self.w_uk_t = uk.transpose(1, 2).contiguous().to(DEV)

    def proj(self, lo, hi):
        s, b, n = self.s, self.batch, hi - lo
        q = torch.zeros(b, n, self.heads, s.dn + s.dr, dtype=self.dtype)
        q[..., :self.dim] = self.q[:, lo:hi, :, :self.dim]
        q[..., s.dn:s.dn + self.rd] = self.q[:, lo:hi, :, self.dim:]
        kv = torch.zeros(b, n, s.cache_cols, dtype=self.dtype)
        kv[..., :self.rank] = self.dkv[:, lo:hi, :self.rank]
        kv[..., s.rp:s.rp + self.rd] = self.dkv[:, lo:hi, self.rank:]
        gate = torch.zeros(b, n, self.gcols, dtype=self.dtype)
        gate[..., :self.heads] = self.gate[:, lo:hi]
        return torch.cat([q.flatten(2), kv, gate], -1).reshape(b * n, -1).contiguous().to(DEV)

    def run(self, cuts, path):
        """Attention outputs [batch, n, heads, vdim] of the tokens cut into portions of the given sizes."""
        s, out, lo = self.s, [], 0
        for c in cuts:
            hi = lo + c
            p = self.proj(lo, hi)
            pos = torch.arange(lo, hi, device=DEV)
            g_off = s.q_cols + s.cache_cols
            q_abs = _mix.latent_append(p, s, s.q_cols, self.table, pos, self.norm_p, self.cache, self.eps,
                                       self.w_uk_t if path == "rows" else None)
            if path == "prefill":
                first = max(lo - s.window + 1, 0)
                c_ = self.cache[:, first:hi, :s.rp].reshape(-1, s.rp)
                kv = (c_.float() @ self.w_ukv.float().t()).to(self.dtype).reshape(self.batch, hi - first, -1)
                y = _mix.latent_prefill(p, s, g_off, kv, self.cache, lo, first)
            else:
                y = _mix.latent_rows(p, s, g_off, self.w_ukv, self.cache, pos, q_abs)
            y = y.reshape(self.batch, c, self.heads, s.vp)
            assert y[..., self.vd:].count_nonzero() == 0   # padding stays zero
            out.append(y[..., :self.vd].cpu())
            lo = hi
        assert lo == self.n
        return torch.cat(out, 1)

    def want(self):
        """The same from the plain implementation's pieces, float64."""
        outs = []
        for b in range(self.batch):
            pos = torch.arange(self.n)
            c = L.rms_norm(self.dkv[b, :, :self.rank].double(), self.norm.double(), self.eps)
            kr = L.rotate_half(self.dkv[b, :, self.rank:].double(), pos, self.rot)
            qn, qr = self.q[b, ..., :self.dim].double(), L.rotate_half(self.q[b, ..., self.dim:].double(), pos, self.rot)
            seen = L.window_mask(self.n, self.window)
            o = torch.empty(self.n, self.heads, self.vd, dtype=torch.float64)
            for h in range(self.heads):
                k, v = c @ self.uk[h].double().T, c @ self.uv[h].double().T
                sc = (qn[:, h] @ k.T + qr[:, h] @ kr.T) * self.s.scale
                sc = sc.masked_fill(~seen, float("-inf"))
                o[:, h] = torch.softmax(sc, -1) @ v * torch.sigmoid(self.gate[b, :, h].double())[:, None]
            outs.append(o)
        return torch.stack(outs)


def paths(shape, dtype):
    out = ["general"]
    if dtype == torch.bfloat16:
        out += ["rows", "prefill"]
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("window,n", [(1, 40), (29, 150), (64, 300), (None, 200)])
def test_latent_attention_whole_block(shape, window, n, dtype):
    case = Case(shape, window, dtype, n, batch=2, seed=n)
    want = case.want()
    for path in paths(shape, dtype):
        log("latent", shape, window, n, dtype, path)
        assert relative_rms(case.run([n], path).flatten(2), want.flatten(2)) < TOL[dtype], path


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_append_writes_the_latent_and_the_rotated_key(dtype):
    case = Case((3, 24, 8, 40, 56), 9, dtype, 30, batch=2)
    case.run([30], "general")
    got = case.cache[:, :30].cpu().double()
    for b in range(2):
        c = L.rms_norm(case.dkv[b, :, :56].double(), case.norm.double(), case.eps)
        kr = L.rotate_half(case.dkv[b, :, 56:].double(), torch.arange(30), case.rot)
        assert relative_rms(got[b, :, :56], c) < TOL[dtype] and relative_rms(got[b, :, 64:72], kr) < TOL[dtype]
    assert got[:, :, 56:64].count_nonzero() == 0 and got[:, :, 72:].count_nonzero() == 0
    assert (case.cache[:, 30:] == 7).all()                # nothing past the block is touched


@pytest.mark.parametrize("cuts", [[2] * 75, [1] * 20 + [130], [100, 2, 3, 45], [17, 16, 33, 64, 20], [149, 1]])
def test_latent_attention_does_not_depend_on_the_portions(cuts):
    for dtype in DTYPES:
        case = Case((5, 64, 40, 96, 200), 37, dtype, 150, seed=4)
        want = case.want()
        for path in paths(None, dtype):
            log("latent portions", cuts[:4], dtype, path)
            assert relative_rms(case.run(cuts, path).flatten(2), want.flatten(2)) < TOL[dtype], path


@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 127, 128, 129])
def test_a_key_that_stands_out_is_seen_exactly_inside_the_window(window):
    """One key matches every query so strongly that whoever sees it returns its value: the queries from its own
    position to window - 1 tokens later do, the one before and the one after do not."""
    n, far = 330, 140
    for dtype in DTYPES:
        case = Case((2, 32, 8, 32, 64), window, dtype, n, seed=9)
        case.q[...] = 0
        case.q[..., 0] = 6.0                              # every query asks for key dimension 0
        case.dkv[...] = case.dkv * 0.5
        case.dkv[:, :, 0] = 0
        case.dkv[:, far, :64] = 0
        case.dkv[:, far, 0] = 3.0                         # the latent that gives a large key dimension 0
        case.uk[...] = 0
        case.uk[:, 0, 0] = 8.0
        case.pack()
        want = case.want()
        alone = torch.zeros(n, dtype=torch.bool)
        alone[far:far + window] = True
        v_far = want[0, far + window - 1, 0] / torch.sigmoid(case.gate[0, far + window - 1, 0].double())
        for path in paths(None, dtype):
            for cuts in ([n], [far] + [1] * (n - far - 40) + [40], [far + window - 1, 1, 1, n - far - window - 1]):
                cuts = [c for c in cuts if c]
                log("window", window, dtype, path, cuts[:3])
                got = case.run(cuts, path)
                assert relative_rms(got.flatten(2), want.flatten(2)) < TOL[dtype] * 2, (path, cuts[:3])
                ungated = got[0, :, 0].double() / torch.sigmoid(case.gate[0, :, 0].double())[:, None]
                hit = (ungated - v_far).norm(dim=-1) < 0.05 * v_far.norm()
                assert torch.equal(hit, alone), (path, window)


def test_first_tokens_and_blocks_that_start_late():
    """Block starts around tile borders, with the first tokens inside and outside the window."""
    for start in (1, 31, 32, 63, 64, 100):
        case = Case((3, 24, 8, 40, 56), 64, torch.bfloat16, start + 129, seed=start)
        want = case.want()
        for path in ("rows", "prefill"):
            log("late block", start, path)
            got = case.run([start, 129], path)
            assert relative_rms(got.flatten(2), want.flatten(2)) < TOL[torch.bfloat16]


@pytest.mark.parametrize("nsplit", [1, 2, 3, 7, 64])
def test_latent_rows_splits(nsplit):
    case = Case((7, 40, 16, 64, 96), 90, torch.bfloat16, 203, batch=3, seed=2)
    want = case.want()[:, 200:]
    case.run([203], "general")
    log("nsplit", nsplit)
    p, pos, s = case.proj(200, 203), torch.arange(200, 203, device=DEV), case.s
    q_abs = _mix.latent_append(p, s, s.q_cols, case.table, pos, case.norm_p, case.cache, case.eps, case.w_uk_t)
    y = _mix.latent_rows(p, s, s.q_cols + s.cache_cols, case.w_ukv, case.cache, pos, q_abs, nsplit)
    assert relative_rms(y.reshape(3, 3, 7, 64).flatten(2), want.flatten(2)) < TOL[torch.bfloat16]


def test_large_scores_of_both_signs():
    """Scores of some hundreds: the running maximum has to be followed."""
    case = Case((2, 64, 16, 64, 96), 150, torch.bfloat16, 260, seed=3, scale=4.0)
    case.q[:, :, :, :] *= torch.linspace(0.1, 3.0, 260).to(torch.bfloat16)[None, :, None, None]
    # (the plain result with keys rounded as the prompt kernel's are: a rounding of a key moves such a score)
    want = case.want()
    for path in ("general", "rows", "prefill"):
        got = case.run([260], path)
        assert torch.isfinite(got.float()).all()
        err = (got.double() - want).norm(dim=-1) / want.norm(dim=-1)
        assert err.median() < 0.05, path


# ---------------------------------------------------------------- lightning attention


def lightning_case(heads, dim, vd, n, dtype, batch=1, seed=0):
    g = torch.Generator().manual_seed(seed)
    dp, vp = pad_to(dim), pad_to(vd)
    q, k = randn(g, batch, n, heads, dim, dtype=dtype), randn(g, batch, n, heads, dim, dtype=dtype)
    v = randn(g, batch, n, heads, vd, dtype=dtype)

    def proj(lo, hi):
        t = torch.zeros(batch, hi - lo, heads * (2 * dp + vp) + 8, dtype=dtype)
        t[..., :heads * dp].unflatten(-1, (heads, dp))[..., :dim] = q[:, lo:hi]
        t[..., heads * dp:2 * heads * dp].unflatten(-1, (heads, dp))[..., :dim] = k[:, lo:hi]
        t[..., 2 * heads * dp:heads * (2 * dp + vp)].unflatten(-1, (heads, vp))[..., :vd] = v[:, lo:hi]
        return t.reshape(batch * (hi - lo), -1).contiguous().to(DEV)

    return q, k, v, dp, vp, proj


def lightning_run(proj, cuts, batch, heads, dp, vp, decay, kernels, nseg=None):
    state = torch.zeros(batch, heads, dp, vp, device=DEV)
    pw, out, lo = _mix.decay_powers(decay).to(DEV), [], 0
    for c, step in zip(cuts, kernels):
        y = _mix.lightning(proj(lo, lo + c), 0, heads * dp, 2 * heads * dp, pw, state, step, nseg)
        out.append(y.reshape(batch, c, heads, vp).cpu())
        lo += c
    return torch.cat(out, 1), state.cpu()


def lightning_want(q, k, v, decay):
    """With silu rounded to the activation type, as the product path does."""
    def act(x):
        return L.silu(x.double()).to(x.dtype).double()
    runs = [L.lightning_scan(act(q[b]), act(k[b]), act(v[b]), decay) for b in range(q.size(0))]
    return torch.stack([r[0] for r in runs]), torch.stack([r[1] for r in runs])


LIGHTNING = [(1, 8, 8), (3, 40, 24), (2, 64, 100), (4, 128, 128), (2, 200, 40), (1, 256, 64)]


@pytest.mark.parametrize("heads,dim,vd", LIGHTNING)
def test_lightning_whole_and_in_portions(heads, dim, vd):
    n, batch = 333, 2
    decay = [0.6, 1.0, 0.999, 0.0][:heads]
    for dtype in DTYPES:
        q, k, v, dp, vp, proj = lightning_case(heads, dim, vd, n, dtype, batch, seed=dim)
        want, state = lightning_want(q, k, v, decay)
        for cuts in ([n], [64] * 5 + [13], [2] * 30 + [273], [63, 65, 1, 1, 127, 76], [128, 200, 5]):
            kernels = {torch.float32: [[True] * len(cuts)],
                       torch.bfloat16: [[True] * len(cuts), [False] * len(cuts), [c < 60 for c in cuts]]}[dtype]
            for steps in kernels:
                log("lightning", heads, dim, vd, dtype, cuts[:3], steps[:3])
                got, s = lightning_run(proj, cuts, batch, heads, dp, vp, decay, steps)
                assert got[..., vd:].count_nonzero() == 0
                assert relative_rms(got[..., :vd].flatten(2), want.flatten(2)) < TOL[dtype]
                # the state itself keeps more than the activations' precision
                assert relative_rms(s[:, :, :dim, :vd], state) < 2e-5
                assert s[:, :, dim:].count_nonzero() == 0 and s[..., vd:].count_nonzero() == 0


@pytest.mark.parametrize("nseg", [1, 2, 3, 5, 6])
def test_lightning_segments(nseg):
    heads, dim, vd, n = 2, 64, 96, 64 * 5 + 9
    decay = [0.98, 1.0]
    q, k, v, dp, vp, proj = lightning_case(heads, dim, vd, n * 2, torch.bfloat16, 2, seed=1)
    want, state = lightning_want(q, k, v, decay)
    log("segments", nseg)
    got, s = lightning_run(proj, [n, n], 2, heads, dp, vp, decay, [False, False], nseg)
    assert relative_rms(got[..., :vd].flatten(2), want.flatten(2)) < TOL[torch.bfloat16]
    assert relative_rms(s[:, :, :dim, :vd], state) < 2e-5


def test_lightning_remembers_one_far_token():
    """One token writes a large value under its own key; with everything else small, a query for that key thousands
    of tokens later reads decay^distance of it."""
    n, far, decay = 3000, 70, [0.9999, 0.99]
    q, k, v, dp, vp, proj = lightning_case(2, 32, 32, n, torch.bfloat16, seed=6)
    q[...], k[...], v[...] = 0, 0, 0
    q[..., 3] = 4.0
    k[:, far, :, 3] = 4.0
    v[:, far, :, 5] = 8.0
    want, _ = lightning_want(q, k, v, decay)
    for cuts, steps in (([n], [False]), ([n], [True]), ([100, 1, 2, 897, 2000], [False, True, True, False, False])):
        got, _ = lightning_run(proj, cuts, 1, 2, dp, vp, decay, steps)
        err = (got[0, far:, :, 5].double() - want[0, far:, :, 5]).abs() / want[0, far:, :, 5]
        assert err[:2000, 0].max() < 5e-3 and err[:300, 1].max() < 5e-3
        assert got[0, :far].count_nonzero() == 0


# ---------------------------------------------------------------- misuse is refused


def test_operands_are_checked():
    case = Case((3, 24, 8, 40, 56), 9, torch.bfloat16, 4)
    p, pos, s = case.proj(0, 4), torch.arange(4, device=DEV), case.s
    with pytest.raises(RuntimeError, match="expected shape"):
        _mix.latent_append(p, s, s.q_cols, case.table, pos[:3], case.norm_p, case.cache, 1e-5)
    with pytest.raises(RuntimeError, match="does not cover"):
        _mix.latent_append(p, s, s.q_cols, case.table[:2], pos, case.norm_p, case.cache, 1e-5)
    with pytest.raises(RuntimeError, match="do not cover"):
        kv = torch.zeros(1, 3, 3 * 96, dtype=torch.bfloat16, device=DEV)
        _mix.latent_prefill(p, s, s.q_cols + s.cache_cols, kv, case.cache, 0, 0)
    with pytest.raises(RuntimeError, match="expected torch.float32"):
        _mix.residual_norm(p, p, case.norm_p, case.norm_p, 1.0, 1e-5)
    with pytest.raises(RuntimeError, match="CUDA tensors"):
        _mix.silu_mul(torch.zeros(2, 16))
