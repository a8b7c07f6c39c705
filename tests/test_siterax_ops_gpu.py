"""The layer-stack kernels alone, against the oracle's functions in float64: residual addition with both norms (as a launch and inside a linear), query / key norm + partial
rotation + append, windowed attention with sink and gates (matrix-core and vector-ALU kernels), the one-token launch (chunk borders, window edges, splits, mixed positions,
garbage past the position), fp32 soft-capped linears."""
import pytest
import torch

from oracle import siterax_oracle as O

pytestmark = pytest.mark.gpu
DT = {"f32": torch.float32, "bf16": torch.bfloat16, "f16": torch.float16}
TOL = {"f32": 3e-5, "bf16": 1.6e-2, "f16": 3e-3}


def _err(got, want):
    got, want = got.double().cpu(), want.double().cpu()
    return ((got - want).abs().max() / want.abs().max().clamp_min(1e-9)).item()


def _pad(x, n):
    return torch.nn.functional.pad(x, (0, n - x.shape[-1]))


@pytest.mark.parametrize("dt", list(DT))
@pytest.mark.parametrize("H,width,rows", [(64, 50, 3), (128, 128, 1), (2048, 2000, 5), (4096, 4096, 2), (8192, 8000, 2)])
@pytest.mark.parametrize("form", ["all", "first", "no_inject", "no_pre"])
def test_residual_norm(cuda, dt, H, width, rows, form):
    from llava_mi355x import ops
    g = torch.Generator().manual_seed(H + rows)
    r = lambda *s: _pad(torch.randn(*s, width, generator=g), H).to(DT[dt]).to(cuda)
    x = _pad(torch.randn(rows, width, generator=g), H).to(cuda)
    y, inj, post, pre = r(rows), r(rows), r(), r()
    if form == "first":
        x = y = None
    if form == "no_inject":
        inj = None
    got, gn = ops.residual_norm(x, y, post if y is not None else None, inj, None if form == "no_pre" else pre, 0.37, 1e-3, width, DT[dt])
    d = lambda t: t.double().cpu()[..., :width]
    want = d(x) if x is not None else 0
    if y is not None:
        want = want + 0.37 * O.rms_norm(d(y), d(post), 1e-3)
    if inj is not None:
        want = want + d(inj)
    assert _err(got[:, :width], want) < 2e-6 and got[:, width:].abs().max().item() == 0 if width < H else True
    assert _err(got[:, :width], want) < 2e-6
    if form != "no_pre":
        assert _err(gn[:, :width], O.rms_norm(want, d(pre), 1e-3)) < TOL[dt] / 2


@pytest.mark.parametrize("dt", ["bf16", "f16"])
@pytest.mark.parametrize("N,H,width,act,form", [(192, 64, 50, 0, "all"), (8, 128, 128, 0, "first"), (640, 2048, 2000, 3, "no_inject"), (1000, 4096, 4096, 0, "all"), (128, 8192, 8100, 3, "all"),
                                                (72, 2112, 2100, 0, "no_x")])
def test_gemv_residual_equals_the_two_launches(cuda, dt, N, H, width, act, form):
    from llava_mi355x import ops
    g = torch.Generator().manual_seed(N)
    r = lambda *s: _pad(torch.randn(*s, width, generator=g), H).to(DT[dt]).to(cuda)
    x = _pad(torch.randn(1, width, generator=g), H).to(cuda)
    y, inj, post, pre = r(1), r(1), r(), r()
    w = _pad(torch.randn(N, width, generator=g) / width ** 0.5, H).to(DT[dt]).to(cuda)
    b = torch.randn(N, generator=g).to(DT[dt]).to(cuda)
    if form == "first":
        x = y = None
    if form == "no_inject":
        inj = None
    if form == "no_x":
        x = None
    p = post if y is not None else None
    x1, xn = ops.residual_norm(x, y, p, inj, pre, 0.37, 1e-5, width, DT[dt])
    two = ops.gemv(xn, w, bias=b, act=act)
    x2, one = ops.gemv_residual(x, y, p, inj, pre, w, 0.37, 1e-5, bias=b, width=width, act=act)
    assert _err(x2, x1) < 2e-6 and _err(one, two) < TOL[dt] / 2


@pytest.mark.parametrize("dt", list(DT))
@pytest.mark.parametrize("M,N,K,form", [(1, 104, 64, 0), (70, 512, 192, 0), (1, 1000, 256, 1), (1, 8, 64, 1), (5, 104, 128, 2), (32, 520, 192, 2)])
@pytest.mark.parametrize("cap", [0.0, 7.5])
def test_linear_f32_soft_cap(cuda, dt, M, N, K, form, cap):
    from llava_mi355x import ops
    if form == 2 and dt == "f32":
        pytest.skip("the decode-batch kernel is 16-bit")
    g = torch.Generator().manual_seed(N)
    x, w = torch.randn(M, K, generator=g).to(DT[dt]), (torch.randn(N, K, generator=g) / 4).to(DT[dt])
    want = x.double() @ w.double().T
    want = cap * torch.tanh(want / cap) if cap else want
    got = ops.linear_f32(x.to(cuda), w.to(cuda), cap, form)
    assert got.dtype == torch.float32 and _err(got, want) < 5e-6


def _qkv(T, H, G, D, dk, dv, stride, dt, seed):
    g = torch.Generator().manual_seed(seed)
    q, k, v = torch.randn(T, H, dk, generator=g), torch.randn(T, G, dk, generator=g), torch.randn(T, G, dv, generator=g)
    row = torch.zeros(T, stride)
    row[:, :H * D] = _pad(q, D).reshape(T, -1); row[:, H * D:(H + G) * D] = _pad(k, D).reshape(T, -1); row[:, (H + G) * D:(H + 2 * G) * D] = _pad(v, D).reshape(T, -1)
    row = row.to(DT[dt])
    un = lambda a, n, d: row[:, a * D:(a + n) * D].reshape(T, n, D)[..., :d].double()
    return row, un(0, H, dk), un(H, G, dk), un(H + G, G, dv)


def _table(rot, n):
    from llava_mi355x.siterax import RotaryConfig, rotary_table
    return rotary_table(RotaryConfig(rot["dims"], rot["base"], rot["scaling"]["factor"]), n)


@pytest.mark.parametrize("dt", list(DT))
@pytest.mark.parametrize("H,G,D,dk,dv,rot,T,pos0", [(4, 2, 64, 48, 64, 32, 70, 5), (2, 1, 128, 96, 128, 96, 130, 0), (3, 3, 128, 80, 72, 20, 64, 100), (2, 1, 256, 200, 160, 128, 33, 7),
                                                    (1, 1, 64, 10, 12, 6, 3, 61), (2, 2, 128, 128, 128, 0, 65, 0), (5, 1, 64, 64, 64, 64, 1, 191)])
def test_qkv_norm_rope_append(cuda, dt, H, G, D, dk, dv, rot, T, pos0):
    from llava_mi355x import ops
    stride, s_max, eps = (H + 2 * G) * D + 64, 256, 1e-4
    row, q, k, v = _qkv(T, H, G, D, dk, dv, stride, dt, 3)
    r = {"dims": rot, "base": 500.0, "scaling": {"factor": 1.7}}
    g = torch.Generator().manual_seed(9)
    qn, kn = (1 + 0.3 * torch.randn(dk, generator=g)).to(DT[dt]), (1 + 0.3 * torch.randn(dk, generator=g)).to(DT[dt])
    kc, vt = torch.zeros(G, s_max, D, dtype=DT[dt], device=cuda), torch.zeros(G, D, s_max, dtype=DT[dt], device=cuda)
    dev = row.to(cuda)
    ops.qkv_norm_rope_kv(dev, kc, vt, _pad(qn, D).to(cuda), _pad(kn, D).to(cuda), _table(r, s_max).to(cuda) if rot else None, pos0, H, G, dk, rot, eps)
    pos = torch.arange(pos0, pos0 + T)
    rope = (lambda x: O.rotate(x, pos, r)) if rot else (lambda x: x)
    wq, wk = rope(O.rms_norm(q, qn.double(), eps)), rope(O.rms_norm(k, kn.double(), eps))
    got_q = dev[:, :H * D].reshape(T, H, D)
    assert _err(got_q[..., :dk], wq) < TOL[dt] and got_q[..., dk:].abs().sum().item() == 0
    assert _err(kc[:, pos0:pos0 + T, :dk].transpose(0, 1), wk) < TOL[dt]
    assert torch.equal(vt[:, :dv, pos0:pos0 + T].permute(2, 0, 1).double().cpu(), v)
    assert kc[:, :pos0].abs().sum().item() == 0 and kc[:, pos0 + T:].abs().sum().item() == 0 and vt[:, :, pos0 + T:].abs().sum().item() == 0
    assert torch.equal(dev[:, H * D:].cpu(), row[:, H * D:])


def _attn_oracle(q, k, v, q_pos0, window, sink, gate, scale):
    """q [T, H, dk] at positions q_pos0 .., k / v [N, G, .] at 0 .. -> [T, H, dv]"""
    T, N, H, G = q.shape[0], k.shape[0], q.shape[1], k.shape[1]
    mask = O.window_mask(q_pos0 + T, window or None)[q_pos0:, :N]
    out = torch.empty(T, H, v.shape[2], dtype=torch.float64)
    for h in range(H):
        s = (q[:, h] @ k[:, h // (H // G)].T) * scale
        p = O.softmax_plus_one(s, mask) if sink else s.masked_fill(~mask, float("-inf")).softmax(-1)
        out[:, h] = p @ v[:, h // (H // G)]
    return out if gate is None else out * torch.sigmoid(gate)[..., None]


CASES = [  # H, G, D, dim, T, q_pos0, window
    (4, 2, 64, 64, 70, 0, 24), (2, 1, 128, 96, 200, 0, 40), (2, 1, 128, 128, 2, 129, 64), (3, 3, 64, 40, 130, 61, 1), (4, 1, 128, 128, 129, 63, 0), (2, 2, 64, 64, 300, 100, 128),
    (2, 1, 128, 80, 257, 0, 257), (1, 1, 64, 64, 1, 0, 8), (2, 1, 256, 200, 90, 30, 33)]


@pytest.mark.parametrize("dt", list(DT))
@pytest.mark.parametrize("rows_form", [False, True])
@pytest.mark.parametrize("H,G,D,dim,T,q_pos0,window", CASES)
def test_window_attention(cuda, dt, rows_form, H, G, D, dim, T, q_pos0, window):
    """random scores; then one standing-out key moved over every query's window edge: seen just inside, not seen just outside"""
    from llava_mi355x import ops
    if rows_form and (dt == "f32" or D == 256):
        pytest.skip("already the only form")
    N, s_max = q_pos0 + T, (q_pos0 + T + 127) // 128 * 128
    g = torch.Generator().manual_seed(T + H)
    q, k, v = (torch.randn(n, h, dim, generator=g).to(DT[dt]) for n, h in ((T, H), (N, G), (N, G)))
    gate = torch.randn(T, H, generator=g).to(DT[dt])
    stride = H * D + 64
    row = torch.zeros(T, stride, dtype=DT[dt]); row[:, :H * D] = _pad(q, D).reshape(T, -1); row[:, H * D:H * D + H] = gate
    scale = 0.7 * dim ** -0.5

    def run(kk, vv, sink, use_gate):
        kc, vt = torch.zeros(G, s_max, D, dtype=DT[dt], device=cuda), torch.zeros(G, D, s_max, dtype=DT[dt], device=cuda)
        kc[:, :N] = _pad(kk, D).transpose(0, 1).to(cuda); vt[:, :, :N] = _pad(vv, D).permute(1, 2, 0).to(cuda)
        got = ops.window_attn(row.to(cuda), kc, vt, q_pos0, H, G, scale, window, sink, H * D if use_gate else -1, rows_form)
        want = _attn_oracle(q.double(), kk.double(), vv.double(), q_pos0, window, sink, gate.double() if use_gate else None, scale)
        got = got.reshape(T, H, D)
        assert D == dim or got[..., dim:].abs().max().item() == 0
        return got[..., :dim], want
    for sink, use_gate in ((True, True), (False, False), (True, False)):
        got, want = run(k, v, sink, use_gate)
        assert _err(got, want) < TOL[dt], (sink, use_gate)
    # very negative scores: the sink takes (almost) everything
    got, want = run(-30 * q[:1, :1].expand(N, G, dim).contiguous(), v, True, False)
    assert (got.double().cpu() - want).abs().max() < TOL[dt] * v.abs().max().double()
    if window:
        for i in sorted({0, T // 3, T - 1}):                            # this query's first visible key and the one before it carry a large value
            first = q_pos0 + i - window + 1
            for j in (first, first - 1):
                if j < 0:
                    continue
                vv = v.clone(); vv[j] = 50.0
                got, want = run(k, vv, True, False)
                assert (got[i].double().cpu() - want[i]).abs().max() < max(TOL[dt] * want[i].abs().max().item(), 0.05)


@pytest.mark.parametrize("dt", list(DT))
@pytest.mark.parametrize("H,G,D,dim,vdim,rot", [(4, 2, 64, 48, 64, 32), (2, 1, 128, 96, 100, 96), (3, 3, 128, 128, 128, 20), (6, 1, 256, 136, 200, 64)])
@pytest.mark.parametrize("window", [0, 1, 40, 128, 200])
@pytest.mark.parametrize("n_split", [1, 2, 5])
def test_one_token_launch(cuda, dt, H, G, D, dim, vdim, rot, window, n_split):
    """mixed positions in one launch (0, chunk borders, far out); keys before the window and everything past the position hold values that would show"""
    from llava_mi355x import ops
    s_max, eps, scale = 640, 1e-5, 0.8 * dim ** -0.5
    positions = [0, 1, 63, 127, 128, 129, 255, 256, 400, 639]
    stride = (H + 2 * G) * D + 64
    n = len(positions)
    row, q, k, v = _qkv(n, H, G, D, dim, vdim, stride, dt, 11)
    g = torch.Generator().manual_seed(5)
    gate = torch.randn(n, H, generator=g).to(DT[dt]); row[:, (H + 2 * G) * D:(H + 2 * G) * D + H] = gate
    qn, kn = (1 + 0.3 * torch.randn(dim, generator=g)).to(DT[dt]), (1 + 0.3 * torch.randn(dim, generator=g)).to(DT[dt])
    r = {"dims": rot, "base": 300.0, "scaling": {"factor": 2.5}}
    kcs, vts, olds = [], [], []
    for i, p in enumerate(positions):
        kk, vv = torch.randn(s_max, G, dim, generator=g).to(DT[dt]), torch.randn(s_max, G, vdim, generator=g).to(DT[dt])
        first = max(0, p - window + 1) if window else 0
        if first > 0:
            vv[first - 1] = 80.0                                         # just outside the window
        kc, vt = _pad(kk, D).transpose(0, 1).contiguous(), _pad(vv, D).permute(1, 2, 0).contiguous()
        kc[:, p:] = float("nan"); vt[:, :, p:] = float("nan")            # never-written rows
        kcs.append(kc.to(cuda)); vts.append(vt.to(cuda)); olds.append((kk[:p].double(), vv[:p].double()))
    words = [torch.tensor([p], dtype=torch.int32, device=cuda) for p in positions]
    got = ops.decode_win(row.to(cuda), kcs, vts, words, _table(r, s_max).to(cuda), H, G, dim, rot, scale, eps, _pad(qn, D).to(cuda), _pad(kn, D).to(cuda), window, True, (H + 2 * G) * D,
                         n_split).reshape(n, H, D)
    rd = lambda x: x.to(DT[dt]).double()
    for i, p in enumerate(positions):
        pos = torch.tensor([p])
        qi = rd(O.rotate(O.rms_norm(q[i:i + 1], qn.double(), eps), pos, r)); ki = rd(O.rotate(O.rms_norm(k[i:i + 1], kn.double(), eps), pos, r))
        want = _attn_oracle(qi, torch.cat([olds[i][0], ki]), torch.cat([olds[i][1], v[i:i + 1]]), p, window, True, gate[i:i + 1].double(), scale)
        assert _err(got[i:i + 1, :, :vdim], want) < TOL[dt], (p, _err(got[i:i + 1, :, :vdim], want))
        assert _err(kcs[i][:, p, :dim], ki[0]) < TOL[dt] and torch.equal(vts[i][:, :vdim, p].double().cpu(), v[i])
        assert torch.equal(kcs[i][:, :p, :dim].double().cpu().transpose(0, 1), olds[i][0]) and bool(torch.isnan(kcs[i][:, p + 1:]).all())


@pytest.mark.parametrize("dt", list(DT))
def test_one_token_launch_matches_the_prompt_kernel(cuda, dt):
    """the same token through the prompt kernels and through the one-token launch: the cache rows are equal, the outputs differ by rounding only"""
    from llava_mi355x import ops
    H, G, D, dim, rot, T, window, eps, scale, s_max = 4, 2, 128, 96, 96, 150, 60, 1e-5, 0.1, 256
    stride = (H + 2 * G) * D + 64
    row, *_ = _qkv(T, H, G, D, dim, dim, stride, dt, 2)
    r = {"dims": rot, "base": 10000.0, "scaling": {"factor": 2.0}}
    w = _pad(torch.ones(dim).to(DT[dt]), D).to(cuda)
    tab = _table(r, s_max).to(cuda)
    mk = lambda: (torch.zeros(G, s_max, D, dtype=DT[dt], device=cuda), torch.zeros(G, D, s_max, dtype=DT[dt], device=cuda))
    (ka, va), (kb, vb) = mk(), mk()
    full, part = row.to(cuda), row[:T - 1].to(cuda)
    ops.qkv_norm_rope_kv(full, ka, va, w, w, tab, 0, H, G, dim, rot, eps)
    a = ops.window_attn(full, ka, va, 0, H, G, scale, window, True, (H + 2 * G) * D)[-1]
    ops.qkv_norm_rope_kv(part, kb, vb, w, w, tab, 0, H, G, dim, rot, eps)
    b = ops.decode_win(row[T - 1:].to(cuda), [kb], [vb], [torch.tensor([T - 1], dtype=torch.int32, device=cuda)], tab, H, G, dim, rot, scale, eps, w, w, window, True, (H + 2 * G) * D, 2)[0]
    assert _err(kb, ka.float()) < TOL[dt] / 2 and torch.equal(va, vb)
    assert _err(b, a.float()) < TOL[dt]


def test_bad_arguments_raise(cuda):
    from llava_mi355x import ops
    from llava_mi355x._C import LmxError
    x = torch.zeros(1, 100, device=cuda)
    with pytest.raises(LmxError):
        ops.residual_norm(x, None, None, None, torch.zeros(100, dtype=torch.bfloat16, device=cuda), 1.0, 1e-5)          # width not a multiple of 8
    kc, vt = torch.zeros(1, 128, 96, device=cuda), torch.zeros(1, 96, 128, device=cuda)
    with pytest.raises(LmxError):
        ops.window_attn(torch.zeros(4, 96, device=cuda), kc, vt, 0, 1, 1, 1.0)                                             # head width 96 is not a padded width
