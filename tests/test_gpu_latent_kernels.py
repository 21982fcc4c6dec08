"""The latent-attention decoder's kernels one by one, through the C ABI, against
the plain float64 statement of each mechanism."""
import ctypes

import numpy as np
import pytest
import torch

import latent_model as lm
import latent_oracle as lo
import mixed_model as mm
import qllm_hip as qh
from kernel_util import BF16, F32, close, on, padded, steps, torch_type

pytestmark = pytest.mark.gpu

EPS = 1e-5


def per_head(device, matrix, heads, padded_rows, transposed):
    """A tensor of `heads` matrices, packed tile after tile."""
    size, width = matrix.shape[0] // heads, matrix.shape[1]
    rows, columns = (width, size) if transposed else (size, width)
    data = torch.zeros(qh.call("qllm_linear_packed_bytes", heads * padded_rows, columns),
                       dtype=torch.uint8, device=device)
    source = on(device, matrix, torch.bfloat16)
    for head in range(heads):
        qh.call("qllm_linear_pack_strided", source.data_ptr() + 2 * head * size * width, rows,
                columns, 1 if transposed else width, width if transposed else 1, qh.ptr(data),
                padded(columns, 64), head * padded_rows // 16, 1, 0, None)
    torch.cuda.synchronize()
    return data


@pytest.mark.parametrize("rows,columns", [(5, 70), (33, 64), (48, 9)])
def test_packing_part_of_a_matrix_and_its_transpose(device, rows, columns):
    rng = np.random.default_rng(rows)
    matrix = mm.bf16(rng.standard_normal((3 * rows, columns)))
    for transposed in (False, True):
        part = matrix[rows:2 * rows]
        part = np.ascontiguousarray(part.T if transposed else part)
        d_part, d_all = on(device, part, torch.bfloat16), on(device, matrix, torch.bfloat16)
        out = [torch.zeros(qh.call("qllm_linear_packed_bytes", *part.shape), dtype=torch.uint8,
                           device=device) for _ in range(2)]
        qh.call("qllm_linear_pack", qh.ptr(d_part), *part.shape, qh.ptr(out[0]),
                padded(part.shape[1], 64), 0, 1, 0, None)
        qh.call("qllm_linear_pack_strided", d_all.data_ptr() + 2 * rows * columns, *part.shape,
                1 if transposed else columns, columns if transposed else 1, qh.ptr(out[1]),
                padded(part.shape[1], 64), 0, 1, 0, None)
        torch.cuda.synchronize()
        assert torch.equal(*out)


# ---- norms behind a sublayer ------------------------------------------------------


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("width,count", [(64, 1), (90, 3), (132, 9), (2052, 4)])
def test_partial_sums_pass_a_norm_into_the_stream(device, element, width, count):
    rng = np.random.default_rng(width)
    rows, stride = 5, padded(width, 64)
    x = rng.standard_normal((rows, width)).astype(np.float32)
    partials = 30.0 * rng.standard_normal((count, rows, padded(width, 4))).astype(np.float32)
    weight, post = rng.standard_normal((2, width)).astype(np.float32)
    d_x, d_partials, d_weight, d_post = (on(device, a) for a in (x, partials, weight, post))
    out = torch.full((rows, stride), 9.0, dtype=torch_type(element), device=device)
    stream = torch.zeros((rows, width), device=device)

    def launch(**changes):
        values = dict(
            input=qh.ptr(d_x), stream_out=qh.ptr(stream), partials=qh.ptr(d_partials),
            partial_count=count, partial_stride=padded(width, 4),
            weight=(ctypes.c_void_p * 2)(qh.ptr(d_weight), None),
            output=(ctypes.c_void_p * 2)(qh.ptr(out), None),
            stride=(ctypes.c_uint32 * 2)(stride, 0), rows=rows, width=width, epsilon=0.5,
            element=element, branch_weight=qh.ptr(d_post), branch_scale=0.3,
            branch_epsilon=2.0)
        values.update(changes)
        qh.call("qllm_stream_norm", ctypes.byref(qh.StreamNormLaunch(**values)), None)
        torch.cuda.synchronize()

    launch()
    added = partials[:, :, :width].astype(np.float64).sum(0)
    want = x + 0.3 * lo.root_mean_square_norm(added, post.astype(np.float64), 2.0)
    close(stream, want, F32)
    close(out[:, :width], lo.root_mean_square_norm(want, weight.astype(np.float64), 0.5),
          element)
    assert torch.all(out[:, width:] == 0)
    # the stream alone
    stream.zero_()
    launch(weight=(ctypes.c_void_p * 2)(None, None), output=(ctypes.c_void_p * 2)(None, None))
    close(stream, want, F32)
    with pytest.raises(qh.QllmError):
        launch(partial_count=0)


# ---- latent attention --------------------------------------------------------------


class Latent:
    """Pages, table, weights and launches of one layer; rows are fed in any
    portions, outputs come back in order."""

    def __init__(self, device, element, heads, dim, rot_dim, rotary, vdim, rank, window,
                 page_tokens=64, context=512, slots=1, seed=0, scale=None, query_rank=0):
        rng = np.random.default_rng(seed)
        self.device, self.element = device, element
        self.heads, self.dim, self.rot_dim, self.vdim, self.rank = (heads, dim, rot_dim, vdim,
                                                                    rank)
        self.window, self.query_rank = window, query_rank
        self.scale = 1.2 / np.sqrt(dim + rot_dim) if scale is None else scale
        self.norm = mm.bf16(1.0 + 0.2 * rng.standard_normal(rank))
        self.key_up = mm.bf16(rng.standard_normal((heads * dim, rank)) / np.sqrt(rank))
        self.value_up = mm.bf16(rng.standard_normal((heads * vdim, rank)) / np.sqrt(rank))
        self.rot = {"dims": rotary, "base": 500.0, "scaling": lm.yarn(4.0, 128, 8.0, 1.0)}
        frequencies, magnitude = (lo.frequencies(**self.rot) if rotary else (np.zeros(1), 1.0))
        self.query_norm = mm.bf16(1.0 + 0.2 * rng.standard_normal(max(query_rank, 1)))
        self.keep = [
            torch.tensor(frequencies, dtype=torch.float64, device=device), on(device, self.norm),
            per_head(device, self.key_up, heads, padded(dim, 32), False),
            per_head(device, self.key_up, heads, padded(rank, 32), True),
            per_head(device, self.value_up, heads, padded(vdim, 16), False),
            on(device, self.query_norm)]
        pages = context // page_tokens
        layer = qh.call("qllm_latent_layer_bytes", page_tokens, rank, rot_dim, element)
        self.pages = [torch.zeros(layer + 64, dtype=torch.uint8, device=device)
                      for _ in range(pages * slots)]
        # pages in no particular order
        order = np.random.default_rng(0).permutation(len(self.pages))
        self.table = torch.tensor([self.pages[i].data_ptr() for i in order],
                                  dtype=torch.int64, device=device)
        self.step = steps(device, 0)
        self.width = heads * (dim + rot_dim)
        self.layer = qh.LatentAttention(
            heads, dim, vdim, rank, rot_dim, rotary, window, self.scale, EPS, magnitude,
            *map(qh.ptr, self.keep[:5]), page_tokens, pages, 64, qh.ptr(self.table),
            qh.ptr(self.step), element)

    def inputs(self, rng, rows):
        """(latent rows with the shared key part, queries, gates)."""
        return (mm.bf16(rng.standard_normal((rows, self.rank + self.rot_dim))),
                mm.bf16(rng.standard_normal((rows, self.width))),
                mm.bf16(rng.standard_normal((rows, self.heads * self.vdim))))

    def run(self, inputs, position, slot=0):
        latent, query, gate = (on(self.device, a) for a in inputs)
        rows = latent.shape[0]
        self.step.copy_(torch.tensor([position, slot, rows, 0], dtype=torch.int32))
        # query latents ahead of the latents, when there are any
        low = torch.randn((rows, self.query_rank), device=self.device)
        projections = torch.cat([low, latent], dim=1).contiguous()
        stride = padded(self.query_rank, 64)
        query_out = torch.full((rows, max(stride, 1)), 5.0, dtype=torch_type(self.element),
                               device=self.device)
        store = qh.LatentStoreLaunch(qh.ptr(projections), projections.shape[1], self.query_rank,
                                     0, self.query_rank, qh.ptr(self.keep[5]),
                                     qh.ptr(query_out), stride, rows)
        qh.call("qllm_latent_store", ctypes.byref(self.layer), ctypes.byref(store), None)
        last = position + rows - 1
        size = qh.call("qllm_latent_attention_workspace_bytes", ctypes.byref(self.layer), rows,
                       last)
        workspace = torch.zeros(max(size, 16), dtype=torch.uint8, device=self.device)
        out = torch.zeros((rows, self.heads * self.vdim + 3), dtype=torch_type(self.element),
                          device=self.device)
        launch = qh.LatentLaunch(
            qh.ptr(query), query.shape[1], qh.ptr(gate), gate.shape[1], qh.ptr(out),
            out.shape[1], rows, last, qh.ptr(workspace), size)
        qh.call("qllm_latent_attention_rows", ctypes.byref(self.layer), ctypes.byref(launch),
                None)
        torch.cuda.synchronize()
        assert torch.all(out[:, self.heads * self.vdim:] == 0)
        if self.query_rank:
            want = lo.root_mean_square_norm(low.double().cpu().numpy(),
                                            self.query_norm.astype(np.float64), EPS)
            close(query_out[:, :self.query_rank], want, self.element, "query latents")
            assert torch.all(query_out[:, self.query_rank:] == 0)
        return out[:, :self.heads * self.vdim].float().cpu().numpy().astype(np.float64)

    def cached(self, latent):
        """What the mathematics says about the cache rows."""
        latent = latent.astype(np.float64)
        c = lo.root_mean_square_norm(latent[:, :self.rank], self.norm.astype(np.float64), EPS)
        shared = latent[:, self.rank:]
        if self.rot["dims"]:
            shared = lo.rotate_halves(shared, range(len(shared)), self.rot)
        return c, shared

    def keys(self, c, head):
        return c @ self.key_up[head * self.dim:(head + 1) * self.dim].T.astype(np.float64)

    def expected(self, inputs, window=None):
        latent, query, gate = (a.astype(np.float64) for a in inputs)
        window = self.window if window is None else window
        rows = latent.shape[0]
        c, shared = self.cached(latent)
        q = query.reshape(rows, self.heads, self.dim + self.rot_dim)
        turned = q[..., self.dim:]
        if self.rot["dims"]:
            turned = lo.rotate_halves(turned, range(rows), self.rot)
        seen = lo.visible(rows, window or None)
        out = []
        for head in range(self.heads):
            v = c @ self.value_up[head * self.vdim:(head + 1) * self.vdim].T.astype(np.float64)
            out.append(lo.attend(np.concatenate([q[:, head, :self.dim], turned[:, head]], axis=1),
                                 np.concatenate([self.keys(c, head), shared], axis=1), v,
                                 self.scale, seen))
        return np.concatenate(out, axis=1) * lo.logistic(gate)


# heads, dim, rot, rotary, vdim, rank, window, page tokens, forms of few and many rows
SHAPES = [
    (1, 16, 0, 0, 16, 16, 0, 32, "split prompt"),
    (4, 48, 16, 16, 40, 56, 37, 64, "split prompt"),
    (3, 40, 24, 16, 33, 100, 1, 32, "split prompt"),
    (16, 128, 64, 64, 128, 512, 100, 64, "split prompt"),
    (20, 64, 0, 0, 72, 200, 0, 96, "split prompt"),
    (2, 160, 64, 32, 112, 256, 70, 64, "split prompt"),
    (8, 200, 64, 64, 144, 130, 50, 64, "split split"),
    (6, 32, 96, 96, 64, 300, 45, 64, "general prompt"),
    (2, 24, 8, 8, 16, 600, 70, 32, "general prompt"),
    (1, 240, 70, 70, 20, 520, 90, 64, "general general"),
    (5, 7, 2, 2, 5, 9, 20, 32, "split prompt"),
    (33, 16, 16, 8, 24, 40, 64, 64, "split prompt"),
]
FORMS = {"general": qh.ATTENTION_GENERAL, "split": qh.ATTENTION_SPLIT,
         "prompt": qh.ATTENTION_PROMPT}


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("shape", SHAPES, ids=lambda s: "x".join(map(str, s[:8])))
def test_latent_attention_in_portions(device, element, shape):
    heads, dim, rot, rotary, vdim, rank, window, page_tokens, forms = shape
    layer = Latent(device, element, heads, dim, rot, rotary, vdim, rank, window,
                   page_tokens=page_tokens, context=page_tokens * (1 + 300 // page_tokens),
                   query_rank=7 * heads)
    for rows, form in zip((1, 40), forms.split()):
        got = qh.call("qllm_latent_attention_form", ctypes.byref(layer.layer), rows)
        assert got == (FORMS["general"] if element == F32 else FORMS[form])
    rng = np.random.default_rng(heads * dim + window)
    inputs = layer.inputs(rng, 258)
    want = layer.expected(inputs)
    at, got = 0, []
    for count in (1, 2, 31, 3, 64, 4, 33, 1, 80, 17, 1, 1, 20):
        got.append(layer.run([a[at:at + count] for a in inputs], at))
        at += count
    assert at == 258
    close(np.concatenate(got), want, element, str(shape), factor=1.5)


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("rows", [1, 2, 20, 64, 150])
@pytest.mark.parametrize("window", [48, 0])
def test_edges_of_windows_and_pages_and_far_keys(device, element, rows, window):
    """One score stands out per case: a key just inside or outside the window, at a
    page's or a tile's border, the first ones, the query itself.  A mask off by one
    changes the output by its whole magnitude."""
    total, query = 420, 419
    layer = Latent(device, element, 3, 64, 32, 32, 48, 96, window, context=448, scale=0.15)
    rng = np.random.default_rng(rows)
    base = layer.inputs(rng, total)
    c, _ = layer.cached(base[0])
    keys = [query, query - 1, 383, 384] + (
        [query - window + 1, query - window, query - window - 1] if window
        else [0, 1, 31, 32, 63, 64, 128, 255, 256])
    for head in (0, 2):
        directions = layer.keys(c, head)
        for key in keys:
            inputs = [a.copy() for a in base]
            place = inputs[1][query].reshape(3, 96)[head]
            place[:] = 0.0
            place[:64] = mm.bf16(16.0 * directions[key] / np.linalg.norm(directions[key]))
            want = layer.expected(inputs)
            if window:
                for wrong, shows in ((window + 1, query - window), (window - 1, query - window + 1)):
                    if key == shows:   # the case would show such a mask
                        other = layer.expected(inputs, wrong)
                        change = np.abs(other[-1] - want[-1]).max() / np.abs(want[-1]).max()
                        assert change > 0.2
            cut = total - rows
            layer.run([a[:cut] for a in inputs], 0)
            got = layer.run([a[cut:] for a in inputs], cut)
            close(got, want[cut:], element, f"head {head} key {key}", factor=2.0)


@pytest.mark.parametrize("element", [F32, BF16])
def test_scores_that_grow_and_shrink_along_the_context(device, element):
    """Later keys outweigh earlier ones by far, and the other way round: sums kept
    so far must be scaled, or keep their weight."""
    layer = Latent(device, element, 2, 64, 0, 0, 32, 64, 0, context=320, scale=1.0)
    rng = np.random.default_rng(3)
    base = layer.inputs(rng, 300)
    c, _ = layer.cached(base[0])
    for order in (1, -1):
        inputs = [a.copy() for a in base]
        for row in range(300):
            for head in range(2):
                # a direction whose products with the keys are set one by one
                keys = layer.keys(c, head)[:row + 1]
                some = keys[::max(1, len(keys) // 12)]
                wish = np.linspace(-30.0, 30.0, len(some))[::order]
                inputs[1][row].reshape(2, 64)[head] = mm.bf16(np.linalg.pinv(some) @ wish)
        want = layer.expected(inputs)
        for counts in ([300], [100, 100, 100], [268, 32], [299, 1]):
            got, at = [], 0
            for count in counts:
                got.append(layer.run([a[at:at + count] for a in inputs], at))
                at += count
            # one key may hold nearly all weight: scores of 30 in bf16 operands
            close(np.concatenate(got), want, element, str(counts),
                  factor=4.0 if element == F32 else 12.0)


@pytest.mark.parametrize("rows", [1, 3, 40])
def test_contexts_of_many_tiles(device, rows):
    """More tiles than workgroups take one each; a key at the far end stands out."""
    total = 9000 + rows
    layer = Latent(device, BF16, 2, 32, 16, 16, 24, 64, 0, page_tokens=256, context=9216,
                   scale=0.2)
    rng = np.random.default_rng(1)
    inputs = layer.inputs(rng, total)
    c, shared = layer.cached(inputs[0])
    for head, far in ((0, 5), (1, 7777)):
        key = layer.keys(c, head)[far]
        place = inputs[1][-1].reshape(2, 48)[head]
        place[:] = 0.0
        place[:32] = mm.bf16(16.0 * key / np.linalg.norm(key))
    layer.run([a[:9000] for a in inputs], 0)
    got = layer.run([a[9000:] for a in inputs], 9000)
    for row in range(9000, total):
        q = inputs[1][row].reshape(2, 48).astype(np.float64)
        # the rotation of this row's position alone
        turned = lo.rotate_halves(q[None, :, 32:], [row], layer.rot)[0]
        want = []
        for head in range(2):
            v = c[:row + 1] @ layer.value_up[head * 24:(head + 1) * 24].T.astype(np.float64)
            keys = np.concatenate([layer.keys(c[:row + 1], head), shared[:row + 1]], axis=1)
            want.append(lo.attend(np.concatenate([q[head, :32], turned[head]])[None], keys, v,
                                  layer.scale, np.ones((1, row + 1), dtype=bool))[0])
        want = np.concatenate(want) * lo.logistic(inputs[2][row].astype(np.float64))
        close(got[row - 9000], want, BF16, str(row), factor=2.0)


def test_pages_and_slots_used_again(device):
    rng = np.random.default_rng(5)
    layer = Latent(device, BF16, 4, 32, 16, 16, 32, 80, 32, context=128, slots=2)
    long = [3.0 * a for a in layer.inputs(rng, 120)]
    short = layer.inputs(rng, 60)
    layer.run(long, 0, slot=1)
    want = layer.expected(short)
    for slot in (1, 0):
        got = np.concatenate([layer.run([a[i:j] for a in short], i, slot=slot)
                              for i, j in ((0, 40), (40, 41), (41, 60))])
        close(got, want, BF16, f"slot {slot}", factor=1.5)


def test_launches_turn_down_what_does_not_fit(device):
    layer = Latent(device, BF16, 4, 32, 16, 16, 32, 80, 32, context=128)
    anything = layer.table.data_ptr()
    bad = qh.LatentStoreLaunch(anything, 95, 0, 0, 0, None, None, 0, 1)
    with pytest.raises(qh.QllmError):
        qh.call("qllm_latent_store", ctypes.byref(layer.layer), ctypes.byref(bad), None)
    for rows in (1, 40):
        launch = qh.LatentLaunch(anything, layer.width, None, 0, anything, 128, rows, 100, None, 0)
        with pytest.raises(qh.QllmError, match="workspace"):
            qh.call("qllm_latent_attention_rows", ctypes.byref(layer.layer),
                    ctypes.byref(launch), None)
    short = qh.LatentLaunch(anything, layer.width - 1, None, 0, anything, 128, 1, 100, None, 0)
    with pytest.raises(qh.QllmError):
        qh.call("qllm_latent_attention_rows", ctypes.byref(layer.layer), ctypes.byref(short),
                None)


# ---- gated linear attention ----------------------------------------------------------


class Gated:
    def __init__(self, device, element, heads, dim, vdim, rank, tau, rng, slots=2):
        self.device, self.element = device, element
        self.heads, self.dim, self.vdim, self.rank, self.tau = heads, dim, vdim, rank, tau
        n, m = heads * dim, heads * vdim
        self.up = mm.bf16(rng.standard_normal((n, rank)) / np.sqrt(rank))
        self.base = mm.bf16(rng.standard_normal(n) + 1.0)
        self.norm = mm.bf16(1.0 + 0.2 * rng.standard_normal(vdim))
        # r k v gate low
        widths = [n, n, m, m, rank]
        self.columns = [sum(widths[:i]) + 3 * i for i in range(5)]
        self.stride = padded(self.columns[4] + rank, 4)
        self.keep = [on(device, self.up, torch.bfloat16), on(device, self.base),
                     on(device, self.norm)]
        self.slot_stride = n * vdim + 12
        self.state = torch.zeros(slots * self.slot_stride, device=device)
        self.step = steps(device, 0)
        up, base, norm = map(qh.ptr, self.keep)
        self.layer = qh.Recurrence(
            kind=qh.RECURRENCE_GATED, heads=heads, dim=dim, rank=rank, gate_kind=1, epsilon=EPS,
            decay_scale=1.0 / tau, decay_up_bf16=up, decay_base=base, norm_weight=norm,
            state=qh.ptr(self.state), slot_stride=self.slot_stride, step=qh.ptr(self.step),
            element=element, vdim=vdim, read_scale=dim ** -0.5)

    def run(self, projections, slot=1):
        rows = projections.shape[0]
        d = on(self.device, projections)
        self.step.copy_(torch.tensor([0, slot, rows, 0], dtype=torch.int32))
        size = qh.call("qllm_recurrence_workspace_bytes", ctypes.byref(self.layer), rows)
        workspace = torch.zeros(max(size, 16), dtype=torch.uint8, device=self.device)
        out = torch.zeros((rows, self.heads * self.vdim), dtype=torch_type(self.element),
                          device=self.device)
        r, k, v, gate, low = self.columns
        launch = qh.RecurrenceLaunch(
            projections=qh.ptr(d), stride=self.stride, r_column=r, k_column=k, v_column=v,
            gate_column=gate, low_column=low, output=qh.ptr(out),
            output_stride=self.heads * self.vdim, rows=rows, workspace=qh.ptr(workspace),
            workspace_bytes=size)
        qh.call("qllm_recurrence_rows", ctypes.byref(self.layer), ctypes.byref(launch), None)
        torch.cuda.synchronize()
        return out.float().cpu().numpy().astype(np.float64)

    def expected(self, projections):
        p = projections.astype(np.float64)
        rows = p.shape[0]
        r, k, v, gate, low = (p[:, c:c + w] for c, w in zip(
            self.columns, [self.heads * self.dim] * 2 + [self.heads * self.vdim] * 2 +
            [self.rank]))
        alpha = lo.channel_decay(low @ self.up.T.astype(np.float64) + self.base, self.tau)
        r, k, alpha = (x.reshape(rows, self.heads, self.dim) for x in (r, k, alpha))
        v = v.reshape(rows, self.heads, self.vdim)
        out, states = np.empty(v.shape), []
        for h in range(self.heads):
            out[:, h], state = lo.gated_recurrence(r[:, h] / np.sqrt(self.dim), k[:, h], v[:, h],
                                                   alpha[:, h], np.zeros((self.dim, self.vdim)))
            states.append(state)
        out = lo.root_mean_square_norm(out, self.norm.astype(np.float64), EPS)
        return out.reshape(rows, -1) * lo.swish(gate), np.stack(states)


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("heads,dim,vdim,rank,tau", [
    (3, 64, 64, 16, 16.0), (2, 24, 40, 8, 4.0), (1, 128, 256, 40, 16.0), (5, 16, 16, 1, 1.0),
    (2, 80, 48, 64, 9.0), (1, 256, 520, 33, 16.0), (7, 5, 3, 3, 2.0), (2, 1, 1, 2, 1.0),
    (1, 40, 1000, 5, 3.0)])
def test_gated_linear_attention_in_portions(device, element, heads, dim, vdim, rank, tau):
    rng = np.random.default_rng(heads * dim + vdim)
    layer = Gated(device, element, heads, dim, vdim, rank, tau, rng)
    projections = mm.bf16(rng.standard_normal((150, layer.stride)))
    want, states = layer.expected(projections)
    at, got = 0, []
    for count in (1, 1, 2, 37, 3, 16, 64, 1, 7, 17, 1):
        got.append(layer.run(projections[at:at + count]))
        at += count
    assert at == 150
    close(np.concatenate(got), want, element, "outputs", factor=2.0)
    n = heads * dim * vdim
    state = layer.state[layer.slot_stride:layer.slot_stride + n].cpu().numpy()
    close(state.reshape(heads, dim, vdim).astype(np.float64), states, F32, "state", factor=4.0)
    # the other slot was not touched
    assert torch.all(layer.state[:layer.slot_stride] == 0)
    # the same prompt in one piece
    layer.state[layer.slot_stride:] = 0
    close(layer.run(projections), want, element, "whole", factor=2.0)


def test_decays_near_both_ends(device):
    """Gates that keep nearly everything over the whole sequence, and gates that
    forget at once (whose logarithm a plain exponential would lose)."""
    rng = np.random.default_rng(2)
    layer = Gated(device, F32, 2, 8, 16, 4, 16.0, rng)
    layer.up[:] = 0.0
    layer.keep[0].zero_()
    layer.base[:] = np.tile([30.0, 12.0, 5.0, 0.0, -20.0, -200.0, -900.0, 3.0], 2)
    layer.keep[1].copy_(on(device, layer.base))
    projections = mm.bf16(rng.standard_normal((140, layer.stride)))
    want, states = layer.expected(projections)
    got = np.concatenate([layer.run(projections[:100]), layer.run(projections[100:101]),
                          layer.run(projections[101:])])
    close(got, want, F32, "outputs", factor=2.0)
    state = layer.state[layer.slot_stride:layer.slot_stride + 2 * 8 * 16].cpu().numpy()
    close(state.reshape(2, 8, 16).astype(np.float64), states, F32, "state", factor=4.0)


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("heads,dim,vdim,tau", [(2, 64, 128, 16.0), (1, 20, 36, 1.0),
                                                (3, 16, 256, 4.0), (1, 130, 8, 16.0),
                                                (1, 32, 300, 8.0)])
def test_long_prompts_in_segments(device, element, heads, dim, vdim, tau):
    rng = np.random.default_rng(dim)
    layer = Gated(device, element, heads, dim, vdim, 6, tau, rng)
    projections = mm.bf16(rng.standard_normal((1300, layer.stride)))
    want, states = layer.expected(projections)
    n = heads * dim * vdim
    for counts in ([1300], [600, 1, 699], [100, 530, 515, 155]):
        layer.state.zero_()
        got, at = [], 0
        for count in counts:
            got.append(layer.run(projections[at:at + count]))
            at += count
        close(np.concatenate(got), want, element, str(counts), factor=2.0)
        state = layer.state[layer.slot_stride:layer.slot_stride + n].cpu().numpy()
        close(state.reshape(heads, dim, vdim).astype(np.float64), states, F32, "state",
              factor=4.0)
        assert torch.all(layer.state[:layer.slot_stride] == 0)
