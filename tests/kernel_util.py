"""Helpers of the kernel tests of model-folder designs: arrays on the device,
tolerances, step words, packed weights."""
import numpy as np
import torch

import qllm_hip as qh

F32, BF16 = qh.ELEMENT_F32, qh.ELEMENT_BF16
# relative to the largest magnitude of the expected values
TOLERANCE = {F32: 2e-5, BF16: 1.2e-2}


def on(device, array, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(array)).to(device=device, dtype=dtype)


def torch_type(element):
    return torch.float32 if element == F32 else torch.bfloat16


def close(got, want, element, what="", factor=1.0):
    got = got.float().cpu().numpy().astype(np.float64) if torch.is_tensor(got) else got
    error = np.abs(got - want).max()
    bound = factor * TOLERANCE[element] * np.abs(want).max()
    assert error <= bound, f"{what}: {error:.3e} exceeds {bound:.3e}"


def steps(device, position, slot=0):
    return torch.tensor([position, slot, 0, 0], dtype=torch.int32, device=device)


def padded(value, to):
    return (value + to - 1) // to * to


def packed(device, parts, rows, columns):
    """parts: (matrix, first_tile, tile_stride, first_column)."""
    data = torch.zeros(qh.call("qllm_linear_packed_bytes", rows, columns),
                       dtype=torch.uint8, device=device)
    for matrix, tile, stride, column in parts:
        source = on(device, matrix, torch.bfloat16)
        qh.call("qllm_linear_pack", qh.ptr(source), *matrix.shape, qh.ptr(data),
                padded(columns, 64), tile, stride, column, None)
    torch.cuda.synchronize()
    return data
