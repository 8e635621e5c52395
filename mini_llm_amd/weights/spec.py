"""What a part says about each of its tensors: shape in the file, role, and how to draw it."""

from __future__ import annotations

from dataclasses import dataclass

MATRIX = "matrix"        # operand of a matrix product: kept in the compute dtype
TABLE = "table"          # rows looked up by index: kept in the compute dtype
VECTOR = "vector"        # bias / norm gain / norm offset: kept in 32-bit
INT_TABLE = "int_table"  # integer table: kept as int32


class FreeDim(int):
    """A dimension that no configuration gives: the file's tensors do. The number itself is what a randomly drawn model takes; a file
    may bring any other (at least 1), the same one wherever a part names the same FreeDim object."""


@dataclass(frozen=True)
class Normal:
    """Draw from N(mean, std)."""

    std: float
    mean: float = 0.0


@dataclass(frozen=True)
class TensorSpec:
    shape: tuple  # as stored in the file (a dimension may be a FreeDim)
    role: str
    init: Normal
    # Stored [in, out] (the Conv1D layout of GPT-2 files); kept transposed, [out, in], which is
    # what the matrix kernels read.
    keep_transposed: bool = False
