"""Sizes that the kernels take, as plain numbers: parts check them when a model is put
together (a model that a kernel would refuse at its first step is refused when it is built),
and `ops.py` checks them again before a launch.  Nothing here touches the GPU."""

MAX_HEAD_DIM = 256  # the attention kernels keep a head's elements in four registers per lane
# the widest row whose partial sums (a product taken in slices of K) the residual add + norm adds
# up: 256 threads x 4 elements x NORM_CHUNKS of norm.hip, and a multiple of 4
MAX_SUMMED_NORM_WIDTH = 8192
# the recurrence with a matrix state keeps a head's key channels in registers, a quarter per thread
MAX_WKV_HEAD_DIM = 256
# the delta rule's walk keeps a column of a head's state in the registers of sixteen lanes, up to sixteen each;
# its convolution keeps a head in a wavefront, four elements a lane
MAX_DELTA_HEAD_DIM = 256
# gated linear attention: as the recurrence with a matrix state, key and value channels each
MAX_GLA_HEAD_DIM = 256
# Mamba-2's recurrence: state and value channels of a head; a wavefront keeps a token's state channels in registers
MAX_SSD_DIM = 256
# heads whose weights are mixed keep a tile of scores, one of weights and their sums in LDS
MAX_TALKING_LDS = 160 * 1024
TALKING_KEYS = 64


def check_talking_sizes(heads: int, head_dim: int) -> None:
    """Raises ValueError for sizes whose heads' weights no kernel mixes."""
    need = 4 * (2 * heads * TALKING_KEYS + heads * head_dim + 2 * heads)
    if need > MAX_TALKING_LDS:
        raise ValueError(f"{heads} heads of {head_dim} elements whose weights are mixed need {need} bytes of LDS, "
                         f"there are {MAX_TALKING_LDS}")


def check_head_dim(head_dim: int, rotary_dim: int = 0) -> None:
    """Raises ValueError for a head size that the attention kernels refuse."""
    if head_dim <= 0:
        raise ValueError(f"head_dim must be positive, not {head_dim}")
    if head_dim > MAX_HEAD_DIM:
        raise ValueError(f"head_dim {head_dim} is larger than the attention kernels take ({MAX_HEAD_DIM})")
    if rotary_dim and (rotary_dim % 2 or rotary_dim > head_dim):
        raise ValueError(f"a rotation over {rotary_dim} elements does not fit a head_dim of {head_dim} (even, within the head)")
