from .configuration import BezuraxConfig  # noqa: F401
from .convert import checkpoint_to_nxd  # noqa: F401
