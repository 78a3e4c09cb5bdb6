"""Building blocks of hybrid decoders (recurrent and attention layers in one stack): mixers that own
their weights and the layout of their cache, hyper-connections, feed-forwards."""

from .context import StepContext  # noqa: F401
from .differential_attention import DifferentialAttentionMixer, interleaved_rope_tables  # noqa: F401
from .gated_delta import GatedDeltaMixer  # noqa: F401
from .hyper_connection import HyperConnection  # noqa: F401
from .mlp import SquaredReluMLP  # noqa: F401
from .channel_delta import ChannelDelta  # noqa: F401
from .experts import RoutedExperts  # noqa: F401
from .parallel_mixer import ParallelMixer  # noqa: F401
from .pooled_attention import PooledAttention  # noqa: F401
