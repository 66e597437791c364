from .linear_attention import FeatureMap, LinearAttention, TaylorExp  # noqa: F401
from .slide_attention import SlidingAttention  # noqa: F401
from .convolution import BaseConv, ShortConvolution  # noqa: F401
from .decay_attention import DecayAttention  # noqa: F401
from .gated_delta import GatedDeltaRule  # noqa: F401
from .latent_attention import LatentAttention  # noqa: F401
from .rglru import RGLRU  # noqa: F401
from .side_by_side import SideBySide  # noqa: F401
from .streaming import StreamConv  # noqa: F401
from .time_mix import TimeMix  # noqa: F401
from .window_attention import WindowAttention  # noqa: F401
