"""Model families: BERT-style sentence encoders, Llama-3-style, latent-attention (Vumuvik), hybrid
(Vugotar, Vunelix) and depth-averaged (Bizetar) decoders."""
from .bert import BertEncoder, pack_sequences  # noqa: F401
from .bizetar import BizetarModel  # noqa: F401
from .cache import AttnMeta, HybridCache, KVCache, LatentCache  # noqa: F401
from .configs import (  # noqa: F401
    DECODERS,
    ENCODERS,
    BizetarConfig,
    DecoderConfig,
    EncoderConfig,
    LatentLayer,
    LatentMixer,
    VugotarConfig,
    VumuvikConfig,
    VunelixConfig,
    decoder_config,
    encoder_config,
    is_decoder,
    is_encoder,
)
from .llama import LlamaModel  # noqa: F401
from .registry import DecoderFamily, decoder_family  # noqa: F401
from .vugotar import VugotarModel  # noqa: F401
from .vumuvik import VumuvikModel  # noqa: F401
from .vunelix import VunelixModel  # noqa: F401
from .weights import (  # noqa: F401
    load_bizetar_checkpoint,
    load_decoder_checkpoint,
    load_encoder_checkpoint,
    load_vugotar_checkpoint,
    load_vumuvik_checkpoint,
    load_vunelix_checkpoint,
    random_bizetar_weights,
    random_decoder_weights,
    random_encoder_weights,
    random_vugotar_weights,
    random_vumuvik_weights,
    random_vunelix_weights,
    shard_decoder_weights,
)
