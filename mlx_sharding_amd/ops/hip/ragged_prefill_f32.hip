// 32-bit instances of the expanded latent attention (fewer shapes: this mode
// is for checking, shapes are padded further instead).
#include "ragged_prefill.h"

extern "C" void launch_latent_attn_long_f32(const LatentLongArgs* a, int nks,
                                            int ndh, hipStream_t stream) {
#define LP_CASE(K, D) \
  case K * 100 + D: latent_attn_long_go<float, K, D>(*a, stream); break
  switch (nks * 100 + ndh) {
    LP_CASE(4, 4); LP_CASE(4, 16);
    LP_CASE(8, 4); LP_CASE(8, 16);
    default: break;
  }
#undef LP_CASE
}
