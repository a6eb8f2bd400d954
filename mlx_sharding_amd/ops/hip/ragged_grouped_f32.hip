// float instances of grouped attention: head sizes up to 64, 128, 256 and (short
// portions only) 512, keys and values apart.
#include "ragged_grouped.h"

extern "C" void launch_grouped_attn_short_f32(const GroupedAttnArgs* a,
                                             int size_k, int size_v,
                                             hipStream_t stream) {
#define GA_CASE(K, V)                                                   \
  case K * 1000 + V:                                                    \
    grouped_attn_short_go<float, K / 32, V / 16>(*a, stream);              \
    break
  switch (size_k * 1000 + size_v) {
    GA_CASE(64, 64); GA_CASE(64, 128); GA_CASE(64, 256);
    GA_CASE(128, 64); GA_CASE(128, 128); GA_CASE(128, 256);
    GA_CASE(256, 64); GA_CASE(256, 128); GA_CASE(256, 256);
    GA_CASE(512, 512);
    default: break;
  }
#undef GA_CASE
}

extern "C" void launch_grouped_attn_long_f32(const GroupedAttnArgs* a,
                                            int size_k, int size_v,
                                            hipStream_t stream) {
#define GA_CASE(K, V)                                                   \
  case K * 1000 + V:                                                    \
    grouped_attn_long_go<float, K / 32, V / 16>(*a, stream);               \
    break
  switch (size_k * 1000 + size_v) {
    GA_CASE(64, 64); GA_CASE(64, 128); GA_CASE(64, 256);
    GA_CASE(128, 64); GA_CASE(128, 128); GA_CASE(128, 256);
    GA_CASE(256, 64); GA_CASE(256, 128); GA_CASE(256, 256);
    default: break;
  }
#undef GA_CASE
}
