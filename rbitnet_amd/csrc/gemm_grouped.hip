// Products in groups: the experts of a routed feed-forward, without gates, for steps of many tokens.  The step's (token, expert) pairs
// are sorted by expert in runs padded to the tiles' rows (rb_route_choose_units), so that a tile of rows belongs to one expert, and
// the tiles are those of the dense product with direct loads into LDS: the way up reads its rows where the tokens lie (a row of a
// tile is any row of h) and leaves the units of the sorted rows; the way down writes every row to its pair's place.
#include "api.h"
#include "gemm_dma.h"

template <int BN, int BM, int WN, int WM, int S, int GR, typename TO>
static int launch_grouped(const bf16_t* x, const bf16_t* w, TO* c, int m_tiles, int n, int k, const float* act, const GemmGroups& groups,
                          hipStream_t s) {
  constexpr int BK = 64;
  const int n_tiles = (n + BN - 1) / BN;
  const long long tiles = (long long)m_tiles * n_tiles;
  RB_REQUIRE(tiles < (1LL << 30), "rb_routed_experts_tiled: too many tiles");
  const size_t lds = (size_t)S * (BN + BM) * BK * sizeof(bf16_t);
  auto kern = gemm_dma_kernel<BN, BM, WN, WM, BK, S, 0, TO, true, GR>;
  static bool configured = false;
  if (!configured) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    RB_REQUIRE(e == hipSuccess, "rb_routed_experts_tiled: cannot reserve %zu bytes of LDS: %s", lds, hipGetErrorString(e));
    configured = true;
  }
  kern<<<dim3((unsigned)((tiles + 7) / 8 * 8)), 64 * (BN / WN) * (BM / WM), lds, s>>>(x, w, c, nullptr, m_tiles * BM, n, k, m_tiles, n_tiles,
                                                                                      k / BK, act, groups);
  return 0;
}

extern "C" int rb_routed_experts_tiled(const void* h, int n_tokens, int top, const int32_t* row_pair, const int32_t* tile_expert, int unit,
                                       int max_rows, const void* w_up, const void* w_down, const float* act, void* y, float* out,
                                       int n_experts, int width, int ff, void* stream) {
  RB_RECORDED(rb_routed_experts_tiled(h, n_tokens, top, row_pair, tile_expert, unit, max_rows, w_up, w_down, act, y, out, n_experts, width,
                                      ff, stream));
  RB_REQUIRE(n_tokens >= 0 && top > 0 && n_experts > 0 && width > 0 && ff > 0 && width % 64 == 0 && ff % 64 == 0,
             "rb_routed_experts_tiled: bad sizes T=%d top=%d experts=%d width=%d ff=%d (sizes are multiples of 64)", n_tokens, top, n_experts,
             width, ff);
  RB_REQUIRE((unit == 64 || unit == 128 || unit == 256) && max_rows >= 0 && max_rows % unit == 0,
             "rb_routed_experts_tiled: runs padded to %d rows not supported (64, 128, 256)", unit);
  // byte offsets inside a tile's operands are 32-bit; those of the gathered rows count from h's first
  RB_REQUIRE((long long)n_tokens * width * 2 < (1LL << 32) && 256LL * width * 2 < (1LL << 32) && 256LL * ff * 2 < (1LL << 32),
             "rb_routed_experts_tiled: %d tokens of %d numbers are too many", n_tokens, width);
  RB_REQUIRE(act != nullptr, "rb_routed_experts_tiled: the units need their activation's numbers");
  auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  RB_REQUIRE(aligned(h) && aligned(w_up) && aligned(w_down) && aligned(y) && aligned(out), "rb_routed_experts_tiled: operands must be 16-byte aligned");
  if (n_tokens == 0 || max_rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const GemmGroups groups = {tile_expert, row_pair, top};
  const int m_tiles = max_rows / unit;
  const bf16_t *x = (const bf16_t*)h, *wu = (const bf16_t*)w_up, *wd = (const bf16_t*)w_down;
  bf16_t* yb = (bf16_t*)y;
  int rc;
#define GR_GO(BN, BM, WN, WM, S)                                                                                    \
  do {                                                                                                              \
    rc = launch_grouped<BN, BM, WN, WM, S, 1, bf16_t>(x, wu, yb, m_tiles, ff, width, act, groups, s);               \
    if (!rc) rc = launch_grouped<BN, BM, WN, WM, S, 2, float>(yb, wd, out, m_tiles, width, ff, nullptr, groups, s); \
  } while (0)
  if (unit == 256) GR_GO(256, 256, 128, 64, 2);
  else if (unit == 128) GR_GO(256, 128, 64, 64, 3);
  else GR_GO(128, 64, 32, 64, 3);
#undef GR_GO
  if (rc) return rc;
  RB_LAUNCH_CHECK();
  return 0;
}
