// The bfloat16 product whose tiles go from memory straight into LDS, as a template: the dense products of gemm_tiled.hip and the
// products in groups of gemm_grouped.hip are instances of it.
#pragma once
#include <type_traits>

#include "gemm_internal.h"

// Which tile a workgroup computes.  Workgroup ids go round robin over the 8 XCDs, each with
// an L2 of its own: every XCD gets a contiguous range of the tile order, and the order runs
// through groups of TG_GROUP_M token tiles, all row tiles of a group before the next group.  The
// 32 workgroups that an XCD runs at a time then cover about 8 x 4 tiles and walk K together,
// so 12 tile rows come from beyond L2 per step for 32 tiles' worth of products.
#define TG_GROUP_M 8
__device__ __forceinline__ bool tile_of_workgroup(int m_tiles, int n_tiles, int* mt, int* nt) {
  const int tiles = m_tiles * n_tiles;
  const int per_xcd = (tiles + 7) / 8;
  const int t = (blockIdx.x % 8) * per_xcd + blockIdx.x / 8;
  if (t >= tiles) return false;
  const int in_group = TG_GROUP_M * n_tiles;
  const int first_m = t / in_group * TG_GROUP_M;
  const int rows = min(m_tiles - first_m, TG_GROUP_M);
  const int r = t % in_group;
  *mt = first_m + r % rows;
  *nt = r / rows;
  return true;
}

// What a lane holds of a 32 x 32 piece when the tokens were the MFMA's rows and W's rows its
// columns: W row first_row + l32 for the 16 tokens mbase + 8 (e / 4) + e % 4 (mbase includes the
// lane's 4 g).  A wave's store then covers 32 consecutive outputs of each of two tokens.  With
// `slab`, the sums go to that slice's [M, N] slab instead, to be added up later in a fixed order.
// row_map (epilogue 0): where in c a row goes.
template <int EPI, typename TO>
__device__ __forceinline__ void store_piece(const f32x16_t& acc, TO* __restrict__ c, float* __restrict__ slab,
                                            int first_row, int l32, int mbase, int m, int n, bool has_act = false,
                                            float ap = 0.f, float an = 0.f, GatePair gp = GatePair{0.f, 0.f},
                                            const int32_t* __restrict__ row_map = nullptr) {
  if (EPI == 0) {
    const int nn = first_row + l32;
    if (nn >= n) return;
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int mm = mbase + 8 * (e / 4) + (e % 4);
      if (mm >= m) continue;
      if (row_map) {                             // the row goes where the map says (-1: nowhere)
        const int to = row_map[mm];
        if (to >= 0) Num<TO>::store(c + (size_t)to * n + nn, acc[e]);
        continue;
      }
      if (slab) slab[(size_t)mm * n + nn] = acc[e];
      else Num<TO>::store(c + (size_t)mm * n + nn, has_act ? xielu_value(acc[e], ap, an) : acc[e]);
    }
  } else {
    // gate rows in lanes 0..15 of a half wave, up rows in lanes 16..31: the two halves swap what
    // the other needs, the lower one finishing the even tokens and the upper one the odd ones
    const int half_n = n / 2;
    const bool upper = (l32 & 16) != 0;
    const int col = first_row / 2 + (l32 & 15);
#pragma unroll
    for (int e = 0; e < 16; e += 2) {
      const float mine = upper ? acc[e + 1] : acc[e];
      const float give = upper ? acc[e] : acc[e + 1];
      const float got = __shfl_xor(give, 16);
      const int mm = mbase + 8 * (e / 4) + (e % 4) + (upper ? 1 : 0);
      const float gate = upper ? got : mine, up = upper ? mine : got;
      if (mm < m && col < half_n) Num<TO>::store(c + (size_t)mm * half_n + col, gated_value(gate, up, gp));
    }
  }
}

// The same product with the tiles brought from memory straight into LDS
// (global_load_lds_dwordx4: no registers, no LDS store instruction), S stages deep.
//
// A wave's load instruction fills 1 KB of LDS in lane order, so rows cannot be padded.  Rows
// of BK elements are kept dense and the 16-byte chunks of a row are permuted instead: chunk c
// of row r lies in slot c ^ swz(r), swz(r) = (r / rows per 256 bytes) % chunks per row.  The
// permutation is applied on the memory side (which chunk a lane fetches), and the 16 lanes of
// a quarter wave that read one chunk column of 16 rows then hit 16 different bank groups.
//
// The loads are inline assembly, so the compiler neither counts nor waits for them: the
// kernel waits itself (s_waitcnt vmcnt) for the stage it is about to read, leaving the
// younger stages in flight.  There is no other memory access in the main loop.
//
// GR: a product in groups (W [groups][N, K], one after another): the tokens' rows are sorted by group in runs padded to BM, so
// that a tile of rows belongs to one group, tile_group[row tile] (-1: none).  GR 1: row r of the tiles is row row_pair[r] / top of x
// (-1: any); c gets the rows in the tiles' order.  GR 2: x holds the rows in the tiles' order; c gets row r at row_pair[r].
struct GemmGroups {
  const int32_t* tile_group;
  const int32_t* row_pair;
  int top;
};
template <int BN, int BM, int WN, int WM, int BK, int S, int EPI, typename TO, bool WF, int GR = 0>
__global__ __launch_bounds__(64 * (BN / WN) * (BM / WM)) void gemm_dma_kernel(const bf16_t* __restrict__ x,
                                                       const bf16_t* __restrict__ w, TO* __restrict__ c,
                                                       float* __restrict__ slabs, int m, int n, int k, int m_tiles,
                                                       int n_tiles, int k_tiles, const float* __restrict__ act,
                                                       GemmGroups groups) {
  extern __shared__ __attribute__((aligned(1024))) unsigned char smem[];
  constexpr int TN = WN / 32, TM = WM / 32;
  constexpr int WAVES_N = BN / WN;
  constexpr int NWAVES = (BN / WN) * (BM / WM);
  constexpr int CPR = BK / 8;                   // 16-byte chunks per row
  constexpr int RPW = 64 / CPR;                 // rows one wave-wide load covers
  constexpr int RPB = 128 / BK;                 // rows per 256 bytes of LDS
  constexpr int W_LOADS = BN / RPW / NWAVES, X_LOADS = BM / RPW / NWAVES;
  constexpr int LOADS = W_LOADS + X_LOADS;      // per thread and stage
  constexpr int STAGE = (BN + BM) * BK;         // elements
  static_assert(BN % (RPW * NWAVES) == 0 && BM % (RPW * NWAVES) == 0, "tile does not divide among the waves");
  static_assert(WN % 32 == 0 && WM % 32 == 0 && BN % WN == 0 && BM % WM == 0, "wave tiles are made of 32 x 32 pieces");
  static_assert(S >= 2 && LOADS * (S - 1) < 64, "too many loads in flight for the counter");
  bf16_t* lds = reinterpret_cast<bf16_t*>(smem);

  int mt, nt;
  if (!tile_of_workgroup(m_tiles, n_tiles, &mt, &nt)) return;
  const int m0 = mt * BM;
  const int n0 = nt * BN;
  int group = 0;
  if (GR) {
    group = groups.tile_group[mt];
    if (group < 0) return;
  }

  const int tid = threadIdx.x;
  const int lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int wn0 = (wave % WAVES_N) * WN;
  const int wm0 = (wave / WAVES_N) * WM;
  const int l32 = lane & 31;
  const int g = lane >> 5;

  f32x16_t acc[TN][TM];
#pragma unroll
  for (int i = 0; i < TN; ++i)
#pragma unroll
    for (int j = 0; j < TM; ++j)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[i][j][e] = 0.f;

  // ---- what this lane fetches: wave-wide load q covers rows q * RPW .. + RPW - 1 of a tile
  const bf16_t* wtile = w + (GR ? (size_t)group * n * k : 0) + (size_t)n0 * k;
  const bf16_t* xtile = GR == 1 ? x : x + (size_t)m0 * k;
  uint32_t woff[W_LOADS], xoff[X_LOADS];        // byte offsets from the tile's first element, without the k-tile
#pragma unroll
  for (int i = 0; i < W_LOADS; ++i) {
    if (WF) {
      // W fragment-major: wave-wide load q fetches one block of 16 rows x 32 depth values, 1 KB in
      // a row, and the stage holds the tile's blocks in the order [BN / 16][BK / 32]
      const int q = wave + NWAVES * i;
      int rt = q / (BK / 32);
      const int kb = q % (BK / 32);
      if (n0 + 16 * rt >= n) rt = 0;            // rows beyond N: any valid tile, never stored
      woff[i] = ((uint32_t)(16 * rt) * (uint32_t)k + (uint32_t)kb * 512u + (uint32_t)lane * 8u) * 2u;
    } else {
      const int row = (wave + NWAVES * i) * RPW + lane / CPR;
      const int chunk = (lane % CPR) ^ ((row / RPB) % CPR);
      int grow = row;
      if (n0 + grow > n - 1) grow = n - 1 - n0;   // rows beyond N: any valid row, never stored
      woff[i] = ((uint32_t)grow * (uint32_t)k + chunk * 8) * 2u;
    }
  }
#pragma unroll
  for (int i = 0; i < X_LOADS; ++i) {
    const int row = (wave + NWAVES * i) * RPW + lane / CPR;
    const int chunk = (lane % CPR) ^ ((row / RPB) % CPR);
    int grow = row;
    if (GR == 1) {
      const int pair = groups.row_pair[m0 + row];
      grow = pair >= 0 ? pair / groups.top : 0;
    } else if (m0 + grow > m - 1) {
      grow = m - 1 - m0;
    }
    xoff[i] = ((uint32_t)grow * (uint32_t)k + chunk * 8) * 2u;
  }
  const uint32_t lds_base = (uint32_t)(uintptr_t)lds;      // LDS byte address of stage 0
  const int kt0 = blockIdx.y * k_tiles;                    // this workgroup's slice of K: k_tiles tiles from here
  // a K tile further on: BK values along a row, or BK / 32 blocks of 1 KB (fragment-major)
  constexpr uint32_t W_KSTEP = WF ? BK * 32 : BK * 2;
  // With one tile of tokens every workgroup reads rows of W that nobody else reads, once: whole
  // lines (fragment-major) past the caches, as the products of few tokens do.  Only where a
  // workgroup's walk along K is long: the short walks of a product cut into many K slices are
  // bound by their first loads, which come sooner through the caches (64 tokens: 28,672 gated rows
  // 51 -> 43 us with such loads, but 4,096 rows in 8 slices of 8 tiles 15 -> 16.6 us).
  // The main loop is compiled for either kind of load (as a run-time choice it stood as eight branches
  // between the MFMAs of a K tile and cost 1.6 % of a long prefill).
  const bool w_once = WF && m_tiles == 1 && k_tiles >= 24;
  auto issue = [&](auto once, int kt) {
    const uint32_t stage = lds_base + (uint32_t)(kt % S) * (STAGE * 2);
    const uint32_t kbytes = (uint32_t)(kt0 + kt) * (BK * 2);
#pragma unroll
    for (int i = 0; i < W_LOADS; ++i) {
      if constexpr (decltype(once)::value)
        load_to_lds16_stream(wtile, woff[i] + (uint32_t)(kt0 + kt) * W_KSTEP,
                             stage + (uint32_t)(wave + NWAVES * i) * 1024u);
      else
        load_to_lds16(wtile, woff[i] + (uint32_t)(kt0 + kt) * W_KSTEP, stage + (uint32_t)(wave + NWAVES * i) * 1024u);
    }
#pragma unroll
    for (int i = 0; i < X_LOADS; ++i)
      load_to_lds16(xtile, xoff[i] + kbytes, stage + (uint32_t)(BN * BK * 2) + (uint32_t)(wave + NWAVES * i) * 1024u);
  };

  // ---- fragments: row base + 32 i + l32, chunk 2 ks + g, found in slot chunk ^ swz(l32)
  constexpr int KSTEPS = BK / 16;
  static_assert(KSTEPS % 2 == 0, "the fragment buffers alternate by depth step");
  const int sw = (l32 / RPB) % CPR;
  // W's fragments.  Rows: row wn0 + 32 i + l32, chunk 2 ks + g in slot chunk ^ sw.  Fragment-major:
  // block [(wn0 + 32 i + l32) / 16][chunk / 4], inside it 16 bytes at 16 ((chunk % 4) * 16 + l32 % 16);
  // the 16 lanes that are served together read 256 bytes in a row.
  const bf16_t* wfrag = WF ? lds + ((size_t)((wn0 + l32) / 16) * (BK / 32) * 64 + (l32 % 16)) * 8
                           : lds + (size_t)(wn0 + l32) * BK;
  constexpr int W_ISTEP = WF ? 2 * (BK / 32) * 512 : 32 * BK;       // 32 rows further on
  auto w_slot = [&](int ks) { return WF ? (((2 * ks + g) / 4) * 64 + ((2 * ks + g) % 4) * 16) * 8 : ((2 * ks + g) ^ sw) * 8; };
  const bf16_t* xfrag = lds + (size_t)BN * BK + (size_t)(wm0 + l32) * BK;
  Frag8 a[2][TN], b[2][TM];
  auto load_frags = [&](int buf2, int kt, int ks) {
    const bf16_t* wb = wfrag + (size_t)(kt % S) * STAGE;
    const bf16_t* xb = xfrag + (size_t)(kt % S) * STAGE;
    const int slot = ((2 * ks + g) ^ sw) * 8;
    const int wslot = w_slot(ks);
#pragma unroll
    for (int i = 0; i < TN; ++i) a[buf2][i].u = *reinterpret_cast<const uint4*>(wb + i * W_ISTEP + wslot);
#pragma unroll
    for (int j = 0; j < TM; ++j) b[buf2][j].u = *reinterpret_cast<const uint4*>(xb + 32 * j * BK + slot);
  };
  // the tokens are the MFMA's rows and W's rows its columns: a lane then holds one column of W's
  // rows for 16 tokens, and a wave's store covers 32 consecutive outputs of a token
  auto mfmas = [&](int buf2) {
#pragma unroll
    for (int i = 0; i < TN; ++i)
#pragma unroll
      for (int j = 0; j < TM; ++j) acc[i][j] = mfma32(b[buf2][j], a[buf2][i], acc[i][j]);
  };

  // ---- main loop.  The barrier that hands over tile kt + 1 stands before the last depth step
  // of tile kt, whose fragments are in registers by then: its MFMAs run while the first
  // fragments of tile kt + 1 come from LDS and while the other waves arrive, and the stage of
  // tile kt is free for tile kt + S from there on.
  // One load of tile kt (number l of the LOADS a wave has), one fragment of a depth step.
  auto issue_one = [&](auto once, int kt, int l) {
    const uint32_t stage = lds_base + (uint32_t)(kt % S) * (STAGE * 2);
    const uint32_t kbytes = (uint32_t)(kt0 + kt) * (BK * 2);
    if (l < W_LOADS) {
      if constexpr (decltype(once)::value)
        load_to_lds16_stream(wtile, woff[l] + (uint32_t)(kt0 + kt) * W_KSTEP,
                             stage + (uint32_t)(wave + NWAVES * l) * 1024u);
      else
        load_to_lds16(wtile, woff[l] + (uint32_t)(kt0 + kt) * W_KSTEP, stage + (uint32_t)(wave + NWAVES * l) * 1024u);
    }
    else
      load_to_lds16(xtile, xoff[l - W_LOADS] + kbytes,
                    stage + (uint32_t)(BN * BK * 2) + (uint32_t)(wave + NWAVES * (l - W_LOADS)) * 1024u);
  };
  // Fragment number f of a depth step, in the order in which the MFMAs first need them:
  // W's first, all of the tokens', the rest of W's.
  auto frag_one = [&](int buf2, int kt, int ks, int f) {
    const int slot = ((2 * ks + g) ^ sw) * 8;
    if (f == 0 || f > TM) {
      const int i = f == 0 ? 0 : f - TM;
      a[buf2][i].u = *reinterpret_cast<const uint4*>(wfrag + (size_t)(kt % S) * STAGE + i * W_ISTEP + w_slot(ks));
    } else {
      b[buf2][f - 1].u = *reinterpret_cast<const uint4*>(xfrag + (size_t)(kt % S) * STAGE + 32 * (f - 1) * BK + slot);
    }
  };
  // A depth step but the last of tile kt: its MFMAs, with the next step's fragments asked for
  // between them, one after each MFMA, so that a wave keeps the matrix core fed by itself (with
  // all the reads in a run before the MFMAs, a wave took 27-30 ns per MFMA where the core takes 16-20,
  // and the two waves of a SIMD, which the barrier keeps in step, did not cover each other).
  constexpr int NM = TN * TM, LASTBUF = (KSTEPS - 1) & 1;
  auto steps_but_last = [&](int kt) {
#pragma unroll
    for (int ks = 0; ks + 1 < KSTEPS; ++ks) {
#pragma unroll
      for (int q = 0; q < NM; ++q) {
        acc[q / TM][q % TM] = mfma32(b[ks & 1][q % TM], a[ks & 1][q / TM], acc[q / TM][q % TM]);
#pragma unroll
        for (int f = q; f < TN + TM; f += NM) frag_one((ks + 1) & 1, kt, ks + 1, f);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
  };
  // The last depth step of tile kt, behind the barrier: between its MFMAs, one at a time, go the
  // loads of tile kt + S and the first fragments of tile kt + 1, so that the matrix core never
  // waits for a run of other instructions (both waves of a SIMD leave the barrier together, and
  // neither covers the other's).
  auto last_step = [&](auto once, int kt, bool fetch) {
#pragma unroll
    for (int q = 0; q < NM; ++q) {
      acc[q / TM][q % TM] = mfma32(b[LASTBUF][q % TM], a[LASTBUF][q / TM], acc[q / TM][q % TM]);
      if (fetch) {
#pragma unroll
        for (int l = q; l < LOADS; l += NM) issue_one(once, kt + S, l);
      }
#pragma unroll
      for (int f = q; f < TN + TM; f += NM) frag_one(0, kt + 1, 0, f);
      __builtin_amdgcn_sched_barrier(0);
    }
  };
  auto hand_over = [&](int kt) {
    // tile kt + 1 must have landed; in the steady state the S - 2 tiles after it stay in flight
    if (S == 2 || kt + S - 1 >= k_tiles) wait_vm<0>();
    else wait_vm<LOADS * (S - 2)>();
    // the last fragments of tile kt are in registers before anyone may overwrite its stage
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __syncthreads();                  // everyone's part of tile kt + 1 is in LDS, and nobody reads tile kt's stage any more
    __builtin_amdgcn_sched_barrier(0);
  };
  auto run = [&](auto once) {
#pragma unroll
    for (int s = 0; s < S; ++s)
      if (s < k_tiles) issue(once, s);
    if (S - 1 < k_tiles) wait_vm<LOADS * (S - 1)>();
    else wait_vm<0>();
    __syncthreads();
    load_frags(0, 0, 0);
    int kt = 0;
    for (; kt + S < k_tiles; ++kt) {
      steps_but_last(kt);
      hand_over(kt);
      last_step(once, kt, true);
    }
    for (; kt + 1 < k_tiles; ++kt) {
      steps_but_last(kt);
      hand_over(kt);
      last_step(once, kt, false);
    }
    steps_but_last(k_tiles - 1);
    mfmas(LASTBUF);
  };
  if (w_once) run(std::true_type{});
  else run(std::false_type{});

  // ---- lane holds, per (i, j): W row n0 + wn0 + 32 i + l32, tokens base + 8 (e / 4) + 4 g + e % 4
  if constexpr (EPI == 1 && sizeof(TO) == 2) {
    // The gated outputs of a piece are 16 columns wide: stored from the registers, a wave's store
    // would write 32 bytes of each of four tokens, and the tile's 80 such stores a lane took 27-35 us
    // of a 320 x 256 tile's 150.  They go through LDS instead (the tiles are done with) and leave
    // as whole rows of the tile, 16 bytes a lane.
    constexpr int HC = BN / 2;              // output columns of the tile
    constexpr int LD = HC + 8;              // 16 bytes of padding: the four tokens of a store hit different banks
    constexpr int CH = HC / 8;              // 16-byte chunks of a row
    static_assert((size_t)BM * LD <= (size_t)S * STAGE, "the tile's outputs do not fit the stages");
    const int half_n = n / 2;
    const GatePair gp = gate_pair(act);
    __syncthreads();                        // everyone has read its last fragments
    const bool upper = (l32 & 16) != 0;
#pragma unroll
    for (int i = 0; i < TN; ++i)
#pragma unroll
      for (int j = 0; j < TM; ++j) {
        // gate rows in lanes 0..15 of a half wave, up rows in lanes 16..31: the two halves swap what
        // the other needs, the lower one finishing the even tokens and the upper one the odd ones
        bf16_t* dst = lds + (size_t)(wm0 + 32 * j + 4 * g + (upper ? 1 : 0)) * LD + (wn0 + 32 * i) / 2 + (l32 & 15);
#pragma unroll
        for (int e = 0; e < 16; e += 2) {
          const float mine = upper ? acc[i][j][e + 1] : acc[i][j][e];
          const float give = upper ? acc[i][j][e] : acc[i][j][e + 1];
          const float got = __shfl_xor(give, 16);
          const float gate = upper ? got : mine, up = upper ? mine : got;
          dst[(size_t)(8 * (e / 4) + (e % 4)) * LD] = f32_to_bf16(gated_value(gate, up, gp));
        }
      }
    __syncthreads();
    const bool wide = (reinterpret_cast<uintptr_t>(c) & 15) == 0 && half_n % 8 == 0;
    for (int q = tid; q < BM * CH; q += 64 * NWAVES) {
      const int row = q / CH, ch = q - row * CH;
      const int mm = m0 + row, col = n0 / 2 + ch * 8;
      if (mm >= m || col >= half_n) continue;
      const bf16_t* src = lds + (size_t)row * LD + ch * 8;
      bf16_t* out = reinterpret_cast<bf16_t*>(c) + (size_t)mm * half_n + col;
      if (wide && col + 8 <= half_n) {
        *reinterpret_cast<uint4*>(out) = *reinterpret_cast<const uint4*>(src);
      } else {
        for (int u = 0; u < 8 && col + u < half_n; ++u) out[u] = src[u];
      }
    }
    return;
  }
  float* slab = slabs ? slabs + (size_t)blockIdx.y * m * n : nullptr;      // this slice of K's partial sums
  const bool has_act = EPI == 0 && act != nullptr && slab == nullptr;      // slices leave the activation to the sum of the slabs
  XieluPair xa = {0.f, 0.f};
  if (has_act) xa = xielu_pair(act);
  const GatePair gp = gate_pair(EPI == 1 ? act : nullptr);
#pragma unroll
  for (int i = 0; i < TN; ++i)
#pragma unroll
    for (int j = 0; j < TM; ++j)
      store_piece<EPI, TO>(acc[i][j], c, slab, n0 + wn0 + 32 * i, l32, m0 + wm0 + 32 * j + 4 * g, m, n, has_act, xa.ap, xa.an, gp,
                           GR == 2 ? groups.row_pair : nullptr);
}

