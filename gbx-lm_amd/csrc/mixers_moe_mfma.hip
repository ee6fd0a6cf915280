// Grouped matrix-core products of routed experts for bf16 prompt portions (mechanism: mixers_moe.hip).
//
// 1. expert_sort_kernel: the step's (row, choice) pairs counted and bucketed by expert on the device (one workgroup, LDS counters):
//    offsets[E + 1], the pair ids in expert order, and the table of row tiles (expert, first pair) the two products walk.  Nothing
//    returns to the host.
// 2. expert_up_kernel:   act[p] = silu(gate_e h) * (up_e h) for the pairs of expert e, 128 pairs x 128 hidden channels per workgroup (256
//    where experts have no gate: the second weight fragment is then another block of 32 channels);
// 3. expert_down_kernel: y[pair] = down_e act[p], 128 pairs x 256 output channels per workgroup.
// Products are computed swapped -- C^T[channel, pair] = mfma(weight rows, activation rows) -- so a lane ends up with four consecutive
// channels of one pair (8-byte stores) and the gate / up pair of a channel sits in the same lane for the activation.
// Weight fragments are 16-byte loads straight from the row-major matrices (every wave has rows of its own); the activation tile,
// which all four waves share, goes global -> registers (one chunk ahead) -> LDS once per workgroup: counters showed the version
// in which every wave fetched it for itself waiting on L2 -> L1 traffic for more than half of its cycles.
// The contraction runs in chunks of 64 elements (a 32-element tail when the size is not a multiple of 64); inside a chunk the lane
// half hb takes the contiguous half [hb * C/2, (hb + 1) * C/2) and feeds it to the chunk's MFMA steps 8 elements at a time -- the
// order of the contraction is free as long as both operands use the same one -- so a lane reads 64 contiguous bytes per chunk.
// The grid is sized for the worst case sum_e ceil(n_e / 128) <= P / 128 + E; surplus workgroups leave at once.
// Steps with few pairs per expert (a batch that decodes) stream weights and little else: expert_skinny_kernel takes tiles of 32 pairs, a
// wave per 32 output channels and no barrier.  A wave moves its own rows -- eight lanes to a row's 128 bytes, so an access touches eight
// cache lines instead of the 64 that loads in fragment order would -- through registers (two chunks in flight) into LDS of its own.
#include <type_traits>
#include "mixers_mfma.h"

namespace gbxm {
namespace {

constexpr int RT = 128;         // pairs per workgroup tile
constexpr int RS = 32;          // and per tile of the skinny form
constexpr int BROW = 128 + 16;  // LDS bytes per activation row of a chunk (+16: conflict-free 16-byte fragment reads)

__global__ __launch_bounds__(1024) void expert_sort_kernel(const int* __restrict__ idx, int* __restrict__ offsets, int* __restrict__ sorted,
                                                          int* __restrict__ tile_tab, int n_tiles, int rt, int P, int E) {
  extern __shared__ int sm[];                 // counts [E] | cursor [E] | first tile [E]
  int* counts = sm;
  int* cursor = sm + E;
  int* first = sm + 2 * E;
  for (int e = threadIdx.x; e < E; e += 1024) counts[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < P; i += 1024) atomicAdd(&counts[idx[i]], 1);
  __syncthreads();
  if (threadIdx.x < 64) {                      // one wave: running sums of pairs and tiles, 64 experts at a time
    int run = 0, tiles = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + threadIdx.x, c = e < E ? counts[e] : 0, t = (c + rt - 1) / rt;
      int sc = c, st = t;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int uc = __shfl_up(sc, o, 64), ut = __shfl_up(st, o, 64);
        if (static_cast<int>(threadIdx.x) >= o) { sc += uc; st += ut; }
      }
      if (e < E) {
        cursor[e] = run + sc - c;
        offsets[e] = run + sc - c;
        first[e] = tiles + st - t;
      }
      run += __shfl(sc, 63, 64);
      tiles += __shfl(st, 63, 64);
    }
    if (threadIdx.x == 0) {
      offsets[E] = run;
      sm[3 * E] = tiles;
    }
  }
  __syncthreads();
  for (int i = threadIdx.x; i < P; i += 1024) sorted[atomicAdd(&cursor[idx[i]], 1)] = i;
  __syncthreads();                             // every cursor now stands at its expert's end
  for (int e = threadIdx.x; e < E; e += 1024) {
    const int nt = (counts[e] + rt - 1) / rt, lo = cursor[e] - counts[e];
    for (int t = 0; t < nt; ++t) { tile_tab[2 * (first[e] + t)] = e; tile_tab[2 * (first[e] + t) + 1] = lo + t * rt; }
  }
  for (int t = sm[3 * E] + threadIdx.x; t < n_tiles; t += 1024) tile_tab[2 * t] = -1;
}

// Workgroup ids go round-robin over the 8 XCDs, each with an L2 of its own: row tile = (id % 8) * (gridDim.x / 8) + id / 8 gives every
// XCD a contiguous run of row tiles, so the row tiles of ONE expert, which read the same weights, run on one XCD next to each other.
// (gridDim.x is a multiple of 8.)
__device__ __forceinline__ int xcd_row_tile() { return (blockIdx.x % 8) * (gridDim.x / 8) + blockIdx.x / 8; }

// Activation tile of a chunk: 128 rows x C elements.  Thread t moves the 16-byte pieces t + 256 i (i < 4): row = piece / 8, column piece
// = piece % 8 (only the first C / 8 column pieces exist in a 32-element tail).
struct BTile {
  const bf16_t* rowp[4];      // this thread's four rows (already offset by its column piece)
  int lds_off[4];
  int cpiece;
  u32x4 regs[4];
  __device__ __forceinline__ void fetch(int k0, int pieces) {
#pragma unroll
    for (int i = 0; i < 4; ++i) regs[i] = cpiece < pieces ? *reinterpret_cast<const u32x4*>(rowp[i] + k0) : u32x4{0, 0, 0, 0};
  }
  __device__ __forceinline__ void park(unsigned char* bl) const {
#pragma unroll
    for (int i = 0; i < 4; ++i) *reinterpret_cast<u32x4*>(bl + lds_off[i]) = regs[i];
  }
};

template <bool GATED>
__global__ __launch_bounds__(256) void expert_up_kernel(const bf16_t* __restrict__ h, const bf16_t* __restrict__ first, const int* __restrict__ offsets,
                                                       const int* __restrict__ sorted, const int* __restrict__ tile_tab, const float* __restrict__ scale,
                                                       bf16_t* __restrict__ act, int K, int F, int top, int kind, float limit) {
  __shared__ __attribute__((aligned(16))) unsigned char bl[RT * BROW];
  const int bt = xcd_row_tile();
  const int e = tile_tab[2 * bt];
  if (e < 0) return;                                                  // (workgroup-uniform)
  const int lo = tile_tab[2 * bt + 1], hi = offsets[e + 1];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 31, hb = lane >> 5;
  const int f0 = GATED ? blockIdx.y * 128 + wave * 32 : blockIdx.y * 256 + wave * 64;
  const bool live = f0 < F;                                           // a wave past the last channel still moves its share of the tile
  const bool second = GATED || f0 + 32 < F;                           // (F is a multiple of 32)
  const bf16_t* wgl = first + (static_cast<int64_t>(e) * (GATED ? 2 : 1) * F + (live ? f0 + r : 0)) * K;
  const bf16_t* wul = GATED ? wgl + static_cast<int64_t>(F) * K : (second ? wgl + static_cast<int64_t>(32) * K : wgl);
  BTile b;
  b.cpiece = tid & 7;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = (tid >> 3) + 32 * i;
    b.rowp[i] = h + static_cast<int64_t>(sorted[min(lo + row, hi - 1)] / top) * K + b.cpiece * 8;
    b.lds_off[i] = row * BROW + b.cpiece * 16;
  }
  f32x16 ag[4], au[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) { ag[j] = f32x16{0}; au[j] = f32x16{0}; }

  auto chunk = [&](int k0, auto steps_c) {
    constexpr int S = decltype(steps_c)::value;                         // MFMA steps of the chunk: 4 (64 elements) or 2 (32)
    const int off = k0 + hb * (S * 8);
    u32x4 fg[S], fu[S];                                                 // weight fragments: requested ahead of the tile hand-over
#pragma unroll
    for (int i = 0; i < S; ++i) {
      fg[i] = *reinterpret_cast<const u32x4*>(wgl + off + i * 8);
      fu[i] = *reinterpret_cast<const u32x4*>(wul + off + i * 8);
    }
    __syncthreads();                                                    // the previous chunk's fragments have been read
    b.park(bl);
    __syncthreads();
    const int kn = k0 + S * 16;
    if (kn < K) b.fetch(kn, kn + 64 <= K ? 8 : 4);                      // the next chunk travels while this one is multiplied
    if (!live) return;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      u32x4 fb[S];
#pragma unroll
      for (int i = 0; i < S; ++i) fb[i] = *reinterpret_cast<const u32x4*>(bl + (j * 32 + r) * BROW + hb * (S * 16) + i * 16);
#pragma unroll
      for (int i = 0; i < S; ++i) {
        ag[j] = mfma_bf16(fg[i], fb[i], ag[j]);
        au[j] = mfma_bf16(fu[i], fb[i], au[j]);
      }
    }
  };
  b.fetch(0, K >= 64 ? 8 : 4);
  int k0 = 0;
  for (; k0 + 64 <= K; k0 += 64) chunk(k0, std::integral_constant<int, 4>{});
  if (k0 < K) chunk(k0, std::integral_constant<int, 2>{});
  if (!live) return;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int row = lo + j * 32 + r;
    if (row >= hi) continue;
    const float sc = scale ? scale[sorted[row]] : 1.f;
    bf16_t* ap = act + static_cast<int64_t>(row) * F + f0 + 4 * hb;
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      float v[4];
      if constexpr (GATED) {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = glu_act<true>(sc * ag[j][4 * q4 + i], sc * au[j][4 * q4 + i], kind, limit, 1.702f);
        *reinterpret_cast<u32x2*>(ap + 8 * q4) = u32x2{pack2(v[0], v[1]), pack2(v[2], v[3])};
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) { const float z = fmaxf(sc * ag[j][4 * q4 + i], 0.f); v[i] = z * z; }
        *reinterpret_cast<u32x2*>(ap + 8 * q4) = u32x2{pack2(v[0], v[1]), pack2(v[2], v[3])};
        if (second) {
#pragma unroll
          for (int i = 0; i < 4; ++i) { const float z = fmaxf(sc * au[j][4 * q4 + i], 0.f); v[i] = z * z; }
          *reinterpret_cast<u32x2*>(ap + 32 + 8 * q4) = u32x2{pack2(v[0], v[1]), pack2(v[2], v[3])};
        }
      }
    }
  }
}

__global__ __launch_bounds__(256) void expert_down_kernel(const bf16_t* __restrict__ act, const bf16_t* __restrict__ down, const int* __restrict__ offsets,
                                                         const int* __restrict__ sorted, const int* __restrict__ tile_tab, bf16_t* __restrict__ y,
                                                         int K, int F) {
  __shared__ __attribute__((aligned(16))) unsigned char bl[RT * BROW];
  const int bt = xcd_row_tile();
  const int e = tile_tab[2 * bt];
  if (e < 0) return;
  const int lo = tile_tab[2 * bt + 1], hi = offsets[e + 1];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 31, hb = lane >> 5;
  const int c0 = blockIdx.y * 256 + wave * 64;
  const bool live = c0 < K;
  const bool second = c0 + 32 < K;                                    // K is a multiple of 32: the wave's second channel block may not exist
  const bf16_t* wl[2];
  wl[0] = down + (static_cast<int64_t>(e) * K + (live ? c0 + r : 0)) * F;
  wl[1] = second ? wl[0] + static_cast<int64_t>(32) * F : wl[0];
  BTile b;
  b.cpiece = tid & 7;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = (tid >> 3) + 32 * i;
    b.rowp[i] = act + static_cast<int64_t>(min(lo + row, hi - 1)) * F + b.cpiece * 8;
    b.lds_off[i] = row * BROW + b.cpiece * 16;
  }
  f32x16 acc[2][4];
#pragma unroll
  for (int c = 0; c < 2; ++c)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[c][j] = f32x16{0};

  auto chunk = [&](int f0_, auto steps_c) {
    constexpr int S = decltype(steps_c)::value;
    const int off = f0_ + hb * (S * 8);
    u32x4 fa[2][S];
#pragma unroll
    for (int i = 0; i < S; ++i) {
      fa[0][i] = *reinterpret_cast<const u32x4*>(wl[0] + off + i * 8);
      fa[1][i] = *reinterpret_cast<const u32x4*>(wl[1] + off + i * 8);
    }
    __syncthreads();
    b.park(bl);
    __syncthreads();
    const int fn = f0_ + S * 16;
    if (fn < F) b.fetch(fn, fn + 64 <= F ? 8 : 4);
    if (!live) return;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      u32x4 fb[S];
#pragma unroll
      for (int i = 0; i < S; ++i) fb[i] = *reinterpret_cast<const u32x4*>(bl + (j * 32 + r) * BROW + hb * (S * 16) + i * 16);
#pragma unroll
      for (int i = 0; i < S; ++i) {
        acc[0][j] = mfma_bf16(fa[0][i], fb[i], acc[0][j]);
        acc[1][j] = mfma_bf16(fa[1][i], fb[i], acc[1][j]);
      }
    }
  };
  b.fetch(0, F >= 64 ? 8 : 4);
  int fc = 0;
  for (; fc + 64 <= F; fc += 64) chunk(fc, std::integral_constant<int, 4>{});
  if (fc < F) chunk(fc, std::integral_constant<int, 2>{});
  if (!live) return;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int row = lo + j * 32 + r;
    if (row >= hi) continue;
    bf16_t* yp = y + static_cast<int64_t>(sorted[row]) * K + c0 + 4 * hb;
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      if (c == 1 && !second) continue;
#pragma unroll
      for (int q4 = 0; q4 < 4; ++q4)
        *reinterpret_cast<u32x2*>(yp + c * 32 + 8 * q4) =
            u32x2{pack2(acc[c][j][4 * q4], acc[c][j][4 * q4 + 1]), pack2(acc[c][j][4 * q4 + 2], acc[c][j][4 * q4 + 3])};
    }
  }
}

// FORM 0: out[pair] = w_e in[position in expert order] (the down product); 1: out[position] = relu(scale w_e in[row])^2; 2: gate rows over up
// rows and their gated activation.  N output channels, C contraction; both multiples of 32.
enum { SKINNY_DOWN = 0, SKINNY_UP = 1, SKINNY_GATED = 2 };

template <int FORM>
__global__ __launch_bounds__(256) void expert_skinny_kernel(const bf16_t* __restrict__ in, const bf16_t* __restrict__ w, const int* __restrict__ offsets,
                                                           const int* __restrict__ sorted, const int* __restrict__ tile_tab, const float* __restrict__ scale,
                                                           bf16_t* __restrict__ out, int N, int C, int top, int kind, float limit) {
  constexpr bool TWO = FORM == SKINNY_GATED;
  const int bt = xcd_row_tile();
  const int e = tile_tab[2 * bt];
  if (e < 0) return;
  const int lo = tile_tab[2 * bt + 1], hi = offsets[e + 1];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 31, hb = lane >> 5;
  const int c0 = blockIdx.y * 128 + wave * 32;
  if (c0 >= N) return;
  const int row = min(lo + r, hi - 1), pair = sorted[row];
  constexpr int PARTS = TWO ? 3 : 2;                                     // weights (twice), activations
  __shared__ __attribute__((aligned(16))) unsigned char lds[4][PARTS][RS * BROW];
  unsigned char* mine = lds[wave][0];
  // this lane's pieces of a chunk: rows lane / 8 + 8 i, 16 bytes at column piece lane % 8 (a 32-element tail has four column pieces)
  const int mrow = lane >> 3, col = lane & 7;
  const bf16_t* wp = w + (static_cast<int64_t>(e) * (TWO ? 2 : 1) * N + c0 + mrow) * C + col * 8;
  const int64_t up = static_cast<int64_t>(N) * C;
  const bf16_t* xp[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int p = min(lo + mrow + 8 * i, hi - 1);
    xp[i] = in + static_cast<int64_t>(FORM == SKINNY_DOWN ? p : sorted[p] / top) * C + col * 8;
  }
  f32x16 acc = f32x16{0}, acc2 = f32x16{0};
  struct Pieces { u32x4 v[PARTS][4]; };
  auto load = [&](Pieces& f, int k0, int cols) {
    const int k = col < cols ? k0 : k0 - 32;                            // (a piece past the tail repeats one inside it; nobody reads it)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f.v[0][i] = *reinterpret_cast<const u32x4*>(wp + static_cast<int64_t>(8 * i) * C + k);
      if constexpr (TWO) f.v[1][i] = *reinterpret_cast<const u32x4*>(wp + up + static_cast<int64_t>(8 * i) * C + k);
      f.v[PARTS - 1][i] = *reinterpret_cast<const u32x4*>(xp[i] + k);
    }
  };
  auto mul = [&](const Pieces& f, auto steps_c) {
    constexpr int S = decltype(steps_c)::value;
    __builtin_amdgcn_wave_barrier();                                    // (a wave's LDS accesses run in program order: its own writes and reads need
#pragma unroll                                                          //  no barrier among waves, only the compiler must keep the order)
    for (int q = 0; q < PARTS; ++q)
#pragma unroll
      for (int i = 0; i < 4; ++i) *reinterpret_cast<u32x4*>(mine + q * (RS * BROW) + (mrow + 8 * i) * BROW + col * 16) = f.v[q][i];
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < S; ++i) {
      const unsigned char* p = mine + r * BROW + (hb * S + i) * 16;
      const u32x4 x = *reinterpret_cast<const u32x4*>(p + (PARTS - 1) * (RS * BROW));
      acc = mfma_bf16(*reinterpret_cast<const u32x4*>(p), x, acc);
      if constexpr (TWO) acc2 = mfma_bf16(*reinterpret_cast<const u32x4*>(p + RS * BROW), x, acc2);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  };
  const std::integral_constant<int, 4> whole;
  const std::integral_constant<int, 2> half;
  const int full = C / 64;
  if (full) {
    Pieces f0, f1;
    load(f0, 0, 8);
    for (int i = 0; i < full; i += 2) {                                 // (the loads past the end repeat the last chunk)
      load(f1, min(i + 1, full - 1) * 64, 8);
      mul(f0, whole);
      load(f0, min(i + 2, full - 1) * 64, 8);
      if (i + 1 < full) mul(f1, whole);
    }
  }
  if (C % 64) {
    Pieces f;
    load(f, full * 64, 4);
    mul(f, half);
  }
  if (lo + r >= hi) return;
  const float sc = FORM != SKINNY_DOWN && scale ? scale[pair] : 1.f;
  bf16_t* op = out + static_cast<int64_t>(FORM == SKINNY_DOWN ? pair : row) * N + c0 + 4 * hb;
#pragma unroll
  for (int q4 = 0; q4 < 4; ++q4) {
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float z = acc[4 * q4 + i];
      if constexpr (FORM == SKINNY_DOWN) v[i] = z;
      else if constexpr (FORM == SKINNY_UP) { const float p = fmaxf(sc * z, 0.f); v[i] = p * p; }
      else v[i] = glu_act<true>(sc * z, sc * acc2[4 * q4 + i], kind, limit, 1.702f);
    }
    *reinterpret_cast<u32x2*>(op + 8 * q4) = u32x2{pack2(v[0], v[1]), pack2(v[2], v[3])};
  }
}

size_t align16(size_t n) { return (n + 15) & ~static_cast<size_t>(15); }
constexpr int64_t MIN_PAIRS = 64;         // below this the weight-streaming row kernels read less
constexpr int64_t SKINNY_PAIRS = 64;      // pairs per expert (on average) up to which the skinny form is taken
int rows_of(int64_t P, int E) { return P <= SKINNY_PAIRS * E ? RS : RT; }
int tiles_of(int64_t P, int E) { return static_cast<int>((P / rows_of(P, E) + E + 7) / 8 * 8); }

}  // namespace

size_t expert_grouped_workspace(int64_t T, int K, int F, int E, int top) {
  const int64_t P = T * top;
  if (P < MIN_PAIRS || K % 32 || F % 32 || E > 4096 || P > 0x3fffffff) return 0;
  return align16(sizeof(int) * (E + 1)) + align16(sizeof(int) * P) + align16(sizeof(int) * 2 * tiles_of(P, E)) + align16(sizeof(bf16_t) * P * F);
}

int launch_expert_grouped(const gbxm_expert_args& a, hipStream_t s) {
  const int K = a.K, F = a.F, E = a.E, top = a.top;
  const size_t need = expert_grouped_workspace(a.T, K, F, E, top);
  if (need == 0) return GBXM_ERR_UNSUPPORTED;
  if (a.ws_bytes < need) return fail(GBXM_ERR_INVALID, "expert_ff: workspace of %zu bytes, %zu needed", a.ws_bytes, need);
  if ((reinterpret_cast<uintptr_t>(a.h) | reinterpret_cast<uintptr_t>(a.first) | reinterpret_cast<uintptr_t>(a.down) | reinterpret_cast<uintptr_t>(a.y) |
       reinterpret_cast<uintptr_t>(a.ws)) % 16)
    return GBXM_ERR_UNSUPPORTED;
  const int P = static_cast<int>(a.T * top);
  const int tiles = tiles_of(P, E);
  unsigned char* w = static_cast<unsigned char*>(a.ws);
  int* offsets = reinterpret_cast<int*>(w);
  w += align16(sizeof(int) * (E + 1));
  int* sorted = reinterpret_cast<int*>(w);
  w += align16(sizeof(int) * P);
  int* tile_tab = reinterpret_cast<int*>(w);
  w += align16(sizeof(int) * 2 * tiles);
  bf16_t* act = reinterpret_cast<bf16_t*>(w);
  expert_sort_kernel<<<1, 1024, (3 * E + 1) * sizeof(int), s>>>(a.idx, offsets, sorted, tile_tab, tiles, rows_of(P, E), P, E);
  const bf16_t* h = static_cast<const bf16_t*>(a.h);
  const bf16_t* first = static_cast<const bf16_t*>(a.first);
  if (rows_of(P, E) == RS) {
    const dim3 up(tiles, (F + 127) / 128), dn(tiles, (K + 127) / 128);
    if (a.kind == GBXM_EXPERT_RELU2)
      expert_skinny_kernel<SKINNY_UP><<<up, 256, 0, s>>>(h, first, offsets, sorted, tile_tab, a.scale, act, F, K, top, a.kind, a.limit);
    else
      expert_skinny_kernel<SKINNY_GATED><<<up, 256, 0, s>>>(h, first, offsets, sorted, tile_tab, a.scale, act, F, K, top, a.kind, a.limit);
    expert_skinny_kernel<SKINNY_DOWN><<<dn, 256, 0, s>>>(act, static_cast<const bf16_t*>(a.down), offsets, sorted, tile_tab, nullptr,
                                                         static_cast<bf16_t*>(a.y), K, F, top, a.kind, a.limit);
    return after_launch("expert_ff (skinny groups)");
  }
  if (a.kind == GBXM_EXPERT_RELU2)
    expert_up_kernel<false><<<dim3(tiles, (F + 255) / 256), 256, 0, s>>>(h, first, offsets, sorted, tile_tab, a.scale, act, K, F, top, a.kind, a.limit);
  else
    expert_up_kernel<true><<<dim3(tiles, (F + 127) / 128), 256, 0, s>>>(h, first, offsets, sorted, tile_tab, a.scale, act, K, F, top, a.kind, a.limit);
  expert_down_kernel<<<dim3(tiles, (K + 255) / 256), 256, 0, s>>>(act, static_cast<const bf16_t*>(a.down), offsets, sorted, tile_tab,
                                                                   static_cast<bf16_t*>(a.y), K, F);
  return after_launch("expert_ff (grouped)");
}

}  // namespace gbxm
