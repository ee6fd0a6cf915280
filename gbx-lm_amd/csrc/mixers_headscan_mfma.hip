// Matrix-core form of the per-head decayed state for bf16 prompt portions (mechanism: mixers_headscan.hip).
//
// A sequence's rows of the step are cut into chunks of 128 (the step's tile table).  With L_t the sum of the logarithms of the decays
// from the chunk's first row to row t, S' the state in front of the chunk and w the write factors,
//
//   o_t = scale ( exp(L_t) S'^T q_t + sum_{s <= t} exp(L_t - L_s) w_s <q_t, k_s> v_s ) + skip v_t
//   S'_next = exp(L_last) S' + sum_s exp(L_last - L_s) w_s k_s v_s^T
//
// 1. chunk_state_kernel   every chunk's own contribution U = sum_s exp(L_last - L_s) w_s v_s k_s^T, all chunks at once;
// 2. chunk_prefix_kernel  the states in front of the chunks, element by element down the chunks of a sequence (in place of the U's), and
//                         the state the sequence leaves in its slot;
// 3. chunk_out_kernel     the read-outs, all chunks at once: a workgroup takes one (chunk, head) and 64 value channels, a wave 32 rows.
//
// q, k and v are bf16 numbers, so products among them are exact in fp32.  What carries more bits -- the states, the decayed scores, the
// weighted values -- enters the bf16 matrix cores as a sum of THREE bf16 numbers (hi + mid + lo hold all 24 bits of an fp32), one
// product each: the results are those of fp32 products up to the order of the sums.  L is summed in fp64 and kept as a pair of floats,
// so differences of large sums keep their bits.
#include <algorithm>
#include "mixers_mfma.h"

namespace gbxm {
namespace {

constexpr int CL = 128;            // rows of a chunk
constexpr int DVS = 64;            // value channels of a workgroup
constexpr int VROW = DVS * 2 + 64; // LDS pitch of a value row: the 4 rows of a transposed block land on disjoint banks

struct ChunkGeo {
  gbxm_head_scan_args a;
  float* ws;                       // [n_tiles][H][dv][dk]: U, then the state in front of the chunk
  float* chunk_decay;              // [n_tiles][H]: exp(L_last)
};

__device__ __forceinline__ void split3(float a, float b, unsigned* p) {
  p[0] = pack2(a, b);
  a -= __uint_as_float(p[0] << 16); b -= __uint_as_float(p[0] & 0xFFFF0000u);
  p[1] = pack2(a, b);
  a -= __uint_as_float(p[1] << 16); b -= __uint_as_float(p[1] & 0xFFFF0000u);
  p[2] = pack2(a, b);
}

// L (as hi + lo) and w of the chunk's rows into LDS; rows past the chunk's end do not decay and write nothing.
struct ChunkDecay {
  float hi[CL], lo[CL], w[CL];
  double first_wave;
};
__device__ __forceinline__ void chunk_decays(const gbxm_head_scan_args& a, int64_t row0, int cn, int h, ChunkDecay& c) {
  const int t = threadIdx.x;
  double l = 0.0;
  if (t < CL) {
    if (a.decay) l = t < cn ? fmax(log(static_cast<double>(a.decay[h])), -1e30) : 0.0;
    else l = t < cn ? static_cast<double>(a.log_decay[(row0 + t) * a.dt_stride + h]) : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double u = __shfl_up(l, o, 64);
      if ((t & 63) >= o) l += u;
    }
    c.w[t] = t < cn ? (a.write ? a.write[(row0 + t) * a.dt_stride + h] : 1.f) : 0.f;
    if (t == 63) c.first_wave = l;
  }
  __syncthreads();
  if (t < CL) {
    if (t >= 64) l += c.first_wave;
    const float hi = static_cast<float>(l);
    c.hi[t] = hi;
    c.lo[t] = static_cast<float>(l - static_cast<double>(hi));
  }
  __syncthreads();
}
// exp(L_t - L_s), s <= t
__device__ __forceinline__ float decay_between(const ChunkDecay& c, int t, int s) { return expf(fminf((c.hi[t] - c.hi[s]) + (c.lo[t] - c.lo[s]), 0.f)); }

// address of the transposed 16-bit block reads (see lds_read_tr): lane -> row 4 (lane / 32) + (lane / 4) % 4, channel 16 ((lane / 16) % 2) + 4 (lane % 4)
__device__ __forceinline__ int tr_offset(int lane, int pitch) { return (4 * (lane >> 5) + ((lane >> 2) & 3)) * pitch + (16 * ((lane >> 4) & 1) + 4 * (lane & 3)) * 2; }
__device__ __forceinline__ u32x4 tr_fragment(const unsigned char* p, int pitch) {
  const u32x2 a = lds_read_tr(p), b = lds_read_tr(p + 8 * pitch);
  return u32x4{a.x, a.y, b.x, b.y};
}

// grid (n_tiles, H * ceil(dv / DVS))
template <int DK>
__global__ __launch_bounds__(256) void chunk_state_kernel(ChunkGeo g) {
  constexpr int KROW = DK * 2 + 64, CT = DK / 32, NTW = 2 * CT / 4;
  __shared__ __attribute__((aligned(16))) unsigned char kl[32 * KROW];
  __shared__ __attribute__((aligned(16))) unsigned char vl[3 * 32 * VROW];
  __shared__ ChunkDecay cd;
  const gbxm_head_scan_args& a = g.a;
  const int slices = (a.dv + DVS - 1) / DVS, h = blockIdx.y / slices, d0 = (blockIdx.y % slices) * DVS;
  const int b = a.tiles[2 * blockIdx.x], t0 = a.tiles[2 * blockIdx.x + 1];
  const int cn = min(CL, a.seq[4 * b + 2] - t0);
  const int64_t row0 = static_cast<int64_t>(a.seq[4 * b + 3]) + t0;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  chunk_decays(a, row0, cn, h, cd);
  if (d0 == 0 && tid == 0) g.chunk_decay[static_cast<int64_t>(blockIdx.x) * a.H + h] = expf(cd.hi[CL - 1] + cd.lo[CL - 1]);
  const bf16_t* rows = static_cast<const bf16_t*>(a.rows) + row0 * a.row_stride;
  const bf16_t* kp = rows + a.off_k + (h / (a.H / a.G)) * a.dk;
  const bf16_t* vp = rows + a.off_v + h * a.dv + d0;
  f32x16 acc[NTW];
#pragma unroll
  for (int i = 0; i < NTW; ++i) acc[i] = f32x16{0};
  const unsigned char* kbase = kl + tr_offset(lane, KROW);
  const unsigned char* vbase = vl + tr_offset(lane, VROW);
  for (int s0 = 0; s0 < cn; s0 += 32) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < DK / 64; ++i) {                     // 32 rows x DK / 8 pieces
      const int p = tid + 256 * i, row = p / (DK / 8), c = (p % (DK / 8)) * 8;
      u32x4 v = u32x4{0, 0, 0, 0};
      if (s0 + row < cn && c < a.dk) v = *reinterpret_cast<const u32x4*>(kp + static_cast<int64_t>(s0 + row) * a.row_stride + c);
      *reinterpret_cast<u32x4*>(kl + row * KROW + c * 2) = v;
    }
    {                                                       // 32 rows x 8 pieces of 8 channels
      const int row = tid >> 3, c = (tid & 7) * 8;
      u32x4 v = u32x4{0, 0, 0, 0};
      float f = 0.f;
      if (s0 + row < cn && d0 + c < a.dv) {
        v = *reinterpret_cast<const u32x4*>(vp + static_cast<int64_t>(s0 + row) * a.row_stride + c);
        f = decay_between(cd, CL - 1, s0 + row) * cd.w[s0 + row];
      }
      u32x4 out[3];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        unsigned q[3];
        split3(__uint_as_float(v[j] << 16) * f, __uint_as_float(v[j] & 0xFFFF0000u) * f, q);
#pragma unroll
        for (int k = 0; k < 3; ++k) out[k][j] = q[k];
      }
#pragma unroll
      for (int k = 0; k < 3; ++k) *reinterpret_cast<u32x4*>(vl + (k * 32 + row) * VROW + c * 2) = out[k];
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      const int id = wave + 4 * i, ct = id % CT, dt = id / CT;
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) {
        const u32x4 kf = tr_fragment(kbase + 16 * tt * KROW + ct * 64, KROW);
#pragma unroll
        for (int k = 0; k < 3; ++k) acc[i] = mfma_bf16(tr_fragment(vbase + (k * 32 + 16 * tt) * VROW + dt * 64, VROW), kf, acc[i]);
      }
    }
  }
  float* u = g.ws + ((static_cast<int64_t>(blockIdx.x) * a.H + h) * a.dv) * a.dk;
  const int r = lane & 31, hb = lane >> 5;
#pragma unroll
  for (int i = 0; i < NTW; ++i) {
    const int id = wave + 4 * i, c = (id % CT) * 32 + r;
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int d = d0 + (id / CT) * 32 + 8 * (e >> 2) + 4 * hb + (e & 3);
      if (c < a.dk && d < a.dv) u[static_cast<int64_t>(d) * a.dk + c] = acc[i][e];
    }
  }
}

// grid (ceil(dv dk / 1024), H, B): a thread owns four neighbouring elements of one head's state and walks the sequence's chunks.
__global__ __launch_bounds__(256) void chunk_prefix_kernel(ChunkGeo g) {
  constexpr int AHEAD = 8;
  const gbxm_head_scan_args& a = g.a;
  const int b = blockIdx.z, h = blockIdx.y;
  const int64_t size = static_cast<int64_t>(a.dv) * a.dk, e = (static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x) * 4;
  if (e >= size) return;
  int first = 0;
  for (int i = 0; i < b; ++i) first += (a.seq[4 * i + 2] + CL - 1) / CL;
  const int slot = a.seq[4 * b], pos0 = a.seq[4 * b + 1], chunks = (a.seq[4 * b + 2] + CL - 1) / CL;
  float4* st = reinterpret_cast<float4*>(a.state + (static_cast<int64_t>(slot) * a.H + h) * size + e);
  float4 s = *st;
  if (pos0 == 0) s = float4{0.f, 0.f, 0.f, 0.f};
  const int64_t step = a.H * size;
  float* p = g.ws + (static_cast<int64_t>(first) * a.H + h) * size + e;
  const float* dp = g.chunk_decay + static_cast<int64_t>(first) * a.H + h;
  for (int c0 = 0; c0 < chunks; c0 += AHEAD) {
    float4 u[AHEAD];
    float d[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const int c = min(c0 + i, chunks - 1);
      u[i] = *reinterpret_cast<const float4*>(p + c * step);
      d[i] = dp[static_cast<int64_t>(c) * a.H];
    }
#pragma unroll
    for (int i = 0; i < AHEAD; ++i)
      if (c0 + i < chunks) {
        *reinterpret_cast<float4*>(p + (c0 + i) * step) = s;
        s.x = s.x * d[i] + u[i].x; s.y = s.y * d[i] + u[i].y; s.z = s.z * d[i] + u[i].z; s.w = s.w * d[i] + u[i].w;
      }
  }
  *st = s;
}

// grid (n_tiles, H * ceil(dv / DVS)).  Products are computed swapped (O^T = V^T P^T), a lane owns one row of the chunk.
template <int DK>
__global__ __launch_bounds__(256) void chunk_out_kernel(ChunkGeo g) {
  constexpr int KROW = DK * 2 + 16, KS = DK / 16;
  constexpr int STATE_BYTES = 3 * 32 * KROW, TILE_BYTES = 32 * KROW + 32 * VROW;
  __shared__ __attribute__((aligned(16))) unsigned char lds[STATE_BYTES > TILE_BYTES ? STATE_BYTES : TILE_BYTES];
  __shared__ ChunkDecay cd;
  unsigned char* vl = lds + 32 * KROW;
  const gbxm_head_scan_args& a = g.a;
  const int slices = (a.dv + DVS - 1) / DVS, h = blockIdx.y / slices, d0 = (blockIdx.y % slices) * DVS;
  const int b = a.tiles[2 * blockIdx.x], t0 = a.tiles[2 * blockIdx.x + 1];
  const int cn = min(CL, a.seq[4 * b + 2] - t0);
  const int64_t row0 = static_cast<int64_t>(a.seq[4 * b + 3]) + t0;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 31, hb = lane >> 5;
  const int ql = wave * 32 + r;
  const bf16_t* rows = static_cast<const bf16_t*>(a.rows) + row0 * a.row_stride;
  const int kv = (h / (a.H / a.G)) * a.dk;
  u32x4 qf[KS];
  {
    const bf16_t* qp = rows + static_cast<int64_t>(min(ql, cn - 1)) * a.row_stride + a.off_q + kv;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int c = ks * 16 + hb * 8;
      qf[ks] = c < a.dk ? *reinterpret_cast<const u32x4*>(qp + c) : u32x4{0, 0, 0, 0};
    }
  }
  chunk_decays(a, row0, cn, h, cd);
  f32x16 o[2] = {f32x16{0}, f32x16{0}};
  if (a.seq[4 * b + 1] + t0 > 0) {                            // (workgroup-uniform) a state in front of the chunk
    const float* s = g.ws + ((static_cast<int64_t>(blockIdx.x) * a.H + h) * a.dv + d0) * a.dk;
#pragma unroll
    for (int dt = 0; dt < 2; ++dt) {
      if (d0 + dt * 32 >= a.dv) break;                        // (uniform)
      __syncthreads();
#pragma unroll
      for (int i = 0; i < DK / 64; ++i) {
        const int p = tid + 256 * i, row = p / (DK / 8), c = (p % (DK / 8)) * 8;
        float4 x0 = float4{0.f, 0.f, 0.f, 0.f}, x1 = x0;
        if (d0 + dt * 32 + row < a.dv && c < a.dk) {
          const float4* sp = reinterpret_cast<const float4*>(s + static_cast<int64_t>(dt * 32 + row) * a.dk + c);
          x0 = sp[0];
          x1 = sp[1];
        }
        const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
        u32x4 out[3];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          unsigned q[3];
          split3(x[2 * j], x[2 * j + 1], q);
#pragma unroll
          for (int k = 0; k < 3; ++k) out[k][j] = q[k];
        }
#pragma unroll
        for (int k = 0; k < 3; ++k) *reinterpret_cast<u32x4*>(lds + (k * 32 + row) * KROW + c * 2) = out[k];
      }
      __syncthreads();
#pragma unroll
      for (int ks = 0; ks < KS; ++ks)
#pragma unroll
        for (int k = 0; k < 3; ++k) o[dt] = mfma_bf16(*reinterpret_cast<const u32x4*>(lds + (k * 32 + r) * KROW + hb * 16 + ks * 32), qf[ks], o[dt]);
    }
    const float et = expf(fminf(cd.hi[ql] + cd.lo[ql], 0.f)) * a.scale;
#pragma unroll
    for (int dt = 0; dt < 2; ++dt)
#pragma unroll
      for (int e = 0; e < 16; ++e) o[dt][e] *= et;
  }
  const float skip = a.skip ? a.skip[h] : 0.f;
  const unsigned char* kbase = lds + r * KROW + hb * 16;
  const unsigned char* vbase = vl + tr_offset(lane, VROW);
  for (int kt = 0; kt * 32 < cn; ++kt) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < DK / 64; ++i) {
      const int p = tid + 256 * i, row = p / (DK / 8), c = (p % (DK / 8)) * 8, s = kt * 32 + row;
      u32x4 v = u32x4{0, 0, 0, 0};
      if (s < cn && c < a.dk) v = *reinterpret_cast<const u32x4*>(rows + static_cast<int64_t>(s) * a.row_stride + a.off_k + kv + c);
      *reinterpret_cast<u32x4*>(lds + row * KROW + c * 2) = v;
    }
    {
      const int row = tid >> 3, c = (tid & 7) * 8, s = kt * 32 + row;
      u32x4 v = u32x4{0, 0, 0, 0};
      if (s < cn && d0 + c < a.dv) v = *reinterpret_cast<const u32x4*>(rows + static_cast<int64_t>(s) * a.row_stride + a.off_v + h * a.dv + d0 + c);
      *reinterpret_cast<u32x4*>(vl + row * VROW + c * 2) = v;
    }
    __syncthreads();
    if (kt > wave) continue;                                  // (wave-uniform) no row of this wave sees these
    f32x16 st = f32x16{0};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) st = mfma_bf16(*reinterpret_cast<const u32x4*>(kbase + ks * 32), qf[ks], st);
    float p[16];
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int s = kt * 32 + 8 * (e >> 2) + 4 * hb + (e & 3);
      p[e] = s <= ql ? st[e] * (decay_between(cd, ql, s) * cd.w[s] * a.scale) : 0.f;
      if (s == ql) p[e] += skip;
    }
    u32x4 pf[3][2];
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        unsigned q[3];
        split3(p[8 * tt + 2 * j], p[8 * tt + 2 * j + 1], q);
#pragma unroll
        for (int k = 0; k < 3; ++k) pf[k][tt][j] = q[k];
      }
#pragma unroll
    for (int dt = 0; dt < 2; ++dt)
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) {
        const u32x4 vf = tr_fragment(vbase + 16 * tt * VROW + dt * 64, VROW);
#pragma unroll
        for (int k = 0; k < 3; ++k) o[dt] = mfma_bf16(vf, pf[k][tt], o[dt]);
      }
  }
  if (ql >= cn) return;
  float* op = a.out + (row0 + ql) * (static_cast<int64_t>(a.H) * a.dv) + h * a.dv + d0;
#pragma unroll
  for (int dt = 0; dt < 2; ++dt)
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      const int d = dt * 32 + 8 * q4 + 4 * hb;
      if (d0 + d < a.dv) *reinterpret_cast<float4*>(op + d) = float4{o[dt][4 * q4], o[dt][4 * q4 + 1], o[dt][4 * q4 + 2], o[dt][4 * q4 + 3]};
    }
}

template <int DK>
int launch_chunks(const ChunkGeo& g, hipStream_t s) {
  const gbxm_head_scan_args& a = g.a;
  const dim3 grid(a.n_tiles, a.H * ((a.dv + DVS - 1) / DVS));
  chunk_state_kernel<DK><<<grid, 256, 0, s>>>(g);
  chunk_prefix_kernel<<<dim3((static_cast<int64_t>(a.dv) * a.dk + 1023) / 1024, a.H, a.B), 256, 0, s>>>(g);
  chunk_out_kernel<DK><<<grid, 256, 0, s>>>(g);
  return after_launch("head_scan (chunks)");
}

bool aligned16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

}  // namespace

size_t head_chunks_workspace(int64_t n_tiles, int H, int dk, int dv) {
  return static_cast<size_t>(n_tiles) * H * (static_cast<size_t>(dk) * dv + 4) * sizeof(float);
}

// true: launch_head_chunks takes this step (bf16, chunk table and workspace given, sizes and addresses on the 16-byte grid)
bool head_chunks_shape(const gbxm_head_scan_args& a) {
  return a.act == GBXM_BF16 && a.tiles && a.n_tiles > 0 && a.q_tile == CL && a.ws && a.ws_bytes >= head_chunks_workspace(a.n_tiles, a.H, a.dk, a.dv) &&
         a.dk % 8 == 0 && a.dv % 8 == 0 && a.dk <= 256 && (a.row_stride | a.off_q | a.off_k | a.off_v) % 8 == 0 && aligned16(a.rows) && aligned16(a.state) &&
         aligned16(a.out) && aligned16(a.ws) && static_cast<int64_t>(a.H) * ((a.dv + DVS - 1) / DVS) <= 65535;
}

int launch_head_chunks(const gbxm_head_scan_args& a, hipStream_t s) {
  float* ws = static_cast<float*>(a.ws);
  const ChunkGeo g{a, ws, ws + static_cast<size_t>(a.n_tiles) * a.H * a.dk * a.dv};
  if (a.dk <= 64) return launch_chunks<64>(g, s);
  if (a.dk <= 128) return launch_chunks<128>(g, s);
  return launch_chunks<256>(g, s);
}

}  // namespace gbxm
