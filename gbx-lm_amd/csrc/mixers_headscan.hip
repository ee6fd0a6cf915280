// Recurrent mixers whose state decays by ONE number per head and token (linear attention with a fixed decay, state space duality):
//
//   S <- d S + w k v^T,   o = scale * S^T q + skip v      (d = decay[h], or exp(log_decay[t][h]); w = write[t][h] or 1; skip[h] or 0)
//
//   ssm_prepare_kernel      short causal convolution + bias + silu over the channels x | B | C (result in the activation dtype), and per
//                           head  w = softplus(dt + dt_bias),  log d = -rate w  (fp32).  In steps where every sequence brings one row it
//                           also moves the convolution's tail on (each thread owns its channels); else conv_tail_kernel does.
//   head_step_kernel<R>     steps of few rows per sequence: a wave takes four state columns (value channels), 16 lanes per column, a lane
//                           holds R x 4 neighbouring key channels; operands straight from the rows.  Bound by the state's traffic.
//   head_scan_kernel<R>     longer portions: the same arithmetic with the operands of a chunk of tokens in LDS, shared by 16 columns, the
//                           next chunk fetched while the current one is computed.
//                           (bf16 prompt portions on the 16-byte grid: chunk kernels on the matrix cores, mixers_headscan_mfma.hip)
//   gate_group_norm_kernel  v = o * silu(z), each of the equal parts of a row scaled by its own root mean square, times a weight.
//
// q, k, v are read from rows of the activation dtype (a projection's rows, or the prepared ones); decays, write factors, the state and
// every sum are fp32.  Sums run in a fixed order: a sequence's result does not depend on what else is in the step.
#include <algorithm>
#include <type_traits>
#include "mixers_common.h"

namespace gbxm {
namespace {

constexpr int NT = 256;

// ------------------------------------------------------------------------------------------------ preparation of state space rows
// grid (rows, splits of the channels).  V channels per thread and pass (4: 8/16-byte accesses; 1: any layout).
template <typename T, bool FAST, int V>
__global__ __launch_bounds__(NT) void ssm_prepare_kernel(gbxm_ssm_prepare_args p) {
  const int64_t t = blockIdx.x;
  const int b = p.tok[2 * t], pos = p.tok[2 * t + 1];
  const int slot = p.seq[4 * b], pos0 = p.seq[4 * b + 1], row0 = p.seq[4 * b + 3];
  const int keep = p.taps - 1, C = p.C;
  const T* y = static_cast<const T*>(p.y);
  const T* x = y + p.off_x;
  const T* cw = static_cast<const T*>(p.conv);                        // [taps][C]
  T* tl = keep ? static_cast<T*>(p.tail) + static_cast<int64_t>(slot) * keep * C : nullptr;
  T* out = static_cast<T*>(p.out) + t * C;
  const int gthread = blockIdx.y * NT + threadIdx.x, n_threads = gridDim.y * NT;
  for (int c = gthread * V; c < C; c += n_threads * V) {
    float acc[V];
#pragma unroll
    for (int i = 0; i < V; ++i) acc[i] = p.bias ? p.bias[c + i] : 0.f;
    for (int j = 0; j < p.taps; ++j) {
      const int src = pos - keep + j;
      if (src < 0) continue;                                          // zeros before the sequence
      float v[V], w[V];
      Lanes<T, V>::load(src >= pos0 ? x + (row0 + (src - pos0)) * p.y_stride + c : tl + static_cast<int64_t>(src - pos0 + keep) * C + c, v);
      Lanes<T, V>::load(cw + static_cast<int64_t>(j) * C + c, w);
#pragma unroll
      for (int i = 0; i < V; ++i) acc[i] += w[i] * v[i];
    }
#pragma unroll
    for (int i = 0; i < V; ++i) acc[i] *= sigmoid_<FAST>(acc[i]);
    Lanes<T, V>::store(out + c, acc);
    if (p.move_tail && keep) {                                        // one row per sequence: nobody else reads these channels of the slot
      float v[V];
      for (int i = 0; i + 1 < keep; ++i) {
        const bool own = pos - keep + 1 + i >= 0;
        Lanes<T, V>::load(tl + static_cast<int64_t>(i + 1) * C + c, v);
#pragma unroll
        for (int k = 0; k < V; ++k) v[k] = own ? v[k] : 0.f;
        Lanes<T, V>::store(tl + static_cast<int64_t>(i) * C + c, v);
      }
      Lanes<T, V>::load(x + t * p.y_stride + c, v);
      Lanes<T, V>::store(tl + static_cast<int64_t>(keep - 1) * C + c, v);
    }
  }
  float* dr = p.dt_out + t * 2 * p.H;
  for (int h = gthread; h < p.H; h += n_threads) {
    const float z = to_f32(y[t * p.y_stride + p.off_dt + h]) + p.dt_bias[h];
    const float w = z > 20.f ? z : log1pf(expf(z));
    dr[h] = -p.rate[h] * w;
    dr[p.H + h] = w;
  }
}

// Sum over the 16 lanes of a row; every lane of the row gets the same bits.
__device__ __forceinline__ float row16_sum(float v) {
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xf, 0xf, false));    // quad_perm [1,0,3,2]
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xf, 0xf, false));    // quad_perm [2,3,0,1]
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x141, 0xf, 0xf, false));   // row_half_mirror
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x140, 0xf, 0xf, false));   // row_mirror
  return v;
}

// ------------------------------------------------------------------------------------------------ few rows per sequence
// grid (ceil(dv / (4 NW)), H, B).  Lane ks of a 16-lane row owns the key channels 64 i + 4 ks + (0..3), i < R.
template <typename T, int R, int NW, bool VEC>
__global__ __launch_bounds__(64 * NW) void head_step_kernel(gbxm_head_scan_args p) {
  const int b = blockIdx.z, h = blockIdx.y;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, ks = lane & 15;
  const int col = blockIdx.x * 4 * NW + wave * 4 + (lane >> 4);
  const int slot = p.seq[4 * b], pos0 = p.seq[4 * b + 1], n = p.seq[4 * b + 2], row0 = p.seq[4 * b + 3];
  const int dk = p.dk, dv = p.dv;
  const bool col_ok = col < dv;
  const int colc = col_ok ? col : dv - 1;
  const int g = h / (p.H / p.G);
  float* sp = p.state + ((static_cast<int64_t>(slot) * p.H + h) * dv + colc) * dk;
  const T* rows = static_cast<const T*>(p.rows) + static_cast<int64_t>(row0) * p.row_stride;
  const T* qp = rows + p.off_q + g * dk;
  const T* kp = rows + p.off_k + g * dk;
  const T* vp = rows + p.off_v + h * dv + colc;
  auto fetch = [&](const auto* base, float* v, int i) {                // 4 channels from 64 i + 4 ks on (zeros past the last channel)
    const int c = 64 * i + 4 * ks;
    using E = std::remove_cv_t<std::remove_pointer_t<decltype(base)>>;
    if constexpr (VEC) {
      Lanes<E, 4>::load(base + (c < dk ? c : 0), v);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = c < dk ? v[j] : 0.f;
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) { const float u = to_f32(base[c + j < dk ? c + j : 0]); v[j] = c + j < dk ? u : 0.f; }
    }
  };
  float S[4 * R];
#pragma unroll
  for (int i = 0; i < R; ++i) fetch(static_cast<const float*>(sp), S + 4 * i, i);
#pragma unroll
  for (int i = 0; i < 4 * R; ++i) S[i] = pos0 > 0 ? S[i] : 0.f;
  const float skip = p.skip ? p.skip[h] : 0.f;
  float* op = p.out + (static_cast<int64_t>(row0) * p.H + h) * dv + colc;
  for (int t = 0; t < n; ++t) {
    float q[4 * R], k[4 * R];
#pragma unroll
    for (int i = 0; i < R; ++i) { fetch(qp, q + 4 * i, i); fetch(kp, k + 4 * i, i); }
    const float v = to_f32(*vp);
    const float d = p.decay ? p.decay[h] : expf(p.log_decay[(row0 + t) * p.dt_stride + h]);
    const float u = p.write ? v * p.write[(row0 + t) * p.dt_stride + h] : v;
    float o = 0.f;
#pragma unroll
    for (int i = 0; i < 4 * R; ++i) { S[i] = S[i] * d + k[i] * u; o += q[i] * S[i]; }
    o = row16_sum(o);
    if (ks == 0 && col_ok) op[static_cast<int64_t>(t) * p.H * dv] = o * p.scale + skip * v;
    qp += p.row_stride; kp += p.row_stride; vp += p.row_stride;
  }
  if (col_ok) {
#pragma unroll
    for (int i = 0; i < R; ++i) {
      const int c = 64 * i + 4 * ks;
      if constexpr (VEC) {
        if (c < dk) Lanes<float, 4>::store(sp + c, S + 4 * i);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c + j < dk) sp[c + j] = S[4 * i + j];
      }
    }
  }
}

// ------------------------------------------------------------------------------------------------ portions
// grid (ceil(dv / 16), H, B), 4 waves.  LDS row of a token: q | k (padded to 64 R channels, zeros past dk) | 16 value columns; decays
// and write factors beside them.  Two buffers: a chunk is fetched into registers before the current one is computed.
template <typename T, int R>
__global__ __launch_bounds__(NT) void head_scan_kernel(gbxm_head_scan_args p) {
  constexpr int DKP = 64 * R, NCOL = 16, ROW = 2 * DKP + NCOL, CH = R <= 1 ? 32 : (R <= 2 ? 16 : (R <= 4 ? 8 : 4));
  constexpr int PF = (CH * ROW + NT - 1) / NT;
  __shared__ __attribute__((aligned(16))) float buf[2][CH * ROW];
  __shared__ float dl[2][CH], wl[2][CH];
  const int b = blockIdx.z, h = blockIdx.y;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, ks = lane & 15;
  const int col0 = blockIdx.x * NCOL, lcol = wave * 4 + (lane >> 4), col = col0 + lcol;
  const int slot = p.seq[4 * b], pos0 = p.seq[4 * b + 1], n = p.seq[4 * b + 2], row0 = p.seq[4 * b + 3];
  const int dk = p.dk, dv = p.dv;
  const bool col_ok = col < dv;
  const int colc = col_ok ? col : dv - 1;
  const int g = h / (p.H / p.G);
  float* sp = p.state + ((static_cast<int64_t>(slot) * p.H + h) * dv + colc) * dk;
  float S[4 * R];
#pragma unroll
  for (int i = 0; i < 4 * R; ++i) {
    const int c = 64 * (i >> 2) + 4 * ks + (i & 3);
    const float s = sp[c < dk ? c : 0];
    S[i] = (pos0 > 0 && c < dk) ? s : 0.f;
  }
  const T* base = static_cast<const T*>(p.rows) + static_cast<int64_t>(row0) * p.row_stride;
  const float* gbase = p.log_decay ? p.log_decay + static_cast<int64_t>(row0) * p.dt_stride + h : nullptr;
  const float* wbase = p.write ? p.write + static_cast<int64_t>(row0) * p.dt_stride + h : nullptr;
  const float d_const = p.decay ? p.decay[h] : 1.f;
  T pf[PF];
  float pd = 0.f, pw = 1.f;
  int offs[PF];
  unsigned loaded = 0;
  static_assert(PF <= 32, "one bit per operand");
#pragma unroll
  for (int i = 0; i < PF; ++i) {
    const int idx = min(static_cast<int>(threadIdx.x) + i * NT, CH * ROW - 1), j = idx % ROW;
    const int seg = j < DKP ? 0 : (j < 2 * DKP ? 1 : 2), jj = j - seg * DKP;
    const bool valid = seg < 2 ? jj < dk : jj < min(dv - col0, NCOL);
    offs[i] = valid ? (seg == 0 ? p.off_q + g * dk + jj : (seg == 1 ? p.off_k + g * dk + jj : p.off_v + h * dv + col0 + jj)) : p.off_q;
    loaded |= static_cast<unsigned>(valid) << i;
  }
  auto fetch = [&](int t0) {                        // rows past the sequence's end are read as its last row (and never used)
    const int last = n - 1 - t0;
    const T* cb = base + static_cast<int64_t>(t0) * p.row_stride;
#pragma unroll
    for (int i = 0; i < PF; ++i) {
      const int tt = min(static_cast<int>(threadIdx.x) + i * NT, CH * ROW - 1) / ROW;
      pf[i] = cb[static_cast<int64_t>(min(tt, last)) * p.row_stride + offs[i]];
    }
    const int64_t row = t0 + min(static_cast<int>(threadIdx.x) % CH, last);
    if (gbase) pd = gbase[row * p.dt_stride];
    if (wbase) pw = wbase[row * p.dt_stride];
  };
  auto park = [&](int w) {
#pragma unroll
    for (int i = 0; i < PF; ++i) {
      const int idx = threadIdx.x + i * NT;
      if (idx < CH * ROW) buf[w][idx] = ((loaded >> i) & 1u) ? to_f32(pf[i]) : 0.f;
    }
    if (threadIdx.x < CH) { dl[w][threadIdx.x] = gbase ? expf(pd) : d_const; wl[w][threadIdx.x] = pw; }
  };
  fetch(0);
  park(0);
  __syncthreads();
  const float skip = p.skip ? p.skip[h] : 0.f;
  float* op = p.out + (static_cast<int64_t>(row0) * p.H + h) * dv + colc;
  int which = 0;
  for (int t0 = 0; t0 < n; t0 += CH, which ^= 1) {
    const bool more = t0 + CH < n;
    if (more) fetch(t0 + CH);
    const float* cur = buf[which];
    const int cn = min(CH, n - t0);
#pragma unroll 2
    for (int tt = 0; tt < cn; ++tt) {
      const float* row = cur + tt * ROW;
      const float v = row[2 * DKP + lcol], d = dl[which][tt], u = v * wl[which][tt];
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < R; ++i) {
        const float4 q = *reinterpret_cast<const float4*>(row + 64 * i + 4 * ks);
        const float4 k = *reinterpret_cast<const float4*>(row + DKP + 64 * i + 4 * ks);
        S[4 * i] = S[4 * i] * d + k.x * u; S[4 * i + 1] = S[4 * i + 1] * d + k.y * u;
        S[4 * i + 2] = S[4 * i + 2] * d + k.z * u; S[4 * i + 3] = S[4 * i + 3] * d + k.w * u;
        o += q.x * S[4 * i]; o += q.y * S[4 * i + 1]; o += q.z * S[4 * i + 2]; o += q.w * S[4 * i + 3];
      }
      o = row16_sum(o);
      if (ks == 0 && col_ok) op[static_cast<int64_t>(t0 + tt) * p.H * dv] = o * p.scale + skip * v;
    }
    if (more) park(which ^ 1);
    __syncthreads();
  }
  if (col_ok) {
#pragma unroll
    for (int i = 0; i < 4 * R; ++i) {
      const int c = 64 * (i >> 2) + 4 * ks + (i & 3);
      if (c < dk) sp[c] = S[i];
    }
  }
}

template <typename T, int NW>
int launch_step(const gbxm_head_scan_args& a, bool vec, hipStream_t s) {
  const dim3 grid((a.dv + 4 * NW - 1) / (4 * NW), a.H, a.B);
  const int R = (a.dk + 63) / 64;
#define GBXM_STEP(N)                                                          \
  do {                                                                        \
    if (vec) head_step_kernel<T, N, NW, true><<<grid, 64 * NW, 0, s>>>(a);    \
    else head_step_kernel<T, N, NW, false><<<grid, 64 * NW, 0, s>>>(a);       \
  } while (0)
  if (R <= 1) GBXM_STEP(1);
  else if (R <= 2) GBXM_STEP(2);
  else if (R <= 4) GBXM_STEP(4);
  else GBXM_STEP(8);
#undef GBXM_STEP
  return after_launch("head_scan (few rows)");
}

template <typename T>
int launch_scan(const gbxm_head_scan_args& a, hipStream_t s) {
  const dim3 grid((a.dv + 15) / 16, a.H, a.B);
  const int R = (a.dk + 63) / 64;
  if (R <= 1) head_scan_kernel<T, 1><<<grid, NT, 0, s>>>(a);
  else if (R <= 2) head_scan_kernel<T, 2><<<grid, NT, 0, s>>>(a);
  else if (R <= 4) head_scan_kernel<T, 4><<<grid, NT, 0, s>>>(a);
  else head_scan_kernel<T, 8><<<grid, NT, 0, s>>>(a);
  return after_launch("head_scan");
}

// ------------------------------------------------------------------------------------------------ gate, then norm in equal parts
constexpr int GR = 16;                 // values a thread keeps between the statistic and its use

template <typename T, bool FAST, int NTH>
__global__ __launch_bounds__(NTH) void gate_group_norm_kernel(const float* __restrict__ o, const T* __restrict__ z, int64_t z_stride,
                                                             const float* __restrict__ w, T* __restrict__ out, int64_t out_stride, int groups, int size,
                                                             float eps) {
  __shared__ float red[NTH / 64];
  const int64_t t = blockIdx.x;
  const int first = blockIdx.y * size;
  const float* x = o + t * groups * size + first;
  const T* zr = z + t * z_stride + first;
  auto value = [&](int c) { const float g = to_f32(zr[c]); return x[c] * (g * sigmoid_<FAST>(g)); };
  float v[GR];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < GR; ++i) {
    const int c = threadIdx.x + i * NTH;
    v[i] = c < size ? value(c) : 0.f;
    ss += v[i] * v[i];
  }
  for (int c = threadIdx.x + GR * NTH; c < size; c += NTH) { const float u = value(c); ss += u * u; }
  ss = block_sum<NTH / 64>(ss, red);
  const float r = 1.f / sqrtf(ss / size + eps);
  T* y = out + t * out_stride + first;
#pragma unroll
  for (int i = 0; i < GR; ++i) {
    const int c = threadIdx.x + i * NTH;
    if (c < size) y[c] = from_f32<T>(v[i] * r * w[first + c]);
  }
  for (int c = threadIdx.x + GR * NTH; c < size; c += NTH) y[c] = from_f32<T>(value(c) * r * w[first + c]);
}

template <typename T, bool FAST>
int launch_gate_norm(const float* o, const void* z, int64_t zs, const float* w, void* out, int64_t os, int64_t T_, int groups, int size, float eps, hipStream_t s) {
  const dim3 grid(T_, groups);
  const T* zp = static_cast<const T*>(z);
  T* op = static_cast<T*>(out);
  if (size <= 256) gate_group_norm_kernel<T, FAST, 64><<<grid, 64, 0, s>>>(o, zp, zs, w, op, os, groups, size, eps);
  else if (size <= 1024) gate_group_norm_kernel<T, FAST, 128><<<grid, 128, 0, s>>>(o, zp, zs, w, op, os, groups, size, eps);
  else gate_group_norm_kernel<T, FAST, 256><<<grid, 256, 0, s>>>(o, zp, zs, w, op, os, groups, size, eps);
  return after_launch("gate_group_norm");
}

bool act_ok(int act) { return act == GBXM_BF16 || act == GBXM_F32; }
bool aligned(const void* p, size_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; }

}  // namespace

bool head_chunks_shape(const gbxm_head_scan_args& a);                       // mixers_headscan_mfma.hip
int launch_head_chunks(const gbxm_head_scan_args& a, hipStream_t s);
size_t head_chunks_workspace(int64_t n_tiles, int H, int dk, int dv);

}  // namespace gbxm

using namespace gbxm;

extern "C" {

int gbxm_ssm_prepare(const gbxm_ssm_prepare_args* a, void* stream) {
  if (!a || !act_ok(a->act) || !a->y || !a->conv || !a->dt_bias || !a->rate || !a->seq || !a->tok || !a->out || !a->dt_out || a->T < 0 || a->C < 1 ||
      a->H < 1 || a->taps < 1 || (a->taps > 1 && !a->tail) || a->off_x < 0 || a->off_dt < 0 || a->off_x + static_cast<int64_t>(a->C) > a->y_stride ||
      a->off_dt + static_cast<int64_t>(a->H) > a->y_stride)
    return fail(GBXM_ERR_INVALID, "ssm_prepare: bad argument");
  if (a->T == 0) return GBXM_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const size_t vb = a->act == GBXM_BF16 ? 8 : 16;
  const bool vec = a->C % 4 == 0 && a->off_x % 4 == 0 && a->y_stride % 4 == 0 && aligned(a->y, vb) && aligned(a->conv, vb) && aligned(a->out, vb) &&
                   (a->taps == 1 || aligned(a->tail, vb));
  const int64_t work = (a->C / (vec ? 4 : 1) + NT - 1) / NT;              // workgroups a row can feed
  const unsigned splits = static_cast<unsigned>(std::max<int64_t>(1, std::min<int64_t>(work, (2048 + a->T - 1) / a->T)));
  const dim3 grid(a->T, splits);
  if (a->act == GBXM_BF16) {
    if (vec) ssm_prepare_kernel<bf16_t, true, 4><<<grid, NT, 0, s>>>(*a);
    else ssm_prepare_kernel<bf16_t, true, 1><<<grid, NT, 0, s>>>(*a);
  } else {
    if (vec) ssm_prepare_kernel<float, false, 4><<<grid, NT, 0, s>>>(*a);
    else ssm_prepare_kernel<float, false, 1><<<grid, NT, 0, s>>>(*a);
  }
  return after_launch("ssm_prepare");
}

size_t gbxm_head_scan_workspace(int64_t T_, int32_t B, int64_t n_tiles, int32_t q_tile, int32_t H, int32_t dk, int32_t dv, int32_t act) {
  if (act != GBXM_BF16 || q_tile != 128 || n_tiles < 1 || T_ < 32 * static_cast<int64_t>(B) || dk % 8 || dv % 8 || dk > 256) return 0;
  return head_chunks_workspace(n_tiles, H, dk, dv);
}

int gbxm_head_scan(const gbxm_head_scan_args* a, void* stream) {
  if (!a || !act_ok(a->act) || !a->rows || !a->state || !a->out || !a->seq || a->B < 0 || a->T < 0 || a->H < 1 || a->G < 1 || a->H % a->G || a->dk < 1 ||
      a->dv < 1 || (!a->decay && !a->log_decay) || ((a->log_decay || a->write) && a->dt_stride < a->H) || a->off_q < 0 || a->off_k < 0 || a->off_v < 0 ||
      a->off_q + static_cast<int64_t>(a->G) * a->dk > a->row_stride || a->off_k + static_cast<int64_t>(a->G) * a->dk > a->row_stride ||
      a->off_v + static_cast<int64_t>(a->H) * a->dv > a->row_stride)
    return fail(GBXM_ERR_INVALID, "head_scan: bad argument");
  if (a->dk > 512) return fail(GBXM_ERR_UNSUPPORTED, "head_scan: %d key channels per head (at most 512)", a->dk);
  if (a->B == 0 || a->T == 0) return GBXM_OK;
  if (a->B > 65535 || a->H > 65535) return fail(GBXM_ERR_UNSUPPORTED, "head_scan: grid");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const bool bf = a->act == GBXM_BF16;
  if (head_chunks_shape(*a)) return launch_head_chunks(*a, s);
  if (a->T >= 8 * static_cast<int64_t>(a->B)) return bf ? launch_scan<bf16_t>(*a, s) : launch_scan<float>(*a, s);
  const size_t vb = bf ? 8 : 16;
  const bool vec = a->dk % 4 == 0 && a->row_stride % 4 == 0 && a->off_q % 4 == 0 && a->off_k % 4 == 0 && aligned(a->rows, vb) && aligned(a->state, 16);
  if (static_cast<int64_t>((a->dv + 15) / 16) * a->H * a->B >= 512) return bf ? launch_step<bf16_t, 4>(*a, vec, s) : launch_step<float, 4>(*a, vec, s);
  return bf ? launch_step<bf16_t, 1>(*a, vec, s) : launch_step<float, 1>(*a, vec, s);
}

int gbxm_gate_group_norm(const float* o, const void* z, int64_t z_stride, const float* w, void* out, int64_t out_stride, int64_t T_, int32_t groups,
                         int32_t size, float eps, int32_t act, void* stream) {
  if (!act_ok(act) || !o || !z || !w || !out || T_ < 0 || groups < 1 || groups > 65535 || size < 1 || z_stride < static_cast<int64_t>(groups) * size ||
      out_stride < static_cast<int64_t>(groups) * size)
    return fail(GBXM_ERR_INVALID, "gate_group_norm: bad argument");
  if (T_ == 0) return GBXM_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  return act == GBXM_BF16 ? launch_gate_norm<bf16_t, true>(o, z, z_stride, w, out, out_stride, T_, groups, size, eps, s)
                          : launch_gate_norm<float, false>(o, z, z_stride, w, out, out_stride, T_, groups, size, eps, s);
}

}  // extern "C"
