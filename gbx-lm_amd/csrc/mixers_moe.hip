// Routed MLPs over dense stacked experts:  y[t][s] = down_e (silu(gate_e h_t) * (up_e h_t)),  e = idx[t][s] -- or another gated
// activation, or experts without a gate, down_e relu(up_e h_t)^2.  With a factor per (row, choice) an expert reads the scaled row: the
// factor meets the fp32 sums of its first products.
//
//   * row kernels -- weight-bandwidth bound: the kernels of decode steps, of fp32 models and of shapes the grouped kernel does not
//     take.  Two launches so that even ONE row spreads over the chip: expert_up_rows (a workgroup = one (row, choice) pair x 8 hidden
//     channels, a wave per channel pair gate / up, lanes across the contraction with 16-byte loads, fp32 sums in a fixed order)
//     leaves the hidden row in the workspace, expert_down_rows (a pair x 16 output channels) consumes it.
//   * grouped matrix-core products for bf16 prompt portions (rows sorted by expert on the device, no host round trip).
#include "mixers_common.h"

namespace gbxm {
namespace {

constexpr int NT = 256, NW = NT / 64;
constexpr int FC = 8;             // hidden channels per workgroup of expert_up_rows
constexpr int KC = 16;            // output channels per workgroup of expert_down_rows

// sum_k w[k] * x[k] over this lane's share of n elements; x in LDS (fp32).  VEC: n is a multiple of the 16-byte vector.
template <typename T, bool VEC>
__device__ __forceinline__ float lane_dot(const T* __restrict__ w, const float* __restrict__ x, int n, int lane) {
  float acc = 0.f;
  if constexpr (VEC) {
    constexpr int PER = 16 / sizeof(T);
    for (int k = lane * PER; k < n; k += 64 * PER) {
      const uint4 raw = *reinterpret_cast<const uint4*>(w + k);
      if constexpr (sizeof(T) == 2) {
        const unsigned u[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          acc += __uint_as_float(u[i] << 16) * x[k + 2 * i];
          acc += __uint_as_float(u[i] & 0xFFFF0000u) * x[k + 2 * i + 1];
        }
      } else {
        acc += __uint_as_float(raw.x) * x[k] + __uint_as_float(raw.y) * x[k + 1] + __uint_as_float(raw.z) * x[k + 2] + __uint_as_float(raw.w) * x[k + 3];
      }
    }
  } else {
    for (int k = lane; k < n; k += 64) acc += to_f32(w[k]) * x[k];
  }
  return acc;
}

// GATED: first = gate rows over up rows, a wave takes one hidden channel at a time; else first = up rows, a wave takes its two channels of
// the workgroup's FC = 2 NW together.
template <typename T, bool FAST, bool VEC, bool GATED>
__global__ __launch_bounds__(NT) void expert_up_rows(const T* __restrict__ h, const T* __restrict__ first, const int* __restrict__ idx,
                                                    const float* __restrict__ scale, T* __restrict__ act, int K, int F, int top, int kind, float limit) {
  static_assert(FC == 2 * NW, "two hidden channels per wave");
  extern __shared__ float hl[];                     // the row [K]
  const int64_t pair = blockIdx.x;
  const int e = idx[pair];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const T* hr = h + (pair / top) * K;
  for (int k = threadIdx.x; k < K; k += NT) hl[k] = to_f32(hr[k]);
  __syncthreads();
  const T* wg = first + static_cast<int64_t>(e) * (GATED ? 2 : 1) * F * K;
  const float sc = scale ? scale[pair] : 1.f;
  if constexpr (!GATED) {
    const int fa = blockIdx.y * FC + wave, fb = fa + NW;
    if (fa >= F) return;
    float a = lane_dot<T, VEC>(wg + static_cast<int64_t>(fa) * K, hl, K, lane);
    float b = lane_dot<T, VEC>(wg + static_cast<int64_t>(min(fb, F - 1)) * K, hl, K, lane);
    a = fmaxf(sc * wave_sum(a), 0.f);
    b = fmaxf(sc * wave_sum(b), 0.f);
    if (lane == 0) {
      act[pair * F + fa] = from_f32<T>(a * a);
      if (fb < F) act[pair * F + fb] = from_f32<T>(b * b);
    }
    return;
  }
  const T* wu = wg + static_cast<int64_t>(F) * K;
  const int f_end = min(F, (static_cast<int>(blockIdx.y) + 1) * FC);
  for (int f = blockIdx.y * FC + wave; f < f_end; f += NW) {
    const float ag = sc * wave_sum(lane_dot<T, VEC>(wg + static_cast<int64_t>(f) * K, hl, K, lane));
    const float au = sc * wave_sum(lane_dot<T, VEC>(wu + static_cast<int64_t>(f) * K, hl, K, lane));
    if (lane == 0) act[pair * F + f] = from_f32<T>(glu_act<FAST>(ag, au, kind, limit, 1.702f));
  }
}

template <typename T, bool VEC>
__global__ __launch_bounds__(NT) void expert_down_rows(const T* __restrict__ act, const T* __restrict__ down, const int* __restrict__ idx,
                                                      T* __restrict__ y, int K, int F) {
  extern __shared__ float al[];                     // the hidden row [F]
  const int64_t pair = blockIdx.x;
  const int e = idx[pair];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  for (int f = threadIdx.x; f < F; f += NT) al[f] = to_f32(act[pair * F + f]);
  __syncthreads();
  const T* wd = down + static_cast<int64_t>(e) * K * F;
  const int c_end = min(K, (static_cast<int>(blockIdx.y) + 1) * KC);
  for (int c = blockIdx.y * KC + wave; c < c_end; c += NW) {
    const float acc = wave_sum(lane_dot<T, VEC>(wd + static_cast<int64_t>(c) * F, al, F, lane));
    if (lane == 0) y[pair * K + c] = from_f32<T>(acc);
  }
}

template <typename T, bool FAST, bool VEC, bool GATED>
int launch_rows(const gbxm_expert_args& a, hipStream_t s) {
  const int64_t P = a.T * a.top;
  const dim3 gu(P, (a.F + FC - 1) / FC), gd(P, (a.K + KC - 1) / KC);
  T* act = static_cast<T*>(a.ws);
  expert_up_rows<T, FAST, VEC, GATED><<<gu, NT, a.K * sizeof(float), s>>>(static_cast<const T*>(a.h), static_cast<const T*>(a.first), a.idx, a.scale, act, a.K,
                                                                         a.F, a.top, a.kind, a.limit);
  expert_down_rows<T, VEC><<<gd, NT, a.F * sizeof(float), s>>>(act, static_cast<const T*>(a.down), a.idx, static_cast<T*>(a.y), a.K, a.F);
  return after_launch("expert_ff (rows)");
}

template <typename T, bool FAST>
int launch_rows(const gbxm_expert_args& a, hipStream_t s) {
  constexpr int PER = 16 / sizeof(T);
  const bool vec = a.K % PER == 0 && a.F % PER == 0 && (reinterpret_cast<uintptr_t>(a.first) | reinterpret_cast<uintptr_t>(a.down)) % 16 == 0;
  if (a.kind == GBXM_EXPERT_RELU2) return vec ? launch_rows<T, FAST, true, false>(a, s) : launch_rows<T, FAST, false, false>(a, s);
  return vec ? launch_rows<T, FAST, true, true>(a, s) : launch_rows<T, FAST, false, true>(a, s);
}

}  // namespace

int launch_expert_grouped(const gbxm_expert_args& a, hipStream_t s);   // mixers_moe_mfma.hip
size_t expert_grouped_workspace(int64_t T, int K, int F, int E, int top);

}  // namespace gbxm

using namespace gbxm;

extern "C" size_t gbxm_expert_glu_workspace(int64_t T_, int32_t K, int32_t F, int32_t E, int32_t top, int32_t act) {
  const size_t rows = static_cast<size_t>(T_) * top * F * (act == GBXM_BF16 ? 2 : 4);      // the hidden rows of the row kernels
  const size_t grouped = act == GBXM_BF16 ? expert_grouped_workspace(T_, K, F, E, top) : 0;
  return grouped > rows ? grouped : rows;
}

extern "C" int gbxm_expert_glu_grouped(int64_t T_, int32_t K, int32_t F, int32_t E, int32_t top, int32_t act) {
  return act == GBXM_BF16 && expert_grouped_workspace(T_, K, F, E, top) > 0;
}

extern "C" int gbxm_expert_ff(const gbxm_expert_args* a, void* stream) {
  if (!a || !a->h || !a->first || !a->down || !a->idx || !a->y || a->K <= 0 || a->F <= 0 || a->E <= 0 || a->top < 1 || a->top > a->E || a->T < 0 ||
      (a->act != GBXM_BF16 && a->act != GBXM_F32) || (a->kind != GBXM_GLU_SILU && a->kind != GBXM_GLU_CLAMPED_SWISH && a->kind != GBXM_EXPERT_RELU2))
    return fail(GBXM_ERR_INVALID, "expert_ff: bad argument");
  if (a->T == 0) return GBXM_OK;
  if (!a->ws || a->ws_bytes < gbxm_expert_glu_workspace(a->T, a->K, a->F, a->E, a->top, a->act)) return fail(GBXM_ERR_INVALID, "expert_ff: workspace too small");
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (a->act == GBXM_BF16) {
    const int rc = launch_expert_grouped(*a, s);
    if (rc != GBXM_ERR_UNSUPPORTED) return rc;
  }
  const int longest = a->K > a->F ? a->K : a->F;
  if (static_cast<size_t>(longest) * sizeof(float) > 64 * 1024) return fail(GBXM_ERR_UNSUPPORTED, "expert_ff: rows of %d channels beyond the row kernels' LDS", longest);
  if (a->T * a->top > 0x7fffffffLL || (a->F + FC - 1) / FC > 65535 || (a->K + KC - 1) / KC > 65535) return fail(GBXM_ERR_UNSUPPORTED, "expert_ff: grid");
  return a->act == GBXM_BF16 ? launch_rows<bf16_t, true>(*a, s) : launch_rows<float, false>(*a, s);
}

extern "C" int gbxm_expert_glu_act(const void* h, const void* gate_up, const void* down, const int32_t* idx, void* y, int64_t T_, int32_t K,
                                   int32_t F, int32_t E, int32_t top, int32_t act, int32_t kind, float limit, void* ws, size_t ws_bytes,
                                   void* stream) {
  if (kind == GBXM_EXPERT_RELU2) return fail(GBXM_ERR_INVALID, "expert_glu: gated experts only");
  const gbxm_expert_args a{h, gate_up, down, idx, nullptr, y, T_, K, F, E, top, act, kind, limit, ws, ws_bytes};
  return gbxm_expert_ff(&a, stream);
}

extern "C" int gbxm_expert_glu(const void* h, const void* gate_up, const void* down, const int32_t* idx, void* y, int64_t T_, int32_t K, int32_t F,
                               int32_t E, int32_t top, int32_t act, void* ws, size_t ws_bytes, void* stream) {
  return gbxm_expert_glu_act(h, gate_up, down, idx, y, T_, K, F, E, top, act, GBXM_GLU_SILU, 0.f, ws, ws_bytes, stream);
}
