// The boundary between two layers whose sublayers read one norm of the stream, and the router of their experts.
//
//   layer_update_kernel   v = (x or 0) + branch + sum_k mix[k] candidate_k + extra;  x <- v;  then the next layer's norm of v in the
//                         activation dtype, or v's image in the activation dtype at a row stride of the caller's (the input of a
//                         product over several rows side by side).  One workgroup per row; four neighbouring channels per thread.
//   router_rows_kernel    fp32 router logits of few rows: a wave per (row, expert), 16-byte loads, sums in a fixed order.
//   route_groups_kernel   softmax over all experts (or a sigmoid of each), the best groups by their largest score, the best experts of those,
//                         their scores as weights; a column past the experts may hold the logit of a gate whose sigmoid is one more weight.
#include "mixers_common.h"

namespace gbxm {
namespace {

constexpr int NT = 256, NW = NT / 64;
constexpr int ZR = 4;              // groups of V channels a thread keeps between the statistic and the norm

template <typename T, int V>
__global__ __launch_bounds__(NT) void layer_update_kernel(gbxm_layer_update_args p) {
  __shared__ float red[NW];
  __shared__ float ml[64];
  const int64_t t = blockIdx.x;
  const int width = p.width, top = p.top;
  const T* a = p.branch ? static_cast<const T*>(p.branch) + t * p.branch_row : nullptr;
  const T* cand = p.cand ? static_cast<const T*>(p.cand) + t * top * width : nullptr;
  const T* ex = p.extra ? static_cast<const T*>(p.extra) + t * width : nullptr;
  float* x = p.x + t * width;
  if (cand && threadIdx.x < top) ml[threadIdx.x] = p.mix ? p.mix[t * p.mix_row + threadIdx.x] : 1.f;
  __syncthreads();
  auto value = [&](int c, float* v) {
    float u[V];
    if (a) {
      Lanes<T, V>::load(a + c, v);
    } else {
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] = 0.f;
    }
    if (cand)
      for (int k = 0; k < top; ++k) {
        Lanes<T, V>::load(cand + static_cast<int64_t>(k) * width + c, u);
#pragma unroll
        for (int i = 0; i < V; ++i) v[i] += ml[k] * u[i];
      }
    if (ex) {
      Lanes<T, V>::load(ex + c, u);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += u[i];
    }
    if (!p.replace) {
      Lanes<float, V>::load(x + c, u);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += u[i];
    }
  };
  T* img = p.image ? static_cast<T*>(p.image) + t * p.image_row : nullptr;
  float z[ZR][V];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < ZR; ++j) {
    const int c = (threadIdx.x + j * NT) * V;
    if (c < width) {
      value(c, z[j]);
      Lanes<float, V>::store(x + c, z[j]);
      if (img) Lanes<T, V>::store(img + c, z[j]);
#pragma unroll
      for (int i = 0; i < V; ++i) ss += z[j][i] * z[j][i];
    }
  }
  for (int c = (threadIdx.x + ZR * NT) * V; c < width; c += NT * V) {
    float v[V];
    value(c, v);
    Lanes<float, V>::store(x + c, v);
    if (img) Lanes<T, V>::store(img + c, v);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += v[i] * v[i];
  }
  if (!p.norm_w) return;
  ss = block_sum<NW>(ss, red);
  const float r = 1.f / sqrtf(ss / width + p.eps);
  T* h = static_cast<T*>(p.h) + t * width;
  auto norm = [&](int c, const float* v) {
    float w[V];
    Lanes<float, V>::load(p.norm_w + c, w);
#pragma unroll
    for (int i = 0; i < V; ++i) w[i] *= v[i] * r;
    Lanes<T, V>::store(h + c, w);
  };
#pragma unroll
  for (int j = 0; j < ZR; ++j) {
    const int c = (threadIdx.x + j * NT) * V;
    if (c < width) norm(c, z[j]);
  }
  for (int c = (threadIdx.x + ZR * NT) * V; c < width; c += NT * V) {        // (a thread re-reads what it wrote)
    float v[V];
    Lanes<float, V>::load(x + c, v);
    norm(c, v);
  }
}

// grid (rows, ceil(E / NW)).  VEC: K a multiple of the 16-byte vectors of both operands.
template <typename T, bool VEC>
__global__ __launch_bounds__(NT) void router_rows_kernel(const T* __restrict__ h, const float* __restrict__ router, float* __restrict__ logits, int K, int E) {
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x & 63, e = blockIdx.y * NW + (threadIdx.x >> 6);
  if (e >= E) return;
  const T* x = h + t * K;
  const float* w = router + static_cast<int64_t>(e) * K;
  float s = 0.f;
  if constexpr (VEC) {
#pragma unroll 4
    for (int k = lane * 4; k < K; k += 256) {
      float a[4], b[4];
      Lanes<T, 4>::load(x + k, a);
      Lanes<float, 4>::load(w + k, b);
#pragma unroll
      for (int i = 0; i < 4; ++i) s += a[i] * b[i];
    }
  } else {
    for (int k = lane; k < K; k += 64) s += to_f32(x[k]) * w[k];
  }
  s = wave_sum(s);
  if (lane == 0) logits[t * E + e] = s;
}

// One workgroup per row.  The choice runs on the logits (softmax keeps their order) and by RANK: an expert counts the candidates in front
// of it -- larger, or equal with a lower index -- so no round waits for another; ranks are a permutation (a logit that is not a number
// counts as the smallest).  LDS: candidate logits [E, padded to 4 with -inf], group maxima [n_groups, padded], partial sums.
__global__ __launch_bounds__(NT) void route_groups_kernel(const float* __restrict__ logits, int64_t row, int* __restrict__ idx, float* __restrict__ weight,
                                                         int64_t weight_row, int E, int top, int n_groups, int keep_groups, int gate, int sigmoid) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float red[NW];
  float* cl = lds;
  float* gl = lds + (E + 3) / 4 * 4;
  const int64_t t = blockIdx.x;
  const int nth = blockDim.x, tid = threadIdx.x;
  const float* lr = logits + t * row;
  auto at = [&](int e) { const float v = lr[e]; return v == v ? v : -INFINITY; };
  for (int e = tid; e < (E + 3) / 4 * 4; e += nth) cl[e] = e < E ? at(e) : -INFINITY;
  __syncthreads();
  auto rank_of = [&](const float* v, int n4, int e, float x) {
    int rank = 0;
#pragma unroll 8
    for (int j = 0; j < n4; ++j) {
      const float4 u = *reinterpret_cast<const float4*>(v + 4 * j);
      const float w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
      for (int k = 0; k < 4; ++k) rank += (w[k] > x || (w[k] == x && 4 * j + k < e)) ? 1 : 0;
    }
    return rank;
  };
  if (sigmoid) {                                       // (its order is the logits' order)
    for (int e = tid; e < E; e += nth) {
      const int rank = rank_of(cl, (E + 3) / 4, e, cl[e]);
      if (rank < top) {
        idx[t * top + rank] = e;
        weight[t * weight_row + rank] = 1.f / (1.f + expf(-cl[e]));
      }
    }
    return;
  }
  float mx = -INFINITY;
  for (int e = tid; e < E; e += nth) mx = fmaxf(mx, cl[e]);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
  if (nth > 64) {
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    for (int i = 0; i < nth / 64; ++i) mx = fmaxf(mx, red[i]);
    __syncthreads();
  }
  float sum = 0.f;
  for (int e = tid; e < E; e += nth) sum += expf(cl[e] - mx);
  sum = wave_sum(sum);
  if (nth > 64) {
    if ((tid & 63) == 0) red[tid >> 6] = sum;
    __syncthreads();
    sum = 0.f;
    for (int i = 0; i < nth / 64; ++i) sum += red[i];
  }
  if (n_groups > 0) {
    const int size = E / n_groups, g4 = (n_groups + 3) / 4;
    for (int g = tid; g < 4 * g4; g += nth) {
      float a = -INFINITY;
      if (g < n_groups)
#pragma unroll 8
        for (int e = g * size; e < (g + 1) * size; ++e) a = fmaxf(a, cl[e]);
      gl[g] = a;
    }
    __syncthreads();
    for (int e = tid; e < E; e += nth) {
      const int g = e / size;
      if (rank_of(gl, g4, g, gl[g]) >= keep_groups) cl[e] = -INFINITY;      // (only this thread reads cl[e] until the barrier)
    }
    __syncthreads();
  }
  for (int e = tid; e < E; e += nth) {
    const float x = cl[e];
    const int rank = rank_of(cl, (E + 3) / 4, e, x);
    if (rank < top) {
      idx[t * top + rank] = e;
      weight[t * weight_row + rank] = expf(x - mx) / sum;
    }
  }
  if (gate && tid == 0) weight[t * weight_row + top] = 1.f / (1.f + expf(-lr[E]));
}

bool act_ok(int act) { return act == GBXM_BF16 || act == GBXM_F32; }
bool aligned(const void* p, size_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; }

}  // namespace
}  // namespace gbxm

using namespace gbxm;

extern "C" {

int gbxm_layer_update(const gbxm_layer_update_args* a, void* stream) {
  if (!a || !act_ok(a->act) || !a->x || !(a->branch || a->cand || a->extra) || a->T < 0 || a->width < 1 || (a->branch && a->branch_row < a->width) ||
      (a->cand && (a->top < 1 || (a->mix && a->mix_row < a->top))) ||
      (a->norm_w && !a->h) || (a->image && a->image_row < a->width))
    return fail(GBXM_ERR_INVALID, "layer_update: bad argument");
  if (a->cand && a->top > 64) return fail(GBXM_ERR_UNSUPPORTED, "layer_update: more than 64 candidate rows");
  if (a->T == 0) return GBXM_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const size_t vb = a->act == GBXM_BF16 ? 8 : 16;
  const bool vec = a->width % 4 == 0 && aligned(a->x, 16) && (!a->branch || (a->branch_row % 4 == 0 && aligned(a->branch, vb))) && (!a->cand || aligned(a->cand, vb)) &&
                   (!a->extra || aligned(a->extra, vb)) && (!a->norm_w || (aligned(a->norm_w, 16) && aligned(a->h, vb))) &&
                   (!a->image || (a->image_row % 4 == 0 && aligned(a->image, vb)));
  if (a->act == GBXM_BF16) {
    if (vec) layer_update_kernel<bf16_t, 4><<<dim3(a->T), NT, 0, s>>>(*a);
    else layer_update_kernel<bf16_t, 1><<<dim3(a->T), NT, 0, s>>>(*a);
  } else {
    if (vec) layer_update_kernel<float, 4><<<dim3(a->T), NT, 0, s>>>(*a);
    else layer_update_kernel<float, 1><<<dim3(a->T), NT, 0, s>>>(*a);
  }
  return after_launch("layer_update");
}

int gbxm_router_rows(const void* h, const float* router, float* logits, int64_t T_, int32_t K, int32_t E, int32_t act, void* stream) {
  if (!act_ok(act) || !h || !router || !logits || T_ < 0 || K < 1 || E < 1) return fail(GBXM_ERR_INVALID, "router_rows: bad argument");
  if ((E + NW - 1) / NW > 65535) return fail(GBXM_ERR_UNSUPPORTED, "router_rows: grid");
  if (T_ == 0) return GBXM_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const dim3 grid(T_, (E + NW - 1) / NW);
  const bool vec = K % 4 == 0 && aligned(h, act == GBXM_BF16 ? 8 : 16) && aligned(router, 16);
  if (act == GBXM_BF16) {
    if (vec) router_rows_kernel<bf16_t, true><<<grid, NT, 0, s>>>(static_cast<const bf16_t*>(h), router, logits, K, E);
    else router_rows_kernel<bf16_t, false><<<grid, NT, 0, s>>>(static_cast<const bf16_t*>(h), router, logits, K, E);
  } else {
    if (vec) router_rows_kernel<float, true><<<grid, NT, 0, s>>>(static_cast<const float*>(h), router, logits, K, E);
    else router_rows_kernel<float, false><<<grid, NT, 0, s>>>(static_cast<const float*>(h), router, logits, K, E);
  }
  return after_launch("router_rows");
}

int gbxm_route_groups(const float* logits, int64_t row, int32_t* idx, float* weight, int64_t weight_row, int64_t T_, int32_t E, int32_t top, int32_t n_groups,
                      int32_t keep_groups, int32_t gate, int32_t sigmoid, void* stream) {
  if (!logits || (sigmoid && (n_groups || gate)) || !idx || !weight || E < 1 || top < 1 || top > E || T_ < 0 || row < E + (gate ? 1 : 0) || weight_row < top + (gate ? 1 : 0) || n_groups < 0 ||
      (n_groups > 0 && (E % n_groups || keep_groups < 1 || keep_groups > n_groups || top > keep_groups * (E / n_groups))))
    return fail(GBXM_ERR_INVALID, "route_groups: bad argument");
  if (E > 8192) return fail(GBXM_ERR_UNSUPPORTED, "route_groups: more than 8192 experts");
  if (T_ == 0) return GBXM_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const size_t lds = ((E + 3) / 4 * 4 + (n_groups + 3) / 4 * 4 + 4) * sizeof(float);
  route_groups_kernel<<<dim3(T_), E <= 64 ? 64 : (E <= 128 ? 128 : NT), lds, s>>>(logits, row, idx, weight, weight_row, E, top, n_groups, keep_groups, gate,
                                                                                          sigmoid);
  return after_launch("route_groups");
}

}  // extern "C"
