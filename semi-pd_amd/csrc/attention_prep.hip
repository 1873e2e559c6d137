// Between the projection GEMM and the attention: angle tables, per-head norms with rotation of queries, keys AND values, pool
// stores, and the means of whole blocks of cached tokens (gfx950, wave64).
//
//  * angle_table_kernel: (cos, sin) of position * freq[i], times a factor, for every row of a batch, fp32.  Computed once per
//    forward pass for every distinct set of frequencies; all layers read it.
//  * head_norm_rope_kv_store_kernel / _vec_kernel: per head q and k to unit RMS times a weight all heads share (no norm without weights), the first
//    rot elements turned in pairs (i, i + rot / 2); values turned over the whole head in pairs (m, m + E / 2); q in place,
//    k and v into the pools.  A layer that reads another layer's cache prepares its queries only (no k / v heads).
//  * block_means_kernel: the mean key and the mean value of every block of `pool` tokens that the batch completes, as the
//    pools hold them.  A mean is not kept as a row of its own: it is cut into pieces of 2^sh elements and piece i lies in the
//    mean pools at the slot of the block's token i -- about 1 / pool of the token rows' memory, handed out and given back with
//    the tokens' own slots, and one contiguous row per head where the tokens' slots are neighbours.  Batches of one row per request take their means inside the preparation launch where that has
//    the vector form.
#include "common.h"

namespace semipd {

__global__ void __launch_bounds__(256) angle_table_kernel(const int64_t* __restrict__ positions, const float* __restrict__ freq,
                                                          int half, int64_t rows, float factor, float2* __restrict__ out) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= rows * half) return;
  const int64_t t = i / half;
  float sn, cs;
  sincosf((float)positions[t] * freq[i - t * half], &sn, &cs);
  out[i] = float2{cs * factor, sn * factor};
}

struct HeadPrepArgs {
  void* qkv; int64_t ld; int64_t num_tokens;
  int H, G, D, E;
  int64_t k_off, v_off;
  const void* q_w; const void* k_w;          // [D] of the activation type, or both NULL: no norm
  float eps;
  const float* qk_cs; int rot;               // [rows, rot / 2] (cos, sin)
  const float* v_cs;                         // [rows, E / 2] (cos, sin) or NULL: values pass
  void* k_pool; void* v_pool; const int64_t* loc;
  // block means
  const int64_t* positions;
  const int32_t* req_to_token; int64_t r2t_stride;
  const int64_t* req_pool_indices; const int64_t* seq_lens;
  const int32_t* q_start; const int32_t* q_len; int64_t batch;
  int pool, k_sh, v_sh;                      // pool 0: no means
  void* kb_pool; void* vb_pool;              // [G, mean_slots, 1 << sh]
  int64_t mean_slots;
};

// One wave per (row, head of q | k | v).
template <typename T>
__global__ void __launch_bounds__(256) head_norm_rope_kv_store_kernel(HeadPrepArgs a) {
  const int lane = threadIdx.x & 63;
  const int units = a.H + 2 * a.G;
  const int64_t id = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (id >= a.num_tokens * units) return;
  const int64_t t = id / units;
  const int u = (int)(id % units), D = a.D, E = a.E, G = a.G;
  T* row = (T*)a.qkv + t * a.ld;
  if (u < a.H + G) {
    const bool is_q = u < a.H;
    T* src = is_q ? row + (int64_t)u * D : row + a.k_off + (int64_t)(u - a.H) * D;
    T* dst = is_q ? src : (T*)a.k_pool + (a.loc[t] * G + (u - a.H)) * D;
    const T* w = (const T*)(is_q ? a.q_w : a.k_w);
    float rs = 1.0f;
    if (w) {
      float ss = 0.f;
      for (int d = lane; d < D; d += 64) {
        const float x = Elem<T>::to_f(src[d]);
        ss += x * x;
      }
      rs = 1.0f / sqrtf(wave_sum(ss) / (float)D + a.eps);
    }
    auto element = [&](int d) { return w ? Elem<T>::to_f(src[d]) * rs * Elem<T>::to_f(w[d]) : Elem<T>::to_f(src[d]); };
    const int half = a.rot >> 1;
    const float2* cs = reinterpret_cast<const float2*>(a.qk_cs) + t * half;
    for (int i = lane; i < half; i += 64) {          // (a pair is read and written by one lane: q in place)
      const float x = element(i), y = element(i + half);
      const float2 c = cs[i];
      dst[i] = Elem<T>::from_f(x * c.x - y * c.y);
      dst[i + half] = Elem<T>::from_f(y * c.x + x * c.y);
    }
    for (int d = a.rot + lane; d < D; d += 64) dst[d] = Elem<T>::from_f(element(d));
  } else {
    const int gv = u - a.H - G;
    const T* src = row + a.v_off + (int64_t)gv * E;
    T* dst = (T*)a.v_pool + (a.loc[t] * G + gv) * E;
    if (a.v_cs == nullptr) {
      for (int e = lane; e < E; e += 64) dst[e] = src[e];
      return;
    }
    const int half = E >> 1;
    const float2* cs = reinterpret_cast<const float2*>(a.v_cs) + t * half;
    for (int i = lane; i < half; i += 64) {
      const float x = Elem<T>::to_f(src[i]), y = Elem<T>::to_f(src[i + half]);
      const float2 c = cs[i];
      dst[i] = Elem<T>::from_f(x * c.x - y * c.y);
      dst[i + half] = Elem<T>::from_f(y * c.x + x * c.y);
    }
  }
}

// 16-bit types, 16-byte accesses: a lane takes two pieces of 8 elements that belong together -- elements 8c .. and 8c + half ..
// of a turned part, or 16 neighbours of the part that passes -- L lanes (a power of two) take a head, 64 / L heads a wave.
// rot, D - rot and E multiples of 16.  MEANS (one row per request): the lanes that write the last token of a block also
// average the block's rows, which they find through the request's row of the table, and store the mean's pieces.
template <typename T, int L, bool MEANS>
__global__ void __launch_bounds__(256) head_norm_rope_kv_store_vec_kernel(HeadPrepArgs a) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = lane % L;
  const int units = a.H + 2 * a.G, D = a.D, E = a.E, G = a.G;
  const int64_t id = ((int64_t)blockIdx.x * 4 + wave) * (64 / L) + lane / L;
  const bool on = id < a.num_tokens * units;          // (lanes of finished units still take part in the shuffles)
  const int64_t t = on ? id / units : 0;
  const int u = on ? (int)(id % units) : 0;
  const bool is_q = u < a.H, is_v = u >= a.H + G;
  const int size = is_v ? E : D, head = is_q ? u : (is_v ? u - a.H - G : u - a.H);
  const bool mine = on && c < (size >> 4);
  T* row = (T*)a.qkv + t * a.ld;
  T* src = is_q ? row + (int64_t)u * D : row + (is_v ? a.v_off : a.k_off) + (int64_t)head * size;
  const int turned = is_v ? (a.v_cs ? E : 0) : a.rot, half = turned >> 1;
  const bool turn = 8 * c < half;
  const int e0 = turn ? 8 * c : turned + 16 * (c - (half >> 3)), e1 = turn ? e0 + half : e0 + 8;
  float x[8], y[8], ss = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) x[i] = y[i] = 0.f;
  if (mine) {
    const Vec16<T> vx = load16(src + e0), vy = load16(src + e1);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      x[i] = Elem<T>::to_f(vx.e[i]);
      y[i] = Elem<T>::to_f(vy.e[i]);
      ss += x[i] * x[i] + y[i] * y[i];
    }
  }
#pragma unroll
  for (int o = L / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
  if (!mine) return;
  const T* w = (const T*)(is_q ? a.q_w : a.k_w);
  if (!is_v && w) {
    const float rs = 1.0f / sqrtf(ss / (float)D + a.eps);
    const Vec16<T> wx = load16(w + e0), wy = load16(w + e1);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      x[i] *= rs * Elem<T>::to_f(wx.e[i]);
      y[i] *= rs * Elem<T>::to_f(wy.e[i]);
    }
  }
  if (turn) {
    const float4* cs = reinterpret_cast<const float4*>((is_v ? a.v_cs : a.qk_cs) + (t * half + e0) * 2);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float4 w = cs[i];
      const float x0 = x[2 * i], y0 = y[2 * i], x1 = x[2 * i + 1], y1 = y[2 * i + 1];
      x[2 * i] = x0 * w.x - y0 * w.y;
      y[2 * i] = y0 * w.x + x0 * w.y;
      x[2 * i + 1] = x1 * w.z - y1 * w.w;
      y[2 * i + 1] = y1 * w.z + x1 * w.w;
    }
  }
  Vec16<T> ox, oy;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    ox.e[i] = Elem<T>::from_f(x[i]);
    oy.e[i] = Elem<T>::from_f(y[i]);
  }
  T* pool = (T*)(is_v ? a.v_pool : a.k_pool) + (int64_t)head * size;
  T* dst = is_q ? src : pool + a.loc[t] * (int64_t)G * size;
  store16(dst + e0, ox);
  store16(dst + e1, oy);
  if constexpr (MEANS) {
    const int64_t pos = a.positions[t];
    if (is_q || (pos + 1) % a.pool != 0) return;
    const int32_t* slots = a.req_to_token + a.req_pool_indices[t] * a.r2t_stride + pos + 1 - a.pool;
    float mx[8], my[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) mx[i] = my[i] = 0.f;
    for (int j = 0; j < a.pool; ++j) {
      Vec16<T> vx = ox, vy = oy;
      if (j + 1 < a.pool) {
        const T* p = pool + (int64_t)slots[j] * G * size;
        vx = load16(p + e0);
        vy = load16(p + e1);
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        mx[i] += Elem<T>::to_f(vx.e[i]);
        my[i] += Elem<T>::to_f(vy.e[i]);
      }
    }
    const float inv = 1.0f / (float)a.pool;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      ox.e[i] = Elem<T>::from_f(mx[i] * inv);
      oy.e[i] = Elem<T>::from_f(my[i] * inv);
    }
    const int sh = is_v ? a.v_sh : a.k_sh, mask = (1 << sh) - 1;
    T* means = (T*)(is_v ? a.vb_pool : a.kb_pool) + ((head * a.mean_slots) << sh);
    // (the last token's slot is the row's own: a padded row of a captured batch points at the dummy slot, whatever its table row says)
    auto slot_of = [&](int i) -> int64_t { return i + 1 < a.pool ? (int64_t)slots[i] : a.loc[t]; };
    store16(means + (slot_of(e0 >> sh) << sh) + (e0 & mask), ox);
    store16(means + (slot_of(e1 >> sh) << sh) + (e1 & mask), oy);
  }
}

// A workgroup per block that the batch completes (workgroups past the last one do nothing), V elements per thread and turn.
template <typename T, int V>
__global__ void __launch_bounds__(256) block_means_kernel(HeadPrepArgs a) {
  int64_t left = blockIdx.x;
  int b = -1;
  int64_t blk = 0;
  const int P = a.pool;
  for (int r0 = 0; r0 < (int)a.batch && b < 0; r0 += 8) {          // eight requests per round trip
    int64_t last[8], n[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const int r = r0 + u;
      last[u] = r < (int)a.batch ? a.seq_lens[r] : 0;
      n[u] = r < (int)a.batch ? (a.q_len ? (int64_t)a.q_len[r] : 1) : 0;
    }
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const int64_t from = last[u] > n[u] ? (last[u] - n[u]) / P : 0, cnt = last[u] > 0 ? last[u] / P - from : 0;
      if (b < 0 && left < cnt) {
        b = r0 + u;
        blk = from + left;
      }
      if (b < 0) left -= cnt;
    }
  }
  if (b < 0) return;
  const int32_t* slots = a.req_to_token + a.req_pool_indices[b] * a.r2t_stride + blk * P;
  const int G = a.G, kn = G * a.D, total = kn + G * a.E;
  const float inv = 1.0f / (float)P;
  for (int i = threadIdx.x * V; i < total; i += blockDim.x * V) {
    const bool is_v = i >= kn;
    const int size = is_v ? a.E : a.D, at = is_v ? i - kn : i, head = at / size, e = at - head * size;
    const T* src = (const T*)(is_v ? a.v_pool : a.k_pool) + at;
    const int64_t ld = (int64_t)G * size;
    float m[V];
#pragma unroll
    for (int u = 0; u < V; ++u) m[u] = 0.f;
    int j = 0;
    if constexpr (V > 1) {
      for (; j + 4 <= P; j += 4) {
        Vec16<T> x[4];
#pragma unroll
        for (int w = 0; w < 4; ++w) x[w] = load16(src + (int64_t)slots[j + w] * ld);
#pragma unroll
        for (int w = 0; w < 4; ++w)
#pragma unroll
          for (int u = 0; u < V; ++u) m[u] += Elem<T>::to_f(x[w].e[u]);
      }
      for (; j < P; ++j) {
        const Vec16<T> x = load16(src + (int64_t)slots[j] * ld);
#pragma unroll
        for (int u = 0; u < V; ++u) m[u] += Elem<T>::to_f(x.e[u]);
      }
    } else {
      for (; j < P; ++j) m[0] += Elem<T>::to_f(src[(int64_t)slots[j] * ld]);
    }
    const int sh = is_v ? a.v_sh : a.k_sh;
    T* dst = (T*)(is_v ? a.vb_pool : a.kb_pool) + ((head * a.mean_slots + slots[e >> sh]) << sh) + (e & ((1 << sh) - 1));
    if constexpr (V > 1) {
      Vec16<T> o;
#pragma unroll
      for (int u = 0; u < V; ++u) o.e[u] = Elem<T>::from_f(m[u] * inv);
      store16(dst, o);
    } else {
      dst[0] = Elem<T>::from_f(m[0] * inv);
    }
  }
}

}  // namespace semipd

using namespace semipd;

extern "C" int semipd_angle_table(const int64_t* positions, const float* freq, int half, int64_t rows, float factor, float* out, void* stream) {
  SEMIPD_CHECK_ARG(rows >= 0 && half >= 0, SEMIPD_EINVAL, "angle_table: bad sizes");
  if (rows == 0 || half == 0) return 0;
  SEMIPD_CHECK_ARG(positions && freq && out, SEMIPD_EINVAL, "angle_table: null pointer");
  const int64_t n = rows * half;
  hipLaunchKernelGGL(angle_table_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, as_stream(stream), positions, freq, half, rows,
                     factor, reinterpret_cast<float2*>(out));
  return launch_status("angle_table");
}

// the power of two a piece of a mean takes up, as a shift
static int piece_shift(int piece) {
  int s = 0;
  while (s < 20 && (1 << s) < piece) ++s;
  return (1 << s) == piece ? s : -1;
}

static int launch_block_means(const HeadPrepArgs& a, int dtype, hipStream_t s) {
  // at most: every whole block among the batch's rows, and one that each request brings to its end
  const int64_t blocks = a.num_tokens / a.pool + a.batch;
  const int64_t V = dtype == SEMIPD_F32 ? 4 : 8;
  const bool vec = a.D % V == 0 && a.E % V == 0 && aligned16(a.k_pool) && aligned16(a.v_pool) && aligned16(a.kb_pool) && aligned16(a.vb_pool);
  const int64_t per = ((int64_t)a.G * (a.D + a.E) + (vec ? V : 1) - 1) / (vec ? V : 1);
  const unsigned threads = (unsigned)(per >= 256 ? 256 : (per + 63) / 64 * 64);
  SEMIPD_DISPATCH_DTYPE(dtype, T, {
    if (vec) hipLaunchKernelGGL((block_means_kernel<T, Elem<T>::kVec>), dim3((unsigned)blocks), dim3(threads), 0, s, a);
    else hipLaunchKernelGGL((block_means_kernel<T, 1>), dim3((unsigned)blocks), dim3(threads), 0, s, a);
  });
  return 0;
}

static int check_means(const char* what, const HeadPrepArgs& a, int k_piece, int v_piece) {
  SEMIPD_CHECK_ARG(a.k_sh >= 0 && a.v_sh >= 0 && (int64_t)k_piece * a.pool >= a.D && (int64_t)v_piece * a.pool >= a.E && k_piece >= 8 &&
                       v_piece >= 8,
                   SEMIPD_ESHAPE, "%s: pieces of %d / %d elements (powers of two from 8 up that cover %d / %d in %d tokens)", what, k_piece,
                   v_piece, a.D, a.E, a.pool);
  SEMIPD_CHECK_ARG(a.kb_pool && a.vb_pool && a.mean_slots > 0 && a.k_pool && a.v_pool && a.req_to_token && a.req_pool_indices && a.seq_lens, SEMIPD_EINVAL,
                   "%s: null pointer", what);
  SEMIPD_CHECK_ARG((a.q_start == nullptr) == (a.q_len == nullptr) && (a.q_start != nullptr || a.num_tokens == a.batch), SEMIPD_EINVAL,
                   "%s: q_start and q_len come together; without them one row per request", what);
  return 0;
}

extern "C" int semipd_head_norm_rope_kv_store(void* qkv, int64_t ld, int64_t num_tokens, int num_q_heads, int num_kv_heads, int qk_dim,
                                              int v_dim, int64_t k_off, int64_t v_off, const void* q_weight, const void* k_weight,
                                              float eps, const float* qk_angles, int rot_dims, const float* v_angles, void* k_pool,
                                              void* v_pool, const int64_t* loc, const int64_t* positions, int pool, void* k_means,
                                              void* v_means, int64_t mean_slots, int k_piece, int v_piece, const int32_t* req_to_token,
                                              int64_t req_to_token_stride, const int64_t* req_pool_indices, const int64_t* seq_lens,
                                              const int32_t* q_start, const int32_t* q_len, int64_t batch, int dtype, void* stream) {
  SEMIPD_CHECK_ARG(num_tokens >= 0 && num_q_heads >= 0 && num_kv_heads >= 0 && num_q_heads + num_kv_heads > 0 && qk_dim > 0,
                   SEMIPD_EINVAL, "head_norm_rope_kv_store: bad sizes");
  if (num_tokens == 0) return 0;
  SEMIPD_CHECK_ARG(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= qk_dim && (num_kv_heads == 0 || (v_dim > 0 && (!v_angles || v_dim % 2 == 0))),
                   SEMIPD_ESHAPE, "head_norm_rope_kv_store: %d turned elements of a head of %d, value heads of %d", rot_dims, qk_dim, v_dim);
  SEMIPD_CHECK_ARG(qkv && (num_q_heads == 0 || num_kv_heads == 0 || (q_weight == nullptr) == (k_weight == nullptr)) &&
                       (rot_dims == 0 || qk_angles) && (num_kv_heads == 0 || (k_pool && v_pool && loc)),
                   SEMIPD_EINVAL, "head_norm_rope_kv_store: null pointer");
  SEMIPD_CHECK_ARG(ld >= (int64_t)num_q_heads * qk_dim &&
                       (num_kv_heads == 0 || (k_off >= (int64_t)num_q_heads * qk_dim && v_off >= k_off + (int64_t)num_kv_heads * qk_dim &&
                                              ld >= v_off + (int64_t)num_kv_heads * v_dim)),
                   SEMIPD_EINVAL, "head_norm_rope_kv_store: column ranges overlap or leave the row");
  SEMIPD_CHECK_ARG(pool == 0 || num_kv_heads > 0, SEMIPD_EINVAL, "head_norm_rope_kv_store: block means without keys");
  HeadPrepArgs a{qkv, ld, num_tokens, num_q_heads, num_kv_heads, qk_dim, v_dim, k_off, v_off, q_weight, k_weight, eps, qk_angles,
                 rot_dims, v_angles, k_pool, v_pool, loc, positions, req_to_token, req_to_token_stride, req_pool_indices, seq_lens,
                 q_start, q_len, batch, pool, piece_shift(k_piece), piece_shift(v_piece), k_means, v_means, mean_slots};
  if (pool > 0) {
    const int rc = check_means("head_norm_rope_kv_store", a, k_piece, v_piece);
    if (rc) return rc;
    SEMIPD_CHECK_ARG(positions, SEMIPD_EINVAL, "head_norm_rope_kv_store: block means need the rows' positions");
  }
  hipStream_t s = as_stream(stream);
  const int64_t items = num_tokens * (num_q_heads + 2 * num_kv_heads);
  const int widest = num_kv_heads > 0 && v_dim > qk_dim ? v_dim : qk_dim;
  int L = 1;
  while (16 * L < widest) L <<= 1;
  const bool half = dtype == SEMIPD_BF16 || dtype == SEMIPD_F16;
  const bool kv_vec = num_kv_heads == 0 || (v_dim % 16 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && aligned16(k_pool) && aligned16(v_pool) &&
                                            aligned16(k_weight) && (pool == 0 || (aligned16(k_means) && aligned16(v_means))));
  const bool vec = half && L <= 64 && qk_dim % 16 == 0 && rot_dims % 16 == 0 && ld % 8 == 0 && aligned16(qkv) &&
                   (num_q_heads == 0 || aligned16(q_weight)) && (rot_dims == 0 || aligned16(qk_angles)) &&
                   (!v_angles || aligned16(v_angles)) && kv_vec;
  const bool fused = vec && pool > 0 && q_start == nullptr;
  if (vec) {
    const int64_t per_block = 4 * (64 / L);
    const dim3 grid((unsigned)((items + per_block - 1) / per_block));
#define SEMIPD_HNR(LL)                                                                                                         \
  SEMIPD_DISPATCH_HALF(dtype, T, {                                                                                            \
    if (fused) hipLaunchKernelGGL((head_norm_rope_kv_store_vec_kernel<T, LL, true>), grid, dim3(256), 0, s, a);               \
    else hipLaunchKernelGGL((head_norm_rope_kv_store_vec_kernel<T, LL, false>), grid, dim3(256), 0, s, a);                    \
  })
    switch (L) {
      case 1: SEMIPD_HNR(1); break;
      case 2: SEMIPD_HNR(2); break;
      case 4: SEMIPD_HNR(4); break;
      case 8: SEMIPD_HNR(8); break;
      case 16: SEMIPD_HNR(16); break;
      case 32: SEMIPD_HNR(32); break;
      default: SEMIPD_HNR(64); break;
    }
#undef SEMIPD_HNR
  } else {
    SEMIPD_DISPATCH_DTYPE(dtype, T, hipLaunchKernelGGL((head_norm_rope_kv_store_kernel<T>), dim3((unsigned)((items + 3) / 4)), dim3(256),
                                                       0, s, a));
  }
  if (pool > 0 && !fused) {
    const int rc = launch_block_means(a, dtype, s);
    if (rc) return rc;
  }
  return launch_status("head_norm_rope_kv_store");
}

extern "C" int semipd_block_means(const void* k_pool, const void* v_pool, int num_kv_heads, int qk_dim, int v_dim, int pool,
                                  void* k_means, void* v_means, int64_t mean_slots, int k_piece, int v_piece, const int32_t* req_to_token,
                                  int64_t req_to_token_stride, const int64_t* req_pool_indices, const int64_t* seq_lens,
                                  const int32_t* q_start, const int32_t* q_len, int64_t batch, int64_t num_tokens, int dtype,
                                  void* stream) {
  SEMIPD_CHECK_ARG(num_kv_heads > 0 && qk_dim > 0 && v_dim > 0 && pool > 0 && batch >= 0 && num_tokens >= 0, SEMIPD_EINVAL,
                   "block_means: bad sizes");
  if (batch == 0 || num_tokens == 0) return 0;
  HeadPrepArgs a{nullptr, 0, num_tokens, 0, num_kv_heads, qk_dim, v_dim, 0, 0, nullptr, nullptr, 0.f, nullptr, 0, nullptr,
                 const_cast<void*>(k_pool), const_cast<void*>(v_pool), nullptr, nullptr, req_to_token, req_to_token_stride,
                 req_pool_indices, seq_lens, q_start, q_len, batch, pool, piece_shift(k_piece), piece_shift(v_piece), k_means, v_means,
                 mean_slots};
  int rc = check_means("block_means", a, k_piece, v_piece);
  if (rc) return rc;
  rc = launch_block_means(a, dtype, as_stream(stream));
  return rc ? rc : launch_status("block_means");
}
